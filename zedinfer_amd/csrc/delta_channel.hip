// The delta rule with a decay per key channel: per head a float32 state S [dim][vdim],
//
//   for every token:  S <- diag(g) S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q
//
// q and k unit vectors per head (q times dim^-1/2), beta in (0, 1) per head, g [heads][dim] in (0, 1), per token.
//
//   zi_channel_inputs    from the stacked projection: convolution, SiLU, unit vectors, beta, and the convolution's tail
//   zi_lowrank_gates     two low-rank projections of float32 rows at once: the decays
//                        g = exp(-exp(a_log_h) * softplus(W_a u_a + bias)) and, as they are, the output gate's W_g u_g
//   zi_delta_channel     the recurrence over the tokens of every entry, state in the request's slot
//
// The recurrence runs token by token in prompts too, in one order of all sums whatever the cut of a prompt into steps
// of several tokens; a token decoded alone takes a kernel of its own, which adds in another order.
#include "zi_common.h"
#include "zi_api.h"

typedef __attribute__((ext_vector_type(8))) __bf16 dc_bf16x8_t;
typedef __attribute__((ext_vector_type(4))) float dc_f32x4_t;
union dc_pack {
    uint4 u;
    dc_bf16x8_t b;
};

__device__ __forceinline__ float dc_decay(float z, float a) {      // exp(-a softplus(z)), a = exp(a_log)
    // softplus(z) = max(z, 0) + ln(1 + e), e = exp(-|z|), in units of ln 2; where 1 + e would drop digits of e the
    // series' first two terms are exact to 32 bits
    const float e = __builtin_amdgcn_exp2f(-fabsf(z) * 1.4426950408889634f);
    const float l = e < 0x1p-11f ? e * fmaf(-0.5f, e, 1.f) * 1.4426950408889634f : __builtin_amdgcn_logf(1.f + e);
    return __builtin_amdgcn_exp2f(-a * fmaf(fmaxf(z, 0.f), 1.4426950408889634f, l));
}

// ---- what the recurrence reads -----------------------------------------------------------------------------------------
// From the stacked projection (float32 rows, or partial sums of them): q, k and v pass a causal convolution over time
// per channel (K taps, the last one the present token's, zeros before the start) and SiLU; every head of q and k
// becomes a unit vector, q also times dim^-1/2; beta = sigmoid.  The convolution's new tail is written here too: the
// first K - 1 tokens of an entry, which reach into the request's tail, all belong to the wavefront that has the entry's
// first token.  A wavefront takes one unit (a head of q or k, 64 I channels of v, or, from partial sums, 64 I of the
// columns that the low-rank gates read, which are only added up) of `per` consecutive tokens, the rows before the
// present one in registers; lane l holds channels l, l + 64, ...
template <int I, int K>
__global__ void __launch_bounds__(256)
channel_inputs_kernel(float* __restrict__ qk, float* __restrict__ v, float* __restrict__ beta, int64_t ld_beta,
                      float* __restrict__ rest, const float* __restrict__ proj, int64_t ld, int splits, int64_t split_stride,
                      const float* __restrict__ conv_w, float* __restrict__ tails, int64_t state_stride,
                      const int32_t* __restrict__ tok_seq, const int32_t* __restrict__ entry_start,
                      const int32_t* __restrict__ entry_len, const int32_t* __restrict__ entry_slot, int n, int heads, int kvh,
                      int dim, int vdim, int taps_rt, int b_at, int rest_at, int rest_cols, int per) {
    const int lane = threadIdx.x & (ZI_WAVE - 1), unit = blockIdx.y * 4 + threadIdx.x / ZI_WAVE;
    const int taps = K > 0 ? K : taps_rt;
    const int qkc = 2 * kvh * dim, Vd = heads * vdim, C = qkc + Vd;
    const int v_units = (Vd + 64 * I - 1) / (64 * I), r_units = (rest_cols + 64 * I - 1) / (64 * I);
    if (unit >= 2 * kvh + v_units + r_units) return;
    const bool is_qk = unit < 2 * kvh, is_rest = unit >= 2 * kvh + v_units;
    // the unit's first channel (column, for the gates' columns) and how many it has
    const int at = is_qk ? unit * dim : (is_rest ? (unit - 2 * kvh - v_units) * 64 * I : qkc + (unit - 2 * kvh) * 64 * I);
    const int count = is_qk ? dim : (is_rest ? rest_cols - at : C - at);
    const int col = is_rest ? rest_at + at : at;
    const int t0 = blockIdx.x * per, t1 = t0 + per < n ? t0 + per : n;
    auto value = [&](int64_t t, int c) __attribute__((always_inline)) {
        const float* p = proj + t * ld + c;
        float x = *p;
        int s = 1;
        for (; s + 4 <= splits; s += 4) {      // four loads in flight; the additions keep their order
            const float a = p[s * split_stride], b = p[(s + 1) * split_stride], d = p[(s + 2) * split_stride], e = p[(s + 3) * split_stride];
            x += a; x += b; x += d; x += e;
        }
        for (; s < splits; ++s) x += p[s * split_stride];
        return x;
    };
    if (is_rest) {
        for (int t = t0; t < t1; ++t)
#pragma unroll
            for (int i = 0; i < I; ++i)
                if (lane + 64 * i < count) rest[(int64_t)t * rest_cols + at + lane + 64 * i] = value(t, col + lane + 64 * i);
        return;
    }
    const float unit_scale = unit < kvh ? 1.f / sqrtf((float)dim) : 1.f;
    auto finish = [&](int64_t t, const float* y) __attribute__((always_inline)) {
        float r = 1.f;
        if (is_qk) {
            float ss = 0.f;
#pragma unroll
            for (int i = 0; i < I; ++i) ss += y[i] * y[i];
            r = unit_scale / sqrtf(zi_wave_sum(ss) + 1e-6f);
        }
        float* dst = is_qk ? qk + t * qkc + at : v + t * Vd + (at - qkc);
#pragma unroll
        for (int i = 0; i < I; ++i)
            if (lane + 64 * i < count) dst[lane + 64 * i] = y[i] * r;
        if (unit == 0)
            for (int h = lane; h < heads; h += ZI_WAVE) beta[t * ld_beta + h] = 1.f / (1.f + expf(-value(t, b_at + h)));
    };
    constexpr int W = K > 1 ? K - 1 : 1;
    float win[W][I], wt[K > 0 ? K : 1][I];
    int ch[I];
#pragma unroll
    for (int i = 0; i < I; ++i) ch[i] = at + (lane + 64 * i < count ? lane + 64 * i : 0);
    if constexpr (K > 0) {
#pragma unroll
        for (int j = 0; j < K; ++j)
#pragma unroll
            for (int i = 0; i < I; ++i) wt[j][i] = conv_w[(int64_t)ch[i] * K + j];
    }
    if constexpr (K > 1) {
        if (per > 1) {
#pragma unroll
            for (int k = 0; k < K - 1; ++k) {
                const int t = t0 - (K - 1) + k;
#pragma unroll
                for (int i = 0; i < I; ++i) win[k][i] = value(t > 0 ? t : 0, ch[i]);      // (of another entry, or none: never used)
            }
        }
    }
    for (int t = t0; t < t1; ++t) {
        const int e = tok_seq[t], start = entry_start[e], local = t - start;
        float cur[I], y[I];
#pragma unroll
        for (int i = 0; i < I; ++i) cur[i] = value(t, ch[i]);
        if (local >= taps - 1) {
#pragma unroll
            for (int i = 0; i < I; ++i) {
                float a = 0.f;
                if constexpr (K > 0) {
                    if constexpr (K > 1) {
#pragma unroll
                        for (int k = 0; k < K - 1; ++k) a += wt[k][i] * (per > 1 ? win[k][i] : value(t - (K - 1) + k, ch[i]));
                    }
                    a += wt[K - 1][i] * cur[i];
                } else {
                    for (int j = 0; j < taps; ++j) a += conv_w[(int64_t)ch[i] * taps + j] * value(t - (taps - 1) + j, ch[i]);
                }
                y[i] = lane + 64 * i < count ? a / (1.f + expf(-a)) : 0.f;
            }
            finish(t, y);
        } else if (local == 0) {
            float* tail = tails + (int64_t)entry_slot[e] * state_stride;
            const int len = entry_len[e], m = len < taps - 1 ? len : taps - 1;
            auto row = [&](int li, int i) __attribute__((always_inline)) {
                return li >= 0 ? value(start + li, ch[i]) : tail[(int64_t)(li + taps - 1) * C + ch[i]];
            };
            for (int i0 = 0; i0 < m; ++i0) {
#pragma unroll
                for (int i = 0; i < I; ++i) {
                    float a = 0.f;
                    for (int j = 0; j < taps; ++j) a += conv_w[(int64_t)ch[i] * taps + j] * row(i0 - (taps - 1) + j, i);
                    y[i] = lane + 64 * i < count ? a / (1.f + expf(-a)) : 0.f;
                }
                finish(start + i0, y);
            }
            // in rising order: row k of the new tail comes from row len + k of the old one or later
#pragma unroll
            for (int i = 0; i < I; ++i)
                if (lane + 64 * i < count)
                    for (int k = 0; k < taps - 1; ++k) tail[(int64_t)k * C + ch[i]] = row(len - (taps - 1) + k, i);
        }
        if constexpr (K > 1) {
#pragma unroll
            for (int i = 0; i < I; ++i) {
#pragma unroll
                for (int k = 0; k + 1 < K - 1; ++k) win[k][i] = win[k + 1][i];
                win[K - 2][i] = cur[i];
            }
        }
    }
}

// proj: float32 [n] rows of stride ld, columns [q | k | v | ...], beta's heads at b_at; or `splits` partial sums of such
// rows, `split_stride` apart.  rest (float32 [n][rest_cols], or null with rest_cols 0): the sums of the columns
// rest_at ... + rest_cols - 1.  tails: the place of [taps - 1][channels] in the slot's row.
extern "C" int zi_channel_inputs(float* qk, float* v, float* beta, int64_t ld_beta, float* rest, const float* proj, int64_t ld,
                                 int splits, int64_t split_stride, const float* conv_w, float* tails, int64_t state_stride,
                                 const int32_t* tok_seq, const int32_t* entry_start, const int32_t* entry_len,
                                 const int32_t* entry_slot, int n, int heads, int kvh, int dim, int vdim, int taps, int b_at,
                                 int rest_at, int rest_cols, hipStream_t stream) {
    ZI_REQUIRE(n >= 0 && heads > 0 && kvh > 0 && heads % kvh == 0 && dim > 0 && dim <= 256 && vdim > 0 && taps >= 1 &&
               ld_beta >= heads && splits >= 1, "channel_inputs: bad sizes");
    const int64_t C = 2LL * kvh * dim + (int64_t)heads * vdim;
    ZI_REQUIRE(b_at >= C && ld >= b_at + heads && rest_cols >= 0 && (!rest_cols || (rest && rest_at >= C && ld >= rest_at + rest_cols)),
               "channel_inputs: the columns do not fit the rows");
    ZI_REQUIRE(taps == 1 || (tails && state_stride >= (int64_t)(taps - 1) * C), "channel_inputs: the state row is too short");
    if (n == 0) return 0;
    const int per = n >= 2048 ? 8 : (n >= 512 ? 4 : (n >= 128 ? 2 : 1));
    const int wide = dim <= 64 ? 1 : (dim <= 128 ? 2 : 4);
    const int units = 2 * kvh + (heads * vdim + 64 * wide - 1) / (64 * wide) + (rest_cols + 64 * wide - 1) / (64 * wide);
    ZI_REQUIRE((units + 3) / 4 <= 65535, "channel_inputs: too many channels");
    const dim3 grid((n + per - 1) / per, (units + 3) / 4);
#define ZI_CI(I, K)                                                                                                        \
    channel_inputs_kernel<I, K><<<grid, 256, 0, stream>>>(qk, v, beta, ld_beta, rest, proj, ld, splits, split_stride, conv_w, \
        tails, state_stride, tok_seq, entry_start, entry_len, entry_slot, n, heads, kvh, dim, vdim, taps, b_at, rest_at,    \
        rest_cols, per)
#define ZI_CI_K(I)                          \
    switch (taps) {                         \
        case 1: ZI_CI(I, 1); break;         \
        case 2: ZI_CI(I, 2); break;         \
        case 3: ZI_CI(I, 3); break;         \
        case 4: ZI_CI(I, 4); break;         \
        default: ZI_CI(I, 0); break;        \
    }
    if (wide == 1) { ZI_CI_K(1) } else if (wide == 2) { ZI_CI_K(2) } else { ZI_CI_K(4) }
#undef ZI_CI_K
#undef ZI_CI
    return zi_check_launch("channel_inputs");
}

// ---- low-rank gates -------------------------------------------------------------------------------------------------
// Matrix cores: the float32 rows u are split into two bfloat16 parts (u = hi + lo within 2^-17 of u), so that the
// product with bfloat16 weights is float32 but for that; ranks are padded to multiples of 32 (zero columns of W).  A
// wavefront makes CT * 16 channels of TM * 16 tokens (CT = 4 for many tokens: u is then split a quarter as often).
template <int TM, int CT>
__global__ void __launch_bounds__(256)
lowrank_gates_cores_kernel(float* __restrict__ out_a, const float* __restrict__ u_a, const zi_bf16* __restrict__ w_a, int Ca,
                           int Ra, const float* __restrict__ bias, const float* __restrict__ a_log, int dim,
                           float* __restrict__ out_g, const float* __restrict__ u_g, const zi_bf16* __restrict__ w_g, int Cg,
                           int Rg, int64_t ldu, int n, int blocks_a) {
    const int lane = threadIdx.x & (ZI_WAVE - 1), wave = threadIdx.x / ZI_WAVE, r = lane & 15, j = lane >> 4;
    const bool decays = (int)blockIdx.x < blocks_a;
    const int C = decays ? Ca : Cg, R = decays ? Ra : Rg;
    const int c0 = ((decays ? blockIdx.x : blockIdx.x - blocks_a) * 4 + wave) * (16 * CT);
    if (c0 >= C) return;
    const zi_bf16* w[CT];
#pragma unroll
    for (int q = 0; q < CT; ++q) w[q] = (decays ? w_a : w_g) + (int64_t)(c0 + q * 16 + r < C ? c0 + q * 16 + r : C - 1) * R;
    const float* u = decays ? u_a : u_g;
    const int t0 = blockIdx.y * (TM * 16);
    dc_f32x4_t acc[CT][TM];
#pragma unroll
    for (int q = 0; q < CT; ++q)
#pragma unroll
        for (int m = 0; m < TM; ++m) acc[q][m] = dc_f32x4_t{0.f, 0.f, 0.f, 0.f};
    for (int k0 = 0; k0 < R; k0 += 32) {
        dc_pack a[CT];
#pragma unroll
        for (int q = 0; q < CT; ++q) a[q].u = *reinterpret_cast<const uint4*>(w[q] + k0 + j * 8);
#pragma unroll
        for (int m = 0; m < TM; ++m) {
            const int t = t0 + m * 16 + r;
            const float* ur = u + (int64_t)(t < n ? t : n - 1) * ldu + k0 + j * 8;
            const float4 x0 = *reinterpret_cast<const float4*>(ur), x1 = *reinterpret_cast<const float4*>(ur + 4);
            const float x[8] = {x0.x, x0.y, x0.z, x0.w, x1.x, x1.y, x1.z, x1.w};
            dc_pack hi, lo;
            uint32_t h[4], l[4];
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                h[i] = zi_pack_bf16x2(x[2 * i], x[2 * i + 1]);
                l[i] = zi_pack_bf16x2(x[2 * i] - __uint_as_float(h[i] << 16), x[2 * i + 1] - __uint_as_float(h[i] & 0xffff0000u));
            }
            hi.u = make_uint4(h[0], h[1], h[2], h[3]);
            lo.u = make_uint4(l[0], l[1], l[2], l[3]);
#pragma unroll
            for (int q = 0; q < CT; ++q) {
                acc[q][m] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a[q].b, hi.b, acc[q][m], 0, 0, 0);
                acc[q][m] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a[q].b, lo.b, acc[q][m], 0, 0, 0);
            }
        }
    }
    // lane (r, j): channels 4j .. + 3 of every 16, of token r of each tile
    float* out = decays ? out_a : out_g;
#pragma unroll
    for (int q = 0; q < CT; ++q) {
    const int cq = c0 + q * 16 + j * 4;
    if (cq >= C) continue;
    float ba[4], ea[4];
#pragma unroll
    for (int e = 0; e < 4; ++e) {
        const int c = cq + e < C ? cq + e : C - 1;
        ba[e] = decays ? bias[c] : 0.f;
        ea[e] = decays ? expf(a_log[c / dim]) : 0.f;
    }
#pragma unroll
    for (int m = 0; m < TM; ++m) {
        const int t = t0 + m * 16 + r;
        if (t >= n) continue;
        float v[4];
#pragma unroll
        for (int e = 0; e < 4; ++e) v[e] = decays ? dc_decay(acc[q][m][e] + ba[e], ea[e]) : acc[q][m][e];
        float* dst = out + (int64_t)t * C + cq;
        if (C % 4 == 0 && cq + 3 < C) {
            *reinterpret_cast<float4*>(dst) = make_float4(v[0], v[1], v[2], v[3]);
        } else {
#pragma unroll
            for (int e = 0; e < 4; ++e)
                if (cq + e < C) dst[e] = v[e];
        }
    }
    }
}

template <typename TW>
__global__ void __launch_bounds__(256)
lowrank_gates_kernel(float* __restrict__ out_a, const float* __restrict__ u_a, const TW* __restrict__ w_a, int Ca, int Ra,
                     const float* __restrict__ bias, const float* __restrict__ a_log, int dim, float* __restrict__ out_g,
                     const float* __restrict__ u_g, const TW* __restrict__ w_g, int Cg, int Rg, int64_t ldu) {
    extern __shared__ float us[];
    const int64_t t = blockIdx.x;
    for (int i = threadIdx.x; i < Ra; i += blockDim.x) us[i] = u_a[t * ldu + i];
    for (int i = threadIdx.x; i < Rg; i += blockDim.x) us[Ra + i] = u_g[t * ldu + i];
    __syncthreads();
    for (int c = threadIdx.x; c < Ca + Cg; c += blockDim.x) {
        const bool decays = c < Ca;
        const int cc = decays ? c : c - Ca, R = decays ? Ra : Rg;
        const TW* w = (decays ? w_a : w_g) + (int64_t)cc * R;
        const float* u = decays ? us : us + Ra;
        float z = 0.f;
        for (int i = 0; i < R; ++i) z += zi_load(w + i) * u[i];
        if (decays) out_a[t * Ca + cc] = dc_decay(z + bias[cc], expf(a_log[cc / dim]));
        else out_g[t * Cg + cc] = z;
    }
}

// u_a [n][Ra], u_g [n][Rg]: float32 columns of one projection (row stride ldu).  w_a [Ca][Ra], w_g [Cg][Rg] of type
// w_dt; bias [Ca], a_log [Ca / dim] float32.  out_a [n][Ca], out_g [n][Cg] float32.
extern "C" int zi_lowrank_gates(float* out_a, const float* u_a, const void* w_a, int Ca, int Ra, const float* bias,
                                const float* a_log, int dim, float* out_g, const float* u_g, const void* w_g, int Cg, int Rg,
                                int w_dt, int64_t ldu, int n, hipStream_t stream) {
    ZI_REQUIRE(n >= 0 && Ca > 0 && Ra > 0 && dim > 0 && Ca % dim == 0 && Cg > 0 && Rg > 0 && ldu >= Ra && ldu >= Rg &&
               Ra + Rg <= 15360, "lowrank_gates: bad sizes");
    if (n == 0) return 0;
    const bool cores = w_dt == ZI_BF16 && Ra % 32 == 0 && Rg % 32 == 0 && ldu % 4 == 0 && ((uintptr_t)u_a % 16) == 0 &&
                       ((uintptr_t)u_g % 16) == 0 && ((uintptr_t)w_a % 16) == 0 && ((uintptr_t)w_g % 16) == 0 &&
                       ((uintptr_t)out_a % 16) == 0 && ((uintptr_t)out_g % 16) == 0;
    if (cores) {
        const bool many = n > 256;
        const int per = many ? 256 : 64, blocks_a = (Ca + per - 1) / per, blocks = blocks_a + (Cg + per - 1) / per;
        ZI_REQUIRE((n + 15) / 16 <= 65535, "lowrank_gates: too many tokens");
        if (many)
            lowrank_gates_cores_kernel<2, 4><<<dim3(blocks, (n + 31) / 32), 256, 0, stream>>>(
                out_a, u_a, (const zi_bf16*)w_a, Ca, Ra, bias, a_log, dim, out_g, u_g, (const zi_bf16*)w_g, Cg, Rg, ldu, n, blocks_a);
        else
            lowrank_gates_cores_kernel<1, 1><<<dim3(blocks, (n + 15) / 16), 256, 0, stream>>>(
                out_a, u_a, (const zi_bf16*)w_a, Ca, Ra, bias, a_log, dim, out_g, u_g, (const zi_bf16*)w_g, Cg, Rg, ldu, n, blocks_a);
        return zi_check_launch("lowrank_gates");
    }
    ZI_DISPATCH_DTYPE(w_dt, TW, {
        lowrank_gates_kernel<TW><<<n, 256, (Ra + Rg) * sizeof(float), stream>>>(out_a, u_a, (const TW*)w_a, Ca, Ra, bias, a_log,
                                                                               dim, out_g, u_g, (const TW*)w_g, Cg, Rg, ldu);
    });
    return zi_check_launch("lowrank_gates");
}

// ---- the recurrence over portions -----------------------------------------------------------------------------------
// A workgroup per (entry, head, WAVES * 64 / PARTS columns of S); a wavefront holds 64 / PARTS columns, lane (c, p) of it
// the R rows 4 PARTS i + 4 p .. + 3 (i < R / 4) of column c, so that the lanes of a column read consecutive bytes of a
// staged row.  (One wavefront a SIMD is all a layer of twelve heads of 128 columns gives the chip, so a token costs what
// its instructions cost one wavefront: 32 lanes a column with 4 rows each, in workgroups that stage 16 tokens at a time,
// take 283 us for 2,048 tokens, 16 lanes with 8 rows and 8 tokens at a time 365; loads two stages ahead changed nothing.)
//  k, q and g of TOKS tokens at a time lie in LDS; the next TOKS tokens' are requested before the present
// ones are worked on.  Tokens past the entry's end stand there with k = q = 0, g = 1 and beta = 0, which leaves S as it
// is to the bit, so the walk has no branch and every token's instructions are the same ones wherever it stands.
// Per token only S^T k is summed over the lanes (in-row lane moves and a swap of rows); the read-outs' sums over the lanes are made
// together after the TOKS tokens.
template <int CTRL>
__device__ __forceinline__ float dc_dpp(float x) {
    return __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(x), CTRL, 0xf, 0xf, true));
}
template <int PARTS>
__device__ __forceinline__ float dc_row_sum(float x) {      // over 16 or 32 neighbouring lanes, in every one of them
    x += dc_dpp<0xB1>(x);       // quad_perm [1, 0, 3, 2]
    x += dc_dpp<0x4E>(x);       // quad_perm [2, 3, 0, 1]
    x += dc_dpp<0x141>(x);      // row_half_mirror
    x += dc_dpp<0x140>(x);      // row_mirror
    if constexpr (PARTS == 32) {      // the sums of rows 0 and 1 (2 and 3) meet in both
        const auto r = __builtin_amdgcn_permlane16_swap(__float_as_uint(x), __float_as_uint(x), false, false);
        x = __uint_as_float(r[0]) + __uint_as_float(r[1]);
    }
    return x;
}

template <int R, int DC_PARTS, int WAVES, int DC_TOKS, int VL>
__global__ void __launch_bounds__(WAVES* ZI_WAVE)
delta_channel_kernel(float* __restrict__ out, const float* __restrict__ qk, const float* __restrict__ v,
                     const float* __restrict__ beta, int64_t ld_beta, const float* __restrict__ g, float* __restrict__ state,
                     int64_t state_stride, const int32_t* __restrict__ entry_start, const int32_t* __restrict__ entry_len,
                     const int32_t* __restrict__ entry_slot, int heads, int kvh, int dim, int vdim) {
    static_assert(DC_PARTS == 16 || DC_PARTS == 32, "a column lies in one row of lanes or in two");
    constexpr int CPW = ZI_WAVE / DC_PARTS;              // columns of a wavefront
    constexpr int D = DC_PARTS * R, COLS = CPW * WAVES, THREADS = WAVES * ZI_WAVE;
    constexpr int PER = DC_TOKS * D / VL / THREADS;      // pieces of VL values of k (or q, or g) of a chunk a thread stages
    static_assert(PER * THREADS * VL == DC_TOKS * D && PER >= 1, "a chunk's rows divide evenly over the threads");
    static_assert(DC_TOKS * COLS <= 2 * THREADS && R % 4 == 0 && DC_TOKS <= DC_PARTS, "values of a chunk: at most two a thread");
    __shared__ __attribute__((aligned(16))) float rows[2][DC_TOKS][3][D];      // k, q, g
    __shared__ float vs[2][DC_TOKS][COLS];
    __shared__ float bs[2][DC_TOKS];
    const int tid = threadIdx.x, lane = tid & (ZI_WAVE - 1), wave = tid / ZI_WAVE;
    const int c = lane / DC_PARTS, p = lane % DC_PARTS;
    const int h = blockIdx.y, e = blockIdx.z;
    const int col0 = blockIdx.x * COLS, col = col0 + wave * CPW + c;
    const bool live = col < vdim;
    const int start = entry_start[e], len = entry_len[e];
    if (len <= 0) return;
    const int kh = h / (heads / kvh), qkc = 2 * kvh * dim;
    float* S_ = state + (int64_t)entry_slot[e] * state_stride + (int64_t)h * dim * vdim;
    float S[R];
#pragma unroll
    for (int i = 0; i < R; ++i) {
        const int d = (i / 4) * (4 * DC_PARTS) + p * 4 + i % 4;
        S[i] = (live && d < dim) ? S_[(int64_t)d * vdim + col] : 0.f;
    }
    float pk[PER][VL], pq[PER][VL], pg[PER][VL], pv[2], pb;
    auto request = [&](int base) __attribute__((always_inline)) {
#pragma unroll
        for (int u = 0; u < PER; ++u) {
            const int idx = (u * THREADS + tid) * VL, tt = idx / D, d = idx % D;
            const bool ok = base + tt < len && d < dim;
            const int64_t t = start + (ok ? base + tt : 0);
            const int dd = ok ? d : 0;
            const float* kr = qk + t * qkc + (int64_t)(kvh + kh) * dim + dd;
            const float* qr = qk + t * qkc + (int64_t)kh * dim + dd;
            const float* gr = g + (t * heads + h) * dim + dd;
            if constexpr (VL == 4) {
                const float4 k4 = *reinterpret_cast<const float4*>(kr), q4 = *reinterpret_cast<const float4*>(qr),
                             g4 = *reinterpret_cast<const float4*>(gr);
                pk[u][0] = k4.x; pk[u][1] = k4.y; pk[u][2] = k4.z; pk[u][3] = k4.w;
                pq[u][0] = q4.x; pq[u][1] = q4.y; pq[u][2] = q4.z; pq[u][3] = q4.w;
                pg[u][0] = g4.x; pg[u][1] = g4.y; pg[u][2] = g4.z; pg[u][3] = g4.w;
            } else {
                pk[u][0] = *kr; pq[u][0] = *qr; pg[u][0] = *gr;
            }
        }
#pragma unroll
        for (int u = 0; u < 2; ++u) {
            const int idx = u * THREADS + tid, tt = idx / COLS, cc = col0 + idx % COLS;
            const bool ok = idx < DC_TOKS * COLS && base + tt < len && cc < vdim;
            pv[u] = v[((int64_t)(start + (ok ? base + tt : 0)) * heads + h) * vdim + (ok ? cc : 0)];
        }
        pb = beta[(int64_t)(start + ((tid < DC_TOKS && base + tid < len) ? base + tid : 0)) * ld_beta + h];
    };
    auto stash = [&](int base, int b) __attribute__((always_inline)) {
#pragma unroll
        for (int u = 0; u < PER; ++u) {
            const int idx = (u * THREADS + tid) * VL, tt = idx / D, d = idx % D;
            const bool ok = base + tt < len && d < dim;
#pragma unroll
            for (int i = 0; i < VL; ++i) {
                rows[b][tt][0][d + i] = ok ? pk[u][i] : 0.f;
                rows[b][tt][1][d + i] = ok ? pq[u][i] : 0.f;
                rows[b][tt][2][d + i] = ok ? pg[u][i] : 1.f;
            }
        }
#pragma unroll
        for (int u = 0; u < 2; ++u) {
            const int idx = u * THREADS + tid;
            if (idx < DC_TOKS * COLS) vs[b][idx / COLS][idx % COLS] = (base + idx / COLS < len && col0 + idx % COLS < vdim) ? pv[u] : 0.f;
        }
        if (tid < DC_TOKS) bs[b][tid] = base + tid < len ? pb : 0.f;
    };
    struct Tok {
        float4 k[R / 4], q[R / 4], g[R / 4];
        float v, beta;
    };
    auto fetch = [&](Tok& x, int b, int tt) __attribute__((always_inline)) {
#pragma unroll
        for (int i = 0; i < R / 4; ++i) {
            x.k[i] = *reinterpret_cast<const float4*>(&rows[b][tt][0][i * (4 * DC_PARTS) + p * 4]);
            x.q[i] = *reinterpret_cast<const float4*>(&rows[b][tt][1][i * (4 * DC_PARTS) + p * 4]);
            x.g[i] = *reinterpret_cast<const float4*>(&rows[b][tt][2][i * (4 * DC_PARTS) + p * 4]);
        }
        x.v = vs[b][tt][wave * CPW + c];
        x.beta = bs[b][tt];
    };
    auto work = [&](const Tok& x) __attribute__((always_inline)) {
        float a0 = 0.f, a1 = 0.f, a2 = 0.f, a3 = 0.f;
#pragma unroll
        for (int i = 0; i < R / 4; ++i) {
            S[4 * i] *= x.g[i].x;
            S[4 * i + 1] *= x.g[i].y;
            S[4 * i + 2] *= x.g[i].z;
            S[4 * i + 3] *= x.g[i].w;
            a0 = fmaf(S[4 * i], x.k[i].x, a0);
            a1 = fmaf(S[4 * i + 1], x.k[i].y, a1);
            a2 = fmaf(S[4 * i + 2], x.k[i].z, a2);
            a3 = fmaf(S[4 * i + 3], x.k[i].w, a3);
        }
        const float a = dc_row_sum<DC_PARTS>((a0 + a1) + (a2 + a3));
        const float u = x.beta * (x.v - a);
        float o0 = 0.f, o1 = 0.f;
#pragma unroll
        for (int i = 0; i < R / 4; ++i) {
            S[4 * i] = fmaf(x.k[i].x, u, S[4 * i]);
            S[4 * i + 1] = fmaf(x.k[i].y, u, S[4 * i + 1]);
            S[4 * i + 2] = fmaf(x.k[i].z, u, S[4 * i + 2]);
            S[4 * i + 3] = fmaf(x.k[i].w, u, S[4 * i + 3]);
            o0 = fmaf(S[4 * i], x.q[i].x, o0);
            o1 = fmaf(S[4 * i + 1], x.q[i].y, o1);
            o0 = fmaf(S[4 * i + 2], x.q[i].z, o0);
            o1 = fmaf(S[4 * i + 3], x.q[i].w, o1);
        }
        return o0 + o1;
    };
    request(0);
    stash(0, 0);
    __syncthreads();
    int cur = 0;
    for (int base = 0; base < len; base += DC_TOKS, cur ^= 1) {
        request(base + DC_TOKS);      // (past the end: the entry's first token again, unused)
        float read[DC_TOKS];
        Tok even, odd;
        fetch(even, cur, 0);
#pragma unroll
        for (int tt = 0; tt < DC_TOKS; tt += 2) {
            fetch(odd, cur, tt + 1);
            read[tt] = work(even);
            if (tt + 2 < DC_TOKS) fetch(even, cur, tt + 2);
            read[tt + 1] = work(odd);
        }
        float mine = 0.f;
#pragma unroll
        for (int tt = 0; tt < DC_TOKS; ++tt) {
            const float total = dc_row_sum<DC_PARTS>(read[tt]);
            if (p == tt) mine = total;
        }
        // lane (c, p) writes token p's read-out of column c
        if (live && p < DC_TOKS && base + p < len) out[((int64_t)(start + base + p) * heads + h) * vdim + col] = mine;
        stash(base + DC_TOKS, cur ^ 1);
        __syncthreads();
    }
    if (live) {
#pragma unroll
        for (int i = 0; i < R; ++i) {
            const int d = (i / 4) * (4 * DC_PARTS) + p * 4 + i % 4;
            if (d < dim) S_[(int64_t)d * vdim + col] = S[i];
        }
    }
}

// ---- steps in which every entry brings one token --------------------------------------------------------------------
// A workgroup per (entry, head, 64 CB columns; four wavefronts for every 64) takes the head's rows through registers
// once: a load instruction of a wavefront covers four rows x 64 columns (lane: row l / 16, columns 4 (l % 16) .. + 3),
// all loads issued before the first is used.  S^T k and S^T q of the decayed state are summed over rows together, and the read-out of the updated
// state is (S^T q) + (k . q) u.  Where a workgroup holds the whole head it can finish it: y = o / rms(o) * w *
// sigmoid(gate), and o itself is then not written.
template <typename TY, int P, int CB>      // passes of 16 rows: dim <= 16 P
__global__ void __launch_bounds__(256 * CB)
delta_channel_step_kernel(TY* __restrict__ y, const float* __restrict__ norm, const float* __restrict__ gate, float eps,
                          float* __restrict__ out, const float* __restrict__ qk, const float* __restrict__ v,
                          const float* __restrict__ beta, int64_t ld_beta, const float* __restrict__ g,
                          float* __restrict__ state, int64_t state_stride, const int32_t* __restrict__ entry_start,
                          const int32_t* __restrict__ entry_len, const int32_t* __restrict__ entry_slot, int heads, int kvh,
                          int dim, int vdim) {
    __shared__ float ks[16 * P], qs[16 * P], gs[16 * P];
    __shared__ float4 pa[CB][4][16], pb[CB][4][16];
    __shared__ float red[16];
    const int h = blockIdx.y, e = blockIdx.z, tid = threadIdx.x, lane = tid & (ZI_WAVE - 1), cb = tid / 256, wave = (tid / ZI_WAVE) % 4;
    if (entry_len[e] != 1) return;
    const int rr = lane / 16, cc = (blockIdx.x * CB + cb) * 64 + (lane % 16) * 4;
    const bool live = cc < vdim;      // vdim is a multiple of 4
    const int64_t t = entry_start[e];
    const int kh = h / (heads / kvh), qkc = 2 * kvh * dim;
    float* S = state + (int64_t)entry_slot[e] * state_stride + (int64_t)h * dim * vdim;
    float4 s[P];
#pragma unroll
    for (int i = 0; i < P; ++i) {
        const int row = i * 16 + wave * 4 + rr;
        const bool ok = live && row < dim;
        s[i] = *reinterpret_cast<const float4*>(S + (ok ? (int64_t)row * vdim + cc : 0));
    }
    const float4 vv = *reinterpret_cast<const float4*>(v + (t * heads + h) * vdim + (live ? cc : 0));
    const float bt = beta[t * ld_beta + h];
    float kq = 0.f;
    for (int d = tid; d < 16 * P; d += 256 * CB) {
        const bool in = d < dim;
        const float kk = in ? qk[t * qkc + (int64_t)(kvh + kh) * dim + d] : 0.f, qq = in ? qk[t * qkc + (int64_t)kh * dim + d] : 0.f;
        ks[d] = kk;
        qs[d] = qq;
        gs[d] = in ? g[(t * heads + h) * dim + d] : 0.f;
        kq += kk * qq;
    }
    kq = zi_block_sum(kq, red);
    __syncthreads();
    float4 a = make_float4(0.f, 0.f, 0.f, 0.f), b = a;
#pragma unroll
    for (int i = 0; i < P; ++i) {
        const int row = i * 16 + wave * 4 + rr;
        const float gg = gs[row], kk = ks[row], qq = qs[row];      // rows past dim: zeros, and so is what follows
        s[i].x *= gg; s[i].y *= gg; s[i].z *= gg; s[i].w *= gg;
        a.x = fmaf(s[i].x, kk, a.x); a.y = fmaf(s[i].y, kk, a.y); a.z = fmaf(s[i].z, kk, a.z); a.w = fmaf(s[i].w, kk, a.w);
        b.x = fmaf(s[i].x, qq, b.x); b.y = fmaf(s[i].y, qq, b.y); b.z = fmaf(s[i].z, qq, b.z); b.w = fmaf(s[i].w, qq, b.w);
    }
#pragma unroll
    for (int o = 16; o <= 32; o *= 2) {
        a.x += __shfl_xor(a.x, o, ZI_WAVE); a.y += __shfl_xor(a.y, o, ZI_WAVE);
        a.z += __shfl_xor(a.z, o, ZI_WAVE); a.w += __shfl_xor(a.w, o, ZI_WAVE);
        b.x += __shfl_xor(b.x, o, ZI_WAVE); b.y += __shfl_xor(b.y, o, ZI_WAVE);
        b.z += __shfl_xor(b.z, o, ZI_WAVE); b.w += __shfl_xor(b.w, o, ZI_WAVE);
    }
    if (rr == 0) {
        pa[cb][wave][lane] = a;
        pb[cb][wave][lane] = b;
    }
    __syncthreads();
    a = pa[cb][0][lane % 16];
    b = pb[cb][0][lane % 16];
#pragma unroll
    for (int w = 1; w < 4; ++w) {
        const float4 x = pa[cb][w][lane % 16], z = pb[cb][w][lane % 16];
        a.x += x.x; a.y += x.y; a.z += x.z; a.w += x.w;
        b.x += z.x; b.y += z.y; b.z += z.z; b.w += z.w;
    }
    const float4 u = make_float4(bt * (vv.x - a.x), bt * (vv.y - a.y), bt * (vv.z - a.z), bt * (vv.w - a.w));
    const float4 o = make_float4(fmaf(kq, u.x, b.x), fmaf(kq, u.y, b.y), fmaf(kq, u.z, b.z), fmaf(kq, u.w, b.w));
    if (y) {      // the workgroup holds the whole head
        const bool one = wave == 0 && rr == 0 && live;
        const float ss = zi_block_sum(one ? o.x * o.x + o.y * o.y + o.z * o.z + o.w * o.w : 0.f, red);
        if (one) {
            const float rstd = 1.f / sqrtf(ss / (float)vdim + eps);
            const float* gr = gate + (t * heads + h) * vdim + cc;
            TY* dst = y + (t * heads + h) * vdim + cc;
            const float ov[4] = {o.x, o.y, o.z, o.w};
#pragma unroll
            for (int i = 0; i < 4; ++i) zi_store(dst + i, ov[i] * rstd * norm[cc + i] / (1.f + expf(-gr[i])));
        }
    } else if (wave == 0 && rr == 0 && live) {
        *reinterpret_cast<float4*>(out + (t * heads + h) * vdim + cc) = o;
    }
    if (!live) return;
#pragma unroll
    for (int i = 0; i < P; ++i) {
        const int row = i * 16 + wave * 4 + rr;
        const float kk = ks[row];
        if (row < dim)
            *reinterpret_cast<float4*>(S + (int64_t)row * vdim + cc) =
                make_float4(fmaf(kk, u.x, s[i].x), fmaf(kk, u.y, s[i].y), fmaf(kk, u.z, s[i].z), fmaf(kk, u.w, s[i].w));
    }
}

// qk [n][2][kvh*dim] (q, then k), v [n][heads*vdim], beta [n] rows of stride ld_beta (heads first), g [n][heads*dim],
// out [n][heads*vdim], all float32.  state: the matrices' place in the slot's row.  single_tokens: the caller says that
// every entry brings one token (entries that do not are then left alone by the kernel for such steps).  y (type y_dt,
// [n][heads*vdim], or null; only for such steps, see zi_delta_channel_finishes): the read-outs normed with the gain
// norm [vdim], times sigmoid(gate), and out is not written.
extern "C" int zi_delta_channel_finishes(int vdim, int64_t state_stride) {
    return vdim > 0 && vdim % 4 == 0 && vdim <= 128 && state_stride % 4 == 0;
}

extern "C" int zi_delta_channel(float* out, const float* qk, const float* v, const float* beta, int64_t ld_beta,
                                const float* g, float* state, int64_t state_stride, const int32_t* entry_start,
                                const int32_t* entry_len, const int32_t* entry_slot, int entries, int heads, int kvh, int dim,
                                int vdim, int single_tokens, void* y, int y_dt, const float* norm, const float* gate, float eps,
                                hipStream_t stream) {
    ZI_REQUIRE(entries >= 0 && entries <= 65535 && heads > 0 && heads <= 65535 && kvh > 0 && heads % kvh == 0 && dim > 0 &&
               vdim > 0 && ld_beta >= heads, "delta_channel: bad sizes");
    ZI_REQUIRE(dim <= 256, "delta_channel: dim %d is more than the 256 rows a wavefront holds", dim);
    ZI_REQUIRE(state_stride >= (int64_t)heads * dim * vdim, "delta_channel: the state row is too short");
    if (entries == 0) return 0;
    const bool a16 = ((uintptr_t)qk % 16) == 0 && ((uintptr_t)g % 16) == 0;
    if (single_tokens && vdim % 4 == 0 && state_stride % 4 == 0 && ((uintptr_t)state % 16) == 0 && ((uintptr_t)v % 16) == 0 &&
        ((uintptr_t)out % 16) == 0) {
        const int cb = y && vdim > 64 ? 2 : 1;
        const dim3 grid((vdim + 64 * cb - 1) / (64 * cb), heads, entries);
        ZI_REQUIRE(!y || (grid.x == 1 && norm && gate && eps > 0.f), "delta_channel: a head of %d values is not finished here", vdim);
#define ZI_DCS2(P, CB)                                                                                                 \
    delta_channel_step_kernel<TY, P, CB><<<grid, 256 * CB, 0, stream>>>((TY*)y, norm, gate, eps, out, qk, v, beta, ld_beta, g, \
        state, state_stride, entry_start, entry_len, entry_slot, heads, kvh, dim, vdim)
#define ZI_DCS(P)                  \
    do {                           \
        if (cb == 2) ZI_DCS2(P, 2); \
        else ZI_DCS2(P, 1);        \
    } while (0)
        ZI_DISPATCH_DTYPE(y ? y_dt : ZI_F32, TY, {
            if (dim <= 32) ZI_DCS(2);
            else if (dim <= 64) ZI_DCS(4);
            else if (dim <= 128) ZI_DCS(8);
            else ZI_DCS(16);
        });
#undef ZI_DCS
#undef ZI_DCS2
        return zi_check_launch("delta_channel_step");
    }
    ZI_REQUIRE(!y, "delta_channel: heads are finished in steps of single tokens only");
#define ZI_DC2(R, PARTS, TOKS, VL)                                                                                      \
    delta_channel_kernel<R, PARTS, 4, TOKS, VL><<<dim3((vdim + 256 / PARTS - 1) / (256 / PARTS), heads, entries), 256, 0, stream>>>( \
        out, qk, v, beta, ld_beta, g, state, state_stride, entry_start, entry_len, entry_slot, heads, kvh, dim, vdim)
    const bool v4 = dim % 4 == 0 && a16;
#define ZI_DC(R, PARTS, TOKS)                  \
    do {                                       \
        if (v4) ZI_DC2(R, PARTS, TOKS, 4);     \
        else ZI_DC2(R, PARTS, TOKS, 1);        \
    } while (0)
    if (dim <= 64) ZI_DC(4, 16, 16);
    else if (dim <= 128) ZI_DC(4, 32, 16);
    else ZI_DC(8, 32, 8);
#undef ZI_DC
#undef ZI_DC2
    return zi_check_launch("delta_channel");
}
