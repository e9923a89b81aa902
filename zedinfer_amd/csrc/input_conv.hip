// The convolution in front of a mixer: what the mixer reads, h, is replaced by h + conv(h), a causal convolution over
// time on each channel,
//
//   y_t[c] = h_t[c] + sum_j taps[j][c] * h_(t - (K-1) + j)[c]          zeros before the sequence's start
//
// with h the normed residual stream.  The last K - 1 rows of h are state of the request: float32, [K-1][H], zero for
// a fresh request.  Everything is float32 arithmetic, rounded once where y is stored.
//
//   zi_stream_scale    resid += the pending terms; scale[t] = 1 / sqrt(mean(resid_t^2) + eps).  The normed rows are not
//                      written: whoever reads them multiplies resid by the row's scale and the channel's gain.
//   zi_input_conv      the convolution over a step's rows (h = x, or x * scale * gain), and the new tails
//   zi_norm_input_conv both in one launch for steps in which every entry brings one token
#include "zi_common.h"
#include "zi_api.h"

#define IC_MAX_TAPS 16
#define IC_RUN 4          // rows of a workgroup in long steps

template <int V>
struct ic_vec {
    float x[V];
};
template <int V>
__device__ __forceinline__ ic_vec<V> ic_zero() {
    ic_vec<V> r;
#pragma unroll
    for (int i = 0; i < V; ++i) r.x[i] = 0.f;
    return r;
}
template <int V>
__device__ __forceinline__ ic_vec<V> ic_load(const float* p) {
    ic_vec<V> r;
    if constexpr (V == 4) {
        const float4 v = *reinterpret_cast<const float4*>(p);
        r.x[0] = v.x; r.x[1] = v.y; r.x[2] = v.z; r.x[3] = v.w;
    } else {
        r.x[0] = *p;
    }
    return r;
}
template <int V>
__device__ __forceinline__ ic_vec<V> ic_load(const zi_bf16* p) {
    ic_vec<V> r;
    if constexpr (V == 4) {
        const uint2 v = *reinterpret_cast<const uint2*>(p);
        r.x[0] = __uint_as_float(v.x << 16); r.x[1] = __uint_as_float(v.x & 0xffff0000u);
        r.x[2] = __uint_as_float(v.y << 16); r.x[3] = __uint_as_float(v.y & 0xffff0000u);
    } else {
        r.x[0] = zi_load(p);
    }
    return r;
}
template <int V>
__device__ __forceinline__ void ic_store(float* p, const ic_vec<V>& v) {
    if constexpr (V == 4) *reinterpret_cast<float4*>(p) = make_float4(v.x[0], v.x[1], v.x[2], v.x[3]);
    else *p = v.x[0];
}
template <int V>
__device__ __forceinline__ void ic_store(zi_bf16* p, const ic_vec<V>& v) {
    if constexpr (V == 4) {
        uint2 w;
        w.x = zi_pack_bf16x2(v.x[0], v.x[1]);
        w.y = zi_pack_bf16x2(v.x[2], v.x[3]);
        *reinterpret_cast<uint2*>(p) = w;
    } else {
        zi_store(p, v.x[0]);
    }
}

// ---- the residual addition and every row's scale -------------------------------------------------------------------
// A workgroup a row, or (ROWS) a wavefront a row.  `splits` terms of the addition (0: none), added in rising order.
template <typename TD, int V, bool ROWS>
__global__ void __launch_bounds__(256)
stream_scale_kernel(float* __restrict__ scale, float* __restrict__ resid, const TD* __restrict__ delta, int splits,
                    int64_t split_stride, int n, int H, float eps) {
    __shared__ float red[16];
    const int64_t row = ROWS ? (int64_t)blockIdx.x * (256 / ZI_WAVE) + threadIdx.x / ZI_WAVE : blockIdx.x;
    if (ROWS && row >= n) return;
    const int first = ROWS ? (threadIdx.x & (ZI_WAVE - 1)) : threadIdx.x, step = ROWS ? ZI_WAVE : 256;
    float* rr = resid + row * H;
    const TD* dr = delta + row * H;
    float ss = 0.f;
#pragma unroll 2
    for (int c = first * V; c < H; c += step * V) {
        ic_vec<V> v = ic_load<V>(rr + c);
        if (splits > 0) {
            ic_vec<V> d = ic_load<V>(dr + c);
            int s = 1;
            for (; s + 4 <= splits; s += 4) {      // four terms' loads in flight; the additions keep their order
                const ic_vec<V> a = ic_load<V>(dr + s * split_stride + c), b = ic_load<V>(dr + (s + 1) * split_stride + c),
                                e = ic_load<V>(dr + (s + 2) * split_stride + c), f = ic_load<V>(dr + (s + 3) * split_stride + c);
#pragma unroll
                for (int i = 0; i < V; ++i) { d.x[i] += a.x[i]; d.x[i] += b.x[i]; d.x[i] += e.x[i]; d.x[i] += f.x[i]; }
            }
            for (; s < splits; ++s) {
                const ic_vec<V> a = ic_load<V>(dr + s * split_stride + c);
#pragma unroll
                for (int i = 0; i < V; ++i) d.x[i] += a.x[i];
            }
#pragma unroll
            for (int i = 0; i < V; ++i) v.x[i] += d.x[i];
            ic_store<V>(rr + c, v);
        }
#pragma unroll
        for (int i = 0; i < V; ++i) ss += v.x[i] * v.x[i];
    }
    ss = ROWS ? zi_wave_sum(ss) : zi_block_sum(ss, red);
    if (first == 0) scale[row] = 1.f / sqrtf(ss / (float)H + eps);
}

static bool ic_aligned(const void* p, int bytes) { return ((uintptr_t)p % bytes) == 0; }

// delta: [n][hidden] of type delta_dt, or `splits` float32 terms `split_stride` apart, or null with splits 0.
extern "C" int zi_stream_scale(float* scale, float* resid, const void* delta, int delta_dt, int splits, int64_t split_stride,
                               int n, int hidden, float eps, hipStream_t stream) {
    ZI_REQUIRE(n >= 0 && hidden > 0 && eps > 0.f && splits >= 0 && (splits == 0 || delta), "stream_scale: bad sizes");
    ZI_REQUIRE(splits <= 1 || (delta_dt == ZI_F32 && split_stride >= (int64_t)n * hidden), "stream_scale: partial sums are float32");
    if (n == 0) return 0;
    const bool v4 = hidden % 4 == 0 && ic_aligned(resid, 16) && split_stride % 4 == 0 &&
                    (!splits || ic_aligned(delta, delta_dt == ZI_F32 ? 16 : 8));
    // a wavefront a row for many rows; in the float32 path (whose addends are float32) one order of the sum of squares
    // whatever the step holds would need one form, but the two differ by rounding only
    const bool rows = n >= 512;
#define ZI_SS(V, ROWS)                                                                                                  \
    stream_scale_kernel<TD, V, ROWS><<<ROWS ? (n + 3) / 4 : n, 256, 0, stream>>>(scale, resid, (const TD*)delta, splits, \
                                                                                 split_stride, n, hidden, eps)
    ZI_DISPATCH_DTYPE(splits ? delta_dt : ZI_F32, TD, {
        if (v4 && rows) ZI_SS(4, true);
        else if (v4) ZI_SS(4, false);
        else if (rows) ZI_SS(1, true);
        else ZI_SS(1, false);
    });
#undef ZI_SS
    return zi_check_launch("stream_scale");
}

// ---- the convolution ------------------------------------------------------------------------------------------------
// A thread owns V channels and walks `per` consecutive rows of the step, keeping the K - 1 rows of h before the present
// one in registers (K known at compile time; K == 0: any number of taps, every row read again).  The first K - 1 tokens
// of an entry, which reach into the request's tail, all belong to the workgroup of the entry's first token: it alone
// reads that tail, and writes the new one afterwards.  With `slots` (every token's place in the cache, negative for
// tokens that have none: padding, which stands behind an entry's own) only an entry's own tokens count for the tail, and
// an entry that has none leaves its slot's tail alone.
template <typename TX, typename TW, typename TO, int V, int K>
__global__ void __launch_bounds__(128)
input_conv_kernel(TO* __restrict__ out, int64_t ldo, const TX* __restrict__ x, int64_t ldx, const float* __restrict__ scale,
                  const TW* __restrict__ gain, float gain_add, const float* __restrict__ conv_w, float* __restrict__ state,
                  int64_t state_stride, const int32_t* __restrict__ tok_seq, const int32_t* __restrict__ entry_start,
                  const int32_t* __restrict__ entry_len, const int32_t* __restrict__ entry_slot,
                  const int32_t* __restrict__ slots, int n, int H, int taps_rt, int per) {
    const int taps = K > 0 ? K : taps_rt;
    const int c = (blockIdx.y * 128 + threadIdx.x) * V;
    if (c >= H) return;
    const int t0 = blockIdx.x * per, t1 = t0 + per < n ? t0 + per : n;
    ic_vec<V> g;
#pragma unroll
    for (int i = 0; i < V; ++i) g.x[i] = 1.f;
    if (scale) {
        g = ic_load<V>(gain + c);
#pragma unroll
        for (int i = 0; i < V; ++i) g.x[i] += gain_add;
    }
    auto h_at = [&](int64_t t) __attribute__((always_inline)) {
        ic_vec<V> v = ic_load<V>(x + t * ldx + c);
        if (scale) {
            const float s = scale[t];
#pragma unroll
            for (int i = 0; i < V; ++i) v.x[i] = v.x[i] * s * g.x[i];
        }
        return v;
    };
    auto weight = [&](int j) __attribute__((always_inline)) { return ic_load<V>(conv_w + (int64_t)j * H + c); };
    constexpr int W = K > 1 ? K - 1 : 1;
    ic_vec<V> win[W], wt[K > 0 ? K : 1];
    if constexpr (K > 0) {
#pragma unroll
        for (int j = 0; j < K; ++j) wt[j] = weight(j);
        if constexpr (K > 1) {
#pragma unroll
            for (int k = 0; k < K - 1; ++k) {
                const int t = t0 - (K - 1) + k;
                win[k] = h_at(t > 0 ? t : 0);      // (rows of another entry, or none: never used)
            }
        }
    }
    if constexpr (K > 1) {
        // a run of rows of one entry that do not reach into the tail: every row's load issued before the first is used
        if (per == IC_RUN && t1 - t0 == IC_RUN) {
            const int e = tok_seq[t0];
            if (tok_seq[t1 - 1] == e && t0 - entry_start[e] >= K - 1) {
                ic_vec<V> h[IC_RUN];
#pragma unroll
                for (int u = 0; u < IC_RUN; ++u) h[u] = h_at(t0 + u);
#pragma unroll
                for (int u = 0; u < IC_RUN; ++u) {
                    ic_vec<V> y = h[u];
#pragma unroll
                    for (int i = 0; i < V; ++i) {
                        float a = 0.f;
#pragma unroll
                        for (int k = 0; k < K; ++k) {
                            const int r = u - (K - 1) + k;      // (known when the loops are unrolled)
                            a += wt[k].x[i] * (r >= 0 ? h[r >= 0 ? r : 0].x[i] : win[r < 0 ? r + K - 1 : 0].x[i]);
                        }
                        y.x[i] += a;
                    }
                    ic_store<V>(out + (int64_t)(t0 + u) * ldo + c, y);
                }
                return;
            }
        }
    }
    for (int t = t0; t < t1; ++t) {
        const int e = tok_seq[t], start = entry_start[e], local = t - start;
        const ic_vec<V> cur = h_at(t);
        if (local >= taps - 1) {
            ic_vec<V> y = cur;
            if constexpr (K > 0) {
#pragma unroll
                for (int i = 0; i < V; ++i) {
                    float a = 0.f;
                    if constexpr (K > 1) {
#pragma unroll
                        for (int k = 0; k < K - 1; ++k) a += wt[k].x[i] * win[k].x[i];
                    }
                    a += wt[K - 1].x[i] * cur.x[i];
                    y.x[i] += a;
                }
            } else {
                ic_vec<V> a = ic_zero<V>();
                for (int j = 0; j < taps; ++j) {
                    const ic_vec<V> hv = h_at(t - (taps - 1) + j), wj = weight(j);
#pragma unroll
                    for (int i = 0; i < V; ++i) a.x[i] += wj.x[i] * hv.x[i];
                }
#pragma unroll
                for (int i = 0; i < V; ++i) y.x[i] += a.x[i];
            }
            ic_store<V>(out + (int64_t)t * ldo + c, y);
        } else if (local == 0) {
            float* tail = state + (int64_t)entry_slot[e] * state_stride + c;
            const int len = entry_len[e];
            const int m = len < taps - 1 ? len : taps - 1;
            for (int i0 = 0; i0 < m; ++i0) {
                ic_vec<V> a = ic_zero<V>(), own = a;
                for (int j = 0; j < taps; ++j) {
                    const int li = i0 - (taps - 1) + j;
                    own = li >= 0 ? h_at(start + li) : ic_load<V>(tail + (int64_t)(li + taps - 1) * H);
                    const ic_vec<V> wj = weight(j);
#pragma unroll
                    for (int i = 0; i < V; ++i) a.x[i] += wj.x[i] * own.x[i];
                }
#pragma unroll
                for (int i = 0; i < V; ++i) a.x[i] = own.x[i] + a.x[i];      // the last tap's row is the token's own
                ic_store<V>(out + (int64_t)(start + i0) * ldo + c, a);
            }
            int real = len;
            if (slots) {
                int lo = 0, hi = len;
                while (lo < hi) {
                    const int mid = (lo + hi) / 2;
                    if (slots[start + mid] >= 0) lo = mid + 1;
                    else hi = mid;
                }
                real = lo;
            }
            // in rising order: row k of the new tail comes from row real + k of the old one or later
            for (int k = 0; real > 0 && k < taps - 1; ++k) {
                const int li = real - (taps - 1) + k;
                ic_store<V>(tail + (int64_t)k * H, li >= 0 ? h_at(start + li) : ic_load<V>(tail + (int64_t)(li + taps - 1) * H));
            }
        }
        if constexpr (K > 1) {
#pragma unroll
            for (int k = 0; k + 1 < K - 1; ++k) win[k] = win[k + 1];
            win[K - 2] = cur;
        }
    }
}

// x: [n][hidden] rows of type x_dt (row stride ldx); with `scale` (float32 [n]) h = x * scale[t] * (gain + gain_add),
// else h = x.  conv_w float32 [taps][hidden], the last row the present token's.  state: float32, the tails' place in
// the slot's row ([taps - 1][hidden] floats there).
extern "C" int zi_input_conv(void* out, int out_dt, int64_t ldo, const void* x, int x_dt, int64_t ldx, const float* scale,
                             const void* gain, int gain_dt, float gain_add, const float* conv_w, float* state,
                             int64_t state_stride, const int32_t* tok_seq, const int32_t* entry_start,
                             const int32_t* entry_len, const int32_t* entry_slot, const int32_t* slots, int n, int hidden,
                             int taps, hipStream_t stream) {
    ZI_REQUIRE(n >= 0 && hidden > 0 && ldx >= hidden && ldo >= hidden && taps >= 1 && taps <= IC_MAX_TAPS,
               "input_conv: bad sizes (at most %d taps)", IC_MAX_TAPS);
    ZI_REQUIRE(!scale || gain, "input_conv: a row's scale comes with the channels' gains");
    ZI_REQUIRE(taps == 1 || (state && state_stride >= (int64_t)(taps - 1) * hidden), "input_conv: the state row is too short");
    ZI_REQUIRE(out != x, "input_conv: the result cannot overwrite its input (a row reads those before it)");
    if (n == 0) return 0;
    const int xe = x_dt == ZI_F32 ? 16 : 8, ge = gain_dt == ZI_F32 ? 16 : 8, oe = out_dt == ZI_F32 ? 16 : 8;
    const bool v4 = hidden % 4 == 0 && ldx % 4 == 0 && ldo % 4 == 0 && state_stride % 4 == 0 && ic_aligned(x, xe) &&
                    ic_aligned(out, oe) && ic_aligned(conv_w, 16) && ic_aligned(state, 16) && (!scale || ic_aligned(gain, ge));
    const int per = n >= 512 ? IC_RUN : (n >= 128 ? 2 : 1);
    const int lanes = v4 ? 4 : 1;
    const dim3 grid((n + per - 1) / per, (hidden + 128 * lanes - 1) / (128 * lanes));
#define ZI_IC(V, K)                                                                                                     \
    input_conv_kernel<TX, TW, TO, V, K><<<grid, 128, 0, stream>>>(                                                      \
        (TO*)out, ldo, (const TX*)x, ldx, scale, (const TW*)gain, gain_add, conv_w, state, state_stride, tok_seq,       \
        entry_start, entry_len, entry_slot, slots, n, hidden, taps, per)
#define ZI_IC_K(V)                          \
    switch (taps) {                         \
        case 1: ZI_IC(V, 1); break;         \
        case 2: ZI_IC(V, 2); break;         \
        case 3: ZI_IC(V, 3); break;         \
        case 4: ZI_IC(V, 4); break;         \
        default: ZI_IC(V, 0); break;        \
    }
    ZI_DISPATCH_DTYPE(x_dt, TX, ZI_DISPATCH_DTYPE(scale ? gain_dt : ZI_F32, TW, ZI_DISPATCH_DTYPE(out_dt, TO, {
        if (v4) { ZI_IC_K(4) } else { ZI_IC_K(1) }
    })));
#undef ZI_IC_K
#undef ZI_IC
    return zi_check_launch("input_conv");
}

// ---- steps of single tokens: addition, norm, convolution and the tail's move in one launch ---------------------------
// A workgroup a row; a thread owns IT groups of four channels and requests everything it needs (the stream, up to 16
// terms of the addition, gains, taps and the tail) before it uses any of it.
template <typename TD, typename TW, typename TO, int IT, int K>
__global__ void __launch_bounds__(1024)
norm_input_conv_kernel(TO* __restrict__ out, float* __restrict__ resid, const TD* __restrict__ delta, int splits,
                       int64_t split_stride, const TW* __restrict__ gain, float gain_add, float eps,
                       const float* __restrict__ conv_w, float* __restrict__ state, int64_t state_stride,
                       const int32_t* __restrict__ tok_seq, const int32_t* __restrict__ entry_slot,
                       const int32_t* __restrict__ slots, int H) {
    __shared__ float red[16];
    const int64_t row = blockIdx.x;
    float* tail = state + (int64_t)entry_slot[tok_seq[row]] * state_stride;
    const bool moves = K > 1 && (!slots || slots[row] >= 0);      // a token without a place in the cache is padding
    ic_vec<4> v[IT], g[IT], w[IT][K], tl[IT][K > 1 ? K - 1 : 1];
    float ss = 0.f;
#pragma unroll
    for (int it = 0; it < IT; ++it) {
        const int c = (it * blockDim.x + threadIdx.x) * 4;
        v[it] = g[it] = ic_zero<4>();
        if (c >= H) continue;
        v[it] = ic_load<4>(resid + row * H + c);
        g[it] = ic_load<4>(gain + c);
        ic_vec<4> d[16];
        const TD* dr = delta + row * H + c;
#pragma unroll
        for (int s = 0; s < 16; ++s) d[s] = s < splits ? ic_load<4>(dr + (int64_t)s * split_stride) : ic_zero<4>();
#pragma unroll
        for (int k = 0; k < K; ++k) w[it][k] = ic_load<4>(conv_w + (int64_t)k * H + c);
#pragma unroll
        for (int k = 0; k + 1 < K; ++k) tl[it][k] = ic_load<4>(tail + (int64_t)k * H + c);
        ic_vec<4> sum = d[0];
#pragma unroll
        for (int s = 1; s < 16; ++s)
#pragma unroll
            for (int i = 0; i < 4; ++i) sum.x[i] += d[s].x[i];
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            v[it].x[i] += sum.x[i];
            ss += v[it].x[i] * v[it].x[i];
        }
        if (splits > 0) ic_store<4>(resid + row * H + c, v[it]);
    }
    ss = zi_block_sum(ss, red);
    const float r = 1.f / sqrtf(ss / (float)H + eps);
#pragma unroll
    for (int it = 0; it < IT; ++it) {
        const int c = (it * blockDim.x + threadIdx.x) * 4;
        if (c >= H) continue;
        ic_vec<4> h, y;
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            h.x[i] = v[it].x[i] * r * (g[it].x[i] + gain_add);
            float a = 0.f;
#pragma unroll
            for (int k = 0; k + 1 < K; ++k) a += w[it][k].x[i] * tl[it][k].x[i];
            a += w[it][K - 1].x[i] * h.x[i];
            y.x[i] = h.x[i] + a;
        }
        ic_store<4>(out + row * H + c, y);
        if (moves) {
#pragma unroll
            for (int k = 0; k + 2 < K; ++k) ic_store<4>(tail + (int64_t)k * H + c, tl[it][k + 1]);
            ic_store<4>(tail + (int64_t)(K - 2) * H + c, h);
        }
    }
}

// 1 when the one-launch form takes these sizes (else: zi_stream_scale, then zi_input_conv).
extern "C" int zi_norm_input_conv_supported(int hidden, int taps, int splits) {
    return hidden > 0 && hidden % 4 == 0 && hidden <= 8192 && taps >= 1 && taps <= 4 && splits >= 0 && splits <= 16;
}

// For steps in which every entry brings one token.  out [n][hidden]; everything else as above.
extern "C" int zi_norm_input_conv(void* out, int out_dt, float* resid, const void* delta, int delta_dt, int splits,
                                  int64_t split_stride, const void* gain, int gain_dt, float gain_add, float eps,
                                  const float* conv_w, float* state, int64_t state_stride, const int32_t* tok_seq,
                                  const int32_t* entry_slot, const int32_t* slots, int n, int hidden, int taps,
                                  hipStream_t stream) {
    ZI_REQUIRE(zi_norm_input_conv_supported(hidden, taps, splits) && n >= 0 && eps > 0.f, "norm_input_conv: unsupported sizes");
    ZI_REQUIRE(splits == 0 || delta, "norm_input_conv: terms without a place");
    ZI_REQUIRE(splits <= 1 || (delta_dt == ZI_F32 && split_stride >= (int64_t)n * hidden), "norm_input_conv: partial sums are float32");
    ZI_REQUIRE(taps == 1 || (state && state_stride >= (int64_t)(taps - 1) * hidden), "norm_input_conv: the state row is too short");
    ZI_REQUIRE(ic_aligned(out, out_dt == ZI_F32 ? 16 : 8) && ic_aligned(resid, 16) && ic_aligned(gain, gain_dt == ZI_F32 ? 16 : 8) &&
                   ic_aligned(conv_w, 16) && ic_aligned(state, 16) && state_stride % 4 == 0 && split_stride % 4 == 0 &&
                   (!splits || ic_aligned(delta, delta_dt == ZI_F32 ? 16 : 8)),
               "norm_input_conv: operands must be aligned to four values");
    if (n == 0) return 0;
    const int vecs = hidden / 4, it = vecs > 1024 ? 2 : 1;
    const int threads = ((vecs + it - 1) / it + ZI_WAVE - 1) / ZI_WAVE * ZI_WAVE;
#define ZI_NIC(IT, K)                                                                                                    \
    norm_input_conv_kernel<TD, TW, TO, IT, K><<<n, threads, 0, stream>>>(                                                \
        (TO*)out, resid, (const TD*)delta, splits, split_stride, (const TW*)gain, gain_add, eps, conv_w, state, state_stride, \
        tok_seq, entry_slot, slots, hidden)
#define ZI_NIC_K(IT)                        \
    switch (taps) {                         \
        case 1: ZI_NIC(IT, 1); break;       \
        case 2: ZI_NIC(IT, 2); break;       \
        case 3: ZI_NIC(IT, 3); break;       \
        default: ZI_NIC(IT, 4); break;      \
    }
    ZI_DISPATCH_DTYPE(splits ? delta_dt : ZI_F32, TD, ZI_DISPATCH_DTYPE(gain_dt, TW, ZI_DISPATCH_DTYPE(out_dt, TO, {
        if (it == 1) { ZI_NIC_K(1) } else { ZI_NIC_K(2) }
    })));
#undef ZI_NIC_K
#undef ZI_NIC
    return zi_check_launch("norm_input_conv");
}
