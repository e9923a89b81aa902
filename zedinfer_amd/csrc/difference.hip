// What stands around the softmax of attention whose heads are differences of `maps` = 2 softmax maps over the same
// values: head h = n(A_1 v - lam A_2 v), n(o) = o / sqrt(mean(o^2) + eps) * factor, times a gate per head and token.
//
// The maps are heads of the ordinary attention kernels: query head h * maps + m, and a key/value head whose key row holds
// every map's key side by side, map m at m * (d / maps), beside one value.  A query row is zero outside its own map's
// part, so its product with the whole key row is its map's score; the keys and values of a head are cached once.  (The
// prompt kernel of the common sizes multiplies a map's part alone and reads only that part.)
//
//   head_norm_store   per query and key map: RMS norm with a gain, rotation of the first dims by a table, into the
//                     padded query rows and the paged key cache; values into the value cache
//   difference_heads  the heads from the maps' attention rows
//   difference_merge  the same straight from the chunks that the decode attention leaves (attention_decode.hip)
//
// All arithmetic is float32.
#include "zi_common.h"
#include "zi_api.h"
#include "zi_paging.h"

#define DF_MAX_D 512

// ---- norm, rotation, store: one wavefront per (token, unit) -------------------------------------------------------
// Units: the nq query maps (head-major), then the nk key maps, then the nkv values; maps = nq / heads = nk / nkv.
template <typename T, typename TP>
__global__ void __launch_bounds__(ZI_WAVE)
head_norm_store_kernel(T* __restrict__ q_out, int64_t ldq, T* __restrict__ kcache, T* __restrict__ vcache,
                       const TP* __restrict__ proj, int64_t ld, int splits, int64_t split_stride,
                       const float* __restrict__ q_gain, const float* __restrict__ k_gain, float eps,
                       const float* __restrict__ table, int rot, const int32_t* __restrict__ slots, int64_t cache_slots,
                       int nq, int nkv, int maps, int dim, int vdim, int d, int page_size, int pad) {
    __shared__ float xs[DF_MAX_D];
    const int t = blockIdx.x, unit = blockIdx.y, lane = threadIdx.x, nk = nkv * maps, part = d / maps;
    const bool is_q = unit < nq, is_v = unit >= nq + nk;
    ZiSlotPlace place = {0, 0, 0};
    if (!is_q) {
        place = zi_slot_place(slots ? slots[t] : -1, cache_slots, page_size);
        if (!place.ok) return;      // padding, or out of range (the host checks the range; never write outside the pool)
    }
    if (is_v) {
        const int g = unit - nq - nk;
        const TP* row = proj + (int64_t)t * ld + (int64_t)(nq + nk) * dim + (int64_t)g * vdim;
        for (int i = lane; i < d; i += ZI_WAVE) {
            float v = 0.f;
            if (i < vdim) {
                v = zi_load(row + i);
                for (int s = 1; s < splits; ++s) v += zi_load(row + s * split_stride + i);
            }
            zi_store(vcache + zi_value_offset(place.page, g, i, place.off, nkv, page_size, d), v);
        }
        return;
    }
    const int u = is_q ? unit : unit - nq, m = u % maps;
    const TP* row = proj + (int64_t)t * ld + (int64_t)unit * dim;
    float ss = 0.f;
    for (int i = lane; i < dim; i += ZI_WAVE) {
        float v = zi_load(row + i);
        for (int s = 1; s < splits; ++s) v += zi_load(row + s * split_stride + i);
        xs[i] = v;
        ss += v * v;
    }
    const float* gain = is_q ? q_gain : k_gain;
    if (gain) {
        const float r = 1.f / sqrtf(zi_wave_sum(ss) / (float)dim + eps);
        for (int i = lane; i < dim; i += ZI_WAVE) xs[i] = xs[i] * r * gain[i];
    }
    __syncthreads();
    // query row u: d values, its own map's at m * part, zeros elsewhere (where asked for); key row: all maps of a head
    T* dst = is_q ? q_out + (int64_t)t * ldq + (int64_t)u * d + m * part
                  : kcache + zi_key_offset(place.page, u / maps, place.off, nkv, page_size, d) + m * part;
    const int half = rot / 2, end = m == maps - 1 ? d - m * part : part;
    for (int i = lane; i < end; i += ZI_WAVE) {
        float v = i < dim ? xs[i] : 0.f;
        if (i < rot) {
            const int pr = i < half ? i : i - half;
            const float c = table[((int64_t)t * half + pr) * 2], s = table[((int64_t)t * half + pr) * 2 + 1];
            v = i < half ? xs[i] * c - xs[i + half] * s : xs[i] * c + xs[i - half] * s;
        }
        zi_store(dst + i, v);
    }
    if (is_q && pad) {
        T* qr = q_out + (int64_t)t * ldq + (int64_t)u * d;
        for (int i = lane; i < d; i += ZI_WAVE)
            if (i < m * part || i >= m * part + end) zi_store(qr + i, 0.f);
    }
}

// ---- the same for many tokens in bfloat16: a workgroup per eight consecutive tokens, 16-byte pieces ------------------
// L = dim / 8 lanes hold a map (a power of two); the partner of a turned piece is another of them.  Values are staged in LDS
// and leave as 16-byte runs of eight tokens where the tokens' slots are a run of a page (the usual case in a prompt).
#define DFT_TOKENS 8
__device__ __forceinline__ void df_unpack(uint4 u, float (&f)[8]) {
    f[0] = __uint_as_float(u.x << 16); f[1] = __uint_as_float(u.x & 0xffff0000u);
    f[2] = __uint_as_float(u.y << 16); f[3] = __uint_as_float(u.y & 0xffff0000u);
    f[4] = __uint_as_float(u.z << 16); f[5] = __uint_as_float(u.z & 0xffff0000u);
    f[6] = __uint_as_float(u.w << 16); f[7] = __uint_as_float(u.w & 0xffff0000u);
}
__device__ __forceinline__ uint4 df_pack(const float (&f)[8]) {
    return make_uint4(zi_pack_bf16x2(f[0], f[1]), zi_pack_bf16x2(f[2], f[3]), zi_pack_bf16x2(f[4], f[5]), zi_pack_bf16x2(f[6], f[7]));
}

template <int L>
__global__ void __launch_bounds__(256)
head_norm_store_tile_kernel(zi_bf16* __restrict__ q_out, int64_t ldq, zi_bf16* __restrict__ kcache, zi_bf16* __restrict__ vcache,
                            const zi_bf16* __restrict__ proj, int64_t ld, const float* __restrict__ q_gain,
                            const float* __restrict__ k_gain, float eps, const float* __restrict__ table, int rot,
                            const int32_t* __restrict__ slots, int64_t cache_slots, int n, int nq, int nkv, int maps, int vdim,
                            int d, int page_size, int pad, int write_kv) {
    extern __shared__ __attribute__((aligned(16))) unsigned char dft_lds[];
    constexpr int dim = L * 8;
    const int half = rot / 2, nk = nkv * maps, part = d / maps, vw = nkv * vdim;
    float* cs = reinterpret_cast<float*>(dft_lds);                                                 // [token][half][cos, sin]
    uint16_t* vt = reinterpret_cast<uint16_t*>(dft_lds + (size_t)DFT_TOKENS * rot * sizeof(float));   // [token][vw]
    const int t0 = blockIdx.x * DFT_TOKENS, tid = threadIdx.x;
    const int nt = (n - t0 < DFT_TOKENS) ? n - t0 : DFT_TOKENS;
    // the last of the tokens' workgroups (gridDim.y) takes keys and values, the others share the queries; without a cache
    // all take queries
    const bool takes_kv = write_kv && blockIdx.y == gridDim.y - 1;
    const int q_groups = gridDim.y - (write_kv ? 1 : 0), q_per = (nq + q_groups - 1) / q_groups;
    const int u_first = takes_kv ? 0 : blockIdx.y * q_per, u_end = takes_kv ? nk : (u_first + q_per < nq ? u_first + q_per : nq);
    for (int i = tid; i < nt * rot; i += 256) cs[i] = table[(int64_t)t0 * rot + i];
    if (takes_kv)
        for (int i = tid; i < nt * (vw / 8); i += 256) {
            const int tt = i / (vw / 8), c8 = i % (vw / 8);
            *reinterpret_cast<uint4*>(vt + tt * vw + c8 * 8) =
                *reinterpret_cast<const uint4*>(proj + (int64_t)(t0 + tt) * ld + (int64_t)(nq + nk) * dim + c8 * 8);
        }
    __syncthreads();
    // the maps of queries and keys: L lanes each.  Every lane of a wavefront goes round the same number of times (the lanes
    // trade values), those past the end on a map that is not stored.
    const int per = u_end - u_first, units = nt * per, li = tid % L, swap = half / 8;
    const bool is_q = !takes_kv;
    for (int i0 = 0; i0 < units; i0 += 256 / L) {
        const int i = i0 + tid / L, ic = i < units ? i : units - 1;
        const int tt = ic / per, u = u_first + ic % per, m = u % maps;
        float x[8], y[8];
        df_unpack(*reinterpret_cast<const uint4*>(proj + (int64_t)(t0 + tt) * ld + (int64_t)((is_q ? 0 : nq) + u) * dim + li * 8), x);
        const float* gain = is_q ? q_gain : k_gain;
        if (gain) {
            float ss = 0.f;
#pragma unroll
            for (int e = 0; e < 8; ++e) ss += x[e] * x[e];
#pragma unroll
            for (int o = 1; o < L; o *= 2) ss += __shfl_xor(ss, o, ZI_WAVE);
            const float rs = 1.f / sqrtf(ss / (float)dim + eps);
            const float4 g0 = *reinterpret_cast<const float4*>(gain + li * 8), g1 = *reinterpret_cast<const float4*>(gain + li * 8 + 4);
            x[0] *= rs * g0.x; x[1] *= rs * g0.y; x[2] *= rs * g0.z; x[3] *= rs * g0.w;
            x[4] *= rs * g1.x; x[5] *= rs * g1.y; x[6] *= rs * g1.z; x[7] *= rs * g1.w;
        }
        // piece li of the turned part pairs with piece li +- swap
#pragma unroll
        for (int e = 0; e < 8; ++e) y[e] = swap ? __shfl(x[e], (tid & (ZI_WAVE - 1)) + (li < swap ? swap : -swap), ZI_WAVE) : 0.f;
        if (li * 8 < rot) {
            const bool first = li < swap;
            const float* c = cs + tt * rot + (first ? li : li - swap) * 16;
#pragma unroll
            for (int e = 0; e < 8; ++e) x[e] = first ? x[e] * c[2 * e] - y[e] * c[2 * e + 1] : x[e] * c[2 * e] + y[e] * c[2 * e + 1];
        }
        if (i >= units) continue;
        const uint4 packed = df_pack(x), zero = make_uint4(0, 0, 0, 0);
        if (is_q) {
            zi_bf16* qr = q_out + (int64_t)(t0 + tt) * ldq + (int64_t)u * d;
            *reinterpret_cast<uint4*>(qr + m * part + li * 8) = packed;
            if (pad)      // everything outside the map's own values
                for (int c8 = li; c8 < d / 8; c8 += L)
                    if (c8 * 8 < m * part || c8 * 8 >= m * part + dim) *reinterpret_cast<uint4*>(qr + c8 * 8) = zero;
        } else {
            const ZiSlotPlace place = zi_slot_place(slots[t0 + tt], cache_slots, page_size);
            if (!place.ok) continue;
            zi_bf16* kr = kcache + zi_key_offset(place.page, u / maps, place.off, nkv, page_size, d);
            *reinterpret_cast<uint4*>(kr + m * part + li * 8) = packed;
            const int end = m == maps - 1 ? d : (m + 1) * part;
            for (int c8 = (m * part + dim) / 8 + li; c8 < end / 8; c8 += L) *reinterpret_cast<uint4*>(kr + c8 * 8) = zero;
        }
    }
    if (!takes_kv) return;
    // values, transposed; dims from vdim on are nobody's
    bool run = nt == DFT_TOKENS;
    const int s0 = slots[t0];
    if (run) {
#pragma unroll
        for (int x = 1; x < DFT_TOKENS; ++x) run = run && slots[t0 + x] == s0 + x;
        run = run && s0 >= 0 && (s0 & 7) == 0 && s0 + DFT_TOKENS <= cache_slots;
    }
    if (run) {
        const int64_t page = s0 / page_size, off = s0 % page_size;
        for (int i = tid; i < nkv * d; i += 256) {
            const int g = i / d, e = i % d, at = g * vdim + e;
            uint4 w = make_uint4(0, 0, 0, 0);
            if (e < vdim) {
                w.x = (uint32_t)vt[0 * vw + at] | ((uint32_t)vt[1 * vw + at] << 16);
                w.y = (uint32_t)vt[2 * vw + at] | ((uint32_t)vt[3 * vw + at] << 16);
                w.z = (uint32_t)vt[4 * vw + at] | ((uint32_t)vt[5 * vw + at] << 16);
                w.w = (uint32_t)vt[6 * vw + at] | ((uint32_t)vt[7 * vw + at] << 16);
            }
            *reinterpret_cast<uint4*>(vcache + zi_value_offset(page, g, e, (int)off, nkv, page_size, d)) = w;
        }
    } else {
        for (int i = tid; i < nt * nkv * d; i += 256) {
            const int tt = i / (nkv * d), g = (i / d) % nkv, e = i % d;
            const ZiSlotPlace place = zi_slot_place(slots[t0 + tt], cache_slots, page_size);
            if (!place.ok) continue;
            vcache[zi_value_offset(place.page, g, e, place.off, nkv, page_size, d)].bits = e < vdim ? vt[tt * vw + g * vdim + e] : (uint16_t)0;
        }
    }
}

#define DF_MANY_TOKENS 256      // from this many tokens on the tile kernel, where it takes the sizes

// proj [n][(nh + nkv) * maps * dim + nkv * vdim (+ more)] of type p_dt (row stride ld), or `splits` float32 partial sums
// `split_stride` apart; q_gain, k_gain float32 [dim] or null (no norm); table float32 [n][rot/2][2] or null when rot is 0.
// q_out [n][nh * maps][d]; the caches (or null: nothing is stored) hold heads of d values, `slots` [n] the tokens' places.
// d / maps >= dim, d >= vdim.  `pad`: query rows are zero outside their map's part (else that part alone is written).
extern "C" int zi_head_norm_store(void* q_out, int dt, int64_t ldq, void* kcache, void* vcache, const void* proj, int p_dt,
                                  int64_t ld, int splits, int64_t split_stride, const float* q_gain, const float* k_gain,
                                  float eps, const float* table, int rot, const int32_t* slots, int64_t cache_slots, int n,
                                  int nh, int nkv, int maps, int dim, int vdim, int d, int page_size, int pad,
                                  hipStream_t stream) {
    ZI_REQUIRE(n >= 0 && nh > 0 && nkv > 0 && maps > 0 && dim > 0 && vdim > 0 && d <= DF_MAX_D && d / maps >= dim && d >= vdim,
               "head_norm_store: bad sizes (heads %d/%d, %d maps, dim %d, vdim %d in heads of %d)", nh, nkv, maps, dim, vdim, d);
    const int64_t units = (int64_t)(nh + nkv) * maps + nkv;
    ZI_REQUIRE(units <= 65535, "head_norm_store: too many heads");
    ZI_REQUIRE(rot >= 0 && rot % 2 == 0 && rot <= dim && (rot == 0 || table), "head_norm_store: %d rotated dims of %d", rot, dim);
    ZI_REQUIRE(ld >= (int64_t)(nh + nkv) * maps * dim + (int64_t)nkv * vdim && ldq >= (int64_t)nh * maps * d && splits >= 1 &&
                   eps > 0.f && (splits == 1 || p_dt == ZI_F32), "head_norm_store: a row is too short");
    ZI_REQUIRE(!kcache || (vcache && slots && page_size > 0 && cache_slots > 0 && cache_slots % page_size == 0), "head_norm_store: a cache without slots");
    if (n == 0) return 0;
    const int nq = nh * maps;
    if (!kcache) { slots = nullptr; page_size = 1; cache_slots = 0; }
    {
        const int L = dim / 8;
        const bool fits = dt == ZI_BF16 && p_dt == ZI_BF16 && splits == 1 && n >= DF_MANY_TOKENS && dim % 8 == 0 && (L & (L - 1)) == 0 &&
                          L <= 32 && (rot / 2) % 8 == 0 && vdim % 8 == 0 && d % 8 == 0 && (d / maps) % 8 == 0 && ld % 8 == 0 && ldq % 8 == 0 &&
                          ((uintptr_t)q_out % 16) == 0 && ((uintptr_t)proj % 16) == 0 && ((uintptr_t)q_gain % 16) == 0 &&
                          ((uintptr_t)k_gain % 16) == 0 && (!kcache || (page_size % 8 == 0 && ((uintptr_t)kcache % 16) == 0 && ((uintptr_t)vcache % 16) == 0));
        const size_t lds = (size_t)DFT_TOKENS * (rot * sizeof(float) + (kcache ? (size_t)nkv * vdim * 2 : 0));
        if (fits && lds <= 48 * 1024) {
#define ZI_DFT(LL)                                                                                                       \
    head_norm_store_tile_kernel<LL><<<dim3((n + DFT_TOKENS - 1) / DFT_TOKENS, kcache ? 4 : 3), 256, lds, stream>>>(        \
        (zi_bf16*)q_out, ldq, (zi_bf16*)kcache, (zi_bf16*)vcache, (const zi_bf16*)proj, ld, q_gain, k_gain, eps, table, rot, slots, \
        cache_slots, n, nq, nkv, maps, vdim, d, page_size, pad, kcache != nullptr)
            switch (L) {
                case 1: ZI_DFT(1); break;
                case 2: ZI_DFT(2); break;
                case 4: ZI_DFT(4); break;
                case 8: ZI_DFT(8); break;
                case 16: ZI_DFT(16); break;
                default: ZI_DFT(32); break;
            }
#undef ZI_DFT
            return zi_check_launch("head_norm_store");
        }
    }
    const dim3 grid(n, kcache ? (unsigned)units : (unsigned)nq);
    ZI_DISPATCH_DTYPE(dt, T, ZI_DISPATCH_DTYPE(p_dt, TP, {
        head_norm_store_kernel<T, TP><<<grid, ZI_WAVE, 0, stream>>>(
            (T*)q_out, ldq, (T*)kcache, (T*)vcache, (const TP*)proj, ld, splits, split_stride, q_gain, k_gain, eps, table, rot,
            slots, cache_slots, nq, nkv, maps, dim, vdim, d, page_size, pad);
    }));
    return zi_check_launch("head_norm_store");
}

// ---- the heads -----------------------------------------------------------------------------------------------------
// A gate per head and token: sigmoid of the sum of `splits` terms `stride` apart at [token][head].
struct DfGate {
    const void* g;      // null: none
    int f32;
    int64_t ld, stride;
    int splits;
};
__device__ __forceinline__ float df_gate(const DfGate& gt, int64_t at) {
    if (!gt.g) return 1.f;
    float v = gt.f32 ? ((const float*)gt.g)[at] : zi_load((const zi_bf16*)gt.g + at);
    for (int s = 1; s < gt.splits; ++s) v += ((const float*)gt.g)[s * gt.stride + at];
    return 1.f / (1.f + expf(-v));
}

// One wavefront per (token, head).
template <typename T>
__global__ void __launch_bounds__(ZI_WAVE)
difference_heads_kernel(T* __restrict__ out, int64_t ldo, const T* __restrict__ att, int64_t lda, int d, int vdim, float lam,
                        float factor, float eps, DfGate gt) {
    const int64_t t = blockIdx.x;
    const int h = blockIdx.y, lane = threadIdx.x;
    const T* a1 = att + t * lda + (int64_t)2 * h * d;
    const T* a2 = a1 + d;
    float ss = 0.f, o[DF_MAX_D / ZI_WAVE];
#pragma unroll
    for (int i = 0; i < DF_MAX_D / ZI_WAVE; ++i) {
        const int e = lane + i * ZI_WAVE;
        o[i] = e < vdim ? zi_load(a1 + e) - lam * zi_load(a2 + e) : 0.f;
        ss += o[i] * o[i];
    }
    const float r = factor / sqrtf(zi_wave_sum(ss) / (float)vdim + eps) * df_gate(gt, t * gt.ld + h);
#pragma unroll
    for (int i = 0; i < DF_MAX_D / ZI_WAVE; ++i) {
        const int e = lane + i * ZI_WAVE;
        if (e < vdim) zi_store(out + t * ldo + (int64_t)h * vdim + e, o[i] * r);
    }
}

// Heads of L * 8 values in bfloat16, L a power of two: L lanes a head, 16-byte pieces.
template <int L>
__global__ void __launch_bounds__(256)
difference_heads_vec_kernel(zi_bf16* __restrict__ out, int64_t ldo, const zi_bf16* __restrict__ att, int64_t lda, int n, int heads,
                            int d, float lam, float factor, float eps, DfGate gt) {
    constexpr int vdim = L * 8;
    const int64_t unit = (int64_t)blockIdx.x * (256 / L) + threadIdx.x / L, last = (int64_t)n * heads - 1;
    const int64_t uc = unit < last ? unit : last, t = uc / heads;
    const int h = (int)(uc % heads), li = threadIdx.x % L;
    const zi_bf16* a1 = att + t * lda + (int64_t)2 * h * d + li * 8;
    float x[8], y[8];
    const uint4 p1 = *reinterpret_cast<const uint4*>(a1), p2 = *reinterpret_cast<const uint4*>(a1 + d);
    const float gate = df_gate(gt, t * gt.ld + h);
    df_unpack(p1, x);
    df_unpack(p2, y);
    float ss = 0.f;
#pragma unroll
    for (int e = 0; e < 8; ++e) {
        x[e] -= lam * y[e];
        ss += x[e] * x[e];
    }
#pragma unroll
    for (int o = 1; o < L; o *= 2) ss += __shfl_xor(ss, o, ZI_WAVE);
    const float r = factor / sqrtf(ss / (float)vdim + eps) * gate;
#pragma unroll
    for (int e = 0; e < 8; ++e) x[e] *= r;
    if (unit <= last) *reinterpret_cast<uint4*>(out + t * ldo + (int64_t)h * vdim + li * 8) = df_pack(x);
}

// att [n][2 * heads][d] (map m of head h is row 2 h + m, its first vdim values count) -> out [n][heads * vdim]: o = a_1 -
// lam a_2, o / sqrt(mean(o^2) + eps) * factor * sigmoid(gate[t][h]); gate of type g_dt (or `g_splits` float32 terms), or null.
extern "C" int zi_difference_heads(void* out, int dt, int64_t ldo, const void* att, int64_t lda, int n, int heads, int d, int vdim,
                                   float lam, float factor, float eps, const void* gate, int g_dt, int64_t ld_gate, int g_splits,
                                   int64_t g_stride, hipStream_t stream) {
    ZI_REQUIRE(n >= 0 && heads > 0 && heads <= 65535 && vdim > 0 && vdim <= d && d <= DF_MAX_D && ldo >= (int64_t)heads * vdim &&
                   lda >= (int64_t)2 * heads * d && eps > 0.f, "difference_heads: bad sizes");
    ZI_REQUIRE(!gate || (ld_gate >= heads && g_splits >= 1 && (g_splits == 1 || g_dt == ZI_F32)), "difference_heads: bad gate");
    if (n == 0) return 0;
    const DfGate gt = {gate, g_dt == ZI_F32, ld_gate, g_stride, g_splits};
    const int L = vdim / 8;
    if (dt == ZI_BF16 && vdim % 8 == 0 && (L & (L - 1)) == 0 && L <= 64 && d % 8 == 0 && lda % 8 == 0 && ldo % 8 == 0 &&
        ((uintptr_t)att % 16) == 0 && ((uintptr_t)out % 16) == 0) {
        const int per = 256 / L;
        const unsigned wgs = (unsigned)(((int64_t)n * heads + per - 1) / per);
#define ZI_DFH(LL)                                                                                                     \
    difference_heads_vec_kernel<LL><<<wgs, 256, 0, stream>>>((zi_bf16*)out, ldo, (const zi_bf16*)att, lda, n, heads, d, lam, factor, eps, gt)
        switch (L) {
            case 1: ZI_DFH(1); break;
            case 2: ZI_DFH(2); break;
            case 4: ZI_DFH(4); break;
            case 8: ZI_DFH(8); break;
            case 16: ZI_DFH(16); break;
            case 32: ZI_DFH(32); break;
            default: ZI_DFH(64); break;
        }
#undef ZI_DFH
        return zi_check_launch("difference_heads");
    }
    ZI_DISPATCH_DTYPE(dt, T, {
        difference_heads_kernel<T><<<dim3(n, heads), ZI_WAVE, 0, stream>>>((T*)out, ldo, (const T*)att, lda, d, vdim, lam, factor, eps, gt);
    });
    return zi_check_launch("difference_heads");
}

// ---- the heads from the decode attention's chunks -------------------------------------------------------------------
// One workgroup of two wavefronts per (token, head), wavefront m merges map m's chunks (rising order); the first makes the head.
__global__ void __launch_bounds__(2 * ZI_WAVE)
difference_merge_kernel(zi_bf16* __restrict__ out, int64_t ldo, const float* __restrict__ part_o, const float* __restrict__ part_ml,
                        const int32_t* __restrict__ tok_pos, int heads, int D, int vdim, int window, int max_chunks, float lam,
                        float factor, float eps, DfGate gt) {
    __shared__ float second[2][ZI_WAVE];
    const int t = blockIdx.x, h = blockIdx.y, lane = threadIdx.x & (ZI_WAVE - 1), m = threadIdx.x / ZI_WAVE;
    const DecSplit sp = dec_split(tok_pos[t], window);
    const bool covered = sp.count <= max_chunks;      // (uniform; chunks the launch did not cover: it shows as NaN)
    float acc[2] = {NAN, NAN};
    const float gate = m == 0 ? df_gate(gt, (int64_t)t * gt.ld + h) : 0.f;
    if (covered) {
        const int64_t slot0 = zi_dec_part_slot(t, 2 * heads, 2 * h + m, 0);
        const float mc = lane < sp.count ? part_ml[(slot0 + lane) * 2] : -INFINITY;
        const float lc = lane < sp.count ? part_ml[(slot0 + lane) * 2 + 1] : 0.f;
        const float M = zi_wave_max(mc);
        const float wc = (mc == -INFINITY) ? 0.f : __builtin_amdgcn_exp2f(mc - M);      // maxima are in base-2 units
        float L = 0.f;
        acc[0] = acc[1] = 0.f;
        for (int c0 = 0; c0 < sp.count; c0 += 8) {
            float po[8][2];      // eight chunks' loads are issued before the first is used
#pragma unroll
            for (int c = 0; c < 8; ++c)
#pragma unroll
                for (int v = 0; v < 2; ++v)
                    po[c][v] = (c0 + c < sp.count && lane + v * ZI_WAVE < vdim) ? part_o[(slot0 + c0 + c) * D + lane + v * ZI_WAVE] : 0.f;
#pragma unroll
            for (int c = 0; c < 8; ++c) {
                const float w = __shfl(wc, (c0 + c) & (ZI_WAVE - 1), ZI_WAVE);      // 0 for chunks past the count
                L += w * __shfl(lc, (c0 + c) & (ZI_WAVE - 1), ZI_WAVE);
                acc[0] += w * po[c][0];
                acc[1] += w * po[c][1];
            }
        }
        const float inv = 1.f / L;
        acc[0] *= inv;
        acc[1] *= inv;
    }
    if (m == 1) {
        second[0][lane] = acc[0];
        second[1][lane] = acc[1];
    }
    __syncthreads();
    if (m == 1) return;
    float o[2], ss = 0.f;
#pragma unroll
    for (int v = 0; v < 2; ++v) {
        o[v] = lane + v * ZI_WAVE < vdim ? acc[v] - lam * second[v][lane] : 0.f;
        ss += o[v] * o[v];
    }
    const float r = factor / sqrtf(zi_wave_sum(ss) / (float)vdim + eps) * gate;
#pragma unroll
    for (int v = 0; v < 2; ++v)
        if (lane + v * ZI_WAVE < vdim) zi_store(out + (int64_t)t * ldo + (int64_t)h * vdim + lane + v * ZI_WAVE, o[v] * r);
}

// The chunks that zi_attention_decode left in `workspace` (out == nullptr, nh = 2 * heads, no token list) for the same n, d,
// tok_pos, window and max_chunks, as finished heads: see zi_difference_heads.  out bfloat16 [n][heads * vdim].
extern "C" int zi_difference_merge(void* out, int64_t ldo, const float* workspace, int64_t workspace_floats, int n,
                                   const int32_t* tok_pos, int window, int max_chunks, int heads, int d, int vdim, float lam,
                                   float factor, float eps, const void* gate, int g_dt, int64_t ld_gate, int g_splits,
                                   int64_t g_stride, hipStream_t stream) {
    ZI_REQUIRE(n >= 0 && n <= 65535 && heads > 0 && heads <= 32767 && d >= 16 && d <= 128 && vdim > 0 && vdim <= d && window >= 0 &&
                   max_chunks >= 1 && max_chunks <= ZI_DEC_MAXC && ldo >= (int64_t)heads * vdim && eps > 0.f, "difference_merge: bad sizes");
    ZI_REQUIRE(!gate || (ld_gate >= heads && g_splits >= 1 && (g_splits == 1 || g_dt == ZI_F32)), "difference_merge: bad gate");
    ZI_REQUIRE(workspace && workspace_floats >= zi_dec_workspace_floats(n, 2 * heads, d) && ((uintptr_t)workspace % 16) == 0,
               "difference_merge: workspace of %lld floats is too small or not aligned", (long long)workspace_floats);
    if (n == 0) return 0;
    const DfGate gt = {gate, g_dt == ZI_F32, ld_gate, g_stride, g_splits};
    difference_merge_kernel<<<dim3(n, heads), 2 * ZI_WAVE, 0, stream>>>((zi_bf16*)out, ldo, workspace,
                                                                       workspace + (int64_t)n * 2 * heads * ZI_DEC_MAXC * d, tok_pos, heads,
                                                                       d, vdim, window, max_chunks, lam, factor, eps, gt);
    return zi_check_launch("difference_merge");
}
