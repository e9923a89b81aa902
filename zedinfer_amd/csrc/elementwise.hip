// Row gathers and elementwise ops: embedding lookup, row gather, residual add,
// SwiGLU.  Arithmetic is done in float32 and rounded once on store.
#include "zi_common.h"
#include "zi_activation.h"
#include "zi_api.h"

// out[i,:] = table[ids[i],:] * scale   (scale 1: reference: src/backend/ops/embedding/cpu/embedding_cpu.cpp:10-23).
// An id outside [0, V) writes NaN into the row so that the fault shows.
template <typename TW, typename TO>
__global__ void embedding_kernel(TO* __restrict__ out, const TW* __restrict__ table,
                                 const int32_t* __restrict__ ids, int H, int V, float scale) {
    const int64_t row = blockIdx.x;
    const int id = ids[row];
    const bool ok = id >= 0 && id < V;
    const TW* src = table + (int64_t)(ok ? id : 0) * H;
    TO* dst = out + row * H;
    for (int j = threadIdx.x; j < H; j += blockDim.x) zi_store(dst + j, ok ? zi_load(src + j) * scale : NAN);
}

extern "C" int zi_embedding_scaled(void* out, int out_dt, const void* table, int table_dt, const int32_t* ids,
                                   int n, int hidden, int vocab, float scale, hipStream_t stream) {
    ZI_REQUIRE(n >= 0 && hidden > 0 && vocab > 0, "embedding: bad sizes n=%d hidden=%d vocab=%d", n, hidden, vocab);
    if (n == 0) return 0;
    ZI_DISPATCH_DTYPE(table_dt, TW, ZI_DISPATCH_DTYPE(out_dt, TO, {
        embedding_kernel<TW, TO><<<n, 256, 0, stream>>>((TO*)out, (const TW*)table, ids, hidden, vocab, scale);
    }));
    return zi_check_launch("embedding");
}

extern "C" int zi_embedding(void* out, int out_dt, const void* table, int table_dt, const int32_t* ids,
                            int n, int hidden, int vocab, hipStream_t stream) {
    return zi_embedding_scaled(out, out_dt, table, table_dt, ids, n, hidden, vocab, 1.f, stream);
}

// out[i,:] = in[idx[i],:]
template <typename T>
__global__ void gather_rows_kernel(T* __restrict__ out, const T* __restrict__ in,
                                   const int32_t* __restrict__ idx, int H, int n_in) {
    const int64_t row = blockIdx.x;
    const int s = idx[row];
    const bool ok = s >= 0 && s < n_in;
    const T* src = in + (int64_t)(ok ? s : 0) * H;
    T* dst = out + row * H;
    for (int j = threadIdx.x; j < H; j += blockDim.x) zi_store(dst + j, ok ? zi_load(src + j) : NAN);
}

extern "C" int zi_gather_rows(void* out, const void* in, int dt, const int32_t* idx, int n_out, int n_in,
                              int hidden, hipStream_t stream) {
    ZI_REQUIRE(n_out >= 0 && n_in >= 0 && hidden > 0, "gather_rows: bad sizes");
    if (n_out == 0) return 0;
    ZI_DISPATCH_DTYPE(dt, T, {
        gather_rows_kernel<T><<<n_out, 256, 0, stream>>>((T*)out, (const T*)in, idx, hidden, n_in);
    });
    return zi_check_launch("gather_rows");
}

// c = a + b, added in float32 (reference: src/backend/ops/add/cpu/add_cpu_opt.cpp:22-24,57-59).
template <typename TA, typename TB, typename TC>
__global__ void add_kernel(TC* __restrict__ c, const TA* __restrict__ a, const TB* __restrict__ b, int64_t n) {
    for (int64_t i = (int64_t)blockIdx.x * blockDim.x + threadIdx.x; i < n; i += (int64_t)gridDim.x * blockDim.x)
        zi_store(c + i, zi_load(a + i) + zi_load(b + i));
}

extern "C" int zi_add(void* c, int c_dt, const void* a, int a_dt, const void* b, int b_dt, int64_t n,
                      hipStream_t stream) {
    ZI_REQUIRE(n >= 0, "add: negative size");
    if (n == 0) return 0;
    const int blocks = (int)((n + 255) / 256 > 65535 ? 65535 : (n + 255) / 256);
    ZI_DISPATCH_DTYPE(a_dt, TA, ZI_DISPATCH_DTYPE(b_dt, TB, ZI_DISPATCH_DTYPE(c_dt, TC, {
        add_kernel<TA, TB, TC><<<blocks, 256, 0, stream>>>((TC*)c, (const TA*)a, (const TB*)b, n);
    })));
    return zi_check_launch("add");
}

// out[i,j] = up[i,j] * gate[i,j] / (1 + exp(-gate[i,j]))
// (reference: src/backend/ops/swiglu/cpu/swiglu_cpu.cpp:9-23).  gate and up are read with their
// own row strides, so both halves of one fused [n, 2I] product can be passed.  With
// `interleave` = B > 0 they are columns of ONE matrix in blocks of B: gate column j sits at
// (j / B) * 2B + j % B of `gate`, up column j another B further (`up` is not used).  The input
// may come as `splits` partial sums (split s at + s * split_stride), added in rising order.
template <typename TI, typename TO>
__global__ void swiglu_kernel(TO* __restrict__ out, const TI* __restrict__ gate, const TI* __restrict__ up,
                              int inter, int64_t ld_gate, int64_t ld_up, int interleave, int splits,
                              int64_t split_stride) {
    const int64_t row = blockIdx.y;
    const TI* g = gate + row * ld_gate;
    const TI* u = interleave > 0 ? g + interleave : up + row * ld_up;
    TO* o = out + row * (int64_t)inter;
    for (int j = blockIdx.x * blockDim.x + threadIdx.x; j < inter; j += gridDim.x * blockDim.x) {
        const int64_t c = interleave > 0 ? (int64_t)(j / interleave) * 2 * interleave + j % interleave : j;
        float gv = zi_load(g + c), uv = zi_load(u + c);
        for (int s = 1; s < splits; ++s) {
            gv += zi_load(g + s * split_stride + c);
            uv += zi_load(u + s * split_stride + c);
        }
        zi_store(o + j, uv * (gv / (1.f + expf(-gv))));
    }
}

// The common case at full speed: bfloat16 in and out, gate and up interleaved in blocks of 8, no
// partial sums.  A thread reads the 16 bytes of 8 gate values and the 16 bytes of their up values and
// writes 16 bytes.
__global__ void __launch_bounds__(256)
swiglu_il8_kernel(zi_bf16* __restrict__ out, const zi_bf16* __restrict__ gu, int64_t n_groups, int groups_per_row,
                  int64_t ld) {
    for (int64_t i = (int64_t)blockIdx.x * blockDim.x + threadIdx.x; i < n_groups; i += (int64_t)gridDim.x * blockDim.x) {
        const int64_t row = i / groups_per_row;
        const int grp = (int)(i - row * groups_per_row);
        const zi_bf16* src = gu + row * ld + (int64_t)grp * 16;
        const uint4 g = *reinterpret_cast<const uint4*>(src);
        const uint4 u = *reinterpret_cast<const uint4*>(src + 8);
        const uint32_t gw[4] = {g.x, g.y, g.z, g.w}, uw[4] = {u.x, u.y, u.z, u.w};
        uint32_t ow[4];
#pragma unroll
        for (int k = 0; k < 4; ++k) {
            const float g0 = __uint_as_float(gw[k] << 16), g1 = __uint_as_float(gw[k] & 0xffff0000u);
            const float u0 = __uint_as_float(uw[k] << 16), u1 = __uint_as_float(uw[k] & 0xffff0000u);
            ow[k] = zi_pack_bf16x2(u0 * (g0 / (1.f + expf(-g0))), u1 * (g1 / (1.f + expf(-g1))));
        }
        *reinterpret_cast<uint4*>(out + i * 8) = make_uint4(ow[0], ow[1], ow[2], ow[3]);
    }
}

// The same from the transposed product: gut [2I, n] holds, for every block of 8 channels, 8 rows of gate
// values over the n tokens and then the 8 rows of their up values (the matrix product of the stacked
// weight with x^T, which the library sometimes makes faster than x with the weight transposed).  Writes
// out [n, I].  A workgroup takes 64 channels x 64 tokens: a thread reads 16 bytes (8 tokens) of the gate
// and up rows of two neighbouring channels, the tile turns in LDS (4-byte words of two channels, rows of
// 33 words), and every token's 64 channels leave as 128 contiguous bytes.  n % 8 == 0, I % 8 == 0.
__global__ void __launch_bounds__(256)
swiglu_il8_t_kernel(zi_bf16* __restrict__ out, const zi_bf16* __restrict__ gut, int n, int inter, int64_t ldt) {
    __shared__ uint32_t tile[64 * 33];
    const int c0 = blockIdx.x * 64, m0 = blockIdx.y * 64, tid = threadIdx.x;
    {
        const int tg = tid % 8, cp = tid / 8;                 // eight tokens, a pair of channels
        const int c = c0 + 2 * cp, m = m0 + tg * 8;
        if (c < inter && m < n) {                              // inter and n are multiples of 8: whole pieces
            const zi_bf16* g = gut + (int64_t)((c / 8) * 16 + c % 8) * ldt + m;
            const uint4 ga = *reinterpret_cast<const uint4*>(g), gb = *reinterpret_cast<const uint4*>(g + ldt);
            const uint4 ua = *reinterpret_cast<const uint4*>(g + 8 * ldt), ub = *reinterpret_cast<const uint4*>(g + 9 * ldt);
            const uint32_t gaw[4] = {ga.x, ga.y, ga.z, ga.w}, gbw[4] = {gb.x, gb.y, gb.z, gb.w};
            const uint32_t uaw[4] = {ua.x, ua.y, ua.z, ua.w}, ubw[4] = {ub.x, ub.y, ub.z, ub.w};
#pragma unroll
            for (int k = 0; k < 8; ++k) {
                const int sh = (k & 1) * 16;
                const float g0 = __uint_as_float((gaw[k / 2] >> sh) << 16), g1 = __uint_as_float((gbw[k / 2] >> sh) << 16);
                const float u0 = __uint_as_float((uaw[k / 2] >> sh) << 16), u1 = __uint_as_float((ubw[k / 2] >> sh) << 16);
                tile[(tg * 8 + k) * 33 + cp] = zi_pack_bf16x2(u0 * (g0 / (1.f + expf(-g0))), u1 * (g1 / (1.f + expf(-g1))));
            }
        }
    }
    __syncthreads();
    {
        const int tok = tid / 4, q = tid % 4;                  // a token, 16 of the 64 channels
        const int m = m0 + tok, c = c0 + q * 16;
        if (m < n && c < inter) {
            const uint32_t* src = tile + tok * 33 + q * 8;
            zi_bf16* dst = out + (int64_t)m * inter + c;
            *reinterpret_cast<uint4*>(dst) = make_uint4(src[0], src[1], src[2], src[3]);
            if (c + 8 < inter) *reinterpret_cast<uint4*>(dst + 8) = make_uint4(src[4], src[5], src[6], src[7]);
        }
    }
}

// out [n, inter] from gut [2 * inter, n] (row stride ldt), bfloat16, gate and up rows in blocks of 8.
extern "C" int zi_swiglu_t(void* out, const void* gut, int dt, int n, int inter, int64_t ldt, hipStream_t stream) {
    ZI_REQUIRE(dt == ZI_BF16, "swiglu_t: bfloat16 only");
    ZI_REQUIRE(n >= 0 && inter > 0 && n % 8 == 0 && inter % 8 == 0 && ldt >= n && ldt % 8 == 0,
               "swiglu_t: tokens %d and channels %d must be multiples of 8 (row stride %lld)", n, inter, (long long)ldt);
    ZI_REQUIRE(((uintptr_t)out % 16) == 0 && ((uintptr_t)gut % 16) == 0, "swiglu_t: pointers must be aligned to 16 bytes");
    if (n == 0) return 0;
    const dim3 grid((inter + 63) / 64, (n + 63) / 64);
    ZI_REQUIRE(grid.y <= 65535, "swiglu_t: too many tokens");
    swiglu_il8_t_kernel<<<grid, 256, 0, stream>>>((zi_bf16*)out, (const zi_bf16*)gut, n, inter, ldt);
    return zi_check_launch("swiglu_t");
}

extern "C" int zi_swiglu(void* out, int out_dt, const void* gate, const void* up, int dt, int n, int inter,
                         int64_t ld_gate, int64_t ld_up, int interleave, int splits, int64_t split_stride,
                         hipStream_t stream) {
    ZI_REQUIRE(n >= 0 && inter > 0 && ld_gate >= inter, "swiglu: bad sizes n=%d inter=%d", n, inter);
    ZI_REQUIRE(interleave >= 0 && (interleave == 0 ? (up != nullptr && ld_up >= inter)
                                                   : (inter % interleave == 0 && ld_gate >= 2 * (int64_t)inter)),
               "swiglu: bad layout (interleave %d)", interleave);
    ZI_REQUIRE(splits >= 1, "swiglu: bad number of partial sums");
    if (n == 0) return 0;
    if (interleave == 8 && splits == 1 && dt == ZI_BF16 && out_dt == ZI_BF16 && ld_gate % 8 == 0 &&
        ((uintptr_t)gate % 16) == 0 && ((uintptr_t)out % 16) == 0) {
        const int64_t groups = (int64_t)n * (inter / 8);
        int64_t blocks = (groups + 255) / 256;
        if (blocks > 16384) blocks = 16384;
        swiglu_il8_kernel<<<(int)blocks, 256, 0, stream>>>((zi_bf16*)out, (const zi_bf16*)gate, groups, inter / 8, ld_gate);
        return zi_check_launch("swiglu");
    }
    ZI_REQUIRE(n <= 65535 * 1024, "swiglu: too many rows");
    int bx = (inter + 255) / 256;
    if (bx > 64) bx = 64;
    // gridDim.y is limited to 65535: fold larger batches.
    for (int r0 = 0; r0 < n; r0 += 65535) {
        const int rows = n - r0 < 65535 ? n - r0 : 65535;
        ZI_DISPATCH_DTYPE(dt, TI, ZI_DISPATCH_DTYPE(out_dt, TO, {
            swiglu_kernel<TI, TO><<<dim3(bx, rows), 256, 0, stream>>>(
                (TO*)out + (int64_t)r0 * inter, (const TI*)gate + (int64_t)r0 * ld_gate,
                up ? (const TI*)up + (int64_t)r0 * ld_up : nullptr, inter, ld_gate, ld_up, interleave, splits,
                split_stride);
        }));
    }
    return zi_check_launch("swiglu");
}

// out = act(gate) * up, element by element, float32 arithmetic: the gated feed-forward's middle for activations
// other than the one the SwiGLU kernels above carry.  act: 0 SiLU, 1 GELU in its tanh form
// 0.5 z (1 + tanh(sqrt(2 / pi) (z + 0.044715 z^3))), 2 GELU with the error function.
template <typename T, typename TO>
__global__ void gated_act_kernel(TO* __restrict__ out, int64_t ldo, const T* __restrict__ gate, const T* __restrict__ up,
                                 int64_t ld_gate, int64_t ld_up, int n, int inter, int act) {
    const int64_t i = (int64_t)blockIdx.x * blockDim.x + threadIdx.x;
    if (i >= (int64_t)n * inter) return;
    const int64_t r = i / inter, c = i % inter;
    zi_store(out + r * ldo + c, zi_activation(zi_load(gate + r * ld_gate + c), act) * zi_load(up + r * ld_up + c));
}

extern "C" int zi_gated_act(void* out, int out_dt, int64_t ldo, const void* gate, const void* up, int dt, int64_t ld_gate,
                            int64_t ld_up, int n, int inter, int act, hipStream_t stream) {
    ZI_REQUIRE(n >= 0 && inter > 0 && ldo >= inter && ld_gate >= inter && ld_up >= inter, "gated_act: bad sizes");
    ZI_REQUIRE(act >= ZI_ACT_SILU && act <= ZI_ACT_GELU_ERF, "gated_act: unknown activation %d", act);
    if (n == 0) return 0;
    const int64_t total = (int64_t)n * inter;
    ZI_DISPATCH_DTYPE(dt, T, ZI_DISPATCH_DTYPE(out_dt, TO, {
        gated_act_kernel<T, TO><<<(unsigned)((total + 255) / 256), 256, 0, stream>>>(
            (TO*)out, ldo, (const T*)gate, (const T*)up, ld_gate, ld_up, n, inter, act);
    }));
    return zi_check_launch("gated_act");
}

// ---- activations of feed-forwards without the SiLU gate ------------------------------------------------------
// Four consecutive values at a time where rows allow it (widths and strides multiples of four, 16-byte aligned).
__device__ __forceinline__ float4 ew_load4(const float* p) { return *reinterpret_cast<const float4*>(p); }
__device__ __forceinline__ float4 ew_load4(const zi_bf16* p) {
    const uint2 r = *reinterpret_cast<const uint2*>(p);
    return make_float4(__uint_as_float(r.x << 16), __uint_as_float(r.x & 0xffff0000u), __uint_as_float(r.y << 16),
                       __uint_as_float(r.y & 0xffff0000u));
}
__device__ __forceinline__ void ew_store4(float* p, float4 v) { *reinterpret_cast<float4*>(p) = v; }
__device__ __forceinline__ void ew_store4(zi_bf16* p, float4 v) {
    uint2 r;
    r.x = zi_pack_bf16x2(v.x, v.y);
    r.y = zi_pack_bf16x2(v.z, v.w);
    *reinterpret_cast<uint2*>(p) = r;
}
static bool ew_rows4(const void* p, int64_t ld, int inter) {
    return inter % 4 == 0 && ld % 4 == 0 && ((uintptr_t)p % 16) == 0;
}

template <typename T, typename TO>
__global__ void relu_squared_vec_kernel(TO* __restrict__ out, int64_t ldo, const T* __restrict__ z, int64_t ldz, int n,
                                        int inter) {
    const int64_t i = (int64_t)blockIdx.x * blockDim.x + threadIdx.x;
    const int q = inter / 4;
    if (i >= (int64_t)n * q) return;
    const int64_t r = i / q, c = (i % q) * 4;
    float4 v = ew_load4(z + r * ldz + c);
    v.x = fmaxf(v.x, 0.f); v.y = fmaxf(v.y, 0.f); v.z = fmaxf(v.z, 0.f); v.w = fmaxf(v.w, 0.f);
    ew_store4(out + r * ldo + c, make_float4(v.x * v.x, v.y * v.y, v.z * v.z, v.w * v.w));
}

template <typename T, typename TO>
__global__ void clamped_glu_vec_kernel(TO* __restrict__ out, int64_t ldo, const T* __restrict__ gate, const T* __restrict__ up,
                                       int64_t ld_gate, int64_t ld_up, int n, int inter, float limit, float alpha,
                                       const float* __restrict__ gate_bias, const float* __restrict__ up_bias) {
    const int64_t i = (int64_t)blockIdx.x * blockDim.x + threadIdx.x;
    const int q = inter / 4;
    if (i >= (int64_t)n * q) return;
    const int64_t r = i / q, c = (i % q) * 4;
    const float4 g4 = ew_load4(gate + r * ld_gate + c), u4 = ew_load4(up + r * ld_up + c);
    float g[4] = {g4.x, g4.y, g4.z, g4.w}, u[4] = {u4.x, u4.y, u4.z, u4.w};
    if (gate_bias) {
#pragma unroll
        for (int k = 0; k < 4; ++k) {
            g[k] += gate_bias[c + k];
            u[k] += up_bias[c + k];
        }
    }
    float o[4];
#pragma unroll
    for (int k = 0; k < 4; ++k) {
        const float gg = fminf(g[k], limit), uu = fminf(fmaxf(u[k], -limit), limit);
        o[k] = gg / (1.f + expf(-alpha * gg)) * (uu + 1.f);
    }
    ew_store4(out + r * ldo + c, make_float4(o[0], o[1], o[2], o[3]));
}

// relu(z)^2 of every element of a [n][inter] operand with dense rows, which may come as `splits` float32 partial
// sums (split s at z + s * split_stride, added in rising order first).
template <typename T, typename TO>
__global__ void relu_squared_kernel(TO* __restrict__ out, int64_t ldo, const T* __restrict__ z, int64_t ldz, int splits,
                                    int64_t split_stride, int n, int inter) {
    const int64_t i = (int64_t)blockIdx.x * blockDim.x + threadIdx.x;
    if (i >= (int64_t)n * inter) return;
    const int64_t r = i / inter, c = i % inter;
    float v = zi_load(z + r * ldz + c);
    for (int s = 1; s < splits; ++s) v += zi_load(z + s * split_stride + r * ldz + c);
    v = fmaxf(v, 0.f);
    zi_store(out + r * ldo + c, v * v);
}

extern "C" int zi_relu_squared(void* out, int out_dt, int64_t ldo, const void* z, int dt, int64_t ldz, int splits,
                               int64_t split_stride, int n, int inter, hipStream_t stream) {
    ZI_REQUIRE(n >= 0 && inter > 0 && ldo >= inter && ldz >= inter && splits >= 1, "relu_squared: bad sizes");
    if (n == 0) return 0;
    const int64_t total = (int64_t)n * inter;
    if (splits == 1 && ew_rows4(z, ldz, inter) && ew_rows4(out, ldo, inter)) {
        ZI_DISPATCH_DTYPE(dt, T, ZI_DISPATCH_DTYPE(out_dt, TO, {
            relu_squared_vec_kernel<T, TO><<<(unsigned)((total / 4 + 255) / 256), 256, 0, stream>>>(
                (TO*)out, ldo, (const T*)z, ldz, n, inter);
        }));
        return zi_check_launch("relu_squared");
    }
    ZI_DISPATCH_DTYPE(dt, T, ZI_DISPATCH_DTYPE(out_dt, TO, {
        relu_squared_kernel<T, TO><<<(unsigned)((total + 255) / 256), 256, 0, stream>>>(
            (TO*)out, ldo, (const T*)z, ldz, splits, split_stride, n, inter);
    }));
    return zi_check_launch("relu_squared");
}

// An activation alone: out = act(z), z [n][inter] with dense rows, possibly as `splits` float32 partial sums (the codes are
// `zi_activate_value`'s).
template <typename T, typename TO>
__global__ void activate_kernel(TO* __restrict__ out, int64_t ldo, const T* __restrict__ z, int64_t ldz, int splits,
                                int64_t split_stride, int n, int inter, int act) {
    const int64_t i = (int64_t)blockIdx.x * blockDim.x + threadIdx.x;
    if (i >= (int64_t)n * inter) return;
    const int64_t r = i / inter, c = i % inter;
    float v = zi_load(z + r * ldz + c);
    for (int s = 1; s < splits; ++s) v += zi_load(z + s * split_stride + r * ldz + c);
    zi_store(out + r * ldo + c, zi_activate_value<sizeof(TO) == 2>(v, act));
}

// Four values a thread, the loads of up to SP terms in flight.
template <typename T, typename TO, int SP>
__global__ void __launch_bounds__(256)
activate_vec_kernel(TO* __restrict__ out, int64_t ldo, const T* __restrict__ z, int64_t ldz, int splits, int64_t split_stride,
                    int inter, int act) {
    const int c = (blockIdx.x * 256 + threadIdx.x) * 4;
    const int64_t r = blockIdx.y;
    if (c >= inter) return;
    float4 t[SP];
#pragma unroll
    for (int s = 0; s < SP; ++s) t[s] = s < splits ? ew_load4(z + s * split_stride + r * ldz + c) : make_float4(0.f, 0.f, 0.f, 0.f);
    float4 v = t[0];
#pragma unroll
    for (int s = 1; s < SP; ++s) { v.x += t[s].x; v.y += t[s].y; v.z += t[s].z; v.w += t[s].w; }
    constexpr bool rough = sizeof(TO) == 2;
    ew_store4(out + r * ldo + c, make_float4(zi_activate_value<rough>(v.x, act), zi_activate_value<rough>(v.y, act), zi_activate_value<rough>(v.z, act),
                                             zi_activate_value<rough>(v.w, act)));
}

extern "C" int zi_activate(void* out, int out_dt, int64_t ldo, const void* z, int dt, int64_t ldz, int splits,
                           int64_t split_stride, int n, int inter, int act, hipStream_t stream) {
    ZI_REQUIRE(n >= 0 && inter > 0 && ldo >= inter && ldz >= inter && splits >= 1 && (splits == 1 || dt == ZI_F32), "activate: bad sizes");
    ZI_REQUIRE(act >= ZI_ACT_SILU && act <= ZI_ACT_RELU2, "activate: unknown activation %d", act);
    if (n == 0) return 0;
    if (splits <= 16 && n <= 65535 && split_stride % 4 == 0 && ew_rows4(z, ldz, inter) && ew_rows4(out, ldo, inter)) {
        const dim3 grid((inter / 4 + 255) / 256, n);
#define ZI_ACTV(SP) activate_vec_kernel<T, TO, SP><<<grid, 256, 0, stream>>>((TO*)out, ldo, (const T*)z, ldz, splits, split_stride, inter, act)
        ZI_DISPATCH_DTYPE(dt, T, ZI_DISPATCH_DTYPE(out_dt, TO, {
            if (splits == 1) ZI_ACTV(1);
            else if (splits <= 4) ZI_ACTV(4);
            else ZI_ACTV(16);
        }));
#undef ZI_ACTV
        return zi_check_launch("activate");
    }
    const int64_t total = (int64_t)n * inter;
    ZI_DISPATCH_DTYPE(dt, T, ZI_DISPATCH_DTYPE(out_dt, TO, {
        activate_kernel<T, TO><<<(unsigned)((total + 255) / 256), 256, 0, stream>>>((TO*)out, ldo, (const T*)z, ldz, splits,
                                                                                    split_stride, n, inter, act);
    }));
    return zi_check_launch("activate");
}

// The clamped gated activation: g = min(gate, limit), u = clamp(up, -limit, limit), out = g sigmoid(alpha g) (u + 1).
// gate and up are [n][inter] with dense rows (column slices of one product are fine), possibly as `splits` float32
// partial sums.
template <typename T, typename TO>
__global__ void clamped_glu_kernel(TO* __restrict__ out, int64_t ldo, const T* __restrict__ gate, const T* __restrict__ up,
                                   int64_t ld_gate, int64_t ld_up, int splits, int64_t split_stride, int n, int inter,
                                   float limit, float alpha, const float* __restrict__ gate_bias,
                                   const float* __restrict__ up_bias) {
    const int64_t i = (int64_t)blockIdx.x * blockDim.x + threadIdx.x;
    if (i >= (int64_t)n * inter) return;
    const int64_t r = i / inter, c = i % inter;
    float g = zi_load(gate + r * ld_gate + c), u = zi_load(up + r * ld_up + c);
    for (int s = 1; s < splits; ++s) {
        g += zi_load(gate + s * split_stride + r * ld_gate + c);
        u += zi_load(up + s * split_stride + r * ld_up + c);
    }
    if (gate_bias) {
        g += gate_bias[c];
        u += up_bias[c];
    }
    g = fminf(g, limit);
    u = fminf(fmaxf(u, -limit), limit);
    zi_store(out + r * ldo + c, g / (1.f + expf(-alpha * g)) * (u + 1.f));
}

extern "C" int zi_clamped_glu(void* out, int out_dt, int64_t ldo, const void* gate, const void* up, int dt, int64_t ld_gate,
                              int64_t ld_up, int splits, int64_t split_stride, int n, int inter, float limit, float alpha,
                              const float* gate_bias, const float* up_bias, hipStream_t stream) {
    ZI_REQUIRE((gate_bias == nullptr) == (up_bias == nullptr), "clamped_glu: biases of both halves or of neither");
    ZI_REQUIRE(n >= 0 && inter > 0 && ldo >= inter && ld_gate >= inter && ld_up >= inter && splits >= 1,
               "clamped_glu: bad sizes");
    ZI_REQUIRE(limit > 0.f, "clamped_glu: the limit must be positive, got %g", (double)limit);
    if (n == 0) return 0;
    const int64_t total = (int64_t)n * inter;
    if (splits == 1 && ew_rows4(gate, ld_gate, inter) && ew_rows4(up, ld_up, inter) && ew_rows4(out, ldo, inter)) {
        ZI_DISPATCH_DTYPE(dt, T, ZI_DISPATCH_DTYPE(out_dt, TO, {
            clamped_glu_vec_kernel<T, TO><<<(unsigned)((total / 4 + 255) / 256), 256, 0, stream>>>(
                (TO*)out, ldo, (const T*)gate, (const T*)up, ld_gate, ld_up, n, inter, limit, alpha, gate_bias, up_bias);
        }));
        return zi_check_launch("clamped_glu");
    }
    ZI_DISPATCH_DTYPE(dt, T, ZI_DISPATCH_DTYPE(out_dt, TO, {
        clamped_glu_kernel<T, TO><<<(unsigned)((total + 255) / 256), 256, 0, stream>>>(
            (TO*)out, ldo, (const T*)gate, (const T*)up, ld_gate, ld_up, splits, split_stride, n, inter, limit, alpha,
            gate_bias, up_bias);
    }));
    return zi_check_launch("clamped_glu");
}

// The same over rows [n][2 inter] (bfloat16) whose gate and up columns alternate in blocks of 8: eight results a thread.
__global__ void __launch_bounds__(256)
clamped_glu_il8_kernel(zi_bf16* __restrict__ out, int64_t ldo, const zi_bf16* __restrict__ gu, int64_t ld, int n, int inter,
                       float limit, float alpha) {
    const int64_t i = (int64_t)blockIdx.x * blockDim.x + threadIdx.x;
    const int blocks = inter / 8;
    if (i >= (int64_t)n * blocks) return;
    const int64_t r = i / blocks, b = i % blocks;
    const uint4 g4 = *reinterpret_cast<const uint4*>(gu + r * ld + b * 16), u4 = *reinterpret_cast<const uint4*>(gu + r * ld + b * 16 + 8);
    const uint32_t gw[4] = {g4.x, g4.y, g4.z, g4.w}, uw[4] = {u4.x, u4.y, u4.z, u4.w};
    uint32_t o[4];
#pragma unroll
    for (int k = 0; k < 4; ++k) {
        float y[2];
#pragma unroll
        for (int z = 0; z < 2; ++z) {
            const float g = fminf(__uint_as_float(z ? gw[k] & 0xffff0000u : gw[k] << 16), limit);
            const float u = fminf(fmaxf(__uint_as_float(z ? uw[k] & 0xffff0000u : uw[k] << 16), -limit), limit);
            y[z] = g / (1.f + expf(-alpha * g)) * (u + 1.f);
        }
        o[k] = zi_pack_bf16x2(y[0], y[1]);
    }
    *reinterpret_cast<uint4*>(out + r * ldo + b * 8) = make_uint4(o[0], o[1], o[2], o[3]);
}

extern "C" int zi_clamped_glu_il8(void* out, int64_t ldo, const void* gu, int64_t ld, int n, int inter, float limit,
                                  float alpha, hipStream_t stream) {
    ZI_REQUIRE(n >= 0 && inter > 0 && inter % 8 == 0 && ldo >= inter && ld >= 2LL * inter && ld % 8 == 0 && ldo % 8 == 0 &&
                   ((uintptr_t)gu % 16) == 0 && ((uintptr_t)out % 16) == 0 && limit > 0.f, "clamped_glu_il8: bad sizes or alignment");
    if (n == 0) return 0;
    const int64_t total = (int64_t)n * (inter / 8);
    clamped_glu_il8_kernel<<<(unsigned)((total + 255) / 256), 256, 0, stream>>>((zi_bf16*)out, ldo, (const zi_bf16*)gu, ld, n,
                                                                               inter, limit, alpha);
    return zi_check_launch("clamped_glu_il8");
}

// x <- cap * tanh(x / cap), float32, in place (the soft cap of logits).
__global__ void softcap_kernel(float* __restrict__ x, int64_t total, float cap) {
    const int64_t i = (int64_t)blockIdx.x * blockDim.x + threadIdx.x;
    if (i < total) x[i] = cap * tanhf(x[i] / cap);
}

extern "C" int zi_softcap(float* x, int64_t total, float cap, hipStream_t stream) {
    ZI_REQUIRE(total >= 0 && cap > 0.f, "softcap: bad sizes or cap %g", (double)cap);
    if (total == 0) return 0;
    softcap_kernel<<<(unsigned)((total + 255) / 256), 256, 0, stream>>>(x, total, cap);
    return zi_check_launch("softcap");
}

// out = x in another storage type (the rounded copy of float32 rows that a matrix product reads).
template <typename T, typename TO>
__global__ void convert_kernel(TO* __restrict__ out, const T* __restrict__ x, int64_t total) {
    const int64_t i = (int64_t)blockIdx.x * blockDim.x + threadIdx.x;
    if (i < total) zi_store(out + i, zi_load(x + i));
}

extern "C" int zi_convert(void* out, int out_dt, const void* x, int dt, int64_t total, hipStream_t stream) {
    ZI_REQUIRE(total >= 0, "convert: bad size");
    if (total == 0) return 0;
    ZI_DISPATCH_DTYPE(dt, T, ZI_DISPATCH_DTYPE(out_dt, TO, {
        convert_kernel<T, TO><<<(unsigned)((total + 255) / 256), 256, 0, stream>>>((TO*)out, (const T*)x, total);
    }));
    return zi_check_launch("convert");
}
