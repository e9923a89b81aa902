// Several residual streams a token, mixed around every sublayer, with the norm that the next sublayer reads.
//
//   X'_t = sum_s M[s][t] X_s + b_t (y * l)          y: the sublayer's result, l: a gain per channel (or none)
//   u    = sum_t a_t X'_t
//   out  = (u - mean(u)) / sqrt(var(u) + eps) * g    (`centered`; else u / sqrt(mean(u^2) + eps) * g)
//
// one launch between two sublayers: the old streams and y are read once, the new streams and the normed row written
// once.  y may come as `splits` float32 terms (partial sums of a product cut along k), added in rising order.  Streams
// that are all equal (before the first sublayer has written) are read from one row each (stream stride 0).  Without y the
// streams stay as they are; without `keep` the new streams are not written (the end of the model: a = 1 for all, and the
// wanted rows picked by `rows`).  Everything is float32; a row's result depends on that row alone.
//
// Few or many rows: a workgroup per row, a thread owns IT groups of four consecutive channels and issues all its loads
// before the first is used.  Rows that are no multiple of 4 wide or not aligned, and more than 4 streams: a thread a channel, u in LDS.
#include "zi_common.h"
#include "zi_api.h"

#define SM_MAX_STREAMS 16
#define SM_MAX_HIDDEN 16384
#define SM_MAX_PLAIN 15360      // of the kernel that keeps u in LDS

__device__ __forceinline__ float4 sm_load4(const float* p) { return *reinterpret_cast<const float4*>(p); }
__device__ __forceinline__ float4 sm_load4(const zi_bf16* p) {
    const uint2 r = *reinterpret_cast<const uint2*>(p);
    return make_float4(__uint_as_float(r.x << 16), __uint_as_float(r.x & 0xffff0000u), __uint_as_float(r.y << 16),
                       __uint_as_float(r.y & 0xffff0000u));
}
__device__ __forceinline__ void sm_store4(float* p, float4 v) { *reinterpret_cast<float4*>(p) = v; }
__device__ __forceinline__ void sm_store4(zi_bf16* p, float4 v) {
    uint2 r;
    r.x = zi_pack_bf16x2(v.x, v.y);
    r.y = zi_pack_bf16x2(v.z, v.w);
    *reinterpret_cast<uint2*>(p) = r;
}
__device__ __forceinline__ float4 sm_fma4(float a, float4 x, float4 acc) {
    return make_float4(fmaf(a, x.x, acc.x), fmaf(a, x.y, acc.y), fmaf(a, x.z, acc.z), fmaf(a, x.w, acc.w));
}

// the row of the inputs that output row `row` is made from (the host checks the list; never read outside the rows)
__device__ __forceinline__ int64_t sm_source(const int32_t* __restrict__ rows, int64_t row, int total_rows) {
    if (!rows) return row;
    const int r = rows[row];
    return r < 0 ? 0 : (r < total_rows ? r : total_rows - 1);
}

// `write`: M [S][S] (from, to), then b [S]; `read`: a [S].
template <typename TY, typename TO, int S, int IT, int SP>
__global__ void __launch_bounds__(1024)
stream_mix_kernel(TO* __restrict__ out, const float* in, int64_t in_stride, float* keep, int64_t keep_stride,
                  const TY* __restrict__ y, int splits, int64_t split_stride, const float* __restrict__ scale,
                  const float* __restrict__ write, const float* __restrict__ read, const float* __restrict__ gain,
                  const int32_t* __restrict__ rows, int total_rows, int H, float eps, int centered) {
    __shared__ float red[16];
    const int64_t row = blockIdx.x, src = sm_source(rows, row, total_rows);
    float4 u[IT];
    float sum = 0.f;
#pragma unroll
    for (int it = 0; it < IT; ++it) {
        const int j = (it * blockDim.x + threadIdx.x) * 4;
        u[it] = make_float4(0.f, 0.f, 0.f, 0.f);
        if (j >= H) continue;
        float4 x[S], t[SP];
#pragma unroll
        for (int s = 0; s < S; ++s) x[s] = sm_load4(in + s * in_stride + src * H + j);
        if (y) {
            const TY* yr = y + src * H + j;
            float4 yv = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
            for (int k = 0; k < SP; ++k) t[k] = k < splits ? sm_load4(yr + (int64_t)k * split_stride) : yv;
            const float4 l = scale ? sm_load4(scale + j) : make_float4(1.f, 1.f, 1.f, 1.f);
            yv = t[0];
#pragma unroll
            for (int k = 1; k < SP; ++k) { yv.x += t[k].x; yv.y += t[k].y; yv.z += t[k].z; yv.w += t[k].w; }
            yv.x *= l.x; yv.y *= l.y; yv.z *= l.z; yv.w *= l.w;
#pragma unroll
            for (int to = 0; to < S; ++to) {
                float4 n = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
                for (int s = 0; s < S; ++s) n = sm_fma4(write[s * S + to], x[s], n);
                n = sm_fma4(write[S * S + to], yv, n);
                if (keep) sm_store4(keep + to * keep_stride + src * H + j, n);
                u[it] = sm_fma4(read[to], n, u[it]);
            }
        } else {
#pragma unroll
            for (int s = 0; s < S; ++s) u[it] = sm_fma4(read[s], x[s], u[it]);
        }
        sum += (u[it].x + u[it].y) + (u[it].z + u[it].w);
    }
    float ss = 0.f;
    if (centered) {
        const float mean = zi_block_sum(sum, red) / (float)H;
#pragma unroll
        for (int it = 0; it < IT; ++it) { u[it].x -= mean; u[it].y -= mean; u[it].z -= mean; u[it].w -= mean; }
    }
#pragma unroll
    for (int it = 0; it < IT; ++it)
        if ((it * blockDim.x + threadIdx.x) * 4 < (unsigned)H)
            ss += (u[it].x * u[it].x + u[it].y * u[it].y) + (u[it].z * u[it].z + u[it].w * u[it].w);
    const float r = 1.f / sqrtf(zi_block_sum(ss, red) / (float)H + eps);
#pragma unroll
    for (int it = 0; it < IT; ++it) {
        const int j = (it * blockDim.x + threadIdx.x) * 4;
        if (j >= H) continue;
        const float4 g = sm_load4(gain + j);
        sm_store4(out + row * H + j, make_float4(u[it].x * r * g.x, u[it].y * r * g.y, u[it].z * r * g.z, u[it].w * r * g.w));
    }
}

// Any width up to SM_MAX_PLAIN, up to MAXS streams (S of them), any number of terms.
template <typename TY, typename TO, int MAXS>
__global__ void __launch_bounds__(256)
stream_mix_plain_kernel(TO* __restrict__ out, const float* in, int64_t in_stride, float* keep, int64_t keep_stride,
                        const TY* __restrict__ y, int splits, int64_t split_stride, const float* __restrict__ scale,
                        const float* __restrict__ write, const float* __restrict__ read, const float* __restrict__ gain,
                        const int32_t* __restrict__ rows, int total_rows, int S, int H, float eps, int centered) {
    extern __shared__ float su[];      // [H]
    __shared__ float red[16];
    const int64_t row = blockIdx.x, src = sm_source(rows, row, total_rows);
    float sum = 0.f;
    for (int j = threadIdx.x; j < H; j += blockDim.x) {
        float x[MAXS], u = 0.f;
#pragma unroll
        for (int s = 0; s < MAXS; ++s) x[s] = s < S ? in[s * in_stride + src * H + j] : 0.f;
        if (y) {
            float yv = zi_load(y + src * H + j);
            for (int k = 1; k < splits; ++k) yv += zi_load(y + (int64_t)k * split_stride + src * H + j);
            if (scale) yv *= scale[j];
            for (int to = 0; to < S; ++to) {
                float n = 0.f;
#pragma unroll
                for (int s = 0; s < MAXS; ++s)
                    if (s < S) n = fmaf(write[s * S + to], x[s], n);
                n = fmaf(write[S * S + to], yv, n);
                if (keep) keep[to * keep_stride + src * H + j] = n;
                u = fmaf(read[to], n, u);
            }
        } else {
#pragma unroll
            for (int s = 0; s < MAXS; ++s)
                if (s < S) u = fmaf(read[s], x[s], u);
        }
        su[j] = u;
        sum += u;
    }
    float mean = 0.f, ss = 0.f;
    if (centered) mean = zi_block_sum(sum, red) / (float)H;
    for (int j = threadIdx.x; j < H; j += blockDim.x) {
        const float d = su[j] - mean;
        ss += d * d;
    }
    const float r = 1.f / sqrtf(zi_block_sum(ss, red) / (float)H + eps);
    for (int j = threadIdx.x; j < H; j += blockDim.x) zi_store(out + row * H + j, (su[j] - mean) * r * gain[j]);
}

extern "C" int zi_stream_mix_max_streams() { return SM_MAX_STREAMS; }

// out [n][hidden]; in, keep: stream s at + s * in_stride (0: all streams equal) / keep_stride, rows hidden apart (keep may
// be `in`, or null: nothing kept); y: null, or [.][hidden] rows (`splits` terms split_stride apart, float32 when there are
// several); scale [hidden] or null; write [streams * streams + streams], read [streams], gain [hidden], all float32;
// rows [n] or null: output row i is made from row rows[i] (of total_rows) of the inputs (then nothing is kept).
extern "C" int zi_stream_mix(void* out, int out_dt, const float* in, int64_t in_stride, float* keep, int64_t keep_stride,
                             const void* y, int y_dt, int splits, int64_t split_stride, const float* scale,
                             const float* write, const float* read, const float* gain, const int32_t* rows, int n,
                             int total_rows, int streams, int hidden, float eps, int centered, hipStream_t stream) {
    ZI_REQUIRE(n >= 0 && hidden > 0 && hidden <= SM_MAX_HIDDEN && streams >= 1 && streams <= SM_MAX_STREAMS,
               "stream_mix: bad sizes (%d rows, %d streams, width %d)", n, streams, hidden);
    ZI_REQUIRE(out && in && read && gain && eps > 0.f, "stream_mix: null argument or bad eps");
    ZI_REQUIRE(!y || (write && splits >= 1 && (splits == 1 || y_dt == ZI_F32)), "stream_mix: several terms are float32, and are written back");
    ZI_REQUIRE(!keep || (y && !rows), "stream_mix: streams are kept where a result is written into all rows");
    ZI_REQUIRE(total_rows >= (rows ? 1 : n), "stream_mix: fewer input rows than outputs");
    ZI_REQUIRE(in_stride >= 0 && (!keep || keep_stride >= (int64_t)n * hidden), "stream_mix: streams overlap");
    if (n == 0) return 0;
    const bool aligned = hidden % 4 == 0 && in_stride % 4 == 0 && keep_stride % 4 == 0 && split_stride % 4 == 0 &&
                         ((uintptr_t)in % 16) == 0 && ((uintptr_t)keep % 16) == 0 && ((uintptr_t)y % 16) == 0 &&
                         ((uintptr_t)scale % 16) == 0 && ((uintptr_t)gain % 16) == 0 && ((uintptr_t)out % 16) == 0;
    if (aligned && streams <= 4 && splits <= 16) {
        const int vecs = hidden / 4, it = vecs > 2048 ? 4 : vecs > 1024 ? 2 : 1;
        const int threads = ((vecs + it - 1) / it + ZI_WAVE - 1) / ZI_WAVE * ZI_WAVE;
#define ZI_SM4(SS, IT, SP)                                                                                             \
    stream_mix_kernel<TY, TO, SS, IT, SP><<<n, threads, 0, stream>>>((TO*)out, in, in_stride, keep, keep_stride, (const TY*)y, \
                                                                     splits, split_stride, scale, write, read, gain, rows, total_rows, hidden, \
                                                                     eps, centered)
#define ZI_SM3(SS, IT)                                                  \
    do {                                                                \
        if (splits <= 1) ZI_SM4(SS, IT, 1);                             \
        else if (splits <= 4) ZI_SM4(SS, IT, 4);                        \
        else ZI_SM4(SS, IT, 16);                                        \
    } while (0)
#define ZI_SM2(SS)                                                      \
    do {                                                                \
        if (it == 1) ZI_SM3(SS, 1);                                     \
        else if (it == 2) ZI_SM3(SS, 2);                                \
        else ZI_SM3(SS, 4);                                             \
    } while (0)
        ZI_DISPATCH_DTYPE(y ? y_dt : ZI_F32, TY, ZI_DISPATCH_DTYPE(out_dt, TO, {
            switch (streams) {
                case 1: ZI_SM2(1); break;
                case 2: ZI_SM2(2); break;
                case 3: ZI_SM2(3); break;
                default: ZI_SM2(4); break;
            }
        }));
#undef ZI_SM2
#undef ZI_SM3
#undef ZI_SM4
        return zi_check_launch("stream_mix");
    }
    ZI_REQUIRE(hidden <= SM_MAX_PLAIN, "stream_mix: width %d with %d streams or unaligned rows", hidden, streams);
    const size_t lds = (size_t)hidden * sizeof(float);
#define ZI_SMP(MAXS)                                                                                                   \
    stream_mix_plain_kernel<TY, TO, MAXS><<<n, 256, lds, stream>>>((TO*)out, in, in_stride, keep, keep_stride, (const TY*)y, \
                                                                   splits, split_stride, scale, write, read, gain, rows, total_rows, streams, \
                                                                   hidden, eps, centered)
    ZI_DISPATCH_DTYPE(y ? y_dt : ZI_F32, TY, ZI_DISPATCH_DTYPE(out_dt, TO, {
        if (streams <= 4) ZI_SMP(4);
        else ZI_SMP(SM_MAX_STREAMS);
    }));
#undef ZI_SMP
    return zi_check_launch("stream_mix");
}
