// Latent attention on the matrix cores (bfloat16 cache, float32 scores and sums; see latent.hip for what is
// computed).  A row is one (token, head); all heads of a token meet the same latents, and neighbouring tokens
// nearly the same, so a workgroup takes 16 rows a wavefront of ONE entry (rows in the order token, head) and walks
// the keys its rows see in blocks of 32:
//
//   stage    the block's latents and key parts, [32][rank + rot], from the pages straight into LDS
//            (global_load_lds_dwordx4), one block ahead, in one of two buffers; where its keys lie in the pool is asked for
//            two blocks ahead, a lane a key, and traded between lanes.  Rows are not padded but swizzled: the 16-byte
//            piece c of row k sits at place c xor la_swizzle(k), so that neither product's reads meet in a bank: sixteen
//            rows' piece c and eight rows' pieces c, c + 1 (c even) lie in different banks
//   scores   S[key][row] = K . Q^T   v_mfma_f32_16x16x32_bf16: first operand the keys' rows from LDS, second the
//            queries, held in registers for the whole walk (KS operands a lane)
//   softmax  a lane holds 8 of a row's 32 scores, the row's other 24 are in 3 lanes: two lane exchanges; running
//            maximum and sum in float32, base 2; a block that all rows of the wavefront see whole needs no mask
//   values   O[dim][row] += C^T . P   the same instruction, contraction over the block's keys in the order in
//            which the lanes hold P (keys 4j..4j+3 and 16+4j..16+4j+3 for lane group j): the latents are read
//            transposed from the same rows (ds_read_b64_tr_b16: sixteen lanes read four keys x sixteen dims and each
//            gets one dim of the four keys), so no second copy of them is made
//
// (Staged through registers, with a transposed copy of the latents written by 2-byte stores, the same walk took 381 us
// for the 2,048 tokens of a layer with 12 heads, rank 512 and a window of 1,024 keys.)
//
// A tile's keys can be cut into chunks over blockIdx.y (decoded tokens: few rows, many keys); the chunks leave
// (maximum, sum, unnormalised O) per row and a second kernel merges them.  The cut is a launch parameter that
// depends on the window and the head count only.  Which tile a workgroup owns it finds itself from the step's
// entry lengths, so the launch is sized by tokens and entries alone.
#include "zi_common.h"
#include "zi_api.h"

typedef __attribute__((ext_vector_type(8))) __bf16 la_bf16x8_t;
typedef __attribute__((ext_vector_type(4))) float la_f32x4_t;
typedef __attribute__((ext_vector_type(4))) unsigned la_u32x4_t;
typedef __attribute__((ext_vector_type(4))) short la_s16x4_t;
union la_pack {
    la_u32x4_t u;
    la_bf16x8_t b;
    la_s16x4_t h[2];
    unsigned w[4];
};

#define LA_BK 32      // keys a block
#define LA_EMPTY -1e30f
#define LA_LOG2E 1.4426950408889634f

__device__ __attribute__((aligned(16))) const unsigned la_zero16[4] = {0u, 0u, 0u, 0u};

// of row k (rows k and k + 16 alike): a permutation of 0 .. 7 over eight rows of one parity, its upper two bits one of 0 .. 3
// over four of them
__device__ __forceinline__ int la_swizzle(int k) { return ((k & 6)) | ((k >> 3) & 1); }

// four keys of one dim from rows of LDS: see above
__device__ __forceinline__ la_s16x4_t la_read_transposed(const char* at) {
    return __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) la_s16x4_t*)at);
}

// SPLIT: all WAVES wavefronts share one tile of 16 rows (decoded tokens): they stage together, each makes the
// scores again (cheap) and every WAVES-th tile of 16 latent dims of the second product.
template <int WAVES, int NT, int KS, bool SPLIT>      // rank <= 16 NT, rank + rot <= 32 KS
__global__ void __launch_bounds__(WAVES* ZI_WAVE, 2)
latent_attention_cores_kernel(void* __restrict__ out, int out_f32, float* __restrict__ partial, const void* __restrict__ qa, int qa_f32,
                              const zi_bf16* __restrict__ c_cache, const zi_bf16* __restrict__ kr_cache,
                              const int32_t* __restrict__ entry_start, const int32_t* __restrict__ entry_len,
                              const int32_t* __restrict__ entry_past, const int32_t* __restrict__ block_tables,
                              int entries, int max_pages, int num_pages, int heads, int rank, int rot, int page_size,
                              int window, float scale, int chunk_keys, int total_rows) {
    constexpr int ROWS = SPLIT ? 16 : WAVES * 16, OT = SPLIT ? (NT + WAVES - 1) / WAVES : NT;
    constexpr int P = KS * 4;                                  // 16-byte pieces of a staged key
    constexpr int KI = LA_BK * P / (WAVES * ZI_WAVE);          // load instructions a wavefront issues per block
    static_assert(P % 8 == 0 && (P * 16) % 256 == 128 && KI * WAVES * ZI_WAVE == LA_BK * P, "whole loads, rows half the banks apart");
    __shared__ __attribute__((aligned(16))) la_u32x4_t buf_a[LA_BK * P];
    __shared__ __attribute__((aligned(16))) la_u32x4_t buf_b[LA_BK * P];
    const int lane = threadIdx.x % ZI_WAVE, wave = threadIdx.x / ZI_WAVE, r = lane % 16, j = lane / 16;
    // the entry whose tiles this one is among: 64 entries at a time, a lane each, their tiles summed up over the lanes
    int tile = blockIdx.x, e = entries;
    for (int e0 = 0; e0 < entries; e0 += ZI_WAVE) {
        const int mine = e0 + lane < entries ? (entry_len[e0 + lane] * heads + ROWS - 1) / ROWS : 0;
        int upto = mine;
#pragma unroll
        for (int d = 1; d < ZI_WAVE; d *= 2) {
            const int below = __shfl_up(upto, d, ZI_WAVE);
            if (lane >= d) upto += below;
        }
        const uint64_t past_it = __ballot(upto > tile);
        if (past_it) {
            const int at = __builtin_ctzll(past_it);
            e = e0 + at;
            tile -= __builtin_amdgcn_readlane(upto - mine, at);
            break;
        }
        tile -= __builtin_amdgcn_readlane(upto, ZI_WAVE - 1);
    }
    if (e >= entries) return;      // the launch is sized for the worst case: the whole workgroup leaves
    const int len = entry_len[e], past = entry_past[e], start = entry_start[e];
    const int erows = len * heads, row0 = tile * ROWS;
    const int32_t* bt = block_tables + (int64_t)e * max_pages;
    const int qw = rank + rot;

    // the tile's keys, and this workgroup's chunk of them
    const int last_row = (row0 + ROWS < erows ? row0 + ROWS : erows) - 1;
    const int pos_first = past + row0 / heads, pos_last = past + last_row / heads;
    const int kmin = (window > 0 && pos_first - window + 1 > 0) ? pos_first - window + 1 : 0;
    int k_lo = kmin, k_hi = pos_last;
    if (chunk_keys > 0) {
        k_lo = kmin + (int)blockIdx.y * chunk_keys;
        if (k_lo + chunk_keys - 1 < k_hi) k_hi = k_lo + chunk_keys - 1;
    }

    // this lane's row; the keys that all rows of the wavefront see are [all_lo, all_hi]
    const int wave_row0 = row0 + (SPLIT ? 0 : wave * 16);
    const int row = wave_row0 + r;
    const bool row_ok = row < erows;
    const int rc = row_ok ? row : last_row;
    const int tok = start + rc / heads, head = rc % heads, pos = past + rc / heads;
    const int lo = (window > 0 && pos - window + 1 > 0) ? pos - window + 1 : 0;
    const int wave_last = wave_row0 + 15 < last_row ? wave_row0 + 15 : last_row;
    const int all_hi = past + (wave_row0 < last_row ? wave_row0 : last_row) / heads, all_pos = past + wave_last / heads;
    const int all_lo = (window > 0 && all_pos - window + 1 > 0) ? all_pos - window + 1 : 0;
    const int64_t grow = (int64_t)tok * heads + head;

    la_pack q[KS];
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
        const int d = ks * 32 + 8 * j;
        q[ks].u = (la_u32x4_t){0u, 0u, 0u, 0u};
        if (d >= qw) continue;      // rank + rot is a multiple of 8: a piece of eight lies inside or outside
        if (qa_f32) {
            const float* qr = (const float*)qa + grow * qw + d;
            const float4 a = *reinterpret_cast<const float4*>(qr), b = *reinterpret_cast<const float4*>(qr + 4);
            q[ks].w[0] = zi_pack_bf16x2(a.x, a.y);
            q[ks].w[1] = zi_pack_bf16x2(a.z, a.w);
            q[ks].w[2] = zi_pack_bf16x2(b.x, b.y);
            q[ks].w[3] = zi_pack_bf16x2(b.z, b.w);
        } else {
            q[ks].u = *reinterpret_cast<const la_u32x4_t*>((const zi_bf16*)qa + grow * qw + d);
        }
    }

    float m = LA_EMPTY, l = 0.f;
    la_f32x4_t o[OT];      // tile tq of this wavefront is the latent dims 16 t ..., t = tq (SPLIT: tq WAVES + wave)
#pragma unroll
    for (int t = 0; t < OT; ++t) o[t] = (la_f32x4_t){0.f, 0.f, 0.f, 0.f};

    // the place in the pool of key kb + lane % 32, or -1: past the end, or a page that is not held
    auto places = [&](int kb) {
        const int kp = kb + (lane & (LA_BK - 1)), kc = kp <= k_hi ? kp : k_hi;
        const int pi = kc / page_size;
        const int page = bt[pi < max_pages ? pi : max_pages - 1];
        return (kp <= k_hi && (unsigned)page < (unsigned)num_pages) ? page * page_size + kc % page_size : -1;
    };
    auto issue = [&](int slots, la_u32x4_t* dst) {
        int ln = lane;      // (what a lane loads is worked out anew every block: kept, it takes the registers of the sums)
        asm volatile("" : "+v"(ln));
#pragma unroll
        for (int i = 0; i < KI; ++i) {
            const int L = (wave * KI + i) * ZI_WAVE + ln, key = L / P, d = ((L % P) ^ la_swizzle(key)) * 8;
            const int slot = __shfl(slots, key, ZI_WAVE);
            const zi_bf16* src = d < rank ? c_cache + (int64_t)slot * rank + d : kr_cache + (int64_t)slot * rot + (d - rank);
            if (slot < 0 || d >= qw) src = reinterpret_cast<const zi_bf16*>(la_zero16);
            __builtin_amdgcn_global_load_lds(src, dst + (wave * KI + i) * ZI_WAVE, 16, 0, 0);
        }
    };
    // where this lane reads in a buffer, in bytes: the keys' rows (k-steps even and odd), and four keys x sixteen dims
    const int sw = la_swizzle(r);      // of rows r and 16 + r
    const int s_even = (r * P + (j ^ sw)) * 16, s_odd = (r * P + ((4 + j) ^ sw)) * 16;
    const int vrow = 4 * j + (r >> 2), vsw = la_swizzle(vrow);
    int v_at[4];
#pragma unroll
    for (int t = 0; t < 4; ++t) v_at[t] = (vrow * P + ((t * 2 + ((r & 3) >> 1)) ^ vsw)) * 16 + (r & 1) * 8;
    const float scale2 = scale * LA_LOG2E;

    auto work = [&](int kb, const la_u32x4_t* buf) {
        const char* base = reinterpret_cast<const char*>(buf);
        la_f32x4_t s[2];
#pragma unroll
        for (int h = 0; h < 2; ++h) {
            s[h] = (la_f32x4_t){0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int ks = 0; ks < KS; ++ks) {
                la_pack a;
                a.u = *reinterpret_cast<const la_u32x4_t*>(base + ((ks & 1) ? s_odd : s_even) + h * (16 * P * 16) + (ks / 2) * 128);
                s[h] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a.b, q[ks].b, s[h], 0, 0, 0);
            }
        }
        // lane (r, j) holds, of row r, the keys kb + 16 h + 4 j + x; in base-2 units from here on
        float mb = LA_EMPTY;
        const bool whole = kb >= all_lo && kb + LA_BK - 1 <= all_hi && kb + LA_BK - 1 <= k_hi;
#pragma unroll
        for (int h = 0; h < 2; ++h)
#pragma unroll
            for (int x = 0; x < 4; ++x) {
                const int kp = kb + 16 * h + 4 * j + x;
                const bool seen = whole || (row_ok && kp >= lo && kp <= pos && kp <= k_hi);
                s[h][x] = seen ? s[h][x] * scale2 : -INFINITY;
                mb = fmaxf(mb, s[h][x]);
            }
        mb = fmaxf(mb, __shfl_xor(mb, 16, ZI_WAVE));
        mb = fmaxf(mb, __shfl_xor(mb, 32, ZI_WAVE));
        const float m_new = fmaxf(m, mb);      // (never below LA_EMPTY, so a key that is not seen weighs 2^-inf = 0)
        const float corr = __builtin_amdgcn_exp2f(m - m_new);
        float sum = 0.f;
#pragma unroll
        for (int h = 0; h < 2; ++h)
#pragma unroll
            for (int x = 0; x < 4; ++x) {
                s[h][x] = __builtin_amdgcn_exp2f(s[h][x] - m_new);
                sum += s[h][x];
            }
        l = l * corr + sum;      // this lane's keys; the row's four lanes are added up at the end
        m = m_new;
        la_pack pb;
        pb.w[0] = zi_pack_bf16x2(s[0][0], s[0][1]);
        pb.w[1] = zi_pack_bf16x2(s[0][2], s[0][3]);
        pb.w[2] = zi_pack_bf16x2(s[1][0], s[1][1]);
        pb.w[3] = zi_pack_bf16x2(s[1][2], s[1][3]);
        if (__any(corr != 1.f)) {      // the running maximum seldom moves after the first blocks
#pragma unroll
            for (int tq = 0; tq < OT; ++tq) o[tq] *= corr;
        }
#pragma unroll
        for (int tq = 0; tq < OT; ++tq) {
            if (SPLIT) {
                const int t = tq * WAVES + wave;
                if (t * 16 < rank) {
                    const char* at = base + (vrow * P + ((t * 2 + ((r & 3) >> 1)) ^ vsw)) * 16 + (r & 1) * 8;
                    la_pack a;
                    a.h[0] = la_read_transposed(at);
                    a.h[1] = la_read_transposed(at + 16 * P * 16);
                    o[tq] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a.b, pb.b, o[tq], 0, 0, 0);
                }
            } else if (tq * 16 < rank) {
                const char* at = base + v_at[tq & 3] + (tq / 4) * 128;
                la_pack a;
                a.h[0] = la_read_transposed(at);
                a.h[1] = la_read_transposed(at + 16 * P * 16);
                o[tq] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a.b, pb.b, o[tq], 0, 0, 0);
            }
        }
    };
    // Two blocks a turn, buffer a then b.  At each barrier the block about to be worked on has arrived (the compiler
    // waits for all loads into LDS before a barrier) and everyone has finished with the other buffer.
    if (k_lo <= k_hi) {
        issue(places(k_lo), buf_a);
        int next = places(k_lo + LA_BK);
        int kb = k_lo;
        while (true) {
            __syncthreads();
            if (kb + LA_BK <= k_hi) {
                issue(next, buf_b);
                next = places(kb + 2 * LA_BK);
            }
            work(kb, buf_a);
            if (kb + LA_BK > k_hi) break;
            kb += LA_BK;
            __syncthreads();
            if (kb + LA_BK <= k_hi) {
                issue(next, buf_a);
                next = places(kb + 2 * LA_BK);
            }
            work(kb, buf_b);
            if (kb + LA_BK > k_hi) break;
            kb += LA_BK;
        }
    }
    l += __shfl_xor(l, 16, ZI_WAVE);
    l += __shfl_xor(l, 32, ZI_WAVE);
    // lane (r, j) holds, of row r, the dims 16 t + 4 j + x (rank is a multiple of 8: four dims lie inside or outside)
    if (!row_ok) return;
    const bool parts = gridDim.y > 1;
    const float inv = parts ? 1.f : 1.f / l;
    const int64_t prow = ((int64_t)blockIdx.y * total_rows + grow) * (rank + 4);      // maximum, sum, two unused, then O
    if (parts && j == 0 && (!SPLIT || wave == 0)) {
        partial[prow] = m;
        partial[prow + 1] = l;
    }
#pragma unroll
    for (int tq = 0; tq < OT; ++tq) {
        const int d = 16 * (SPLIT ? tq * WAVES + wave : tq) + 4 * j;
        if (d >= rank) continue;
        const la_f32x4_t v = o[tq] * inv;
        if (parts) {
            *reinterpret_cast<la_f32x4_t*>(partial + prow + 4 + d) = v;
        } else if (out_f32) {
            *reinterpret_cast<la_f32x4_t*>((float*)out + grow * rank + d) = v;
        } else {
            uint2 w;
            w.x = zi_pack_bf16x2(v[0], v[1]);
            w.y = zi_pack_bf16x2(v[2], v[3]);
            *reinterpret_cast<uint2*>((zi_bf16*)out + grow * rank + d) = w;
        }
    }
}

// out[row] = sum_c O_c 2^(m_c - M) / sum_c l_c 2^(m_c - M), chunks in rising order.  A thread owns four dims; the loads of
// eight chunks travel together.
#define LA_MAX_CHUNKS 4096
__global__ void __launch_bounds__(128)
latent_attention_merge_kernel(void* __restrict__ out, int out_f32, const float* __restrict__ partial, int chunks, int total_rows,
                              int rank) {
    __shared__ float weight[128];
    const int64_t row = blockIdx.x, stride = (int64_t)total_rows * (rank + 4);
    const float* p0 = partial + row * (rank + 4);
    const int tid = threadIdx.x, lane = tid & (ZI_WAVE - 1);
    const int d = tid * 4;
    // every wavefront makes the maximum and the sum: lane c takes chunks c, c + 64, ...
    float M = LA_EMPTY;
    for (int c = lane; c < chunks; c += ZI_WAVE) M = fmaxf(M, p0[c * stride]);
    M = zi_wave_max(M);
    float L = 0.f;
    for (int c = lane; c < chunks; c += ZI_WAVE) L += p0[c * stride + 1] * __builtin_amdgcn_exp2f(p0[c * stride] - M);
    const float inv = 1.f / zi_wave_sum(L);
    la_f32x4_t acc = (la_f32x4_t){0.f, 0.f, 0.f, 0.f};
    for (int c0 = 0; c0 < chunks; c0 += 128) {
        __syncthreads();
        if (c0 + tid < chunks) weight[tid] = __builtin_amdgcn_exp2f(p0[(c0 + tid) * stride] - M);
        __syncthreads();
        const int count = chunks - c0 < 128 ? chunks - c0 : 128;
        if (d >= rank) continue;
        for (int c = 0; c < count; c += 8) {
            la_f32x4_t v[8];
#pragma unroll
            for (int u = 0; u < 8; ++u) v[u] = *reinterpret_cast<const la_f32x4_t*>(p0 + (c0 + (c + u < count ? c + u : c)) * stride + 4 + d);
#pragma unroll
            for (int u = 0; u < 8; ++u) acc += v[u] * (c + u < count ? weight[c + u] : 0.f);
        }
    }
    if (d >= rank) return;
    acc *= inv;
    if (out_f32) {
        *reinterpret_cast<la_f32x4_t*>((float*)out + row * rank + d) = acc;
    } else {
        uint2 w;
        w.x = zi_pack_bf16x2(acc[0], acc[1]);
        w.y = zi_pack_bf16x2(acc[2], acc[3]);
        *reinterpret_cast<uint2*>((zi_bf16*)out + row * rank + d) = w;
    }
}

extern "C" int zi_latent_attention_cores_supported(int dt, int rank, int rot) {
    return dt == ZI_BF16 && rank > 0 && rank % 8 == 0 && rot >= 0 && rot % 8 == 0 && rank <= 512 && rank + rot <= 576;
}

// Rows of a tile for `waves` wavefronts, and the most tiles a step of n tokens in `entries` entries has.
extern "C" int zi_latent_attention_cores_tiles(int n, int entries, int heads, int waves) {
    const int64_t rows = 16 * waves;
    const int64_t by_entry = ((int64_t)n * heads + rows - 1) / rows + entries, by_token = (int64_t)n * ((heads + rows - 1) / rows);
    return (int)(by_entry < by_token ? by_entry : by_token);
}

// qa [n][heads][rank + rot] and out [n][heads][rank], each float32 or bfloat16; partial: chunks * n * heads * (rank + 4) floats.
extern "C" int zi_latent_attention_cores(void* out, int out_dt, float* partial, int64_t partial_floats, const void* qa, int qa_dt,
                                         const void* c_cache, const void* kr_cache, const int32_t* entry_start,
                                         const int32_t* entry_len, const int32_t* entry_past, const int32_t* block_tables,
                                         int entries, int n, int max_pages, int num_pages, int heads, int rank, int rot,
                                         int page_size, int window, float scale, int waves, int chunk_keys, int chunks,
                                         hipStream_t stream) {
    ZI_REQUIRE(zi_latent_attention_cores_supported(ZI_BF16, rank, rot), "latent_attention_cores: rank %d, rot %d not taken",
               rank, rot);
    ZI_REQUIRE(n >= 0 && entries > 0 && heads > 0 && page_size > 0 && max_pages > 0 && num_pages > 0 && window >= 0 &&
                   (int64_t)num_pages * page_size < (1ll << 31), "latent_attention_cores: bad sizes");
    ZI_REQUIRE((out_dt == ZI_F32 || out_dt == ZI_BF16) && (qa_dt == ZI_F32 || qa_dt == ZI_BF16) && ((uintptr_t)qa % 16) == 0 &&
                   ((uintptr_t)out % 16) == 0 && ((uintptr_t)partial % 16) == 0 && ((uintptr_t)c_cache % 16) == 0 && ((uintptr_t)kr_cache % 16) == 0,
               "latent_attention_cores: unknown types, or addresses that are not aligned to 16 bytes");
    ZI_REQUIRE(waves == 1 || waves == 4, "latent_attention_cores: 1 or 4 wavefronts a workgroup");
    ZI_REQUIRE(chunks >= 1 && chunks <= LA_MAX_CHUNKS && (chunks == 1) == (chunk_keys == 0) && chunk_keys >= 0,
               "latent_attention_cores: bad cut (%d chunks of %d keys)", chunks, chunk_keys);
    if (chunks > 1) {
        // every key a tile's rows see lies in one of the chunks
        const int tokens_in_tile = (16 * waves + heads - 1) / heads + 1;
        // (without a window the caller sees to it that the chunks reach the last key of every entry)
        ZI_REQUIRE(window == 0 || (int64_t)chunks * chunk_keys >= (int64_t)window + tokens_in_tile,
                   "latent_attention_cores: %d chunks of %d keys do not cover a window of %d", chunks, chunk_keys, window);
        ZI_REQUIRE(partial && partial_floats >= (int64_t)chunks * n * heads * (rank + 4),
                   "latent_attention_cores: the workspace is too small");
    }
    if (n == 0) return 0;
    const int total_rows = n * heads;
    const dim3 grid(zi_latent_attention_cores_tiles(n, entries, heads, waves), chunks);
#define ZI_LA_LAUNCH(W, NT, KS)                                                                                       \
    latent_attention_cores_kernel<4, NT, KS, W == 1><<<grid, 4 * ZI_WAVE, 0, stream>>>(                                \
        out, out_dt == ZI_F32, partial, qa, qa_dt == ZI_F32, (const zi_bf16*)c_cache, (const zi_bf16*)kr_cache, entry_start, entry_len, \
        entry_past, block_tables, entries, max_pages, num_pages, heads, rank, rot, page_size, window, scale, chunk_keys, total_rows)
#define ZI_LA_SIZES(W)                                                       \
    do {                                                                     \
        if (rank <= 128 && rank + rot <= 192) ZI_LA_LAUNCH(W, 8, 6);         \
        else if (rank <= 256 && rank + rot <= 320) ZI_LA_LAUNCH(W, 16, 10);  \
        else ZI_LA_LAUNCH(W, 32, 18);                                        \
    } while (0)
    if (waves == 1) ZI_LA_SIZES(1);
    else ZI_LA_SIZES(4);
#undef ZI_LA_SIZES
#undef ZI_LA_LAUNCH
    int rc = zi_check_launch("latent_attention_cores");
    if (rc != 0 || chunks == 1) return rc;
    latent_attention_merge_kernel<<<total_rows, 128, 0, stream>>>(out, out_dt == ZI_F32, partial, chunks, total_rows, rank);
    return zi_check_launch("latent_attention_merge");
}

// ---- a product per head on the matrix cores ---------------------------------------------------------------------
// out[t][h][i] = sum_k w[h][i][k] x[t][h][k]: w bfloat16 [heads][N][K] (k runs fastest), x float32 (rounded to bfloat16 as
// it is loaded) or bfloat16 with row stride ldx and head stride xs, out float32 or bfloat16 with row stride ldo and head stride
// os.  It carries the queries through W_uk (w = W_uk of the head, transposed at load) and the attended latents through W_uv.
// GATED: out *= sigmoid(gate[t][h * N + i]), the gate bfloat16 or the sum of `splits` float32 terms.
// Operands straight from memory.  Many tokens: a wavefront owns 32 tokens x 64 outputs (every operand serves several
// products), the four wavefronts of a workgroup take neighbouring tokens of one head.  Few: 16 x 16, k dealt over the
// four wavefronts in runs of 32 and added up in their order.
struct LaGate {
    const void* g;
    int f32, splits;
    int64_t ld, stride;
};

__device__ __forceinline__ la_pack la_load8(const float* p) {
    const float4 lo = *reinterpret_cast<const float4*>(p), hi = *reinterpret_cast<const float4*>(p + 4);
    la_pack b;
    b.w[0] = zi_pack_bf16x2(lo.x, lo.y);
    b.w[1] = zi_pack_bf16x2(lo.z, lo.w);
    b.w[2] = zi_pack_bf16x2(hi.x, hi.y);
    b.w[3] = zi_pack_bf16x2(hi.z, hi.w);
    return b;
}
__device__ __forceinline__ la_pack la_load8(const zi_bf16* p) {
    la_pack b;
    b.u = *reinterpret_cast<const la_u32x4_t*>(p);
    return b;
}

// four gates of one token and head, columns n0 .. n0 + 3 (clamped to the head)
__device__ __forceinline__ la_f32x4_t la_gates(const LaGate& gt, int64_t t, int h, int n0, int N) {
    const int64_t at = t * gt.ld + (int64_t)h * N;
    la_f32x4_t g;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const int col = n0 + i < N ? n0 + i : N - 1;
        g[i] = gt.f32 ? ((const float*)gt.g)[at + col] : zi_load((const zi_bf16*)gt.g + at + col);
    }
    if (gt.f32) {
        int s = 1;
        for (; s + 3 < gt.splits; s += 4) {      // four terms in flight, added in their order
            la_f32x4_t v[4];
#pragma unroll
            for (int u = 0; u < 4; ++u)
#pragma unroll
                for (int i = 0; i < 4; ++i) v[u][i] = ((const float*)gt.g)[(s + u) * gt.stride + at + (n0 + i < N ? n0 + i : N - 1)];
#pragma unroll
            for (int u = 0; u < 4; ++u) g += v[u];
        }
        for (; s < gt.splits; ++s)
#pragma unroll
            for (int i = 0; i < 4; ++i) g[i] += ((const float*)gt.g)[s * gt.stride + at + (n0 + i < N ? n0 + i : N - 1)];
    }
    return g;
}
template <typename TO>
__device__ __forceinline__ void la_store4(TO* orow, la_f32x4_t v, int left) {
#pragma unroll
    for (int i = 0; i < 4; ++i)
        if (i < left) zi_store(orow + i, v[i]);
}
__device__ __forceinline__ void la_gate4(la_f32x4_t& v, const la_f32x4_t& g) {
#pragma unroll
    for (int i = 0; i < 4; ++i) v[i] = v[i] / (1.f + expf(-g[i]));
}

template <typename TX, typename TO, bool GATED>
__global__ void __launch_bounds__(4 * ZI_WAVE)
headwise_linear_few_kernel(TO* __restrict__ out, int64_t ldo, int os, const TX* __restrict__ x, int64_t ldx, int xs,
                           const zi_bf16* __restrict__ w, int n, int N, int K, LaGate gt) {
    __shared__ la_f32x4_t part[3][ZI_WAVE];
    const int t0 = blockIdx.x * 16, h = blockIdx.y, n0 = blockIdx.z * 16;
    const int lane = threadIdx.x % ZI_WAVE, wave = threadIdx.x / ZI_WAVE, r = lane % 16, j = lane / 16;
    const zi_bf16* wrow = w + ((int64_t)h * N + (n0 + r < N ? n0 + r : N - 1)) * K;
    const int64_t t = t0 + r < n ? t0 + r : n - 1;
    const TX* xrow = x + t * ldx + (int64_t)h * xs;
    la_f32x4_t acc = (la_f32x4_t){0.f, 0.f, 0.f, 0.f}, gate = acc;
    if (GATED && wave == 0) gate = la_gates(gt, t, h, n0 + 4 * j, N);      // asked for before the product, used after it
#pragma unroll 4
    for (int k0 = wave * 32; k0 < K; k0 += 128) {
        const int k = k0 + 8 * j, kc = k < K ? k : 0;      // K is a multiple of 8
        const unsigned mask = 0u - (unsigned)(k < K);
        la_pack a = la_load8(wrow + kc), b = la_load8(xrow + kc);
        a.u &= mask;
        b.u &= mask;
        acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a.b, b.b, acc, 0, 0, 0);
    }
    if (wave > 0) part[wave - 1][lane] = acc;
    __syncthreads();
    if (wave > 0) return;
#pragma unroll
    for (int u = 0; u < 3; ++u) acc += part[u][lane];
    if (t0 + r >= n || n0 + 4 * j >= N) return;
    if constexpr (GATED) la_gate4(acc, gate);
    la_store4(out + t * ldo + (int64_t)h * os + n0 + 4 * j, acc, N - n0 - 4 * j);
}

template <typename TX, typename TO, bool GATED>
__global__ void __launch_bounds__(4 * ZI_WAVE)
headwise_linear_many_kernel(TO* __restrict__ out, int64_t ldo, int os, const TX* __restrict__ x, int64_t ldx, int xs,
                            const zi_bf16* __restrict__ w, int n, int N, int K, LaGate gt) {
    constexpr int TM = 2, TN = 4;      // tiles of 16 tokens and of 16 outputs
    const int lane = threadIdx.x % ZI_WAVE, wave = threadIdx.x / ZI_WAVE, r = lane % 16, j = lane / 16;
    const int t0 = (blockIdx.x * 4 + wave) * (16 * TM), h = blockIdx.y, n0 = blockIdx.z * (16 * TN);
    if (t0 >= n) return;
    const zi_bf16* wrow[TN];
    const TX* xrow[TM];
#pragma unroll
    for (int c = 0; c < TN; ++c) {
        const int i = n0 + c * 16 + r;
        wrow[c] = w + ((int64_t)h * N + (i < N ? i : N - 1)) * K;
    }
#pragma unroll
    for (int c = 0; c < TM; ++c) {
        const int t = t0 + c * 16 + r;
        xrow[c] = x + (int64_t)(t < n ? t : n - 1) * ldx + (int64_t)h * xs;
    }
    la_f32x4_t acc[TM][TN];
#pragma unroll
    for (int a = 0; a < TM; ++a)
#pragma unroll
        for (int c = 0; c < TN; ++c) acc[a][c] = (la_f32x4_t){0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
    for (int k0 = 0; k0 < K; k0 += 32) {
        const int k = k0 + 8 * j, kc = k < K ? k : 0;
        const unsigned mask = 0u - (unsigned)(k < K);
        la_pack a[TN], b[TM];
#pragma unroll
        for (int c = 0; c < TN; ++c) a[c] = la_load8(wrow[c] + kc);
#pragma unroll
        for (int c = 0; c < TM; ++c) b[c] = la_load8(xrow[c] + kc);
#pragma unroll
        for (int c = 0; c < TN; ++c) a[c].u &= mask;
#pragma unroll
        for (int c = 0; c < TM; ++c) b[c].u &= mask;
#pragma unroll
        for (int m = 0; m < TM; ++m)
#pragma unroll
            for (int c = 0; c < TN; ++c) acc[m][c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a[c].b, b[m].b, acc[m][c], 0, 0, 0);
    }
#pragma unroll
    for (int m = 0; m < TM; ++m) {
        const int t = t0 + m * 16 + r;
        if (t >= n) continue;
#pragma unroll
        for (int c = 0; c < TN; ++c) {
            const int i = n0 + c * 16 + 4 * j;
            if (i >= N) continue;
            if constexpr (GATED) la_gate4(acc[m][c], la_gates(gt, t, h, i, N));
            TO* dst = out + (int64_t)t * ldo + (int64_t)h * os + i;
            if (sizeof(TO) == 2 && i + 3 < N && ((uintptr_t)dst % 8) == 0) {
                uint2 p;
                p.x = zi_pack_bf16x2(acc[m][c][0], acc[m][c][1]);
                p.y = zi_pack_bf16x2(acc[m][c][2], acc[m][c][3]);
                *reinterpret_cast<uint2*>(dst) = p;
            } else {
                la_store4(dst, acc[m][c], N - i);
            }
        }
    }
}

// (either storage type of x)
extern "C" int zi_headwise_linear_supported(int w_dt, int K, int64_t ldx, int xs) {
    return w_dt == ZI_BF16 && K > 0 && K % 8 == 0 && ldx % 8 == 0 && xs % 8 == 0;
}

#define LA_MANY_TOKENS 128      // from this many tokens on the kernel for many

extern "C" int zi_headwise_linear_gated(void* out, int out_dt, int64_t ldo, int os, const void* x, int x_dt, int64_t ldx, int xs,
                                        const void* w, int n, int heads, int N, int K, const void* gate, int g_dt,
                                        int64_t ld_gate, int g_splits, int64_t g_stride, hipStream_t stream) {
    ZI_REQUIRE(n >= 0 && heads > 0 && heads <= 65535 && N > 0 && (N + 15) / 16 <= 65535, "headwise_linear: bad sizes");
    ZI_REQUIRE(zi_headwise_linear_supported(ZI_BF16, K, ldx, xs) && ((uintptr_t)x % 16) == 0 && ((uintptr_t)w % 16) == 0,
               "headwise_linear: K %d, row stride %lld, head stride %d or an address is not aligned", K, (long long)ldx, xs);
    ZI_REQUIRE(xs >= K && os >= N && ldx >= (int64_t)(heads - 1) * xs + K && ldo >= (int64_t)(heads - 1) * os + N,
               "headwise_linear: strides too small");
    ZI_REQUIRE(!gate || (ld_gate >= (int64_t)heads * N && g_splits >= 1 && (g_dt == ZI_F32 || (g_dt == ZI_BF16 && g_splits == 1))),
               "headwise_linear: bad gate");
    if (n == 0) return 0;
    const bool many = n >= LA_MANY_TOKENS;
    const dim3 grid(many ? (n + 127) / 128 : (n + 15) / 16, heads, many ? (N + 63) / 64 : (N + 15) / 16);
    const LaGate gt = {gate, g_dt == ZI_F32, g_splits, ld_gate, g_stride};
#define ZI_HW(KERNEL, GATED) KERNEL<TX, TO, GATED><<<grid, 4 * ZI_WAVE, 0, stream>>>((TO*)out, ldo, os, (const TX*)x, ldx, xs, (const zi_bf16*)w, n, N, K, gt)
    ZI_DISPATCH_DTYPE(x_dt, TX, ZI_DISPATCH_DTYPE(out_dt, TO, {
        if (many && gate) ZI_HW(headwise_linear_many_kernel, true);
        else if (many) ZI_HW(headwise_linear_many_kernel, false);
        else if (gate) ZI_HW(headwise_linear_few_kernel, true);
        else ZI_HW(headwise_linear_few_kernel, false);
    }));
#undef ZI_HW
    return zi_check_launch("headwise_linear");
}

extern "C" int zi_headwise_linear(void* out, int out_dt, int64_t ldo, int os, const void* x, int x_dt, int64_t ldx, int xs,
                                  const void* w, int n, int heads, int N, int K, hipStream_t stream) {
    return zi_headwise_linear_gated(out, out_dt, ldo, os, x, x_dt, ldx, xs, w, n, heads, N, K, nullptr, ZI_F32, 0, 1, 0, stream);
}

// qa[t][h][rank + ...] = the rotated part of every head's query, turned in neighbouring pairs.
template <typename T, typename TO>
__global__ void latent_query_rot_kernel(TO* __restrict__ qa, const T* __restrict__ q, int64_t ldq,
                                        const float* __restrict__ table, int n, int heads, int dim, int rank, int rot) {
    const int half = rot / 2;
    const int64_t i = (int64_t)blockIdx.x * blockDim.x + threadIdx.x;
    if (i >= (int64_t)n * heads * half) return;
    const int p = (int)(i % half), h = (int)((i / half) % heads);
    const int64_t t = i / ((int64_t)half * heads);
    const T* qr = q + t * ldq + (int64_t)h * (dim + rot) + dim + 2 * p;
    const float u = zi_load(qr), v = zi_load(qr + 1);
    const float c = table[(t * half + p) * 2], s = table[(t * half + p) * 2 + 1];
    TO* o = qa + (t * heads + h) * (rank + rot) + rank + 2 * p;
    zi_store(o, u * c - v * s);
    zi_store(o + 1, v * c + u * s);
}

extern "C" int zi_latent_query_rot(void* qa, int qa_dt, const void* q, int dt, int64_t ldq, const float* table, int n, int heads,
                                   int dim, int rank, int rot, hipStream_t stream) {
    ZI_REQUIRE(n >= 0 && heads > 0 && dim > 0 && rank > 0 && rot >= 0 && rot % 2 == 0 && ldq >= (int64_t)heads * (dim + rot),
               "latent_query_rot: bad sizes");
    const int64_t total = (int64_t)n * heads * (rot / 2);
    if (total == 0) return 0;
    ZI_REQUIRE(table, "latent_query_rot: no table of angles");
    ZI_DISPATCH_DTYPE(dt, T, ZI_DISPATCH_DTYPE(qa_dt, TO, {
        latent_query_rot_kernel<T, TO><<<(unsigned)((total + 255) / 256), 256, 0, stream>>>((TO*)qa, (const T*)q, ldq, table, n, heads,
                                                                                             dim, rank, rot);
    }));
    return zi_check_launch("latent_query_rot");
}

// Few tokens: qa[t][h] = (W_uk[h]^T q_plain, turn(q_rot)) from the query product's float32 partial sums, one launch.
// x [splits][n][heads * (dim + rot)] (row stride ldx); w bfloat16 [heads][rank][dim].  Workgroups as in
// headwise_linear_few_kernel (the terms are added as they are loaded); the last of a head's (blockIdx.z) turns the rotated part.
template <typename TO>
__global__ void __launch_bounds__(4 * ZI_WAVE)
latent_query_sums_kernel(TO* __restrict__ qa, const float* __restrict__ x, int splits, int64_t split_stride, int64_t ldx,
                         const zi_bf16* __restrict__ w, const float* __restrict__ table, int n, int heads, int dim, int rank, int rot) {
    __shared__ la_f32x4_t part[3][ZI_WAVE];
    const int t0 = blockIdx.x * 16, h = blockIdx.y;
    const int out_w = rank + rot, xs = dim + rot;
    if (blockIdx.z == gridDim.z - 1) {
        const int half = rot / 2;
        for (int i = threadIdx.x; i < 16 * half; i += 4 * ZI_WAVE) {
            const int t = t0 + i / half, p = i % half;
            if (t >= n) continue;
            const float* at = x + (int64_t)t * ldx + (int64_t)h * xs + dim + 2 * p;
            float u = at[0], v = at[1];
            for (int s = 1; s < splits; ++s) {
                u += at[s * split_stride];
                v += at[s * split_stride + 1];
            }
            const float c = table[((int64_t)t * half + p) * 2], sn = table[((int64_t)t * half + p) * 2 + 1];
            TO* o = qa + ((int64_t)t * heads + h) * out_w + rank + 2 * p;
            zi_store(o, u * c - v * sn);
            zi_store(o + 1, v * c + u * sn);
        }
        return;
    }
    const int n0 = blockIdx.z * 16;
    const int lane = threadIdx.x % ZI_WAVE, wave = threadIdx.x / ZI_WAVE, r = lane % 16, j = lane / 16;
    const zi_bf16* wrow = w + ((int64_t)h * rank + (n0 + r < rank ? n0 + r : rank - 1)) * dim;
    const int64_t t = t0 + r < n ? t0 + r : n - 1;
    const float* xrow = x + t * ldx + (int64_t)h * xs;
    la_f32x4_t acc = (la_f32x4_t){0.f, 0.f, 0.f, 0.f};
    for (int k0 = wave * 32; k0 < dim; k0 += 128) {
        const int k = k0 + 8 * j, kc = k < dim ? k : 0;
        const unsigned mask = 0u - (unsigned)(k < dim);
        la_pack a = la_load8(wrow + kc), b;
        float4 lo = *reinterpret_cast<const float4*>(xrow + kc), hi = *reinterpret_cast<const float4*>(xrow + kc + 4);
        for (int s0 = 1; s0 < splits; s0 += 4) {      // four terms in flight, added in their order
            float4 l4[4], h4[4];
#pragma unroll
            for (int u = 0; u < 4; ++u) {
                const float* at = xrow + (int64_t)(s0 + u < splits ? s0 + u : 0) * split_stride + kc;
                l4[u] = *reinterpret_cast<const float4*>(at);
                h4[u] = *reinterpret_cast<const float4*>(at + 4);
            }
#pragma unroll
            for (int u = 0; u < 4; ++u) {
                if (s0 + u >= splits) break;
                lo.x += l4[u].x; lo.y += l4[u].y; lo.z += l4[u].z; lo.w += l4[u].w;
                hi.x += h4[u].x; hi.y += h4[u].y; hi.z += h4[u].z; hi.w += h4[u].w;
            }
        }
        b.w[0] = zi_pack_bf16x2(lo.x, lo.y);
        b.w[1] = zi_pack_bf16x2(lo.z, lo.w);
        b.w[2] = zi_pack_bf16x2(hi.x, hi.y);
        b.w[3] = zi_pack_bf16x2(hi.z, hi.w);
        a.u &= mask;
        b.u &= mask;
        acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a.b, b.b, acc, 0, 0, 0);
    }
    if (wave > 0) part[wave - 1][lane] = acc;
    __syncthreads();
    if (wave > 0) return;
#pragma unroll
    for (int u = 0; u < 3; ++u) acc += part[u][lane];
    if (t0 + r >= n || n0 + 4 * j >= rank) return;
    la_store4(qa + (t * heads + h) * out_w + n0 + 4 * j, acc, rank - n0 - 4 * j);
}

extern "C" int zi_latent_query_sums(void* qa, int qa_dt, const float* x, int splits, int64_t split_stride, int64_t ldx, const void* w,
                                    const float* table, int n, int heads, int dim, int rank, int rot, hipStream_t stream) {
    ZI_REQUIRE(n >= 0 && heads > 0 && heads <= 65535 && dim > 0 && rank > 0 && rot >= 0 && rot % 2 == 0 && splits >= 1 &&
                   ldx >= (int64_t)heads * (dim + rot) && (rank + 15) / 16 < 65535, "latent_query_sums: bad sizes");
    ZI_REQUIRE(zi_headwise_linear_supported(ZI_BF16, dim, ldx, dim + rot) && split_stride % 4 == 0 && ((uintptr_t)x % 16) == 0 && ((uintptr_t)w % 16) == 0,
               "latent_query_sums: sizes in eights and aligned rows are needed");
    ZI_REQUIRE(rot == 0 || table, "latent_query_sums: no table of angles");
    if (n == 0) return 0;
    const dim3 grid((n + 15) / 16, heads, (rank + 15) / 16 + 1);
    ZI_DISPATCH_DTYPE(qa_dt, TO, {
        latent_query_sums_kernel<TO><<<grid, 4 * ZI_WAVE, 0, stream>>>((TO*)qa, x, splits, split_stride, ldx, (const zi_bf16*)w, table, n,
                                                                       heads, dim, rank, rot);
    });
    return zi_check_launch("latent_query_sums");
}
