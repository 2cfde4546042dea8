// Attention over the paged KV cache with a causal mask, narrowed to the query's chunk or to a sliding window, and with an
// optional sink per head: a score without key or value that only takes its share of the softmax.  Cache rows are
// [block][kv head][token][row], a row being a head's dim (vdim) elements and zero padding.
//   attn_tile_kernel     prompts in bf16: 128 query tokens of one head per workgroup, both products on the matrix cores; keys
//                        and values from the cache, or of latent attention expanded per head (DENSE)
//   attn_decode_kernel   decode in bf16: the query heads of a kv head are the columns of the same products
//   latent_decode_kernel decode of latent attention in bf16: one cache row is key and value of all heads
//   attn_rows_kernel     any sizes, both element types: one wave per (query token, head), arithmetic on the vector ALU
#include <algorithm>

#include "hybrid_common.hpp"

namespace nqh {
namespace {

constexpr float kLog2e = 1.4426950408889634f;
constexpr float kNegBig = -3.0e38f;
constexpr int kMaxDim = 512;      // value elements of a head
constexpr int kMaxKeyDim = 1024;
constexpr int kTileRows = 128;   // query tokens per tile of a prompt pass

// First position that the token at position p sees; 0: no chunks, no window.
__device__ __forceinline__ int first_visible(int p, int chunk, int window) {
    const int c = chunk > 0 ? p / chunk * chunk : 0;
    return window > 0 ? max(c, p - window + 1) : c;
}

// ---------------------------------------------------------------------------------------------------
// Lanes walk the visible keys 64 at a time (a lane scores one key), then the value columns.  With `context_lens` row b is
// the last of context_lens[b] tokens of sequence b; otherwise a workgroup takes the tile (segment, first row) of a prompt
// pass, see nqh_attention_prefill.
template <typename T>
__global__ __launch_bounds__(256) void attn_rows_kernel(
    const typename T::elem* __restrict__ q, const typename T::elem* __restrict__ k_cache,
    const typename T::elem* __restrict__ v_cache, const int32_t* __restrict__ block_table,
    const int32_t* __restrict__ context_lens, const int32_t* __restrict__ segments, const int32_t* __restrict__ tiles,
    const typename T::elem* __restrict__ sink, typename T::elem* __restrict__ out, int64_t items, int tile_groups, int heads,
    int kv_heads, int dim, int vdim, int k_row, int v_row, int block_size, int max_blocks, int num_blocks, int chunk, int window,
    float scale) {
    __shared__ float s_q[4][kMaxKeyDim];
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
    int64_t row, pos;
    int h, seq;
    bool live;
    if (context_lens) {
        const int64_t item = (int64_t)blockIdx.x * 4 + wave;
        live = item < items;
        row = live ? item / heads : 0;
        h = live ? (int)(item % heads) : 0;
        seq = (int)row;
        pos = context_lens[row] - 1;
    } else {
        const int tile = blockIdx.x / tile_groups, i = (blockIdx.x % tile_groups) * 4 + wave;
        seq = tiles[2 * tile];
        const int in_seg = tiles[2 * tile + 1] + i / heads;
        live = i / heads < kTileRows && in_seg < segments[3 * seq + 1];
        h = i % heads;
        row = segments[3 * seq] + (live ? in_seg : 0);
        pos = (int64_t)segments[3 * seq + 2] + (live ? in_seg : 0);
    }
    for (int d = lane; d < dim; d += 64) s_q[wave][d] = T::load(q + (row * heads + h) * k_row + d) * scale * kLog2e;
    __syncthreads();
    if (!live) return;
    const int g = h / (heads / kv_heads);
    const int64_t cap = (int64_t)max_blocks * block_size;
    pos = pos < 0 ? 0 : (pos >= cap ? cap - 1 : pos);
    const int lo = first_visible((int)pos, chunk, window), hi = (int)pos + 1;
    const int32_t* table = block_table + (int64_t)seq * max_blocks;
    float m = sink ? T::load(sink + h) * kLog2e : kNegBig, l = sink ? 1.f : 0.f, acc[kMaxDim / 64];
#pragma unroll
    for (int c = 0; c < kMaxDim / 64; ++c) acc[c] = 0.f;
    for (int j0 = lo; j0 < hi; j0 += 64) {
        const int j = j0 + lane;
        const bool ok = j < hi;
        const int jc = ok ? j : hi - 1;
        int blk = table[jc / block_size];
        blk = blk < 0 ? 0 : (blk >= num_blocks ? num_blocks - 1 : blk);
        const int64_t tok = ((int64_t)blk * kv_heads + g) * block_size + jc % block_size;
        const typename T::elem* kp = k_cache + tok * k_row;
        float s = 0.f;
        for (int d = 0; d < dim; ++d) s += s_q[wave][d] * T::load(kp + d);
        s = ok ? s : kNegBig;
        const float mn = fmaxf(m, wave_max(s));
        const float c = exp2f(m - mn), p = ok ? exp2f(s - mn) : 0.f;
        m = mn;
        l = l * c + wave_sum(p);
#pragma unroll
        for (int e = 0; e < kMaxDim / 64; ++e) acc[e] *= c;
        const int n = min(64, hi - j0);
        for (int u = 0; u < n; ++u) {
            const float pu = __shfl(p, u);
            const int64_t tu = __shfl((int)tok, u);   // blocks * block_size fits 31 bits (checked on the host)
#pragma unroll
            for (int e = 0; e < kMaxDim / 64; ++e) {
                const int d = e * 64 + lane;
                if (d < vdim) acc[e] += pu * T::load(v_cache + tu * v_row + d);
            }
        }
    }
#pragma unroll
    for (int e = 0; e < kMaxDim / 64; ++e) {
        const int d = e * 64 + lane;
        if (d < vdim) T::store(out + (row * heads + h) * vdim + d, acc[e] / l);
    }
}

// ---------------------------------------------------------------------------------------------------
// Matrix-core forms.  Scores of 16 keys x 16 columns (queries or heads) are S^T = K q^T, so a lane holds the scores of
// column lane % 16 and keys 4 (lane / 16) + r -- which is where the B operand of out^T = V^T P^T wants that column's
// probabilities (the order of the keys inside the contraction is free as long as both operands agree), so they never
// leave their registers.  The A operand of the second product needs several keys of one value dim per lane: V tiles
// come back from LDS through the transposing read (in each group of 16 lanes, lane 4q + c receives element c of the
// four 8-byte pieces that lanes q, q + 4, q + 8, q + 12 point at).
//
// LDS rows are R elements (a cache row), brought by load-to-LDS, which writes linearly: 16-byte piece n of the tile is
// row n / (R / 8), position n % (R / 8).  A K row is stored rotated by row / kTurn pieces, a V row by row / kTurn windows
// of 16 dims, kTurn being the number of rows after which the bank of a row's start repeats: the 16 rows of one operand
// read then fall on different banks.
#define NQH_GPTR(p) ((__attribute__((address_space(1))) void*)(p))
#define NQH_LPTR(p) ((__attribute__((address_space(3))) void*)(p))
typedef short s16x4 __attribute__((ext_vector_type(4)));

template <int R>
struct RowLayout {
    static constexpr int kPieces = R / 8, kWindows = R / 16;
    static constexpr int kTurn = kWindows % 8 == 0 ? 1 : (kWindows % 4 == 0 ? 2 : 4);
    static_assert(R % 32 == 0, "cache rows");
    // source element of the piece stored at position `pos` of row `row`
    static __device__ __forceinline__ int k_source(int row, int pos) {
        return 8 * ((pos + kPieces - (row / kTurn) % kPieces) % kPieces);
    }
    static __device__ __forceinline__ int v_source(int row, int pos) {
        return 16 * (((pos >> 1) + kWindows - (row / kTurn) % kWindows) % kWindows) + 8 * (pos & 1);
    }
    // byte offset of piece `piece` of K row `row`, and of the 16-dim window `w` of V row `row`
    static __device__ __forceinline__ int k_at(int row, int piece) {
        return row * (2 * R) + 16 * ((piece + row / kTurn) % kPieces);
    }
    static __device__ __forceinline__ int v_at(int row, int w) {
        return row * (2 * R) + 32 * ((w + row / kTurn) % kWindows);
    }
};

// Eight keys of 16 value dims as an A operand: keys tok .. tok + 3 (tok already holds 4 * (lane / 16)) and tok + 16 ..
template <int R>
__device__ __forceinline__ u32x4 value_operand(const unsigned char* v_tile, int tile_row, int w, int lane) {
    const int lo = lane & 15, hi = lane >> 4, row = tile_row + 4 * hi + (lo >> 2), quad = (lo & 3) * 8;
    const unsigned char* p0 = v_tile + RowLayout<R>::v_at(row, w) + quad;
    const unsigned char* p1 = v_tile + RowLayout<R>::v_at(row + 16, w) + quad;
    const s16x4 a = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s16x4*)p0);
    const s16x4 b = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s16x4*)p1);
    const u32x2 ua = __builtin_bit_cast(u32x2, a), ub = __builtin_bit_cast(u32x2, b);
    return u32x4{ua[0], ua[1], ub[0], ub[1]};
}

// Rows of latents.  One of 512 elements is a load-to-LDS of its own, so rows can lie 1040 bytes apart instead of being
// rotated: the places of all operands of a lane then differ by constants.
template <int R>
struct LatentLayout {
    static constexpr int kLoadBytes = R == 512 ? 1040 : 1024, kTile = 32 * R * 2 / 1024 * kLoadBytes;
    static __device__ __forceinline__ int source(int row, int pos) { return R == 512 ? 8 * pos : RowLayout<R>::k_source(row, pos); }
    static __device__ __forceinline__ int at(int row, int piece) {
        return R == 512 ? row * kLoadBytes + 16 * piece : RowLayout<R>::k_at(row, piece);
    }
};
// value_operand from such rows.
template <int R>
__device__ __forceinline__ u32x4 latent_operand(const unsigned char* tile, int w, int lane) {
    const int lo = lane & 15, hi = lane >> 4, row = 4 * hi + (lo >> 2), sub = (lo & 3) >> 1, half = (lo & 1) * 8;
    const unsigned char* p0 = tile + LatentLayout<R>::at(row, 2 * w + sub) + half;
    const unsigned char* p1 = tile + LatentLayout<R>::at(row + 16, 2 * w + sub) + half;
    const s16x4 a = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s16x4*)p0);
    const s16x4 b = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s16x4*)p1);
    const u32x2 ua = __builtin_bit_cast(u32x2, a), ub = __builtin_bit_cast(u32x2, b);
    return u32x4{ua[0], ua[1], ub[0], ub[1]};
}

__device__ const u32x4 g_zero_piece = {0u, 0u, 0u, 0u};   // what lies past the end of an unpadded row

// Keys and values of all heads, expanded from latents: token j of a segment is row first[segment] + j of `kv`, which holds
// the heads' unrotated keys and, from `v_at` on, their values, and of `rot`, the rotated key part that all heads share.
struct DenseKV {
    const uint16_t *kv, *rot;
    const int32_t* first;
    int64_t kv_stride, rot_stride, v_at;
    int dim, rot_dim;
};

__device__ __forceinline__ float exp2_raw(float x) { return __builtin_amdgcn_exp2f(x); }

// Prompt attention.  Four waves of 32 queries; tiles of KT keys, double-buffered; every wave skips the tiles none of its
// queries sees.  Cache rows are addressed key by key, so a tile may start anywhere and straddle cache blocks.  R, RV: key and
// value elements of a row in LDS.
template <int R, int RV, int KT, bool DENSE>
__global__ __launch_bounds__(256) void attn_tile_kernel(
    const uint16_t* __restrict__ q, const uint16_t* __restrict__ k_cache, const uint16_t* __restrict__ v_cache,
    const int32_t* __restrict__ block_tables, const int32_t* __restrict__ segments, const int32_t* __restrict__ tiles,
    const uint16_t* __restrict__ sink, DenseKV dense, uint16_t* __restrict__ out, int heads, int kv_heads, int vdim,
    int block_size, int max_blocks, int num_blocks, int chunk, int window, float scale, int q_tiles) {
    using L = RowLayout<R>;
    using LV = RowLayout<RV>;
    constexpr int kBytes = KT * R * 2, kLoads = KT * L::kPieces / 256;
    constexpr int vBytes = KT * RV * 2, vLoads = KT * LV::kPieces / 256, kBuffer = kBytes + vBytes;
    static_assert(KT % 32 == 0 && KT * L::kPieces % 256 == 0 && KT * LV::kPieces % 256 == 0, "whole load-to-LDS instructions");
    // one array: with several the compiler waits for every load-to-LDS in flight before any LDS read
    __shared__ __attribute__((aligned(1024))) unsigned char s_mem[2 * kBuffer + (DENSE ? 0 : 2 * KT * 4)];   // [buffer][K | V], rows
    int* s_row = reinterpret_cast<int*>(s_mem + 2 * kBuffer);                                   // [buffer][KT]
    // contiguous runs of (kv head, query tile, head of the group) per XCD: a kv head's cache is read through one L2
    const int per = gridDim.x >> 3, id = (blockIdx.x & 7) * per + (blockIdx.x >> 3);
    if (id >= q_tiles * heads) return;
    const int group = heads / kv_heads;
    const int g = id / (q_tiles * group), rest = id - g * q_tiles * group;
    const int qt = rest / group, h = g * group + rest % group;
    const int seg = tiles[2 * qt], q0 = tiles[2 * qt + 1];
    const int rows = segments[3 * seg + 1], start = segments[3 * seg + 2];
    const int32_t* block_table = DENSE ? nullptr : block_tables + (int64_t)seg * max_blocks;
    q += (int64_t)segments[3 * seg] * heads * R;
    out += (int64_t)segments[3 * seg] * heads * vdim;
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int lo = lane & 15, hi = lane >> 4;
    auto visible_from = [&](int p) { return first_visible(p, chunk, window); };

    const int q_last = min(q0 + kTileRows, rows) - 1;
    const int k_begin = visible_from(start + q0), k_end = start + q_last + 1;
    const int wq0 = q0 + wave * 32;                                  // this wave's first query row
    const bool wave_live = wq0 <= q_last;
    const int w_first = start + min(wq0, q_last), w_last = start + min(wq0 + 31, q_last);
    const int see_lo = visible_from(w_first), full_lo = visible_from(w_last);
    int pos[2], low[2];                                              // per column: query position, first visible key
    u32x4 bq[2][R / 32];
#pragma unroll
    for (int c = 0; c < 2; ++c) {
        const int row = min(wq0 + 16 * c + lo, q_last);
        pos[c] = start + row;
        low[c] = visible_from(pos[c]);
        const uint16_t* p = q + ((int64_t)row * heads + h) * R + 8 * hi;
#pragma unroll
        for (int s = 0; s < R / 32; ++s) bq[c][s] = *reinterpret_cast<const u32x4*>(p + 32 * s);
    }
    // cache rows of a tile's keys (past the end those of the last visible key): the block number is fetched ahead of the
    // tile's other loads and turned into a row once they are under way
    const int key = (int)threadIdx.x % KT;
    int next_block = 0;
    auto fetch_block = [&](int t0) {
        if constexpr (!DENSE) next_block = block_table[min(t0 + key, k_end - 1) / block_size];
    };
    auto put_row = [&](int t0, int buf) {
        if constexpr (DENSE) return;
        const int blk = next_block < 0 ? 0 : (next_block >= num_blocks ? num_blocks - 1 : next_block);
        if (threadIdx.x < KT) s_row[buf * KT + key] = (blk * kv_heads + g) * block_size + min(t0 + key, k_end - 1) % block_size;
    };
    const int64_t dense_first = DENSE ? dense.first[seg] : 0;
    const uint16_t* dense_k = dense.kv + (int64_t)h * dense.dim;
    const uint16_t* dense_v = dense.kv + dense.v_at + (int64_t)h * vdim;
    auto stage_dense = [&](int t0, int buf) {
        unsigned char* base = s_mem + buf * kBuffer;
#pragma unroll
        for (int i = 0; i < kLoads; ++i) {
            const int n = (i * 4 + wave) * 64 + lane, row = n / L::kPieces, e = L::k_source(row, n % L::kPieces);
            const int64_t at = dense_first + min(t0 + row, k_end - 1);
            const uint16_t* src = e < dense.dim ? dense_k + at * dense.kv_stride + e
                                  : e < dense.dim + dense.rot_dim ? dense.rot + at * dense.rot_stride + (e - dense.dim)
                                                                  : (const uint16_t*)&g_zero_piece;
            __builtin_amdgcn_global_load_lds(NQH_GPTR(src), NQH_LPTR(base + (i * 4 + wave) * 1024), 16, 0, 0);
        }
#pragma unroll
        for (int i = 0; i < vLoads; ++i) {
            const int n = (i * 4 + wave) * 64 + lane, row = n / LV::kPieces, e = LV::v_source(row, n % LV::kPieces);
            const int64_t at = dense_first + min(t0 + row, k_end - 1);
            const uint16_t* src = e < vdim ? dense_v + at * dense.kv_stride + e : (const uint16_t*)&g_zero_piece;
            __builtin_amdgcn_global_load_lds(NQH_GPTR(src), NQH_LPTR(base + kBytes + (i * 4 + wave) * 1024), 16, 0, 0);
        }
    };
    auto stage = [&](int t0, int buf) {
        if constexpr (DENSE) {
            stage_dense(t0, buf);
            return;
        }
        static_assert(DENSE || R == RV, "cache rows of keys and values are equally wide");
        unsigned char* base = s_mem + buf * kBuffer;
#pragma unroll
        for (int i = 0; i < kLoads; ++i) {
            const int n = (i * 4 + wave) * 64 + lane, row = n / L::kPieces, p = n % L::kPieces;
            const int64_t at = (int64_t)s_row[buf * KT + row] * R;
            __builtin_amdgcn_global_load_lds(NQH_GPTR(k_cache + at + L::k_source(row, p)),
                                             NQH_LPTR(base + (i * 4 + wave) * 1024), 16, 0, 0);
            __builtin_amdgcn_global_load_lds(NQH_GPTR(v_cache + at + L::v_source(row, p)),
                                             NQH_LPTR(base + kBytes + (i * 4 + wave) * 1024), 16, 0, 0);
        }
    };
    const float sc = scale * kLog2e;
    // a sink is where the running softmax starts; a column's sum is spread over four lanes, one of which counts it
    const float m0 = sink ? Bf::to_f32(sink[h]) * kLog2e : kNegBig, l0 = sink && hi == 0 ? 1.f : 0.f;
    float m[2] = {m0, m0}, l[2] = {l0, l0};
    f32x4 acc[2][RV / 16];
#pragma unroll
    for (int c = 0; c < 2; ++c)
#pragma unroll
        for (int w = 0; w < RV / 16; ++w) acc[c][w] = f32x4{0.f, 0.f, 0.f, 0.f};

    fetch_block(k_begin);
    put_row(k_begin, 0);
    fetch_block(k_begin + KT);
    __syncthreads();
    stage(k_begin, 0);
    put_row(k_begin + KT, 1);
    int buf = 0;
    for (int t0 = k_begin; t0 < k_end; t0 += KT) {
        __builtin_amdgcn_s_waitcnt(0x0F70);   // this wave's part of the tile has landed
        __syncthreads();
        const bool more = t0 + KT < k_end;
        if (more) {
            fetch_block(t0 + 2 * KT);
            stage(t0 + KT, buf ^ 1);
        }
        const unsigned char *k_tile = s_mem + buf * kBuffer, *v_tile = k_tile + kBytes;
        if (wave_live && t0 <= w_last && t0 + KT > see_lo) {
            const bool masked = t0 + KT - 1 > w_first || t0 < full_lo;
            f32x4 st[2][KT / 16];
#pragma unroll
            for (int a = 0; a < KT / 16; ++a) {
                st[0][a] = st[1][a] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
                for (int s = 0; s < R / 32; ++s) {
                    const u32x4 ka = *reinterpret_cast<const u32x4*>(k_tile + L::k_at(16 * a + lo, 4 * s + hi));
                    st[0][a] = Bf::mfma16(ka, bq[0][s], st[0][a]);
                    st[1][a] = Bf::mfma16(ka, bq[1][s], st[1][a]);
                }
            }
            u32x4 pb[2][KT / 32];
#pragma unroll
            for (int c = 0; c < 2; ++c) {
                float mx = kNegBig;
#pragma unroll
                for (int a = 0; a < KT / 16; ++a)
#pragma unroll
                    for (int r = 0; r < 4; ++r) {
                        float s = st[c][a][r] * sc;
                        if (masked) {
                            const int j = t0 + 16 * a + 4 * hi + r;
                            s = (j <= pos[c] && j >= low[c]) ? s : -__builtin_inff();
                        }
                        st[c][a][r] = s;
                        mx = fmaxf(mx, s);
                    }
                mx = fmaxf(mx, __shfl_xor(mx, 16));
                mx = fmaxf(mx, __shfl_xor(mx, 32));
                const float mn = fmaxf(m[c], mx);
                if (__any(mn > m[c])) {
                    const float f = exp2_raw(m[c] - mn);
                    m[c] = mn;
                    l[c] *= f;
#pragma unroll
                    for (int w = 0; w < RV / 16; ++w)
#pragma unroll
                        for (int r = 0; r < 4; ++r) acc[c][w][r] *= f;
                }
#pragma unroll
                for (int u = 0; u < KT / 32; ++u) {
                    float p[2][4];
#pragma unroll
                    for (int a = 0; a < 2; ++a)
#pragma unroll
                        for (int r = 0; r < 4; ++r) {
                            p[a][r] = exp2_raw(st[c][2 * u + a][r] - mn);   // exp2(-inf) = 0: mn is finite always
                            l[c] += p[a][r];
                        }
                    pb[c][u] = u32x4{Bf::pack2(p[0][0], p[0][1]), Bf::pack2(p[0][2], p[0][3]), Bf::pack2(p[1][0], p[1][1]),
                                     Bf::pack2(p[1][2], p[1][3])};
                }
            }
#pragma unroll
            for (int u = 0; u < KT / 32; ++u)
#pragma unroll
                for (int w = 0; w < RV / 16; ++w) {
                    const u32x4 va = value_operand<RV>(v_tile, 32 * u, w, lane);
                    acc[0][w] = Bf::mfma16(va, pb[0][u], acc[0][w]);
                    acc[1][w] = Bf::mfma16(va, pb[1][u], acc[1][w]);
                }
        }
        if (more) put_row(t0 + 2 * KT, buf);   // the slots were last read by the stage before this one
        buf ^= 1;
    }
    if (!wave_live) return;
#pragma unroll
    for (int c = 0; c < 2; ++c) {
        float t = l[c];
        t += __shfl_xor(t, 16);
        t += __shfl_xor(t, 32);
        const float inv = 1.f / t;
        const int row = wq0 + 16 * c + lo;
        if (row > q_last) continue;
        uint16_t* dst = out + ((int64_t)row * heads + h) * vdim;
#pragma unroll
        for (int w = 0; w < RV / 16; ++w) {
            const int d = 16 * w + 4 * hi;
            float v[4];
#pragma unroll
            for (int r = 0; r < 4; ++r) v[r] = acc[c][w][r] * inv;
            if (vdim % 4 == 0) {
                if (d < vdim) store_vec<Bf, 4>(dst + d, v);
            } else {
#pragma unroll
                for (int r = 0; r < 4; ++r)
                    if (d + r < vdim) Bf::store(dst + d + r, v[r]);
            }
        }
    }
}

// Decode attention.  Workgroup = (sequence, kv head, 16 of its query heads, context split); a wave takes tiles of 32 keys
// through its own part of LDS, no barriers until the merge.
template <int R, int WAVES>
__global__ __launch_bounds__(64 * WAVES) void attn_decode_kernel(
    const uint16_t* __restrict__ q, const uint16_t* __restrict__ k_cache, const uint16_t* __restrict__ v_cache,
    const int32_t* __restrict__ block_table, const int32_t* __restrict__ context_lens, const uint16_t* __restrict__ sink,
    uint16_t* __restrict__ out, float* __restrict__ partial, int heads, int kv_heads, int vdim, int block_size, int max_blocks,
    int num_blocks, int chunk, int window, float scale, int splits, int head_tiles) {
    using L = RowLayout<R>;
    constexpr int RS = R + 4;                             // width of a result row
    constexpr int TT = 32, kBytes = TT * R * 2, kLoads = kBytes / 1024;
    constexpr int kWave = 2 * kBytes + 1024;
    static_assert(16 * RS * 4 <= kWave, "the per-wave results reuse the wave's tiles");
    __shared__ __attribute__((aligned(1024))) unsigned char s_raw[WAVES * kWave];
    const int sp = blockIdx.x % splits, ht = blockIdx.x / splits % head_tiles;
    const int g = blockIdx.x / (splits * head_tiles) % kv_heads, b = blockIdx.x / (splits * head_tiles * kv_heads);
    const int group = heads / kv_heads, h0 = g * group + 16 * ht, n_heads = min(16, group - 16 * ht);
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int lo = lane & 15, hi = lane >> 4;
    int ctx = context_lens[b];
    ctx = ctx < 1 ? 1 : (ctx > max_blocks * block_size ? max_blocks * block_size : ctx);
    const int first = first_visible(ctx - 1, chunk, window);
    const int per = ((ctx - first + splits - 1) / splits + TT - 1) / TT * TT;
    const int t0 = first + sp * per, t1 = min(ctx, t0 + per);
    unsigned char* kt = s_raw + wave * kWave;
    unsigned char* vt = kt + kBytes;

    u32x4 bq[R / 32];
#pragma unroll
    for (int s = 0; s < R / 32; ++s) {
        // columns past the heads repeat the last one; their results are not stored
        bq[s] = *reinterpret_cast<const u32x4*>(q + ((int64_t)b * heads + h0 + min(lo, n_heads - 1)) * R + 32 * s + 8 * hi);
    }
    const float sc = scale * kLog2e;
    float m = kNegBig, l = 0.f;
    if (sink && sp == 0 && wave == 0) {       // counted once: by one wave of one split, in one of a column's four lanes
        m = Bf::to_f32(sink[h0 + min(lo, n_heads - 1)]) * kLog2e;
        l = hi == 0 ? 1.f : 0.f;
    }
    f32x4 acc[R / 16];
#pragma unroll
    for (int w = 0; w < R / 16; ++w) acc[w] = f32x4{0.f, 0.f, 0.f, 0.f};
    const int32_t* table = block_table + (int64_t)b * max_blocks;
    for (int tb = t0 + wave * TT; tb < t1; tb += WAVES * TT) {
        // the cache row of key tb + lane % 32 (past the split's end the last key stands in)
        const int j = min(tb + (lane & 31), t1 - 1);
        int blk = table[j / block_size];
        blk = blk < 0 ? 0 : (blk >= num_blocks ? num_blocks - 1 : blk);
        const int my_row = (blk * kv_heads + g) * block_size + j % block_size;
#pragma unroll
        for (int i = 0; i < kLoads; ++i) {
            const int n = i * 64 + lane, row = n / L::kPieces;
            const int64_t base = (int64_t)__shfl(my_row, row) * R;
            __builtin_amdgcn_global_load_lds(NQH_GPTR(k_cache + base + L::k_source(row, n % L::kPieces)),
                                             NQH_LPTR(kt + i * 1024), 16, 0, 0);
        }
#pragma unroll
        for (int i = 0; i < kLoads; ++i) {
            const int n = i * 64 + lane, row = n / L::kPieces;
            const int64_t base = (int64_t)__shfl(my_row, row) * R;
            __builtin_amdgcn_global_load_lds(NQH_GPTR(v_cache + base + L::v_source(row, n % L::kPieces)),
                                             NQH_LPTR(vt + i * 1024), 16, 0, 0);
        }
        // a wave's loads return in order: with at most the V tile's outstanding, the K tile has landed
        asm volatile("s_waitcnt vmcnt(%0)" : : "n"(kLoads) : "memory");
        f32x4 st[2];
        st[0] = st[1] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int a = 0; a < 2; ++a)
#pragma unroll
            for (int s = 0; s < R / 32; ++s)
                st[a] = Bf::mfma16(*reinterpret_cast<const u32x4*>(kt + L::k_at(16 * a + lo, 4 * s + hi)), bq[s], st[a]);
        float mx = kNegBig;
#pragma unroll
        for (int a = 0; a < 2; ++a)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                st[a][r] = tb + 16 * a + 4 * hi + r < t1 ? st[a][r] * sc : -__builtin_inff();
                mx = fmaxf(mx, st[a][r]);
            }
        mx = fmaxf(mx, __shfl_xor(mx, 16));
        mx = fmaxf(mx, __shfl_xor(mx, 32));
        const float mn = fmaxf(m, mx);
        const float f = exp2_raw(m - mn);
        m = mn;
        float p[2][4], ps = 0.f;
#pragma unroll
        for (int a = 0; a < 2; ++a)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                p[a][r] = exp2_raw(st[a][r] - mn);
                ps += p[a][r];
            }
        l = l * f + ps;
        const u32x4 pb = u32x4{Bf::pack2(p[0][0], p[0][1]), Bf::pack2(p[0][2], p[0][3]), Bf::pack2(p[1][0], p[1][1]),
                               Bf::pack2(p[1][2], p[1][3])};
#pragma unroll
        for (int w = 0; w < R / 16; ++w)
#pragma unroll
            for (int r = 0; r < 4; ++r) acc[w][r] *= f;
        asm volatile("s_waitcnt vmcnt(0)" : : : "memory");
#pragma unroll
        for (int w = 0; w < R / 16; ++w) acc[w] = Bf::mfma16(value_operand<R>(vt, 0, w, lane), pb, acc[w]);
        asm volatile("s_waitcnt lgkmcnt(0)" : : : "memory");   // the tile is free for the next loads
    }
    l += __shfl_xor(l, 16);
    l += __shfl_xor(l, 32);
    // per-wave results [head][RS] over the wave's own tiles, then merged over the waves
    float* mine = reinterpret_cast<float*>(kt);
#pragma unroll
    for (int w = 0; w < R / 16; ++w)
#pragma unroll
        for (int r = 0; r < 4; ++r) mine[lo * RS + 16 * w + 4 * hi + r] = acc[w][r];
    if (hi == 0) {
        mine[lo * RS + R] = m;
        mine[lo * RS + R + 1] = l;
    }
    __syncthreads();
    // per head: what each wave's result counts (in place of its maximum), and what is known of the whole split
    if (threadIdx.x < n_heads) {
        const int h = threadIdx.x;
        float* o[WAVES];
        float mm = kNegBig, lt = 0.f;
#pragma unroll
        for (int w = 0; w < WAVES; ++w) {
            o[w] = reinterpret_cast<float*>(s_raw + w * kWave) + h * RS + R;
            mm = fmaxf(mm, o[w][0]);
        }
#pragma unroll
        for (int w = 0; w < WAVES; ++w) {
            o[w][0] = exp2_raw(o[w][0] - mm);
            lt += o[w][1] * o[w][0];
        }
        if (splits == 1) {
#pragma unroll
            for (int w = 0; w < WAVES; ++w) o[w][0] /= lt;
        } else {
            float* dst = partial + (((int64_t)b * heads + h0 + h) * splits + sp) * (vdim + 4) + vdim;
            dst[0] = mm;
            dst[1] = lt;
        }
    }
    __syncthreads();
    const int quads = (vdim + 3) >> 2;
    for (int i = threadIdx.x; i < n_heads * quads; i += 64 * WAVES) {
        const int h = i / quads, d = (i - h * quads) * 4;
        f32x4 at = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int w = 0; w < WAVES; ++w) {
            const float* o = reinterpret_cast<const float*>(s_raw + w * kWave) + h * RS;
            const f32x4 v = *reinterpret_cast<const f32x4*>(o + d);
            const float f = o[R];
#pragma unroll
            for (int e = 0; e < 4; ++e) at[e] += v[e] * f;
        }
        const int64_t head = (int64_t)b * heads + h0 + h;
        const float r[4] = {at[0], at[1], at[2], at[3]};
        if (splits == 1) {
            uint16_t* dst = out + head * vdim + d;
            if (vdim % 4 == 0) {
                store_vec<Bf, 4>(dst, r);
            } else {
                for (int e = 0; e < 4; ++e)
                    if (d + e < vdim) Bf::store(dst + e, r[e]);
            }
        } else {
            float* dst = partial + (head * splits + sp) * (vdim + 4) + d;
            if (vdim % 4 == 0) {
                *reinterpret_cast<f32x4*>(dst) = at;
            } else {
                for (int e = 0; e < 4; ++e)
                    if (d + e < vdim) dst[e] = r[e];
            }
        }
    }
}

// Decode attention over latent rows of R elements, the first RL of which are the value.  Workgroup = (sequence, 16 HT heads,
// context split): tiles of 32 keys, double-buffered, that all four waves read; a wave has one tile of 16 heads and a part of
// the value elements, so nothing is merged between waves (those that share heads repeat the scores).  Latents and rotated
// parts lie in two LDS tiles whose row widths are powers of two: a load-to-LDS takes whole rows and needs next to no address
// arithmetic.
template <int RL, int R, int HT>
__global__ __launch_bounds__(256, 2) void latent_decode_kernel(
    const uint16_t* __restrict__ q, const uint16_t* __restrict__ cache, const int32_t* __restrict__ block_table,
    const int32_t* __restrict__ context_lens, uint16_t* __restrict__ out, float* __restrict__ partial, int heads, int rank,
    int block_size, int max_blocks, int num_blocks, float scale, int splits, int head_groups) {
    using LL = LatentLayout<RL>;
    using LR = LatentLayout<R - RL>;
    constexpr int TT = 32, kRot = LL::kTile, kBuffer = kRot + LR::kTile, kLoads = RL / 64, kPieces = RL / 8, rPieces = (R - RL) / 8;
    constexpr int kParts = 4 / HT, kWindows = RL / 16 / kParts;
    static_assert(2 * kBuffer <= 80 * 1024, "two workgroups per CU");
    __shared__ __attribute__((aligned(1024))) unsigned char s_mem[2 * kBuffer];
    const int sp = blockIdx.x % splits, hg = blockIdx.x / splits % head_groups, b = blockIdx.x / (splits * head_groups);
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int lo = lane & 15, hi = lane >> 4, part = wave / HT;
    const int h0 = hg * 16 * HT + wave % HT * 16, head = min(h0 + lo, heads - 1);   // columns past the heads repeat the last
    int ctx = context_lens[b];
    ctx = ctx < 1 ? 1 : (ctx > max_blocks * block_size ? max_blocks * block_size : ctx);
    const int tiles = (ctx + TT - 1) / TT;               // dealt evenly
    const int t0 = (int)((int64_t)tiles * sp / splits) * TT, t1 = min(ctx, (int)((int64_t)tiles * (sp + 1) / splits) * TT);
    const int32_t* table = block_table + (int64_t)b * max_blocks;
    u32x4 bq[R / 32];
#pragma unroll
    for (int s = 0; s < R / 32; ++s)
        bq[s] = *reinterpret_cast<const u32x4*>(q + ((int64_t)b * heads + head) * R + 32 * s + 8 * hi);
    // the cache row of key tb + lane % 32 (past the split's end the last key stands in); the block number is fetched ahead
    int next_block = 0;
    auto key_of = [&](int tb) { return max(min(tb + (lane & 31), t1 - 1), 0); };
    auto fetch_block = [&](int tb) { next_block = table[key_of(tb) / block_size]; };
    auto stage = [&](int tb, int buf) {
        const int blk = next_block < 0 ? 0 : (next_block >= num_blocks ? num_blocks - 1 : next_block);
        const int my_row = blk * block_size + key_of(tb) % block_size;
        unsigned char* base = s_mem + buf * kBuffer;
        // every shuffle comes before the first load: the compiler has LDS instructions wait for loads-to-LDS
        int rows[kLoads];
#pragma unroll
        for (int i = 0; i < kLoads; ++i) {                          // a wave brings eight rows
            const int at = wave * kLoads + i;
            rows[i] = kPieces == 64 ? __builtin_amdgcn_readlane(my_row, at) : __shfl(my_row, (at * 64 + lane) / kPieces);
        }
        const int rn = wave * 64 + lane, rot_row = __shfl(my_row, min(rn / rPieces, TT - 1));
#pragma unroll
        for (int i = 0; i < kLoads; ++i) {
            const int at = wave * kLoads + i, n = at * 64 + lane;
            __builtin_amdgcn_global_load_lds(NQH_GPTR(cache + (int64_t)rows[i] * R + LL::source(n / kPieces, n % kPieces)),
                                             NQH_LPTR(base + at * LL::kLoadBytes), 16, 0, 0);
        }
        if (wave < rPieces / 2)                                     // 32 x 32 elements are two loads, 32 x 64 four
            __builtin_amdgcn_global_load_lds(NQH_GPTR(cache + (int64_t)rot_row * R + RL + LR::source(rn / rPieces, rn % rPieces)),
                                             NQH_LPTR(base + kRot + wave * 1024), 16, 0, 0);
    };
    const float sc = scale * kLog2e;
    float m = kNegBig, l = 0.f;
    f32x4 acc[kWindows];
#pragma unroll
    for (int w = 0; w < kWindows; ++w) acc[w] = f32x4{0.f, 0.f, 0.f, 0.f};
    fetch_block(t0);
    if (t0 < t1) stage(t0, 0);
    fetch_block(t0 + TT);
    int buf = 0;
    for (int tb = t0; tb < t1; tb += TT) {
        __builtin_amdgcn_s_waitcnt(0x0F70);   // this wave's part of the tile has landed
        __syncthreads();
        if (tb + TT < t1) {
            stage(tb + TT, buf ^ 1);
            fetch_block(tb + 2 * TT);
        }
        const unsigned char* tile = s_mem + buf * kBuffer;
        f32x4 st[2];
        st[0] = st[1] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int s = 0; s < R / 32; ++s)
#pragma unroll
            for (int a = 0; a < 2; ++a) {
                const int row = 16 * a + lo;
                const unsigned char* p = s < RL / 32 ? tile + LL::at(row, 4 * s + hi)
                                                     : tile + kRot + LR::at(row, 4 * (s - RL / 32) + hi);
                st[a] = Bf::mfma16(*reinterpret_cast<const u32x4*>(p), bq[s], st[a]);
            }
        float mx = kNegBig;
#pragma unroll
        for (int a = 0; a < 2; ++a)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                st[a][r] = tb + 16 * a + 4 * hi + r < t1 ? st[a][r] * sc : -__builtin_inff();
                mx = fmaxf(mx, st[a][r]);
            }
        mx = fmaxf(mx, __shfl_xor(mx, 16));
        mx = fmaxf(mx, __shfl_xor(mx, 32));
        const float mn = fmaxf(m, mx);
        if (__any(mn > m)) {
            const float f = exp2_raw(m - mn);
            m = mn;
            l *= f;
#pragma unroll
            for (int w = 0; w < kWindows; ++w)
#pragma unroll
                for (int r = 0; r < 4; ++r) acc[w][r] *= f;
        }
        float p[2][4];
#pragma unroll
        for (int a = 0; a < 2; ++a)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                p[a][r] = exp2_raw(st[a][r] - mn);
                l += p[a][r];
            }
        const u32x4 pb = u32x4{Bf::pack2(p[0][0], p[0][1]), Bf::pack2(p[0][2], p[0][3]), Bf::pack2(p[1][0], p[1][1]),
                               Bf::pack2(p[1][2], p[1][3])};
#pragma unroll
        for (int w = 0; w < kWindows; ++w)
            acc[w] = Bf::mfma16(latent_operand<RL>(tile, part * kWindows + w, lane), pb, acc[w]);
        buf ^= 1;
    }
    l += __shfl_xor(l, 16);
    l += __shfl_xor(l, 32);
    if (h0 + lo >= heads) return;
    const int64_t row = (int64_t)b * heads + head;
    float* dst = splits > 1 ? partial + (row * splits + sp) * (rank + 4) : nullptr;
    if (dst && part == 0 && hi == 0) {
        dst[rank] = m;
        dst[rank + 1] = l;
    }
    const float inv = splits > 1 ? 1.f : 1.f / l;
#pragma unroll
    for (int w = 0; w < kWindows; ++w) {
        const int d = 16 * (part * kWindows + w) + 4 * hi;
        const float v[4] = {acc[w][0] * inv, acc[w][1] * inv, acc[w][2] * inv, acc[w][3] * inv};
        if (rank % 4 == 0) {
            if (d >= rank) continue;
            if (dst) store_vec<Fp, 4>(dst + d, v);
            else store_vec<Bf, 4>(out + row * rank + d, v);
        } else {
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                if (d + r >= rank) continue;
                if (dst) dst[d + r] = v[r];
                else Bf::store(out + row * rank + d + r, v[r]);
            }
        }
    }
}

// One workgroup per head; `splits` is at most 64, U of them are loaded together.
template <int U>
__global__ __launch_bounds__(512) void attn_merge_kernel(const float* __restrict__ partial, uint16_t* __restrict__ out,
                                                         int vdim, int splits) {
    __shared__ float s_share[64];
    const int64_t head = blockIdx.x;
    const float* p = partial + head * splits * (vdim + 4);
    if (threadIdx.x < 64) {
        const int s = min((int)threadIdx.x, splits - 1);           // lanes past the splits repeat the last
        const float m = p[s * (vdim + 4) + vdim], l = p[s * (vdim + 4) + vdim + 1];
        const float mm = wave_max(m), f = (int)threadIdx.x < splits ? exp2_raw(m - mm) : 0.f;
        s_share[threadIdx.x] = f / wave_sum(l * f);
    }
    __syncthreads();
    for (int d = threadIdx.x; d < vdim; d += blockDim.x) {
        float at = 0.f;
        for (int s0 = 0; s0 < splits; s0 += U) {
            float v[U];
#pragma unroll
            for (int u = 0; u < U; ++u) v[u] = p[min(s0 + u, splits - 1) * (vdim + 4) + d];
#pragma unroll
            for (int u = 0; u < U; ++u) at += v[u] * s_share[min(s0 + u, 63)];    // zero past the splits
        }
        Bf::store(out + head * vdim + d, at);
    }
}

void launch_merge(const void* partial, void* out, int64_t head_rows, int64_t vdim, int splits, void* stream) {
    const auto kernel = splits <= 4 ? attn_merge_kernel<4> : splits <= 8 ? attn_merge_kernel<8> : attn_merge_kernel<16>;
    kernel<<<dim3((unsigned)head_rows), dim3(vdim > 256 ? 512 : 256), 0, (hipStream_t)stream>>>(
        (const float*)partial, (uint16_t*)out, (int)vdim, splits);
}

// Whether the matrix-core forms take this problem: bf16, equal cache rows of a width they exist for.
bool matrix_form(int64_t k_row, int64_t v_row, int dtype) {
    return dtype == NQH_BF16 && k_row == v_row &&
           (k_row == 32 || k_row == 64 || k_row == 96 || k_row == 128 || k_row == 192 || k_row == 256);
}
constexpr int decode_waves(int row) { return row > 128 ? 2 : 4; }
int64_t most_keys(int64_t max_context, int64_t chunk, int64_t window) {
    const int64_t n = chunk > 0 ? std::min(chunk, max_context) : max_context;
    return window > 0 ? std::min(window, n) : n;
}
// Context splits: about 2048 waves on the chip, at least 512 keys a split (the merge is a launch of its own).
int decode_splits(int64_t batch, int64_t heads, int64_t kv_heads, int waves, int64_t longest) {
    const int64_t groups = batch * kv_heads * cdiv(heads / kv_heads, 16);
    const int64_t want = 2048 / std::max<int64_t>(1, groups * waves);
    return (int)std::max<int64_t>(1, std::min({want, longest / 512, (int64_t)64}));
}
#define NQH_WITH_ROW(row, ...)                        \
    do {                                              \
        switch (row) {                                \
            case 32: { constexpr int R = 32; __VA_ARGS__; } break;    \
            case 64: { constexpr int R = 64; __VA_ARGS__; } break;    \
            case 96: { constexpr int R = 96; __VA_ARGS__; } break;    \
            case 128: { constexpr int R = 128; __VA_ARGS__; } break;  \
            case 192: { constexpr int R = 192; __VA_ARGS__; } break;  \
            default: { constexpr int R = 256; __VA_ARGS__; } break;   \
        }                                             \
    } while (0)

int check_attention(const char* fn, const void* q, const void* k, const void* v, const int32_t* table, const void* out,
                    int64_t rows, int64_t heads, int64_t kv_heads, int64_t dim, int64_t vdim, int64_t k_row,
                    int64_t v_row, int64_t block_size, int64_t max_blocks, int64_t num_blocks, int64_t chunk, int64_t window,
                    int dtype) {
    if (!q || !k || !v || !table || !out) return fail(NQH_ERR_ARG, fn, "null pointer");
    if (!dtype_ok(dtype)) return fail(NQH_ERR_ARG, fn, "dtype must be NQH_BF16 or NQH_F32");
    if (rows <= 0 || heads <= 0 || kv_heads <= 0 || heads % kv_heads != 0 || dim <= 0 || vdim <= 0 || block_size <= 0 ||
        max_blocks <= 0 || num_blocks <= 0 || chunk < 0 || window < 0)
        return fail(NQH_ERR_ARG, fn, "sizes must be positive, heads a multiple of kv_heads, chunk and window >= 0");
    if (k_row < dim || v_row < vdim) return fail(NQH_ERR_ARG, fn, "cache rows are narrower than a head");
    if (dim > kMaxKeyDim || vdim > kMaxDim)
        return fail(NQH_ERR_UNSUPPORTED, fn, "head dims above %d (keys) or %d (values)", kMaxKeyDim, kMaxDim);
    if (block_size * max_blocks > kMaxI32 || num_blocks * kv_heads * block_size > kMaxI32 || chunk > kMaxI32 || window > kMaxI32 ||
        cdiv(rows * heads, 4) > kMaxI32)
        return fail(NQH_ERR_ARG, fn, "problem too large");
    return NQH_OK;
}

}  // namespace
}  // namespace nqh

using namespace nqh;

extern "C" int64_t nqh_attention_tile_rows(void) { return kTileRows; }

extern "C" int nqh_attention_prefill(const void* q, const void* k_cache, const void* v_cache, const int32_t* block_tables,
                                     const int32_t* segments, const int32_t* tiles, const void* sink, void* out,
                                     int64_t rows, int64_t num_tiles, int64_t heads, int64_t kv_heads, int64_t dim,
                                     int64_t vdim, int64_t k_row, int64_t v_row, int64_t block_size, int64_t max_blocks,
                                     int64_t num_blocks, int64_t chunk, int64_t window, float scale, int dtype,
                                     void* stream) {
    const char* fn = "nqh_attention_prefill";
    const int rc = check_attention(fn, q, k_cache, v_cache, block_tables, out, rows, heads, kv_heads, dim, vdim, k_row,
                                   v_row, block_size, max_blocks, num_blocks, chunk, window, dtype);
    if (rc != NQH_OK) return rc;
    if (!segments || !tiles) return fail(NQH_ERR_ARG, fn, "null pointer");
    const int64_t tile_groups = cdiv(kTileRows * heads, 4), groups = cdiv(num_tiles * heads, 8) * 8;
    if (num_tiles <= 0 || groups > kMaxI32 || num_tiles * tile_groups > kMaxI32)
        return fail(NQH_ERR_ARG, fn, "the number of tiles must be positive and the problem not too large");
    (void)hipGetLastError();
    if (matrix_form(k_row, v_row, dtype)) {
        if (!aligned(q, 16) || !aligned(k_cache, 16) || !aligned(v_cache, 16) || !aligned(out, 8))
            return fail(NQH_ERR_ARG, fn, "misaligned pointer");
        NQH_WITH_ROW(k_row, {
            constexpr int KT = R >= 192 ? 32 : 64;
            attn_tile_kernel<R, R, KT, false><<<dim3((unsigned)groups), dim3(256), 0, (hipStream_t)stream>>>(
                (const uint16_t*)q, (const uint16_t*)k_cache, (const uint16_t*)v_cache, block_tables, segments, tiles,
                (const uint16_t*)sink, DenseKV{}, (uint16_t*)out, (int)heads, (int)kv_heads, (int)vdim, (int)block_size,
                (int)max_blocks, (int)num_blocks, (int)chunk, (int)window, scale, (int)num_tiles);
        });
        return launched(fn);
    }
    NQH_WITH_TYPE(dtype, {
        using E = typename T::elem;
        attn_rows_kernel<T><<<dim3((unsigned)(num_tiles * tile_groups)), dim3(256), 0, (hipStream_t)stream>>>(
            (const E*)q, (const E*)k_cache, (const E*)v_cache, block_tables, nullptr, segments, tiles, (const E*)sink,
            (E*)out, 0, (int)tile_groups, (int)heads, (int)kv_heads, (int)dim, (int)vdim, (int)k_row, (int)v_row,
            (int)block_size, (int)max_blocks, (int)num_blocks, (int)chunk, (int)window, scale);
    });
    return launched(fn);
}

extern "C" size_t nqh_attention_decode_workspace_bytes(int64_t batch, int64_t heads, int64_t kv_heads, int64_t v_row,
                                                       int64_t max_context, int64_t chunk, int64_t window, int dtype) {
    if (batch <= 0 || heads <= 0 || kv_heads <= 0 || v_row <= 0 || !matrix_form(v_row, v_row, dtype)) return 0;
    const int splits = decode_splits(batch, heads, kv_heads, decode_waves((int)v_row), most_keys(max_context, chunk, window));
    return splits > 1 ? (size_t)(batch * heads * splits * (v_row + 4)) * sizeof(float) : 0;
}

extern "C" int nqh_attention_decode(const void* q, const void* k_cache, const void* v_cache, const int32_t* block_table,
                                    const int32_t* context_lens, const void* sink, void* out, int64_t batch,
                                    int64_t heads, int64_t kv_heads, int64_t dim, int64_t vdim, int64_t k_row, int64_t v_row,
                                    int64_t block_size, int64_t max_blocks, int64_t num_blocks, int64_t chunk, int64_t window,
                                    float scale, int dtype, void* workspace, size_t workspace_bytes, void* stream) {
    const char* fn = "nqh_attention_decode";
    const int rc = check_attention(fn, q, k_cache, v_cache, block_table, out, batch, heads, kv_heads, dim, vdim, k_row,
                                   v_row, block_size, max_blocks, num_blocks, chunk, window, dtype);
    if (rc != NQH_OK) return rc;
    if (!context_lens) return fail(NQH_ERR_ARG, fn, "null pointer");
    (void)hipGetLastError();
    if (matrix_form(k_row, v_row, dtype)) {
        if (!aligned(q, 16) || !aligned(k_cache, 16) || !aligned(v_cache, 16))
            return fail(NQH_ERR_ARG, fn, "misaligned pointer");
        const int64_t max_context = block_size * max_blocks, head_tiles = cdiv(heads / kv_heads, 16);
        const int splits = decode_splits(batch, heads, kv_heads, decode_waves((int)v_row), most_keys(max_context, chunk, window));
        const size_t need = splits > 1 ? (size_t)(batch * heads * splits * (vdim + 4)) * sizeof(float) : 0;
        if (need && (!workspace || workspace_bytes < need || !aligned(workspace, 16)))
            return fail(NQH_ERR_WORKSPACE, fn, "workspace of %zu bytes needed, %zu given", need, workspace ? workspace_bytes : 0);
        const int64_t groups = batch * kv_heads * head_tiles * splits;
        if (groups > kMaxI32 || batch * heads > kMaxI32) return fail(NQH_ERR_ARG, fn, "problem too large");
        NQH_WITH_ROW(k_row, {
            constexpr int WAVES = decode_waves(R);
            attn_decode_kernel<R, WAVES><<<dim3((unsigned)groups), dim3(64 * WAVES), 0, (hipStream_t)stream>>>(
                (const uint16_t*)q, (const uint16_t*)k_cache, (const uint16_t*)v_cache, block_table, context_lens,
                (const uint16_t*)sink, (uint16_t*)out, (float*)workspace, (int)heads, (int)kv_heads, (int)vdim, (int)block_size,
                (int)max_blocks, (int)num_blocks, (int)chunk, (int)window, scale, splits, (int)head_tiles);
        });
        if (splits > 1) launch_merge(workspace, out, batch * heads, vdim, splits, stream);
        return launched(fn);
    }
    NQH_WITH_TYPE(dtype, {
        using E = typename T::elem;
        attn_rows_kernel<T><<<dim3((unsigned)cdiv(batch * heads, 4)), dim3(256), 0, (hipStream_t)stream>>>(
            (const E*)q, (const E*)k_cache, (const E*)v_cache, block_table, context_lens, nullptr, nullptr,
            (const E*)sink, (E*)out, batch * heads, 1, (int)heads, (int)kv_heads, (int)dim, (int)vdim, (int)k_row, (int)v_row,
            (int)block_size, (int)max_blocks, (int)num_blocks, (int)chunk, (int)window, scale);
    });
    return launched(fn);
}

// ---- latent attention --------------------------------------------------------------------------------------------------
// Row layouts of the matrix-core decode form: RL latent elements, then the rotated part in 32 or 64.
#define NQH_WITH_LATENT(rl, rr, ...)                                                            \
    do {                                                                                        \
        if ((rl) == 64 && (rr) == 32) { constexpr int RL = 64, R = 96; __VA_ARGS__; }           \
        else if ((rl) == 64) { constexpr int RL = 64, R = 128; __VA_ARGS__; }                   \
        else if ((rl) == 128 && (rr) == 32) { constexpr int RL = 128, R = 160; __VA_ARGS__; }   \
        else if ((rl) == 128) { constexpr int RL = 128, R = 192; __VA_ARGS__; }                 \
        else if ((rl) == 256 && (rr) == 32) { constexpr int RL = 256, R = 288; __VA_ARGS__; }   \
        else if ((rl) == 256) { constexpr int RL = 256, R = 320; __VA_ARGS__; }                 \
        else if ((rr) == 32) { constexpr int RL = 512, R = 544; __VA_ARGS__; }                  \
        else { constexpr int RL = 512, R = 576; __VA_ARGS__; }                                  \
    } while (0)
// Heads per workgroup are 16 or 32.  Context splits: two workgroups per CU, at least two tiles of 32 keys each.
static int64_t latent_head_groups(int64_t heads) { return heads <= 16 ? 1 : cdiv(heads, 32); }
static int latent_splits(int64_t batch, int64_t heads, int64_t longest) {
    const int64_t want = 512 / std::max<int64_t>(1, batch * latent_head_groups(heads));
    return (int)std::max<int64_t>(1, std::min({want, longest / 64, (int64_t)64}));
}
static bool latent_matrix_form(int64_t rot_at, int64_t row, int dtype) {
    return dtype == NQH_BF16 && (rot_at == 64 || rot_at == 128 || rot_at == 256 || rot_at == 512) &&
           (row - rot_at == 32 || row - rot_at == 64);
}

extern "C" size_t nqh_latent_attention_decode_workspace_bytes(int64_t batch, int64_t heads, int64_t rank, int64_t rot_at,
                                                              int64_t row, int64_t max_context, int dtype) {
    if (batch <= 0 || heads <= 0 || rank <= 0 || !latent_matrix_form(rot_at, row, dtype)) return 0;
    const int splits = latent_splits(batch, heads, max_context);
    return splits > 1 ? (size_t)(batch * heads * splits * (rank + 4)) * sizeof(float) : 0;
}

extern "C" int nqh_latent_attention_decode(const void* q, const void* cache, const int32_t* block_table,
                                           const int32_t* context_lens, void* out, int64_t batch, int64_t heads, int64_t rank,
                                           int64_t rot_at, int64_t row, int64_t block_size, int64_t max_blocks,
                                           int64_t num_blocks, float scale, int dtype, void* workspace,
                                           size_t workspace_bytes, void* stream) {
    const char* fn = "nqh_latent_attention_decode";
    const int rc = check_attention(fn, q, cache, cache, block_table, out, batch, heads, 1, row, rank, row, row, block_size,
                                   max_blocks, num_blocks, 0, 0, dtype);
    if (rc != NQH_OK) return rc;
    if (!context_lens) return fail(NQH_ERR_ARG, fn, "null pointer");
    if (rot_at < rank || rot_at > row) return fail(NQH_ERR_ARG, fn, "the rotated part lies outside the row or in the latent");
    (void)hipGetLastError();
    if (!latent_matrix_form(rot_at, row, dtype)) {
        NQH_WITH_TYPE(dtype, {
            using E = typename T::elem;
            attn_rows_kernel<T><<<dim3((unsigned)cdiv(batch * heads, 4)), dim3(256), 0, (hipStream_t)stream>>>(
                (const E*)q, (const E*)cache, (const E*)cache, block_table, context_lens, nullptr, nullptr, (const E*)nullptr,
                (E*)out, batch * heads, 1, (int)heads, 1, (int)row, (int)rank, (int)row, (int)row, (int)block_size,
                (int)max_blocks, (int)num_blocks, 0, 0, scale);
        });
        return launched(fn);
    }
    if (!aligned(q, 16) || !aligned(cache, 16)) return fail(NQH_ERR_ARG, fn, "misaligned pointer");
    const int64_t head_groups = latent_head_groups(heads);
    const int splits = latent_splits(batch, heads, block_size * max_blocks);
    const size_t need = splits > 1 ? (size_t)(batch * heads * splits * (rank + 4)) * sizeof(float) : 0;
    if (need && (!workspace || workspace_bytes < need || !aligned(workspace, 16)))
        return fail(NQH_ERR_WORKSPACE, fn, "workspace of %zu bytes needed, %zu given", need, workspace ? workspace_bytes : 0);
    const int64_t groups = batch * head_groups * splits;
    if (groups > kMaxI32 || batch * heads > kMaxI32) return fail(NQH_ERR_ARG, fn, "problem too large");
    NQH_WITH_LATENT(rot_at, row - rot_at, {
        const auto kernel = heads <= 16 ? latent_decode_kernel<RL, R, 1> : latent_decode_kernel<RL, R, 2>;
        kernel<<<dim3((unsigned)groups), dim3(256), 0, (hipStream_t)stream>>>(
            (const uint16_t*)q, (const uint16_t*)cache, block_table, context_lens, (uint16_t*)out, (float*)workspace, (int)heads,
            (int)rank, (int)block_size, (int)max_blocks, (int)num_blocks, scale, splits, (int)head_groups);
    });
    if (splits > 1) launch_merge(workspace, out, batch * heads, rank, splits, stream);
    return launched(fn);
}

// Key rows of 64, 128, 192 or 256 elements and value rows of 64, 128 or 256 (not more than the keys').
static int64_t dense_row(int64_t n) { return n <= 64 ? 64 : n <= 128 ? 128 : n <= 192 ? 192 : 256; }

extern "C" int64_t nqh_latent_attention_prefill_query_row(int64_t dim, int64_t rot_dim, int64_t vdim, int dtype) {
    if (dtype != NQH_BF16 || dim <= 0 || rot_dim < 0 || vdim <= 0 || dim % 8 || rot_dim % 8 || vdim % 8) return 0;
    if (dim + rot_dim > 256 || vdim > 256) return 0;
    return std::max(dense_row(dim + rot_dim), vdim > 128 ? (int64_t)256 : dense_row(vdim));
}

extern "C" int nqh_latent_attention_prefill(const void* q, const void* kv, int64_t kv_stride, const void* rot,
                                            int64_t rot_stride, const int32_t* first, const int32_t* segments,
                                            const int32_t* tiles, void* out, int64_t rows, int64_t num_tiles, int64_t heads,
                                            int64_t dim, int64_t rot_dim, int64_t vdim, float scale, void* stream) {
    const char* fn = "nqh_latent_attention_prefill";
    if (!q || !kv || !rot || !first || !segments || !tiles || !out) return fail(NQH_ERR_ARG, fn, "null pointer");
    const int64_t row = nqh_latent_attention_prefill_query_row(dim, rot_dim, vdim, NQH_BF16);
    if (!row) return fail(NQH_ERR_UNSUPPORTED, fn, "head sizes must be multiples of 8, at most 256 for keys and values each");
    const int64_t groups = cdiv(num_tiles * heads, 8) * 8;
    if (rows <= 0 || heads <= 0 || num_tiles <= 0 || groups > kMaxI32 || kv_stride < heads * (dim + vdim) ||
        rot_stride < rot_dim || kv_stride % 8 || rot_stride % 8)
        return fail(NQH_ERR_ARG, fn, "sizes must be positive, row strides multiples of 8 and as wide as the rows");
    if (!aligned(q, 16) || !aligned(kv, 16) || !aligned(rot, 16) || !aligned(out, 8))
        return fail(NQH_ERR_ARG, fn, "misaligned pointer");
    const DenseKV dense{(const uint16_t*)kv, (const uint16_t*)rot, first, kv_stride, rot_stride, heads * dim, (int)dim, (int)rot_dim};
    (void)hipGetLastError();
#define NQH_GO(R, RV, KT)                                                                                                   \
    attn_tile_kernel<R, RV, KT, true><<<dim3((unsigned)groups), dim3(256), 0, (hipStream_t)stream>>>(                        \
        (const uint16_t*)q, nullptr, nullptr, nullptr, segments, tiles, nullptr, dense, (uint16_t*)out, (int)heads,          \
        (int)heads, (int)vdim, 1, 0, 0, 0, 0, scale, (int)num_tiles)
    if (row == 64) NQH_GO(64, 64, 64);
    else if (row == 128 && vdim <= 64) NQH_GO(128, 64, 64);
    else if (row == 128) NQH_GO(128, 128, 64);
    else if (row == 192 && vdim <= 64) NQH_GO(192, 64, 32);
    else if (row == 192) NQH_GO(192, 128, 64);
    else if (vdim <= 128) NQH_GO(256, 128, 32);
    else NQH_GO(256, 256, 32);
#undef NQH_GO
    return launched(fn);
}
