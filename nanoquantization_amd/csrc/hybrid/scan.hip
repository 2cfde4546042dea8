// Selective scan (Gu and Dao, "Mamba: Linear-Time Sequence Modeling with Selective State Spaces") with the short causal
// convolution in front of it.  Per channel c and state n:
//   S[c, n] = exp(dt_c A[c, n]) S[c, n] + dt_c x_c B_n,   y_c = (sum_n S[c, n] C_n + D_c x_c) silu(z_c),   A = -exp(A_log)
// The state lies [slot][n][channel], the convolution's last inputs [slot][taps - 1][channel], both fp32 and neither cleared:
// before position 0 both count as zero.
//   conv_silu_kernel      convolution and silu of a prompt pass
//   conv_step_kernel      of one token per sequence; moves the stored inputs on
//   scan_dt*_kernel       dt = softplus(W low + b)
//   scan_piece_kernel     the recurrence over a piece of a sequence: only its final state from zero, or the outputs
//   scan_chain_kernel     the states at the pieces' starts, from what the pieces contribute
//   scan_step_kernel      one token per sequence
// A piece decays a state by exp(A sum of dt) altogether, so the chain needs one number per channel and piece besides the
// contributions.
#include <algorithm>

#include "hybrid_common.hpp"

namespace nqh {
namespace {

constexpr int kMaxTaps = 16;
constexpr int kMinPiece = 32;          // not below kMaxTaps - 1: only a sequence's first piece reaches into the stored inputs
constexpr int kLaneStates = 16;        // states a lane holds in the prompt kernels
constexpr int kMaxState = 256;
constexpr int kTokens = 8;             // tokens whose operands are fetched together
constexpr float kLog2e = 1.4426950408889634f;

struct Piece {
    int first, rows, slot, fresh, index, count;      // as in the list of nqh_gla_prefill
};
__device__ __forceinline__ Piece load_piece_desc(const int32_t* pieces, int p) {
    const int32_t* d = pieces + 6 * (int64_t)p;
    return Piece{d[0], d[1], d[2], d[3], d[4], d[5]};
}

// ---- convolution -----------------------------------------------------------------------------------------------------
// x rows x_stride apart.  Workgroup: 256 * V channels of 8 tokens of a piece.
template <typename T, int V>
__global__ __launch_bounds__(256) void conv_silu_kernel(const typename T::elem* __restrict__ x, int64_t x_stride,
                                                        const typename T::elem* __restrict__ w,
                                                        const typename T::elem* __restrict__ bias,
                                                        const float* __restrict__ tail, const int32_t* __restrict__ pieces,
                                                        typename T::elem* __restrict__ out, int channels, int taps) {
    const Piece pc = load_piece_desc(pieces, blockIdx.y);
    const int c = (blockIdx.x * 256 + threadIdx.x) * V;
    if (c >= channels) return;
    const bool start = pc.index == 0;
    float b[V];
#pragma unroll
    for (int e = 0; e < V; ++e) b[e] = T::load(bias + c + e);
    for (int r0 = blockIdx.z * 8; r0 < min(pc.rows, (int)blockIdx.z * 8 + 8); ++r0) {
        float a[V];
#pragma unroll
        for (int e = 0; e < V; ++e) a[e] = b[e];
        for (int k = 0; k < taps; ++k) {
            const int at = r0 - (taps - 1) + k;
            float v[V];
            if (at >= 0 || !start) {
                load_vec<T, V>(x + (pc.first + at) * x_stride + c, v);
            } else if (pc.fresh) {
                continue;
            } else {
                const float* t = tail + ((int64_t)pc.slot * (taps - 1) + taps - 1 + at) * channels + c;
#pragma unroll
                for (int e = 0; e < V; ++e) v[e] = t[e];
            }
#pragma unroll
            for (int e = 0; e < V; ++e) a[e] += T::load(w + (int64_t)(c + e) * taps + k) * v[e];
        }
#pragma unroll
        for (int e = 0; e < V; ++e) a[e] = silu_quick(a[e]);
        store_vec<T, V>(out + (int64_t)(pc.first + r0) * channels + c, a);
    }
}

// Up to four taps: the weights and the rows that kConvRows tokens need are in registers before the first is used.
constexpr int kConvRows = 16;
// 16 bytes of a row as they lie in memory.
template <typename T>
struct Raw16;
template <>
struct Raw16<Bf> {
    using type = u32x4;
    static __device__ __forceinline__ float get(type v, int e) { return Bf::to_f32((uint16_t)(v[e >> 1] >> (16 * (e & 1)))); }
};
template <>
struct Raw16<Fp> {
    using type = f32x4;
    static __device__ __forceinline__ float get(type v, int e) { return v[e]; }
};

template <typename T, int V>
__global__ __launch_bounds__(256) void conv4_silu_kernel(const typename T::elem* __restrict__ x, int64_t x_stride,
                                                         const typename T::elem* __restrict__ w,
                                                         const typename T::elem* __restrict__ bias,
                                                         const float* __restrict__ tail, const int32_t* __restrict__ pieces,
                                                         typename T::elem* __restrict__ out, int channels, int taps) {
    const Piece pc = load_piece_desc(pieces, blockIdx.y);
    const int c = (blockIdx.x * 256 + threadIdx.x) * V, r0 = blockIdx.z * kConvRows;
    if (c >= channels || r0 >= pc.rows) return;
    using Raw = Raw16<T>;
    typename Raw::type v[kConvRows + 3];
    float ahead[3][V], wt[4][V], b[V];
#pragma unroll
    for (int j = 0; j < kConvRows + 3; ++j) {      // rows ahead of the sequence's tokens are replaced below
        const int at = min(r0 + j - 3, pc.rows - 1);
        v[j] = *reinterpret_cast<const typename Raw::type*>(x + (int64_t)max(pc.first + at, pc.index == 0 ? pc.first : 0) * x_stride + c);
    }
    load_vec<T, V>(bias + c, b);
#pragma unroll
    for (int k = 0; k < 4; ++k)                    // tap k of four; the missing ones in front are zero
#pragma unroll
        for (int e = 0; e < V; ++e) {
            const float f = T::load(w + (int64_t)(c + e) * taps + max(k - (4 - taps), 0));
            wt[k][e] = k >= 4 - taps ? f : 0.f;
        }
#pragma unroll
    for (int j = 0; j < 3; ++j)
#pragma unroll
        for (int e = 0; e < V; ++e) ahead[j][e] = Raw::get(v[j], e);
    if (r0 == 0 && pc.index == 0) {
#pragma unroll
        for (int j = 0; j < 3; ++j) {
            const int k = j - (4 - taps);          // place in the stored inputs
#pragma unroll
            for (int e = 0; e < V; ++e)
                ahead[j][e] = k < 0 || pc.fresh ? 0.f : tail[((int64_t)pc.slot * (taps - 1) + k) * channels + c + e];
        }
    }
#pragma unroll
    for (int j = 0; j < kConvRows; ++j) {
        float a[V];
#pragma unroll
        for (int e = 0; e < V; ++e) {
            const float now = Raw::get(v[j + 3], e);
            a[e] = b[e] + wt[0][e] * ahead[0][e] + wt[1][e] * ahead[1][e] + wt[2][e] * ahead[2][e] + wt[3][e] * now;
            ahead[0][e] = ahead[1][e];
            ahead[1][e] = ahead[2][e];
            ahead[2][e] = now;
            a[e] = silu_quick(a[e]);
        }
        if (r0 + j < pc.rows) store_vec<T, V>(out + (int64_t)(pc.first + r0 + j) * channels + c, a);
    }
}

template <typename T>
__global__ __launch_bounds__(256) void conv_step_kernel(const typename T::elem* __restrict__ x, int64_t x_stride,
                                                        const typename T::elem* __restrict__ w,
                                                        const typename T::elem* __restrict__ bias, float* __restrict__ tail,
                                                        const int32_t* __restrict__ slots, const int64_t* __restrict__ positions,
                                                        const uint8_t* __restrict__ active,
                                                        typename T::elem* __restrict__ out, int num_slots, int channels,
                                                        int taps) {
    const int row = blockIdx.y, c = blockIdx.x * 256 + threadIdx.x;
    if (c >= channels) return;
    const int slot = slots[row];
    const bool live = active[row] && slot >= 0 && slot < num_slots, fresh = positions[row] <= 0;
    const float now = T::load(x + row * x_stride + c);
    float a = T::load(bias + c) + T::load(w + (int64_t)c * taps + taps - 1) * now;
    float* t = tail + (int64_t)(live ? slot : 0) * (taps - 1) * channels + c;
    if (live) {
        for (int k = 0; k < taps - 1; ++k) {
            const float v = fresh ? 0.f : t[(int64_t)k * channels];
            a += T::load(w + (int64_t)c * taps + k) * v;
            if (k > 0) t[(int64_t)(k - 1) * channels] = v;
        }
        if (taps > 1) t[(int64_t)(taps - 2) * channels] = now;
    }
    T::store(out + (int64_t)row * channels + c, live ? silu_quick(a) : 0.f);
}

// ---- step sizes --------------------------------------------------------------------------------------------------------
// dt [rows, channels] fp32.  Matrix cores: the workgroup's four waves lie 2 x 2, a wave takes 16 CT channels of 16 RT rows and
// has the next step's operands in flight.
template <int CT, int RT>
__global__ __launch_bounds__(256) void scan_dt_kernel(const uint16_t* __restrict__ low, int64_t low_stride,
                                                      const uint16_t* __restrict__ w, const uint16_t* __restrict__ bias,
                                                      float* __restrict__ dt, int rows, int channels, int rank) {
    const int lane = threadIdx.x & 63, lo = lane & 15, hi = lane >> 4, wave = threadIdx.x >> 6;
    const int c0 = blockIdx.x * 32 * CT + (wave & 1) * 16 * CT;
    const int64_t r0 = (int64_t)blockIdx.y * 32 * RT + (wave >> 1) * 16 * RT;
    if (c0 >= channels || r0 >= rows) return;
    const uint16_t *wr[CT], *xr[RT];
    f32x4 acc[CT][RT];
#pragma unroll
    for (int i = 0; i < CT; ++i) wr[i] = w + (int64_t)min(c0 + 16 * i + lo, channels - 1) * rank;
#pragma unroll
    for (int m = 0; m < RT; ++m) {
        xr[m] = low + min(r0 + 16 * m + lo, (int64_t)rows - 1) * low_stride;
#pragma unroll
        for (int i = 0; i < CT; ++i) acc[i][m] = f32x4{0.f, 0.f, 0.f, 0.f};
    }
    u32x4 a[2][CT], b[2][RT];
    auto load = [&](u32x4 (&as)[CT], u32x4 (&bs)[RT], int k0) {
        const int k = k0 + 8 * hi, kc = min(k, rank - 8);
#pragma unroll
        for (int i = 0; i < CT; ++i) as[i] = *reinterpret_cast<const u32x4*>(wr[i] + kc);
#pragma unroll
        for (int m = 0; m < RT; ++m) bs[m] = *reinterpret_cast<const u32x4*>(xr[m] + kc);
    };
    auto multiply = [&](const u32x4 (&as)[CT], u32x4 (&bs)[RT], int k0) {
        if (k0 + 32 > rank) {                                     // the weights repeat past the end, the inputs are zero
#pragma unroll
            for (int m = 0; m < RT; ++m)
                if (k0 + 8 * hi >= rank) bs[m] = u32x4{0u, 0u, 0u, 0u};
        }
#pragma unroll
        for (int i = 0; i < CT; ++i)
#pragma unroll
            for (int m = 0; m < RT; ++m) acc[i][m] = Bf::mfma16(as[i], bs[m], acc[i][m]);
    };
    load(a[0], b[0], 0);
    for (int k0 = 0; k0 < rank; k0 += 64) {
        if (k0 + 32 < rank) load(a[1], b[1], k0 + 32);
        multiply(a[0], b[0], k0);
        if (k0 + 64 < rank) load(a[0], b[0], k0 + 64);
        if (k0 + 32 < rank) multiply(a[1], b[1], k0 + 32);
    }
#pragma unroll
    for (int i = 0; i < CT; ++i) {
        const int c = c0 + 16 * i + 4 * hi;
        float bv[4];
#pragma unroll
        for (int e = 0; e < 4; ++e) bv[e] = Bf::to_f32(bias[min(c + e, channels - 1)]);
#pragma unroll
        for (int m = 0; m < RT; ++m) {
            const int64_t r = r0 + 16 * m + lo;
            if (r >= rows) continue;
            float v[4];
#pragma unroll
            for (int e = 0; e < 4; ++e) v[e] = softplus_f32(acc[i][m][e] + bv[e]);
            float* dst = dt + r * channels + c;
            if (channels % 4 == 0) {
                if (c < channels) store_vec<Fp, 4>(dst, v);
            } else {
#pragma unroll
                for (int e = 0; e < 4; ++e)
                    if (c + e < channels) dst[e] = v[e];
            }
        }
    }
}

// The same for passes of many rows: 128 channels x 128 rows, operands through LDS in stages of 64 contraction elements,
// double-buffered.  LDS rows are 128 bytes; 16-byte piece p of row r lies at position (p + r / 2) % 8, so that the 16 rows of
// an operand read fall on different banks.
#define NQH_GPTR(p) ((__attribute__((address_space(1))) void*)(p))
#define NQH_LPTR(p) ((__attribute__((address_space(3))) void*)(p))
__device__ const u32x4 g_zero_piece = {0u, 0u, 0u, 0u};   // what lies past the end of a row

__global__ __launch_bounds__(256) void scan_dt_tile_kernel(const uint16_t* __restrict__ low, int64_t low_stride,
                                                           const uint16_t* __restrict__ w, const uint16_t* __restrict__ bias,
                                                           float* __restrict__ dt, int rows, int channels, int rank) {
    constexpr int kTile = 128 * 128;                     // bytes of one operand's stage
    __shared__ __attribute__((aligned(1024))) unsigned char s_mem[4 * kTile];      // [buffer][weights | rows]
    const int lane = threadIdx.x & 63, lo = lane & 15, hi = lane >> 4;
    const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int c0 = blockIdx.x * 128, wc = (wave & 1) * 64, wr = (wave >> 1) * 64;
    const int64_t r0 = (int64_t)blockIdx.y * 128;
    const uint16_t *w_src[4], *x_src[4];
    int k_src[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const int n = (i * 4 + wave) * 64 + lane, row = n >> 3;
        k_src[i] = 8 * (((n & 7) - (row >> 1)) & 7);
        w_src[i] = w + (int64_t)min(c0 + row, channels - 1) * rank;
        x_src[i] = low + min(r0 + row, (int64_t)rows - 1) * low_stride;
    }
    auto stage = [&](int k0, int buf) {
        unsigned char* base = s_mem + buf * 2 * kTile + wave * 1024;
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int k = k0 + k_src[i];
            const void* a = k < rank ? (const void*)(w_src[i] + k) : (const void*)&g_zero_piece;
            const void* b = k < rank ? (const void*)(x_src[i] + k) : (const void*)&g_zero_piece;
            __builtin_amdgcn_global_load_lds(NQH_GPTR(a), NQH_LPTR(base + i * 4096), 16, 0, 0);
            __builtin_amdgcn_global_load_lds(NQH_GPTR(b), NQH_LPTR(base + kTile + i * 4096), 16, 0, 0);
        }
    };
    f32x4 acc[4][4];
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int m = 0; m < 4; ++m) acc[i][m] = f32x4{0.f, 0.f, 0.f, 0.f};
    stage(0, 0);
    int buf = 0;
    for (int k0 = 0; k0 < rank; k0 += 64) {
        __builtin_amdgcn_s_waitcnt(0x0F70);              // this wave's part of the stage has landed
        __syncthreads();
        if (k0 + 64 < rank) stage(k0 + 64, buf ^ 1);
        const unsigned char* base = s_mem + buf * 2 * kTile;
#pragma unroll
        for (int s = 0; s < 2; ++s) {
            u32x4 a[4], b[4];
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int ra = wc + 16 * i + lo, rb = wr + 16 * i + lo;
                a[i] = *reinterpret_cast<const u32x4*>(base + ra * 128 + ((4 * s + hi + (ra >> 1)) & 7) * 16);
                b[i] = *reinterpret_cast<const u32x4*>(base + kTile + rb * 128 + ((4 * s + hi + (rb >> 1)) & 7) * 16);
            }
#pragma unroll
            for (int i = 0; i < 4; ++i)
#pragma unroll
                for (int m = 0; m < 4; ++m) acc[i][m] = Bf::mfma16(a[i], b[m], acc[i][m]);
        }
        buf ^= 1;
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const int c = c0 + wc + 16 * i + 4 * hi;
        float bv[4];
#pragma unroll
        for (int e = 0; e < 4; ++e) bv[e] = Bf::to_f32(bias[min(c + e, channels - 1)]);
#pragma unroll
        for (int m = 0; m < 4; ++m) {
            const int64_t r = r0 + wr + 16 * m + lo;
            if (r >= rows || c >= channels) continue;
            float v[4];
#pragma unroll
            for (int e = 0; e < 4; ++e) v[e] = softplus_f32(acc[i][m][e] + bv[e]);
            store_vec<Fp, 4>(dt + r * channels + c, v);  // the number of channels is a multiple of 4
        }
    }
}

template <typename T>
__global__ __launch_bounds__(256) void scan_dt_any_kernel(const typename T::elem* __restrict__ low, int64_t low_stride,
                                                          const typename T::elem* __restrict__ w,
                                                          const typename T::elem* __restrict__ bias, float* __restrict__ dt,
                                                          int channels, int rank) {
    const int c = blockIdx.x * 256 + threadIdx.x;
    const int64_t r = blockIdx.y;
    if (c >= channels) return;
    float a = 0.f;
    for (int k = 0; k < rank; ++k) a += T::load(low + r * low_stride + k) * T::load(w + (int64_t)c * rank + k);
    dt[r * channels + c] = softplus_f32(a + T::load(bias + c));
}

// ---- the recurrence over a piece -----------------------------------------------------------------------------------------
// LPC lanes per channel, kLaneStates states each; 256 / LPC channels per workgroup.
template <typename T, int LPC, bool OUT>
__global__ __launch_bounds__(256) void scan_piece_kernel(
    const typename T::elem* __restrict__ x, const float* __restrict__ dt, const typename T::elem* __restrict__ bc,
    int64_t bc_stride, const typename T::elem* __restrict__ z, int64_t z_stride, const typename T::elem* __restrict__ a_log,
    const typename T::elem* __restrict__ d_skip, const typename T::elem* __restrict__ conv_in, int64_t conv_stride,
    float* __restrict__ state, float* __restrict__ tail, float* __restrict__ ws_state, float* __restrict__ ws_dt,
    const int32_t* __restrict__ pieces, typename T::elem* __restrict__ out, int channels, int states, int taps) {
    constexpr int CPG = 256 / LPC, NP = LPC * kLaneStates;
    __shared__ __attribute__((aligned(16))) float s_bc[2][kTokens][2][NP];
    const Piece pc = load_piece_desc(pieces, blockIdx.y);
    if (!OUT && pc.index == pc.count - 1) return;                 // nobody follows it
    const int sub = threadIdx.x % LPC, n0 = sub * kLaneStates;
    const int cw = blockIdx.x * CPG + threadIdx.x / LPC, c = min(cw, channels - 1);
    const bool live = cw < channels;
    float S[kLaneStates], A[kLaneStates];
    // of several pieces the first too: the last one overwrites the slot
    const float* init = pc.count > 1 ? ws_state + (int64_t)blockIdx.y * states * channels
                                     : (pc.fresh ? nullptr : state + (int64_t)pc.slot * states * channels);
#pragma unroll
    for (int i = 0; i < kLaneStates; ++i) {
        const int n = n0 + i, nc = min(n, states - 1);
        A[i] = n < states ? -expf(T::load(a_log + (int64_t)c * states + nc)) * kLog2e : 0.f;
        S[i] = OUT && init && n < states ? init[(int64_t)nc * channels + c] : 0.f;
    }
    const float D = OUT ? T::load(d_skip + c) : 0.f;
    float dt_sum = 0.f;
    float xv[kTokens], dv[kTokens], zv[kTokens];
    const int last = pc.rows - 1;
    auto fetch = [&](int t0) {
#pragma unroll
        for (int u = 0; u < kTokens; ++u) {
            const int64_t r = pc.first + min(t0 + u, last);
            xv[u] = T::load(x + r * channels + c);
            dv[u] = dt[r * channels + c];
            if constexpr (OUT) zv[u] = T::load(z + r * z_stride + c);
        }
    };
    constexpr int kBc = (kTokens * 2 * NP + 255) / 256;
    float bcv[kBc];
    auto fetch_bc = [&](int t0) {
#pragma unroll
        for (int j = 0; j < kBc; ++j) {
            const int i = j * 256 + threadIdx.x, u = min(i / (2 * NP), kTokens - 1), which = i / NP % 2, n = i % NP;
            const int64_t r = pc.first + min(t0 + u, last);
            const float v = T::load(bc + r * bc_stride + which * states + min(n, states - 1));
            bcv[j] = n < states ? v : 0.f;
        }
    };
    auto put_bc = [&](int buf) {
#pragma unroll
        for (int j = 0; j < kBc; ++j) {
            const int i = j * 256 + threadIdx.x;
            if (kTokens * 2 * NP % 256 == 0 || i < kTokens * 2 * NP) (&s_bc[buf][0][0][0])[i] = bcv[j];
        }
    };
    fetch_bc(0);
    fetch(0);
    int buf = 0;
    for (int t0 = 0; t0 < pc.rows; t0 += kTokens) {
        put_bc(buf);
        __syncthreads();
        float xc[kTokens], dc[kTokens], zc[kTokens];
#pragma unroll
        for (int u = 0; u < kTokens; ++u) {
            xc[u] = xv[u];
            dc[u] = t0 + u <= last ? dv[u] : 0.f;                 // a step of size zero changes nothing
            if constexpr (OUT) zc[u] = zv[u];
        }
        if (t0 + kTokens < pc.rows) {
            fetch_bc(t0 + kTokens);
            fetch(t0 + kTokens);
        }
#pragma unroll
        for (int u = 0; u < kTokens; ++u) {
            const float d = dc[u], dx = d * xc[u];
            dt_sum += d;
            float y = 0.f;
#pragma unroll
            for (int i = 0; i < kLaneStates; i += 4) {
                const f32x4 b = *reinterpret_cast<const f32x4*>(&s_bc[buf][u][0][n0 + i]);
                f32x4 cc = f32x4{0.f, 0.f, 0.f, 0.f};
                if constexpr (OUT) cc = *reinterpret_cast<const f32x4*>(&s_bc[buf][u][1][n0 + i]);
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    S[i + e] = __builtin_amdgcn_exp2f(d * A[i + e]) * S[i + e] + dx * b[e];
                    if constexpr (OUT) y += S[i + e] * cc[e];
                }
            }
            if constexpr (OUT) {
#pragma unroll
                for (int o = 1; o < LPC; o <<= 1) y += __shfl_xor(y, o);
                if (sub == 0 && live && t0 + u <= last)
                    T::store(out + (int64_t)(pc.first + t0 + u) * channels + c, (y + D * xc[u]) * silu_quick(zc[u]));
            }
        }
        buf ^= 1;
    }
    if (!live) return;
    if constexpr (OUT) {
        if (pc.index != pc.count - 1) return;
        float* dst = state + (int64_t)pc.slot * states * channels;
#pragma unroll
        for (int i = 0; i < kLaneStates; ++i)
            if (n0 + i < states) dst[(int64_t)(n0 + i) * channels + c] = S[i];
        if (sub != 0) return;
        // the convolution's inputs of the sequence's last tokens; rows of earlier pieces lie ahead of this one's
        const int have = pc.index > 0 ? taps - 1 : min(pc.rows, taps - 1), keep = taps - 1 - have;
        float* t = tail + (int64_t)pc.slot * (taps - 1) * channels + c;
        for (int k = 0; k < taps - 1; ++k) {
            float v;
            if (k < keep) v = pc.fresh ? 0.f : t[(int64_t)(k + have) * channels];
            else v = T::load(conv_in + (int64_t)(pc.first + pc.rows - (taps - 1) + k) * conv_stride + c);
            t[(int64_t)k * channels] = v;
        }
    } else {
        float* dst = ws_state + ((int64_t)blockIdx.y + 1) * states * channels;   // where the next piece starts from
#pragma unroll
        for (int i = 0; i < kLaneStates; ++i)
            if (n0 + i < states) dst[(int64_t)(n0 + i) * channels + c] = S[i];
        if (sub == 0) ws_dt[(int64_t)blockIdx.y * channels + c] = dt_sum;
    }
}

// ws_state[p] holds what the piece before p contributes (nothing for a first one) and receives the state in front of p.
template <typename T>
__global__ __launch_bounds__(256) void scan_chain_kernel(const float* __restrict__ state, float* __restrict__ ws_state,
                                                         const float* __restrict__ ws_dt,
                                                         const typename T::elem* __restrict__ a_log,
                                                         const int32_t* __restrict__ pieces, int channels, int states) {
    const Piece pc = load_piece_desc(pieces, blockIdx.z);
    const int c = blockIdx.x * 256 + threadIdx.x, n = blockIdx.y;
    if (pc.index != 0 || pc.count < 2 || c >= channels) return;
    const int64_t at = (int64_t)n * channels + c, size = (int64_t)states * channels;
    const float A = -expf(T::load(a_log + (int64_t)c * states + n)) * kLog2e;
    float S = pc.fresh ? 0.f : state[pc.slot * size + at];
    const int64_t p0 = blockIdx.z;
    ws_state[p0 * size + at] = S;
    for (int p = 0; p < pc.count - 1; p += 8) {          // eight pieces' operands in flight
        float d[8], v[8];
#pragma unroll
        for (int u = 0; u < 8; ++u) {
            const int64_t q = p0 + min(p + u, pc.count - 2);
            d[u] = ws_dt[q * channels + c];
            v[u] = ws_state[(q + 1) * size + at];
        }
#pragma unroll
        for (int u = 0; u < 8; ++u) {
            if (p + u >= pc.count - 1) break;
            S = __builtin_amdgcn_exp2f(A * d[u]) * S + v[u];
            ws_state[(p0 + p + u + 1) * size + at] = S;
        }
    }
}

// ---- one token per sequence ------------------------------------------------------------------------------------------------
// Workgroup: 64 channels of ROWS rows; its four waves share the states.
template <typename T, int ROWS>
__global__ __launch_bounds__(256) void scan_step_kernel(
    const typename T::elem* __restrict__ x, const float* __restrict__ dt, const typename T::elem* __restrict__ bc,
    int64_t bc_stride, const typename T::elem* __restrict__ z, int64_t z_stride, const typename T::elem* __restrict__ a_log,
    const typename T::elem* __restrict__ d_skip, float* __restrict__ state, const int32_t* __restrict__ slots,
    const int64_t* __restrict__ positions, const uint8_t* __restrict__ active, typename T::elem* __restrict__ out, int batch,
    int num_slots, int channels, int states) {
    __shared__ float s_y[4][ROWS][64];
    const int row0 = blockIdx.y * ROWS, lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int cw = blockIdx.x * 64 + lane, c = min(cw, channels - 1);
    const int64_t size = (int64_t)states * channels;
    int slot[ROWS];
    bool ok[ROWS], fresh[ROWS];
    float d[ROWS], dx[ROWS], y[ROWS];
#pragma unroll
    for (int r = 0; r < ROWS; ++r) {
        const int row = min(row0 + r, batch - 1);
        slot[r] = slots[row];
        ok[r] = row0 + r < batch && active[row] && slot[r] >= 0 && slot[r] < num_slots;
        fresh[r] = positions[row] <= 0;
        slot[r] = ok[r] ? slot[r] : 0;
        d[r] = dt[(int64_t)row * channels + c];
        dx[r] = d[r] * T::load(x + (int64_t)row * channels + c);
        y[r] = 0.f;
    }
    for (int n0 = wave; n0 < states; n0 += 16) {              // four of this wave's states of every row in flight
        float s[ROWS][4], a[4];
#pragma unroll
        for (int u = 0; u < 4; ++u) {
            const int n = min(n0 + 4 * u, states - 1);
            a[u] = T::load(a_log + (int64_t)c * states + n);
#pragma unroll
            for (int r = 0; r < ROWS; ++r) s[r][u] = state[slot[r] * size + (int64_t)n * channels + c];
        }
#pragma unroll
        for (int u = 0; u < 4; ++u) {
            const int n = n0 + 4 * u;
            if (n >= states) break;
            const float A = -expf(a[u]) * kLog2e;
#pragma unroll
            for (int r = 0; r < ROWS; ++r) {
                const typename T::elem* B = bc + min(row0 + r, batch - 1) * bc_stride;
                const float v = __builtin_amdgcn_exp2f(d[r] * A) * (fresh[r] ? 0.f : s[r][u]) + dx[r] * T::load(B + n);
                y[r] += v * T::load(B + states + n);
                if (ok[r] && cw < channels) state[slot[r] * size + (int64_t)n * channels + c] = v;
            }
        }
    }
#pragma unroll
    for (int r = 0; r < ROWS; ++r) s_y[wave][r][lane] = y[r];
    __syncthreads();
    for (int r = wave; r < ROWS; r += 4) {
        const int64_t row = row0 + r;
        if (row >= batch || cw >= channels) continue;
        const bool live = active[row] && slots[row] >= 0 && slots[row] < num_slots;
        const float v = s_y[0][r][lane] + s_y[1][r][lane] + s_y[2][r][lane] + s_y[3][r][lane] +
                        T::load(d_skip + c) * T::load(x + row * channels + c);
        T::store(out + row * channels + c, live ? v * silu_quick(T::load(z + row * z_stride + c)) : 0.f);
    }
}

int lanes_per_channel(int64_t states) {
    int l = 1;
    while (l * kLaneStates < states) l *= 2;
    return l;
}
int check_scan(const char* fn, int64_t channels, int64_t states, int64_t taps, int dtype) {
    if (!dtype_ok(dtype)) return fail(NQH_ERR_ARG, fn, "dtype must be NQH_BF16 or NQH_F32");
    if (channels <= 0 || channels > kMaxI32 - 256 || states <= 0 || taps <= 0)
        return fail(NQH_ERR_ARG, fn, "sizes must be positive 31-bit counts");
    if (states > kMaxState || taps > kMaxTaps)
        return fail(NQH_ERR_UNSUPPORTED, fn, "at most %d states per channel and %d taps", kMaxState, kMaxTaps);
    return NQH_OK;
}

}  // namespace
}  // namespace nqh

using namespace nqh;

extern "C" int64_t nqh_scan_piece_rows(int64_t rows, int64_t channels, int64_t states) {
    // Four workgroups per CU keep the vector ALU busy; more pieces than that only cost, each but a sequence's last runs twice.
    const int64_t groups = cdiv(channels, 256 / lanes_per_channel(states));
    const int64_t size = std::max<int64_t>(kMinPiece, cdiv(cdiv(rows * groups, 1024), 32) * 32);
    return size;
}
extern "C" size_t nqh_scan_workspace_bytes(int64_t num_pieces, int64_t channels, int64_t states) {
    if (num_pieces <= 0 || channels <= 0 || states <= 0) return 0;
    return (size_t)(num_pieces * channels * (states + 1)) * sizeof(float);
}

extern "C" int nqh_conv_silu(const void* x, int64_t x_stride, const void* weight, const void* bias, const float* tail,
                             const int32_t* pieces, int64_t num_pieces, int64_t longest, void* out, int64_t channels,
                             int64_t taps, int dtype, void* stream) {
    const char* fn = "nqh_conv_silu";
    const int rc = check_scan(fn, channels, 1, taps, dtype);
    if (rc != NQH_OK) return rc;
    if (!x || !weight || !bias || (!tail && taps > 1) || !pieces || !out) return fail(NQH_ERR_ARG, fn, "null pointer");
    if (num_pieces <= 0 || num_pieces > 65535 || longest <= 0 || cdiv(longest, 8) > 65535 || x_stride < channels)
        return fail(NQH_ERR_ARG, fn, "1 to 65535 pieces, and x rows at least as wide as the channels");
    (void)hipGetLastError();
#define NQH_GO(KERNEL, V, ROWS)                                                                                            \
    KERNEL<T, V><<<dim3((unsigned)cdiv(channels, 256 * V), (unsigned)num_pieces, (unsigned)cdiv(longest, ROWS)), dim3(256), 0, \
                   (hipStream_t)stream>>>((const E*)x, x_stride, (const E*)weight, (const E*)bias, tail, pieces, (E*)out,   \
                                          (int)channels, (int)taps)
    NQH_WITH_TYPE(dtype, {
        using E = typename T::elem;
        constexpr int V = 16 / sizeof(E);
        const bool vec = channels % V == 0 && x_stride % V == 0 && aligned(x, 16) && aligned(bias, 16) && aligned(out, 16);
        if (taps <= 4 && vec) NQH_GO(conv4_silu_kernel, V, kConvRows);
        else if (vec) NQH_GO(conv_silu_kernel, V, 8);
        else NQH_GO(conv_silu_kernel, 1, 8);
    });
#undef NQH_GO
    return launched(fn);
}

extern "C" int nqh_conv_step(const void* x, int64_t x_stride, const void* weight, const void* bias, float* tail,
                             const int32_t* state_slots, const int64_t* positions, const uint8_t* active, void* out,
                             int64_t batch, int64_t num_slots, int64_t channels, int64_t taps, int dtype, void* stream) {
    const char* fn = "nqh_conv_step";
    const int rc = check_scan(fn, channels, 1, taps, dtype);
    if (rc != NQH_OK) return rc;
    if (!x || !weight || !bias || (!tail && taps > 1) || !state_slots || !positions || !active || !out)
        return fail(NQH_ERR_ARG, fn, "null pointer");
    if (batch <= 0 || batch > 65535 || num_slots <= 0 || num_slots > kMaxI32 || x_stride < channels)
        return fail(NQH_ERR_ARG, fn, "1 to 65535 rows at least as wide as the channels, and some slots");
    (void)hipGetLastError();
    NQH_WITH_TYPE(dtype, {
        using E = typename T::elem;
        conv_step_kernel<T><<<dim3((unsigned)cdiv(channels, 256), (unsigned)batch), dim3(256), 0, (hipStream_t)stream>>>(
            (const E*)x, x_stride, (const E*)weight, (const E*)bias, tail, state_slots, positions, active, (E*)out,
            (int)num_slots, (int)channels, (int)taps);
    });
    return launched(fn);
}

extern "C" int nqh_scan_dt(const void* low, int64_t low_stride, const void* weight, const void* bias, float* dt, int64_t rows,
                           int64_t channels, int64_t rank, int dtype, void* stream) {
    const char* fn = "nqh_scan_dt";
    const int rc = check_scan(fn, channels, 1, 1, dtype);
    if (rc != NQH_OK) return rc;
    if (!low || !weight || !bias || !dt) return fail(NQH_ERR_ARG, fn, "null pointer");
    if (rows <= 0 || rows > kMaxI32 - 64 || rank <= 0 || rank > kMaxI32 || low_stride < rank)
        return fail(NQH_ERR_ARG, fn, "sizes must be positive 31-bit counts and the rows as wide as the rank");
    const bool matrix = dtype == NQH_BF16 && rank % 8 == 0 && low_stride % 8 == 0 && aligned(low, 16) && aligned(weight, 16) &&
                        aligned(dt, 16);
    if (cdiv(rows, 128) > 65535 || (!matrix && rows > 65535)) return fail(NQH_ERR_UNSUPPORTED, fn, "too many rows");
    (void)hipGetLastError();
    if (matrix) {
#define NQH_GO(CT, RT)                                                                                                    \
    scan_dt_kernel<CT, RT><<<dim3((unsigned)cdiv(channels, 32 * CT), (unsigned)cdiv(rows, 32 * RT)), dim3(256), 0,         \
                             (hipStream_t)stream>>>((const uint16_t*)low, low_stride, (const uint16_t*)weight,             \
                                                    (const uint16_t*)bias, dt, (int)rows, (int)channels, (int)rank)
        if (rows <= 64) NQH_GO(1, 1);
        else if (channels % 4 != 0 || rows < 512) NQH_GO(2, 4);
        else
            scan_dt_tile_kernel<<<dim3((unsigned)cdiv(channels, 128), (unsigned)cdiv(rows, 128)), dim3(256), 0,
                                  (hipStream_t)stream>>>((const uint16_t*)low, low_stride, (const uint16_t*)weight,
                                                         (const uint16_t*)bias, dt, (int)rows, (int)channels, (int)rank);
#undef NQH_GO
        return launched(fn);
    }
    NQH_WITH_TYPE(dtype, {
        using E = typename T::elem;
        scan_dt_any_kernel<T><<<dim3((unsigned)cdiv(channels, 256), (unsigned)rows), dim3(256), 0, (hipStream_t)stream>>>(
            (const E*)low, low_stride, (const E*)weight, (const E*)bias, dt, (int)channels, (int)rank);
    });
    return launched(fn);
}

extern "C" int nqh_scan_prefill(const void* x, const float* dt, const void* bc, int64_t bc_stride, const void* z,
                                int64_t z_stride, const void* a_log, const void* d_skip, const void* conv_in,
                                int64_t conv_stride, float* state, float* tail, const int32_t* pieces, int64_t num_pieces,
                                int chained, void* out, int64_t channels, int64_t states, int64_t taps, int dtype,
                                void* workspace, size_t workspace_bytes, void* stream) {
    const char* fn = "nqh_scan_prefill";
    const int rc = check_scan(fn, channels, states, taps, dtype);
    if (rc != NQH_OK) return rc;
    if (!x || !dt || !bc || !z || !a_log || !d_skip || !conv_in || !state || (!tail && taps > 1) || !pieces || !out)
        return fail(NQH_ERR_ARG, fn, "null pointer");
    if (num_pieces <= 0 || num_pieces > 65535 || bc_stride < 2 * states || z_stride < channels || conv_stride < channels)
        return fail(NQH_ERR_ARG, fn, "1 to 65535 pieces, and rows at least as wide as what they hold");
    const size_t need = chained ? nqh_scan_workspace_bytes(num_pieces, channels, states) : 0;
    if (need && (!workspace || workspace_bytes < need || !aligned(workspace, 4)))
        return fail(NQH_ERR_WORKSPACE, fn, "workspace of %zu bytes needed, %zu given", need, workspace ? workspace_bytes : 0);
    float* ws_state = (float*)workspace;
    float* ws_dt = chained ? ws_state + num_pieces * channels * states : nullptr;
    const int lpc = lanes_per_channel(states);
    const dim3 grid((unsigned)cdiv(channels, 256 / lpc), (unsigned)num_pieces);
    (void)hipGetLastError();
#define NQH_RUN(LPC, OUT)                                                                                                  \
    scan_piece_kernel<T, LPC, OUT><<<grid, dim3(256), 0, (hipStream_t)stream>>>(                                           \
        (const E*)x, dt, (const E*)bc, bc_stride, (const E*)z, z_stride, (const E*)a_log, (const E*)d_skip,                \
        (const E*)conv_in, conv_stride, state, tail, ws_state, ws_dt, pieces, (E*)out, (int)channels, (int)states, (int)taps)
#define NQH_LANES(OUT)                   \
    do {                                 \
        if (lpc == 1) NQH_RUN(1, OUT);   \
        else if (lpc == 2) NQH_RUN(2, OUT); \
        else if (lpc == 4) NQH_RUN(4, OUT); \
        else if (lpc == 8) NQH_RUN(8, OUT); \
        else NQH_RUN(16, OUT);           \
    } while (0)
    NQH_WITH_TYPE(dtype, {
        using E = typename T::elem;
        if (chained) {
            NQH_LANES(false);
            scan_chain_kernel<T><<<dim3((unsigned)cdiv(channels, 256), (unsigned)states, (unsigned)num_pieces), dim3(256), 0,
                                   (hipStream_t)stream>>>(state, ws_state, ws_dt, (const E*)a_log, pieces, (int)channels,
                                                          (int)states);
        }
        NQH_LANES(true);
    });
#undef NQH_LANES
#undef NQH_RUN
    return launched(fn);
}

extern "C" int nqh_scan_step(const void* x, const float* dt, const void* bc, int64_t bc_stride, const void* z, int64_t z_stride,
                             const void* a_log, const void* d_skip, float* state, const int32_t* state_slots,
                             const int64_t* positions, const uint8_t* active, void* out, int64_t batch, int64_t num_slots,
                             int64_t channels, int64_t states, int dtype, void* stream) {
    const char* fn = "nqh_scan_step";
    const int rc = check_scan(fn, channels, states, 1, dtype);
    if (rc != NQH_OK) return rc;
    if (!x || !dt || !bc || !z || !a_log || !d_skip || !state || !state_slots || !positions || !active || !out)
        return fail(NQH_ERR_ARG, fn, "null pointer");
    if (batch <= 0 || batch > 65535 || num_slots <= 0 || num_slots > kMaxI32 || bc_stride < 2 * states || z_stride < channels)
        return fail(NQH_ERR_ARG, fn, "1 to 65535 rows at least as wide as what they hold, and some slots");
    (void)hipGetLastError();
    NQH_WITH_TYPE(dtype, {
        using E = typename T::elem;
        const int rows = batch >= 32 ? 4 : 1;                 // several rows share the exponentials of a_log
        const auto kernel = rows == 4 ? scan_step_kernel<T, 4> : scan_step_kernel<T, 1>;
        kernel<<<dim3((unsigned)cdiv(channels, 64), (unsigned)cdiv(batch, rows)), dim3(256), 0, (hipStream_t)stream>>>(
            (const E*)x, dt, (const E*)bc, bc_stride, (const E*)z, z_stride, (const E*)a_log, (const E*)d_skip, state,
            state_slots, positions, active, (E*)out, (int)batch, (int)num_slots, (int)channels, (int)states);
    });
    return launched(fn);
}
