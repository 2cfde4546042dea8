// Dense linear for few rows: y = act(x W^T (+ bias)), bf16 operands, fp32 accumulation.
//   up to 16 rows    skinny_linear_kernel: both operands straight from memory, the waves split the contraction; also for more
//                    rows of few features, 16 at a time, where the next would leave most of the chip idle
//   17 to 64 rows    wide_linear_kernel: the activations, by now as many bytes per workgroup as its weights, go through LDS
#include "skinny.hpp"

namespace nqh {
namespace {

template <bool F32OUT>
__global__ __launch_bounds__(1024) void skinny_linear_kernel(const uint16_t* __restrict__ x, const uint16_t* __restrict__ w,
                                                             const uint16_t* __restrict__ bias, void* __restrict__ y,
                                                             int rows, int n_out, int n_in, int act, float param) {
    extern __shared__ __attribute__((aligned(16))) float s_sum[];
    const int lane = threadIdx.x & 63, lo = lane & 15, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int waves = blockDim.x >> 6, n0 = blockIdx.x * 16, r0 = blockIdx.y * 16;
    rows -= r0;
    x += (int64_t)r0 * n_in;
    const uint16_t* w_row[1] = {w + (int64_t)min(n0 + lo, n_out - 1) * n_in};
    const uint16_t* x_row[1] = {x + (int64_t)min(lo, rows - 1) * n_in};
    f32x4 acc[1][1] = {{f32x4{0.f, 0.f, 0.f, 0.f}}};
    skinny_accumulate<1, 1>(acc, w_row, x_row, n_in, wave, waves);
    skinny_reduce<1, 1>(acc, s_sum, wave, waves);
    const int t = threadIdx.x >> 4, n = n0 + (threadIdx.x & 15);
    if (threadIdx.x < 256 && t < rows && n < n_out) {
        const float v = activation_f32(s_sum[threadIdx.x] + (bias ? Bf::to_f32(bias[n]) : 0.f), act, param);
        if constexpr (F32OUT) reinterpret_cast<float*>(y)[(int64_t)(r0 + t) * n_out + n] = v;
        else reinterpret_cast<uint16_t*>(y)[(int64_t)(r0 + t) * n_out + n] = Bf::from_f32(v);
    }
}

// 16 MT rows, 16 NT output features per workgroup; its eight waves are NT features tiles x KS parts of every stage of
// KS * 128 contraction elements.  The stage's activations are brought to LDS once (rows of 128 elements, 16-byte piece p of
// row r at position (p + r) % 16: the 16 rows of an operand read fall on all banks once), double-buffered; the weights
// stream into registers, one stage ahead.
#define NQH_GPTR(p) ((__attribute__((address_space(1))) void*)(p))
#define NQH_LPTR(p) ((__attribute__((address_space(3))) void*)(p))
__device__ const u32x4 g_zero_piece = {0u, 0u, 0u, 0u};   // what lies past the end of a row

template <int MT, int NT, bool F32OUT>
__global__ __launch_bounds__(512) void wide_linear_kernel(const uint16_t* __restrict__ x, const uint16_t* __restrict__ w,
                                                          const uint16_t* __restrict__ bias, void* __restrict__ y, int rows,
                                                          int n_out, int n_in, int act, float param) {
    constexpr int KS = 8 / NT, kPart = 16 * MT * 256, kBuf = KS * kPart, kLoads = kBuf / 1024 / 8;
    extern __shared__ __attribute__((aligned(1024))) unsigned char s_x[];   // [buffer][part][row][256 bytes]
    const int lane = threadIdx.x & 63, lo = lane & 15, hi = lane >> 4;
    const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), nt = wave % NT, part = wave / NT;
    const int n0 = blockIdx.x * 16 * NT;
    const uint16_t* w_row = w + (int64_t)min(n0 + 16 * nt + lo, n_out - 1) * n_in;
    auto stage = [&](int k0, int buf) {
#pragma unroll
        for (int i = 0; i < kLoads; ++i) {
            const int block = i * 8 + wave;                       // 1 KiB: four rows of one part
            const int p = block / (4 * MT), row = block % (4 * MT) * 4 + (lane >> 4);
            const int k = k0 + p * kPiece + 8 * (((lane & 15) - row) & 15);
            const void* src = k < n_in ? (const void*)(x + (int64_t)min(row, rows - 1) * n_in + k) : (const void*)&g_zero_piece;
            __builtin_amdgcn_global_load_lds(NQH_GPTR(src), NQH_LPTR(s_x + buf * kBuf + block * 1024), 16, 0, 0);
        }
    };
    f32x4 acc[MT];
#pragma unroll
    for (int m = 0; m < MT; ++m) acc[m] = f32x4{0.f, 0.f, 0.f, 0.f};
    u32x4 cur[4], nxt[4];
    stage(0, 0);
    load_piece_clamped(cur, w_row, part * kPiece, hi, n_in);      // the activations are zero past the end
    int buf = 0;
    for (int k0 = 0; k0 < n_in; k0 += KS * kPiece) {
        __builtin_amdgcn_s_waitcnt(0x0F70);   // this wave's part of the stage and its weights have landed
        __syncthreads();
        if (k0 + KS * kPiece < n_in) {
            load_piece_clamped(nxt, w_row, k0 + (KS + part) * kPiece, hi, n_in);
            stage(k0 + KS * kPiece, buf ^ 1);
        }
        const unsigned char* base = s_x + buf * kBuf + part * kPart;
#pragma unroll
        for (int s = 0; s < 4; ++s)
#pragma unroll
            for (int m = 0; m < MT; ++m) {
                const int row = 16 * m + lo;
                const u32x4 xf = *reinterpret_cast<const u32x4*>(base + row * 256 + ((4 * s + hi + row) & 15) * 16);
                acc[m] = Bf::mfma16(cur[s], xf, acc[m]);
            }
#pragma unroll
        for (int s = 0; s < 4; ++s) cur[s] = nxt[s];
        buf ^= 1;
    }
    __syncthreads();                          // the stages are read: their memory takes the parts' sums [part][nt][row][16]
    float* sums = reinterpret_cast<float*>(s_x);
#pragma unroll
    for (int m = 0; m < MT; ++m)
        *reinterpret_cast<f32x4*>(sums + ((part * NT + nt) * 16 * MT + 16 * m + lo) * 16 + 4 * hi) = acc[m];
    __syncthreads();
    for (int i = threadIdx.x; i < NT * MT * 256; i += 512) {
        const int j = i / (MT * 256), t = i / 16 % (16 * MT), n = n0 + 16 * j + (i & 15);
        if (t >= rows || n >= n_out) continue;
        float v = bias ? Bf::to_f32(bias[n]) : 0.f;
#pragma unroll
        for (int p = 0; p < KS; ++p) v += sums[p * NT * MT * 256 + i];
        v = activation_f32(v, act, param);
        if constexpr (F32OUT) reinterpret_cast<float*>(y)[(int64_t)t * n_out + n] = v;
        else reinterpret_cast<uint16_t*>(y)[(int64_t)t * n_out + n] = Bf::from_f32(v);
    }
}

template <int MT, int NT>
int launch_wide(const char* fn, const void* x, const void* w, const void* bias, void* y, int64_t rows, int64_t n_out,
                int64_t n_in, int out_f32, int act, float param, void* stream) {
    constexpr int lds = 2 * (8 / NT) * 16 * MT * 256;
    const auto kernel = out_f32 ? wide_linear_kernel<MT, NT, true> : wide_linear_kernel<MT, NT, false>;
    if (lds > 65536) {
        const hipError_t e = hipFuncSetAttribute((const void*)kernel, hipFuncAttributeMaxDynamicSharedMemorySize, lds);
        if (e != hipSuccess) return fail(NQH_ERR_HIP, fn, "%s", hipGetErrorString(e));
    }
    kernel<<<dim3((unsigned)cdiv(n_out, 16 * NT)), dim3(512), lds, (hipStream_t)stream>>>(
        (const uint16_t*)x, (const uint16_t*)w, (const uint16_t*)bias, y, (int)rows, (int)n_out, (int)n_in, act, param);
    return launched(fn);
}

}  // namespace
}  // namespace nqh

using namespace nqh;

extern "C" int nqh_skinny_linear(const void* x, const void* weight, const void* bias, void* y, int64_t rows,
                                 int64_t out_features, int64_t in_features, int out_f32, int act, float param,
                                 void* stream) {
    const char* fn = "nqh_skinny_linear";
    if (!x || !weight || !y || !aligned(x, 16) || !aligned(weight, 16))
        return fail(NQH_ERR_ARG, fn, "null or misaligned pointer");
    if (rows <= 0 || rows > 64 || out_features <= 0 || in_features <= 0 || in_features % 8 != 0 ||
        out_features > kMaxI32 - 16 || in_features > (1 << 30))
        return fail(NQH_ERR_ARG, fn, "1 to 64 rows and an in_features that is a multiple of 8");
    if (act < NQH_ACT_NONE || act > NQH_ACT_SOFTCAP || (act == NQH_ACT_SOFTCAP && !(param > 0.f)))
        return fail(NQH_ERR_ARG, fn, "unknown activation, or a cap that is not positive");
    (void)hipGetLastError();
    if (rows > 16 && out_features > 1024) {
        const bool narrow = out_features <= 8192;      // fewer features per workgroup: more workgroups
        if (rows <= 32)
            return narrow ? launch_wide<2, 2>(fn, x, weight, bias, y, rows, out_features, in_features, out_f32, act, param, stream)
                          : launch_wide<2, 4>(fn, x, weight, bias, y, rows, out_features, in_features, out_f32, act, param, stream);
        return narrow ? launch_wide<4, 2>(fn, x, weight, bias, y, rows, out_features, in_features, out_f32, act, param, stream)
                      : launch_wide<4, 4>(fn, x, weight, bias, y, rows, out_features, in_features, out_f32, act, param, stream);
    }
    const int64_t groups = cdiv(out_features, 16);
    const int waves = skinny_waves(groups * cdiv(rows, 16), in_features);
    const size_t lds = (size_t)waves * 256 * sizeof(float);
    const dim3 grid((unsigned)groups, (unsigned)cdiv(rows, 16)), block((unsigned)waves * 64);
    if (out_f32)
        skinny_linear_kernel<true><<<grid, block, lds, (hipStream_t)stream>>>(
            (const uint16_t*)x, (const uint16_t*)weight, (const uint16_t*)bias, y, (int)rows, (int)out_features, (int)in_features,
            act, param);
    else
        skinny_linear_kernel<false><<<grid, block, lds, (hipStream_t)stream>>>(
            (const uint16_t*)x, (const uint16_t*)weight, (const uint16_t*)bias, y, (int)rows, (int)out_features, (int)in_features,
            act, param);
    return launched(fn);
}
