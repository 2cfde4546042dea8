// Shared device/host helpers of the hybrid-decoder kernels (libnq_hybrid.so).
#pragma once

#include "../awq_common.hpp"
#include "../../../include/nq_hybrid_ops.h"

namespace nqh {

using awq::as_f32_result;
using awq::cdiv;
using awq::f32x4;
using awq::f32x16;
using awq::u32x2;
using awq::u32x4;

// Element types of a call: bf16 (matrix products on the matrix cores, fp32 accumulation) and fp32 (everything in fp32).
struct Bf : awq::BF16 {
    using elem = uint16_t;
    static __device__ __forceinline__ float load(const elem* p) { return to_f32(*p); }
    static __device__ __forceinline__ void store(elem* p, float v) { *p = from_f32(v); }
    static __device__ __forceinline__ float round(float v) { return to_f32(from_f32(v)); }
};
struct Fp {
    using elem = float;
    static __device__ __forceinline__ float load(const elem* p) { return *p; }
    static __device__ __forceinline__ void store(elem* p, float v) { *p = v; }
    static __device__ __forceinline__ float round(float v) { return v; }
};

// V consecutive elements <-> fp32, one access; p aligned to the access.
template <typename T, int V>
__device__ __forceinline__ void load_vec(const typename T::elem* p, float (&f)[V]) {
    if constexpr (sizeof(typename T::elem) == 4) {
        if constexpr (V % 4 == 0) {
#pragma unroll
            for (int i = 0; i < V; i += 4) {
                const f32x4 v = *reinterpret_cast<const f32x4*>(p + i);
                f[i] = v[0]; f[i + 1] = v[1]; f[i + 2] = v[2]; f[i + 3] = v[3];
            }
        } else {
#pragma unroll
            for (int i = 0; i < V; ++i) f[i] = T::load(p + i);
        }
    } else if constexpr (V % 8 == 0) {
#pragma unroll
        for (int i = 0; i < V; i += 8) {
            const u32x4 v = *reinterpret_cast<const u32x4*>(p + i);
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                const uint32_t w = v[j];
                f[i + 2 * j] = T::to_f32((uint16_t)(w & 0xFFFFu));
                f[i + 2 * j + 1] = T::to_f32((uint16_t)(w >> 16));
            }
        }
    } else if constexpr (V == 4) {
        const u32x2 v = *reinterpret_cast<const u32x2*>(p);
#pragma unroll
        for (int j = 0; j < 2; ++j) {
            const uint32_t w = v[j];
            f[2 * j] = T::to_f32((uint16_t)(w & 0xFFFFu));
            f[2 * j + 1] = T::to_f32((uint16_t)(w >> 16));
        }
    } else {
#pragma unroll
        for (int i = 0; i < V; ++i) f[i] = T::load(p + i);
    }
}
template <typename T, int V>
__device__ __forceinline__ void store_vec(typename T::elem* p, const float (&f)[V]) {
    if constexpr (sizeof(typename T::elem) == 4) {
        if constexpr (V % 4 == 0) {
#pragma unroll
            for (int i = 0; i < V; i += 4) *reinterpret_cast<f32x4*>(p + i) = f32x4{f[i], f[i + 1], f[i + 2], f[i + 3]};
        } else {
#pragma unroll
            for (int i = 0; i < V; ++i) T::store(p + i, f[i]);
        }
    } else if constexpr (V % 8 == 0) {
#pragma unroll
        for (int i = 0; i < V; i += 8)
            *reinterpret_cast<u32x4*>(p + i) = u32x4{T::pack2(f[i], f[i + 1]), T::pack2(f[i + 2], f[i + 3]),
                                                     T::pack2(f[i + 4], f[i + 5]), T::pack2(f[i + 6], f[i + 7])};
    } else if constexpr (V == 4) {
        *reinterpret_cast<u32x2*>(p) = u32x2{T::pack2(f[0], f[1]), T::pack2(f[2], f[3])};
    } else {
#pragma unroll
        for (int i = 0; i < V; ++i) T::store(p + i, f[i]);
    }
}

// V = 4 consecutive elements as they lie in memory, to be fetched early and unpacked late.
template <typename T>
struct Raw4;
template <>
struct Raw4<Bf> {
    using type = u32x2;
    static __device__ __forceinline__ float get(type v, int e) { return Bf::to_f32((uint16_t)(v[e >> 1] >> (16 * (e & 1)))); }
    static __device__ __forceinline__ type pack(const uint16_t (&f)[4]) {
        return type{(uint32_t)f[0] | (uint32_t)f[1] << 16, (uint32_t)f[2] | (uint32_t)f[3] << 16};
    }
};
template <>
struct Raw4<Fp> {
    using type = f32x4;
    static __device__ __forceinline__ float get(type v, int e) { return v[e]; }
    static __device__ __forceinline__ type pack(const float (&f)[4]) { return type{f[0], f[1], f[2], f[3]}; }
};

__device__ __forceinline__ float wave_sum(float v) {
#pragma unroll
    for (int o = 32; o >= 1; o >>= 1) v += __shfl_xor(v, o);
    return v;
}
__device__ __forceinline__ float wave_max(float v) {
#pragma unroll
    for (int o = 32; o >= 1; o >>= 1) v = fmaxf(v, __shfl_xor(v, o));
    return v;
}
// Sum over a workgroup of WAVES waves; s: WAVES floats that nobody else touches between two barriers.
template <int WAVES>
__device__ __forceinline__ float block_sum(float v, float* s) {
    v = wave_sum(v);
    if ((threadIdx.x & 63) == 0) s[threadIdx.x >> 6] = v;
    __syncthreads();
    float t = 0.f;
#pragma unroll
    for (int w = 0; w < WAVES; ++w) t += s[w];
    return t;
}

__device__ __forceinline__ float sigmoid_f32(float z) { return 1.f / (1.f + expf(-z)); }
__device__ __forceinline__ float silu_f32(float z) { return z / (1.f + expf(-z)); }
// The same by the hardware's 2^x and reciprocal (about one ulp each), for kernels that the exact division would slow down.
__device__ __forceinline__ float silu_quick(float z) {
    return z * __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(z * -1.4426950408889634f));
}
// sigmoid(z)^(1 / tau) = 2^(-(log2(1 + e^-|z|) + max(-z, 0) log2 e) / tau).  log(1 + x) as log(u) x / (u - 1) with
// u = 1 + x rounded keeps its relative precision for small x (Goldberg, "What every computer scientist should know about
// floating-point arithmetic", theorem 4).
__device__ __forceinline__ float decay_f32(float z, float inv_tau) {
    constexpr float kLog2e_ = 1.4426950408889634f;
    const float x = __builtin_amdgcn_exp2f(-fabsf(z) * kLog2e_);
    const float u = as_f32_result(1.f + x), um1 = as_f32_result(u - 1.f);
    const float l = um1 == 0.f ? x * kLog2e_ : __builtin_amdgcn_logf(u) * (x * __builtin_amdgcn_rcpf(um1));
    return __builtin_amdgcn_exp2f(-(l + fmaxf(-z, 0.f) * kLog2e_) * inv_tau);
}

// log(1 + e^z) = max(z, 0) + log(1 + e^-|z|), the logarithm as above.
__device__ __forceinline__ float softplus_f32(float z) {
    constexpr float kLog2e_ = 1.4426950408889634f, kLn2_ = 0.6931471805599453f;
    const float x = __builtin_amdgcn_exp2f(-fabsf(z) * kLog2e_);
    const float u = as_f32_result(1.f + x), um1 = as_f32_result(u - 1.f);
    const float l = um1 == 0.f ? x : kLn2_ * __builtin_amdgcn_logf(u) * (x * __builtin_amdgcn_rcpf(um1));
    return fmaxf(z, 0.f) + l;
}
// What may follow a matrix product (nqh_activation); param: the cap of NQH_ACT_SOFTCAP.
__device__ __forceinline__ float activation_f32(float v, int act, float param) {
    if (act == NQH_ACT_RELU2) {
        v = fmaxf(v, 0.f);
        return v * v;
    }
    return act == NQH_ACT_SOFTCAP ? param * tanhf(v / param) : v;
}

// ---- host-side error plumbing ---------------------------------------------------------------------
int fail(int status, const char* fn, const char* fmt, ...);
int launched(const char* fn);   // status of the launch just made
static inline bool aligned(const void* p, size_t n) { return (reinterpret_cast<uintptr_t>(p) & (n - 1)) == 0; }
static inline bool dtype_ok(int dtype) { return dtype == NQH_BF16 || dtype == NQH_F32; }
constexpr int64_t kMaxI32 = 0x7fffffff;

}  // namespace nqh

// Runs the statement with T bound to the element type of the call.
#define NQH_WITH_TYPE(dtype, ...)             \
    do {                                      \
        if ((dtype) == NQH_BF16) {            \
            using T = nqh::Bf;                \
            __VA_ARGS__;                      \
        } else {                              \
            using T = nqh::Fp;                \
            __VA_ARGS__;                      \
        }                                     \
    } while (0)
