// Hyper-connections: the residual is `streams` copies of the token's row, a sublayer reads a weighted sum of them, and its
// output and the old streams are mixed into the new ones.  The write of one sublayer, the read of the next and its norm are
// one launch.  Byte mover: one workgroup per token row, a thread owns the same elements of every stream.
#include "hybrid_common.hpp"

namespace nqh {
namespace {

constexpr int kMaxStreams = 8;
constexpr int kMaxWidth = 8192;

// S: streams held in registers (`streams` of them exist), V elements per thread and step, P steps.
template <typename T, int S, int V, int THREADS, int P>
__global__ __launch_bounds__(THREADS) void hyper_norm_kernel(
    float* __restrict__ x, const int64_t* __restrict__ ids, const typename T::elem* __restrict__ table, int64_t table_rows,
    const typename T::elem* __restrict__ y, const typename T::elem* __restrict__ mix, const typename T::elem* __restrict__ w_out,
    const typename T::elem* __restrict__ w_in, const typename T::elem* __restrict__ norm_w, typename T::elem* __restrict__ h,
    int streams, int width, float eps) {
    constexpr int WAVES = THREADS / 64;
    __shared__ float s_red[WAVES];
    const int64_t row = blockIdx.x;
    float* xr = x + row * streams * width;
    float v[S][P][V], yv[P][V], wn[P][V];
    int64_t src = 0;
    if (ids) {
        src = ids[row];
        src = (src < 0 ? 0 : (src >= table_rows ? table_rows - 1 : src)) * width;
    }
#pragma unroll
    for (int p = 0; p < P; ++p) {          // every load is under way before the first is used
        const int i = (p * THREADS + threadIdx.x) * V;
#pragma unroll
        for (int e = 0; e < V; ++e) {
            yv[p][e] = wn[p][e] = 0.f;
#pragma unroll
            for (int s = 0; s < S; ++s) v[s][p][e] = 0.f;
        }
        if (i < width) {
            if (ids) {
                load_vec<T, V>(table + src + i, v[0][p]);
            } else {
#pragma unroll
                for (int s = 0; s < S; ++s)
                    if (s < streams) load_vec<Fp, V>(xr + (int64_t)s * width + i, v[s][p]);
            }
            if (y) load_vec<T, V>(y + row * width + i, yv[p]);
            if (h) load_vec<T, V>(norm_w + i, wn[p]);
        }
    }
    float win[S];
#pragma unroll
    for (int s = 0; s < S; ++s) win[s] = s < streams ? (w_in ? T::load(w_in + s) : 1.f) : 0.f;
    if (ids) {
#pragma unroll
        for (int s = 1; s < S; ++s)
#pragma unroll
            for (int p = 0; p < P; ++p)
#pragma unroll
                for (int e = 0; e < V; ++e) v[s][p][e] = v[0][p][e];
    }
    if (y) {
        float m[S][S], wo[S];
#pragma unroll
        for (int t = 0; t < S; ++t) {
            wo[t] = t < streams ? T::load(w_out + t) : 0.f;
#pragma unroll
            for (int s = 0; s < S; ++s) m[s][t] = (s < streams && t < streams) ? T::load(mix + s * streams + t) : 0.f;
        }
#pragma unroll
        for (int p = 0; p < P; ++p)
#pragma unroll
            for (int e = 0; e < V; ++e) {
                float o[S];
#pragma unroll
                for (int s = 0; s < S; ++s) o[s] = v[s][p][e];
#pragma unroll
                for (int t = 0; t < S; ++t) {
                    float a = wo[t] * yv[p][e];
#pragma unroll
                    for (int s = 0; s < S; ++s) a += m[s][t] * o[s];
                    v[t][p][e] = a;
                }
            }
    }
    float ss = 0.f;
#pragma unroll
    for (int p = 0; p < P; ++p) {
        const int i = (p * THREADS + threadIdx.x) * V;
        if (i < width && (y || ids)) {
#pragma unroll
            for (int s = 0; s < S; ++s)
                if (s < streams) store_vec<Fp, V>(xr + (int64_t)s * width + i, v[s][p]);
        }
#pragma unroll
        for (int e = 0; e < V; ++e) {
            float u = 0.f;
#pragma unroll
            for (int s = 0; s < S; ++s) u += win[s] * v[s][p][e];
            yv[p][e] = u;
            ss += u * u;                   // elements past the width are zero
        }
    }
    if (!h) return;
    const float r = rsqrtf(block_sum<WAVES>(ss, s_red) / (float)width + eps);
#pragma unroll
    for (int p = 0; p < P; ++p) {
        const int i = (p * THREADS + threadIdx.x) * V;
#pragma unroll
        for (int e = 0; e < V; ++e) yv[p][e] *= r * wn[p][e];
        if (i < width) store_vec<T, V>(h + row * width + i, yv[p]);
    }
}

template <typename T, int S>
void launch_hyper(float* x, const int64_t* ids, const void* table, int64_t table_rows, const void* y, const void* mix,
                  const void* w_out, const void* w_in, const void* norm_w, void* h, int64_t rows, int64_t streams,
                  int64_t width, float eps, bool vec, hipStream_t st) {
    using E = typename T::elem;
#define NQH_GO(V, THREADS, P)                                                                                              \
    hyper_norm_kernel<T, S, V, THREADS, P><<<dim3((unsigned)rows), dim3(THREADS), 0, st>>>(                                \
        x, ids, (const E*)table, table_rows, (const E*)y, (const E*)mix, (const E*)w_out, (const E*)w_in, (const E*)norm_w, \
        (E*)h, (int)streams, (int)width, eps)
    if (!vec) NQH_GO(1, 1024, 8);
    else if (width <= 1024) NQH_GO(4, 256, 1);
    else if (width <= 2048) NQH_GO(4, 512, 1);
    else if (width <= 4096) NQH_GO(4, 1024, 1);
    else NQH_GO(4, 1024, 2);
#undef NQH_GO
}

// Element-wise functions of a matrix product's result, in place.
template <typename T, int V>
__global__ __launch_bounds__(256) void activate_kernel(typename T::elem* __restrict__ x, int64_t n, int act, float param) {
    const int64_t i = ((int64_t)blockIdx.x * 256 + threadIdx.x) * V;
    if (i >= n) return;
    float v[V];
    load_vec<T, V>(x + i, v);
#pragma unroll
    for (int e = 0; e < V; ++e) v[e] = activation_f32(v[e], act, param);
    store_vec<T, V>(x + i, v);
}

}  // namespace
}  // namespace nqh

using namespace nqh;

extern "C" int64_t nqh_hyper_max_streams(void) { return kMaxStreams; }

extern "C" int nqh_hyper_norm(float* x, const int64_t* ids, const void* table, int64_t table_rows, const void* y,
                              const void* mix, const void* w_out, const void* w_in, const void* norm_weight, void* h,
                              int64_t rows, int64_t streams, int64_t width, float eps, int dtype, void* stream) {
    const char* fn = "nqh_hyper_norm";
    if (!x || (ids && (!table || table_rows <= 0)) || (y && (!mix || !w_out)) || (h && !norm_weight))
        return fail(NQH_ERR_ARG, fn, "null pointer");
    if (!dtype_ok(dtype)) return fail(NQH_ERR_ARG, fn, "dtype must be NQH_BF16 or NQH_F32");
    if (rows <= 0 || rows > kMaxI32 || width <= 0 || streams <= 0) return fail(NQH_ERR_ARG, fn, "sizes must be positive");
    if (width > kMaxWidth || streams > kMaxStreams)
        return fail(NQH_ERR_UNSUPPORTED, fn, "at most width %d and %d streams", kMaxWidth, kMaxStreams);
    const bool vec = width % 4 == 0 && aligned(x, 16) && aligned(y, 16) && aligned(table, 16) && aligned(norm_weight, 16) &&
                     aligned(h, 16);
    (void)hipGetLastError();
#define NQH_STREAMS(S) \
    launch_hyper<T, S>(x, ids, table, table_rows, y, mix, w_out, w_in, norm_weight, h, rows, streams, width, eps, vec, (hipStream_t)stream)
    NQH_WITH_TYPE(dtype, {
        if (streams == 1) NQH_STREAMS(1);
        else if (streams == 2) NQH_STREAMS(2);
        else if (streams <= 4) NQH_STREAMS(4);
        else NQH_STREAMS(8);
    });
#undef NQH_STREAMS
    return launched(fn);
}

extern "C" int nqh_activate(void* x, int64_t count, int act, float param, int dtype, void* stream) {
    const char* fn = "nqh_activate";
    if (!x) return fail(NQH_ERR_ARG, fn, "null pointer");
    if (!dtype_ok(dtype)) return fail(NQH_ERR_ARG, fn, "dtype must be NQH_BF16 or NQH_F32");
    if (count <= 0 || cdiv(count, 256) > kMaxI32) return fail(NQH_ERR_ARG, fn, "count must be positive and not too large");
    if (act < NQH_ACT_NONE || act > NQH_ACT_SOFTCAP || (act == NQH_ACT_SOFTCAP && !(param > 0.f)))
        return fail(NQH_ERR_ARG, fn, "unknown activation, or a cap that is not positive");
    (void)hipGetLastError();
    NQH_WITH_TYPE(dtype, {
        using E = typename T::elem;
        if (count % 8 == 0 && aligned(x, 16))
            activate_kernel<T, 8><<<dim3((unsigned)cdiv(count, 2048)), dim3(256), 0, (hipStream_t)stream>>>((E*)x, count, act, param);
        else
            activate_kernel<T, 1><<<dim3((unsigned)cdiv(count, 256)), dim3(256), 0, (hipStream_t)stream>>>((E*)x, count, act, param);
    });
    return launched(fn);
}
