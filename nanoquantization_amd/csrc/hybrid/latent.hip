// Latent attention around the attention kernels: the norm of the latent, rotary and cache write of a projection row, the
// gathering of cached rows for a prompt pass, and products with a matrix per head (queries into the latent space, read-outs
// out of it).  A cache row is one token's latent, zero padding up to rot_at, the rotated key part, zero padding.
#include "skinny.hpp"

namespace nqh {
namespace {

// One workgroup per token row.  proj: queries [heads][dim | rot_dim], latent [rank], rotated key part [rot_dim].
// q_out [heads][q_row]: with copy_plain the unrotated part goes to 0 .. dim - 1; the rotated one goes to rot_q ..; the rest
// from `lead` on (what neither this kernel nor the absorbing product fills) is zeroed.
template <typename T>
__global__ __launch_bounds__(256) void latent_store_kernel(
    const typename T::elem* __restrict__ proj, const typename T::elem* __restrict__ norm_w, const float* __restrict__ cos_sin,
    const int64_t* __restrict__ positions, const int64_t* __restrict__ slots, typename T::elem* __restrict__ q_out,
    typename T::elem* __restrict__ cache, int heads, int dim, int rot_dim, int rank, int q_row, int rot_q, int copy_plain,
    int row, int rot_at, int64_t max_positions, int64_t num_slots, float eps) {
    __shared__ float s_red[4];
    const int64_t r = blockIdx.x;
    const int head = dim + rot_dim, nq = heads * head, half = rot_dim >> 1;
    const typename T::elem* src = proj + r * (nq + rank + rot_dim);
    const int64_t slot = slots[r];
    const bool slot_ok = slot >= 0 && slot < num_slots;
    int64_t pos = positions[r];
    pos = pos < 0 ? 0 : (pos >= max_positions ? max_positions - 1 : pos);
    const float* cs = cos_sin + pos * rot_dim;
    if (slot_ok) {       // the same for the whole workgroup
        typename T::elem* dst = cache + slot * row;
        float ss = 0.f;
        for (int i = threadIdx.x; i < rank; i += 256) {
            const float a = T::load(src + nq + i);
            ss += a * a;
        }
        const float f = rsqrtf(block_sum<4>(ss, s_red) / (float)rank + eps);
        for (int i = threadIdx.x; i < rank; i += 256) T::store(dst + i, T::load(src + nq + i) * f * T::load(norm_w + i));
        for (int i = threadIdx.x; i < half; i += 256) {
            const float c = cs[i], s = cs[half + i];
            const float u = T::load(src + nq + rank + 2 * i), v = T::load(src + nq + rank + 2 * i + 1);
            T::store(dst + rot_at + 2 * i, u * c - v * s);
            T::store(dst + rot_at + 2 * i + 1, v * c + u * s);
        }
    }
    typename T::elem* q = q_out + r * heads * q_row;
    for (int i = threadIdx.x; i < heads * half; i += 256) {
        const int h = i / half, p = i - h * half;
        const float c = cs[p], s = cs[half + p];
        const float u = T::load(src + h * head + dim + 2 * p), v = T::load(src + h * head + dim + 2 * p + 1);
        T::store(q + h * q_row + rot_q + 2 * p, u * c - v * s);
        T::store(q + h * q_row + rot_q + 2 * p + 1, v * c + u * s);
    }
    if (copy_plain) {
        if (dim % 8 == 0 && rot_dim % 8 == 0 && q_row % 8 == 0 && rank % 8 == 0) {   // rows and heads are aligned then
            const int per = dim >> 3;
            for (int i = threadIdx.x; i < heads * per; i += 256) {
                const int h = i / per, d = (i - h * per) * 8;
                float a[8];
                load_vec<T, 8>(src + h * head + d, a);
                store_vec<T, 8>(q + h * q_row + d, a);
            }
        } else {
            for (int i = threadIdx.x; i < heads * dim; i += 256) {
                const int h = i / dim, d = i - h * dim;
                q[h * q_row + d] = src[h * head + d];
            }
        }
    }
    const int lead = copy_plain ? dim : rank, gap = rot_q - lead, tail = q_row - rot_q - rot_dim, pad = gap + tail;
    for (int i = threadIdx.x; i < heads * pad; i += 256) {
        const int h = i / pad, d = i - h * pad;
        T::store(q + h * q_row + (d < gap ? lead + d : rot_q + rot_dim + d - gap), 0.f);
    }
}

// Cached rows of all segments' contexts, one after the other and without padding: out[first[s] + j] = latent | rotated part of
// token j of segment s.  Workgroup (16 tokens, segment).
__global__ __launch_bounds__(256) void latent_gather_kernel(const uint16_t* __restrict__ cache, const int32_t* __restrict__ tables,
                                                            const int32_t* __restrict__ segments,
                                                            const int32_t* __restrict__ first, uint16_t* __restrict__ out,
                                                            int rank, int rot_dim, int row, int rot_at, int block_size,
                                                            int max_blocks, int num_blocks) {
    const int seg = blockIdx.y, ctx = min(segments[3 * seg + 1] + segments[3 * seg + 2], max_blocks * block_size);
    const int width = rank + rot_dim, per = width >> 3;
    for (int i = threadIdx.x; i < 16 * per; i += 256) {
        const int j = blockIdx.x * 16 + i / per, e = i % per * 8;
        if (j >= ctx) return;
        int blk = tables[(int64_t)seg * max_blocks + j / block_size];
        blk = blk < 0 ? 0 : (blk >= num_blocks ? num_blocks - 1 : blk);
        const uint16_t* src = cache + ((int64_t)blk * block_size + j % block_size) * row;
        *reinterpret_cast<u32x4*>(out + ((int64_t)first[seg] + j) * width + e) =
            *reinterpret_cast<const u32x4*>(src + (e < rank ? e : rot_at + e - rank));
    }
}

// y[r, h, :] = w[h] x[r, h, :].  Matrix cores: workgroup = (16 outputs, head, 16 rows).
__global__ __launch_bounds__(256) void head_linear_kernel(const uint16_t* __restrict__ x, const uint16_t* __restrict__ w,
                                                          uint16_t* __restrict__ y, int rows, int n_out, int n_in,
                                                          int64_t x_row, int64_t x_head, int64_t y_row, int64_t y_head) {
    extern __shared__ __attribute__((aligned(16))) float s_sum[];
    const int lane = threadIdx.x & 63, lo = lane & 15, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int waves = blockDim.x >> 6, n0 = blockIdx.x * 16, h = blockIdx.y, r0 = blockIdx.z * 16;
    const uint16_t* w_row[1] = {w + ((int64_t)h * n_out + min(n0 + lo, n_out - 1)) * n_in};
    const uint16_t* x_at[1] = {x + (int64_t)min(r0 + lo, rows - 1) * x_row + h * x_head};
    f32x4 acc[1][1] = {{f32x4{0.f, 0.f, 0.f, 0.f}}};
    skinny_accumulate<1, 1>(acc, w_row, x_at, n_in, wave, waves);
    skinny_reduce<1, 1>(acc, s_sum, wave, waves);
    for (int i = threadIdx.x; i < 256; i += blockDim.x) {
        const int t = r0 + (i >> 4), n = n0 + (i & 15);
        if (t < rows && n < n_out) Bf::store(y + (int64_t)t * y_row + h * y_head + n, s_sum[i]);
    }
}

// Any sizes, both element types: one thread per output.
template <typename T>
__global__ __launch_bounds__(256) void head_linear_any_kernel(const typename T::elem* __restrict__ x,
                                                              const typename T::elem* __restrict__ w,
                                                              typename T::elem* __restrict__ y, int rows, int n_out, int n_in,
                                                              int64_t x_row, int64_t x_head, int64_t y_row, int64_t y_head) {
    const int n = blockIdx.x * 256 + threadIdx.x, h = blockIdx.y, r = blockIdx.z;
    if (n >= n_out) return;
    const typename T::elem* xr = x + (int64_t)r * x_row + h * x_head;
    const typename T::elem* wr = w + ((int64_t)h * n_out + n) * n_in;
    float a = 0.f;
    for (int k = 0; k < n_in; ++k) a += T::load(xr + k) * T::load(wr + k);
    T::store(y + (int64_t)r * y_row + h * y_head + n, a);
}

}  // namespace
}  // namespace nqh

using namespace nqh;

extern "C" int nqh_latent_store(const void* proj, const void* norm_weight, const float* cos_sin, const int64_t* positions,
                                const int64_t* slots, void* q_out, void* cache, int64_t rows, int64_t heads, int64_t dim,
                                int64_t rot_dim, int64_t rank, int64_t q_row, int64_t rot_q, int copy_plain, int64_t row,
                                int64_t rot_at, int64_t max_positions, int64_t num_slots, float eps, int dtype, void* stream) {
    const char* fn = "nqh_latent_store";
    if (!proj || !norm_weight || !cos_sin || !positions || !slots || !q_out || !cache)
        return fail(NQH_ERR_ARG, fn, "null pointer");
    if (!dtype_ok(dtype)) return fail(NQH_ERR_ARG, fn, "dtype must be NQH_BF16 or NQH_F32");
    if (rows <= 0 || rows > kMaxI32 || heads <= 0 || dim <= 0 || rot_dim <= 0 || rot_dim % 2 || rank <= 0 || max_positions <= 0 ||
        num_slots <= 0 || heads * q_row > kMaxI32 || heads * (dim + rot_dim) + rank + rot_dim > kMaxI32)
        return fail(NQH_ERR_ARG, fn, "sizes must be positive 31-bit counts and rot_dim even");
    if (rot_q < (copy_plain ? dim : rank) || q_row < rot_q + rot_dim || rot_at < rank || row < rot_at + rot_dim)
        return fail(NQH_ERR_ARG, fn, "the parts of a query or cache row overlap or exceed it");
    if (copy_plain && (!aligned(proj, 16) || !aligned(q_out, 16))) return fail(NQH_ERR_ARG, fn, "misaligned pointer");
    (void)hipGetLastError();
    NQH_WITH_TYPE(dtype, {
        using E = typename T::elem;
        latent_store_kernel<T><<<dim3((unsigned)rows), dim3(256), 0, (hipStream_t)stream>>>(
            (const E*)proj, (const E*)norm_weight, cos_sin, positions, slots, (E*)q_out, (E*)cache, (int)heads, (int)dim,
            (int)rot_dim, (int)rank, (int)q_row, (int)rot_q, copy_plain, (int)row, (int)rot_at, max_positions, num_slots, eps);
    });
    return launched(fn);
}

extern "C" int nqh_latent_gather(const void* cache, const int32_t* tables, const int32_t* segments, const int32_t* first,
                                 void* out, int64_t num_segments, int64_t longest, int64_t rank, int64_t rot_dim, int64_t row,
                                 int64_t rot_at, int64_t block_size, int64_t max_blocks, int64_t num_blocks, void* stream) {
    const char* fn = "nqh_latent_gather";
    if (!cache || !tables || !segments || !first || !out || !aligned(cache, 16) || !aligned(out, 16))
        return fail(NQH_ERR_ARG, fn, "null or misaligned pointer");
    if (num_segments <= 0 || num_segments > 65535 || longest <= 0 || longest > block_size * max_blocks || rank <= 0 ||
        rot_dim <= 0 || block_size <= 0 || max_blocks <= 0 || num_blocks <= 0 || block_size * max_blocks > kMaxI32)
        return fail(NQH_ERR_ARG, fn, "sizes must be positive, at most 65535 segments, contexts inside their block tables");
    if (rank % 8 || rot_dim % 8 || row % 8 || rot_at % 8 || rot_at < rank || row < rot_at + rot_dim || row > kMaxI32)
        return fail(NQH_ERR_UNSUPPORTED, fn, "sizes and places in a row must be multiples of 8");
    (void)hipGetLastError();
    latent_gather_kernel<<<dim3((unsigned)cdiv(longest, 16), (unsigned)num_segments), dim3(256), 0, (hipStream_t)stream>>>(
        (const uint16_t*)cache, tables, segments, first, (uint16_t*)out, (int)rank, (int)rot_dim, (int)row, (int)rot_at,
        (int)block_size, (int)max_blocks, (int)num_blocks);
    return launched(fn);
}

extern "C" int nqh_head_linear(const void* x, const void* weight, void* y, int64_t rows, int64_t heads, int64_t out_features,
                               int64_t in_features, int64_t x_row, int64_t x_head, int64_t y_row, int64_t y_head, int dtype,
                               void* stream) {
    const char* fn = "nqh_head_linear";
    if (!x || !weight || !y) return fail(NQH_ERR_ARG, fn, "null pointer");
    if (!dtype_ok(dtype)) return fail(NQH_ERR_ARG, fn, "dtype must be NQH_BF16 or NQH_F32");
    if (rows <= 0 || heads <= 0 || heads > 65535 || out_features <= 0 || in_features <= 0 || rows > kMaxI32 ||
        heads * out_features > kMaxI32 || in_features > (1 << 30) || x_row < 0 || x_head < 0 || y_row < 0 || y_head < 0)
        return fail(NQH_ERR_ARG, fn, "sizes must be positive 31-bit counts, at most 65535 heads");
    const bool matrix = dtype == NQH_BF16 && in_features % 8 == 0 && x_row % 8 == 0 && x_head % 8 == 0 && aligned(x, 16) &&
                        aligned(weight, 16);
    if (cdiv(rows, 16) > 65535 || (!matrix && rows > 65535)) return fail(NQH_ERR_UNSUPPORTED, fn, "too many rows");
    (void)hipGetLastError();
    if (matrix) {
        const int waves = (int)(in_features <= kPiece ? 1 : in_features <= 2 * kPiece ? 2 : 4);
        head_linear_kernel<<<dim3((unsigned)cdiv(out_features, 16), (unsigned)heads, (unsigned)cdiv(rows, 16)), dim3(64 * waves),
                             waves * 256 * sizeof(float), (hipStream_t)stream>>>(
            (const uint16_t*)x, (const uint16_t*)weight, (uint16_t*)y, (int)rows, (int)out_features, (int)in_features, x_row,
            x_head, y_row, y_head);
        return launched(fn);
    }
    NQH_WITH_TYPE(dtype, {
        using E = typename T::elem;
        head_linear_any_kernel<T><<<dim3((unsigned)cdiv(out_features, 256), (unsigned)heads, (unsigned)rows), dim3(256), 0,
                                    (hipStream_t)stream>>>((const E*)x, (const E*)weight, (E*)y, (int)rows, (int)out_features,
                                                           (int)in_features, x_row, x_head, y_row, y_head);
    });
    return launched(fn);
}
