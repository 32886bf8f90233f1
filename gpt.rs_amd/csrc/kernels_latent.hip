// Latent attention: keys and values of all heads are linear images of one cached row per position, [latent | rotated key
// part].  Also the rotation tables and the interleaved (pairwise) rotation it uses.
//
// This file's first part are the stand-alone kernels of the CustomCall targets, for any sizes and either element type.
#include "kernels.hpp"
#include "device_utils.hpp"

namespace gptrs {
namespace k {

namespace {

inline int64_t cdiv_l(int64_t a, int64_t b) { return (a + b - 1) / b; }

// the angle is formed and reduced in f64: at position 10^5 an f32 product is off by 0.004 rad
__global__ __launch_bounds__(256) void rope_table_kernel(const int32_t* __restrict__ pos, const float* __restrict__ freqs, float mag,
                                                         float* __restrict__ out, int64_t rows, int64_t half) {
    const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (i >= rows * half) return;
    const int64_t r = i / half, c = i % half;
    double sn, cs;
    sincos((double)pos[r] * (double)freqs[c], &sn, &cs);
    out[r * 2 * half + c] = (float)cs * mag;
    out[r * 2 * half + half + c] = (float)sn * mag;
}

template <typename T>
__global__ __launch_bounds__(256) void rope_pairs_kernel(const T* __restrict__ x, const float* __restrict__ table, T* __restrict__ y, int64_t pairs,
                                                         int64_t per_row, int64_t head_dim, int64_t offset, int64_t half) {
    const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;   // element pair; head_dim and offset are even
    if (i >= pairs) return;
    const int64_t r = (2 * i) / per_row, d = (2 * i) % head_dim - offset;
    float u = Elem<T>::ld(x, 2 * i), v = Elem<T>::ld(x, 2 * i + 1);
    if (d >= 0 && d < 2 * half) {
        const float c = table[r * 2 * half + d / 2], s = table[r * 2 * half + half + d / 2];
        const float a = u * c - v * s, b = v * c + u * s;
        u = a; v = b;
    }
    Elem<T>::st(y, 2 * i, u);
    Elem<T>::st(y, 2 * i + 1, v);
}

// Workgroup = row.
template <typename T>
__global__ __launch_bounds__(256) void latent_rows_kernel(const float* __restrict__ raw, const float* __restrict__ gain, const float* __restrict__ table,
                                                          T* __restrict__ y, int64_t rank, int64_t half, float eps) {
    __shared__ float red[16];
    const int64_t w = rank + 2 * half;
    const float* row = raw + (int64_t)blockIdx.x * w;
    const float* tab = table + (int64_t)blockIdx.x * 2 * half;
    T* out = y + (int64_t)blockIdx.x * w;
    float q = 0.f;
    for (int64_t i = threadIdx.x; i < rank; i += 256) q += row[i] * row[i];
    const float inv = 1.0f / sqrtf(block_sum(q, red) / (float)rank + eps);
    for (int64_t i = threadIdx.x; i < rank; i += 256) Elem<T>::st(out, i, (row[i] * inv) * gain[i]);
    for (int64_t i = threadIdx.x; i < half; i += 256) {
        const float u = row[rank + 2 * i], v = row[rank + 2 * i + 1], c = tab[i], s = tab[half + i];
        Elem<T>::st(out, rank + 2 * i, u * c - v * s);
        Elem<T>::st(out, rank + 2 * i + 1, v * c + u * s);
    }
}

// Workgroup = head x query.  Keys in tiles of 256, one per thread; online softmax; the weighted latent in LDS.
template <typename T>
__global__ __launch_bounds__(256) void latent_attn_kernel(LatentAttnArgs a) {
    extern __shared__ float lat_lds[];
    float* q = lat_lds;                          // [dim + rot]
    float* ql = q + a.dim + a.rot;               // [rank] W_uk^T q_n
    float* acc = ql + a.rank;                    // [rank]
    float* pr = acc + a.rank;                    // [256]
    float* red = pr + 256;                       // [16]
    const int t = threadIdx.x;
    const int64_t i = blockIdx.x, h = blockIdx.y, hd = a.dim + a.rot, w = a.rank + a.rot;
    const T* qrow = (const T*)a.q + (i * a.heads + h) * hd;
    for (int64_t d = t; d < hd; d += 256) q[d] = Elem<T>::ld(qrow, d);
    __syncthreads();
    for (int64_t r = t; r < a.rank; r += 256) {
        const T* wr = (const T*)a.w_uk + r * a.heads * a.dim + h * a.dim;
        float s = 0.f;
        for (int64_t d = 0; d < a.dim; ++d) s += q[d] * Elem<T>::ld(wr, d);
        ql[r] = s;
        acc[r] = 0.f;
    }
    __syncthreads();
    int64_t n = (int64_t)a.start[0] + i + 1;
    n = n < 1 ? 1 : (n > a.capacity ? a.capacity : n);
    float m = -INFINITY, l = 0.f;
    for (int64_t j0 = 0; j0 < n; j0 += 256) {
        const int64_t j = j0 + t;
        float s = -INFINITY;
        if (j < n) {
            const T* row = (const T*)a.rows + j * w;
            s = 0.f;
            for (int64_t r = 0; r < a.rank; ++r) s += ql[r] * Elem<T>::ld(row, r);
            for (int64_t r = 0; r < a.rot; ++r) s += q[a.dim + r] * Elem<T>::ld(row, a.rank + r);
            s *= a.scale;
        }
        const float mn = fmaxf(m, block_max(s, red));
        const float corr = expf(m - mn), p = expf(s - mn);
        pr[t] = p;
        l = l * corr + block_sum(p, red);
        m = mn;
        const int nj = (int)(n - j0 < 256 ? n - j0 : 256);
        for (int64_t r = t; r < a.rank; r += 256) {
            float v = acc[r] * corr;
            for (int jj = 0; jj < nj; ++jj) v += pr[jj] * Elem<T>::ld((const T*)a.rows, (j0 + jj) * w + r);
            acc[r] = v;
        }
        __syncthreads();
    }
    const float inv = 1.0f / l;
    for (int64_t v = t; v < a.vdim; v += 256) {
        const T* wv = (const T*)a.w_uv + h * a.vdim + v;
        float s = 0.f;
        for (int64_t r = 0; r < a.rank; ++r) s += (acc[r] * inv) * Elem<T>::ld(wv, r * a.heads * a.vdim);
        Elem<T>::st((T*)a.ctx, (i * a.heads + h) * a.vdim + v, s);
    }
}

template <typename T>
__global__ __launch_bounds__(256) void latent_attn_x_kernel(LatentAttnXArgs a) {
    extern __shared__ float lat_lds[];
    float* q = lat_lds;                          // [dim + rot]
    float* acc = q + a.dim + a.rot;              // [vdim]
    float* pr = acc + a.vdim;                    // [256]
    float* red = pr + 256;                       // [16]
    const int t = threadIdx.x;
    const int64_t i = blockIdx.x, h = blockIdx.y, hd = a.dim + a.rot, w = a.rank + a.rot;
    const T* qrow = (const T*)a.q + (i * a.heads + h) * hd;
    for (int64_t d = t; d < hd; d += 256) q[d] = Elem<T>::ld(qrow, d);
    for (int64_t v = t; v < a.vdim; v += 256) acc[v] = 0.f;
    __syncthreads();
    const int64_t n = a.l - a.t + i + 1;
    float m = -INFINITY, l = 0.f;
    for (int64_t j0 = 0; j0 < n; j0 += 256) {
        const int64_t j = j0 + t;
        float s = -INFINITY;
        if (j < n) {
            const T* kr = (const T*)a.k + (j * a.heads + h) * a.dim;
            const T* rr = (const T*)a.rows + j * w + a.rank;
            s = 0.f;
            for (int64_t d = 0; d < a.dim; ++d) s += q[d] * Elem<T>::ld(kr, d);
            for (int64_t d = 0; d < a.rot; ++d) s += q[a.dim + d] * Elem<T>::ld(rr, d);
            s *= a.scale;
        }
        const float mn = fmaxf(m, block_max(s, red));
        const float corr = expf(m - mn), p = expf(s - mn);
        pr[t] = p;
        l = l * corr + block_sum(p, red);
        m = mn;
        const int nj = (int)(n - j0 < 256 ? n - j0 : 256);
        for (int64_t v = t; v < a.vdim; v += 256) {
            float o = acc[v] * corr;
            for (int jj = 0; jj < nj; ++jj) o += pr[jj] * Elem<T>::ld((const T*)a.v, ((j0 + jj) * a.heads + h) * a.vdim + v);
            acc[v] = o;
        }
        __syncthreads();
    }
    const float inv = 1.0f / l;
    for (int64_t v = t; v < a.vdim; v += 256) Elem<T>::st((T*)a.ctx, (i * a.heads + h) * a.vdim + v, acc[v] * inv);
}

template <typename F>
void with_lds(F kern, size_t bytes) { (void)hipFuncSetAttribute((const void*)kern, hipFuncAttributeMaxDynamicSharedMemorySize, (int)bytes); }

}  // namespace

void rope_table(hipStream_t s, const int32_t* positions, const float* freqs, float magnitude, float* out, int64_t rows, int64_t half) {
    if (rows <= 0 || half <= 0) return;
    rope_table_kernel<<<(unsigned)cdiv_l(rows * half, 256), 256, 0, s>>>(positions, freqs, magnitude, out, rows, half);
}
void rope_pairs(hipStream_t s, int dtype, const void* x, const float* table, void* y, int64_t rows, int64_t heads, int64_t head_dim, int64_t offset,
                int64_t half) {
    const int64_t per_row = heads * head_dim, pairs = rows * per_row / 2;
    if (pairs <= 0) return;
    const unsigned g = (unsigned)cdiv_l(pairs, 256);
    if (dtype == 0) rope_pairs_kernel<float><<<g, 256, 0, s>>>((const float*)x, table, (float*)y, pairs, per_row, head_dim, offset, half);
    else rope_pairs_kernel<bf16_t><<<g, 256, 0, s>>>((const bf16_t*)x, table, (bf16_t*)y, pairs, per_row, head_dim, offset, half);
}
void latent_rows(hipStream_t s, int dtype, const float* raw, const float* gain, const float* table, void* y, int64_t rows, int64_t rank, int64_t half,
                 float eps) {
    if (rows <= 0) return;
    if (dtype == 0) latent_rows_kernel<float><<<(unsigned)rows, 256, 0, s>>>(raw, gain, table, (float*)y, rank, half, eps);
    else latent_rows_kernel<bf16_t><<<(unsigned)rows, 256, 0, s>>>(raw, gain, table, (bf16_t*)y, rank, half, eps);
}
void latent_attn(hipStream_t s, const LatentAttnArgs& a) {
    if (a.t <= 0) return;
    const size_t lds = (size_t)(a.dim + a.rot + 2 * a.rank + 256 + 16) * sizeof(float);
    const dim3 grid((unsigned)a.t, (unsigned)a.heads);
    if (a.dtype == 0) { with_lds(latent_attn_kernel<float>, lds); latent_attn_kernel<float><<<grid, 256, lds, s>>>(a); }
    else { with_lds(latent_attn_kernel<bf16_t>, lds); latent_attn_kernel<bf16_t><<<grid, 256, lds, s>>>(a); }
}
void latent_attn_expanded(hipStream_t s, const LatentAttnXArgs& a) {
    if (a.t <= 0) return;
    const size_t lds = (size_t)(a.dim + a.rot + a.vdim + 256 + 16) * sizeof(float);
    const dim3 grid((unsigned)a.t, (unsigned)a.heads);
    if (a.dtype == 0) { with_lds(latent_attn_x_kernel<float>, lds); latent_attn_x_kernel<float><<<grid, 256, lds, s>>>(a); }
    else { with_lds(latent_attn_x_kernel<bf16_t>, lds); latent_attn_x_kernel<bf16_t><<<grid, 256, lds, s>>>(a); }
}

}  // namespace k
}  // namespace gptrs
