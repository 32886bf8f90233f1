// Latent attention: keys and values of all heads are linear images of one cached row per position, [latent | rotated key
// part].  Also the rotation tables and the interleaved (pairwise) rotation it uses.
//
// The second part are the launches of Mix::LatentDecode and Mix::LatentPrefill (bf16; f32 and sizes outside their tilings run
// the stand-alone kernels sequence by sequence).
//
// This file's first part are the stand-alone kernels of the CustomCall targets, for any sizes and either element type.
#include <algorithm>

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

// Workgroup = row.  starts (one row): the row goes to place starts[1] of y, which holds `capacity` rows.
template <typename T>
__global__ __launch_bounds__(256) void latent_rows_kernel(const float* __restrict__ raw, const float* __restrict__ gain, const float* __restrict__ table,
                                                          T* __restrict__ y, int64_t rank, int64_t half, float eps, const int32_t* __restrict__ starts,
                                                          int64_t capacity) {
    __shared__ float red[16];
    const int64_t w = rank + 2 * half;
    const float* row = raw + (int64_t)blockIdx.x * w;
    const float* tab = table + (int64_t)blockIdx.x * 2 * half;
    int64_t at = blockIdx.x;
    if (starts) at = starts[1] < 0 ? 0 : (starts[1] > capacity - 1 ? capacity - 1 : starts[1]);
    T* out = y + at * w;
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

// ---------------------------------------------------------------------------- decode (bf16)
constexpr int kPrepRows = 64;    // latent dimensions per workgroup of the query part
constexpr int kTileP = 64;       // cache rows per step of the attention part
constexpr int kHeadTile = 16;

// Blocks [0, heads * rank / 64): W_uk^T q_n of one head and 64 latent dimensions, for every sequence (the first of a head
// also rotates the q_r part); blocks behind them, one per sequence: the step's cache row.
// ql bf16 [nseq][heads][rank + rot].
__global__ __launch_bounds__(256) void latent_prep_kernel(LatentDecodeArgs a, bf16_t* __restrict__ ql) {
    extern __shared__ float lat_lds[];
    const int t = threadIdx.x;
    const int rank = (int)a.rank, rot = (int)a.rot, dim = (int)a.dim, H = (int)a.heads, hd = dim + rot, w = rank + rot;
    const int rc = (rank + kPrepRows - 1) / kPrepRows;
    if ((int)blockIdx.x >= H * rc) {
        float* red = lat_lds;
        const int b = blockIdx.x - H * rc;
        const float* raw = a.raw + (int64_t)b * w;
        const float* tab = a.table + (int64_t)b * rot;
        int64_t at = a.starts[3 * b + 1];
        at = at < 0 ? 0 : (at > a.capacity - 1 ? a.capacity - 1 : at);
        bf16_t* out = (bf16_t*)a.cache[b] + at * w;
        float q = 0.f;
        for (int i = t; i < rank; i += 256) q += raw[i] * raw[i];
        const float inv = 1.0f / sqrtf(block_sum(q, red) / (float)rank + a.eps);
        for (int i = t; i < rank; i += 256) out[i] = f32_to_bf16((raw[i] * inv) * a.gain[i]);
        for (int i = t; i < rot / 2; i += 256) {
            const float u = raw[rank + 2 * i], v = raw[rank + 2 * i + 1], c = tab[i], s = tab[rot / 2 + i];
            out[rank + 2 * i] = f32_to_bf16(u * c - v * s);
            out[rank + 2 * i + 1] = f32_to_bf16(v * c + u * s);
        }
        return;
    }
    const int h = blockIdx.x / rc, r0 = (blockIdx.x % rc) * kPrepRows;
    const int l16 = t & 15, g = t >> 4;          // 16 groups of 16 lanes; a group takes latent dimensions r0 + g + 16 j
    float* q = lat_lds;                          // [nseq][dim]
    for (int i = t; i < (int)a.nseq * dim; i += 256)
        q[i] = bf16_to_f32(((const bf16_t*)a.x)[((int64_t)(i / dim) * H + h) * hd + i % dim]);
    if (r0 == 0)
        for (int i = t; i < (int)a.nseq * (rot / 2); i += 256) {
            const int b = i / (rot / 2), j = i % (rot / 2);
            const bf16_t* xr = (const bf16_t*)a.x + ((int64_t)b * H + h) * hd + dim;
            const float u = bf16_to_f32(xr[2 * j]), v = bf16_to_f32(xr[2 * j + 1]);
            const float c = a.table[(int64_t)b * rot + j], s = a.table[(int64_t)b * rot + rot / 2 + j];
            bf16_t* o = ql + ((int64_t)b * H + h) * w + rank;
            o[2 * j] = f32_to_bf16(u * c - v * s);
            o[2 * j + 1] = f32_to_bf16(v * c + u * s);
        }
    __syncthreads();
    const bf16_t* wk = (const bf16_t*)a.w_uk;
    const int64_t ldw = (int64_t)H * dim;
    constexpr int J = kPrepRows / 16;
    for (int b = 0; b < (int)a.nseq; ++b) {
        float s[J];
#pragma unroll
        for (int j = 0; j < J; ++j) s[j] = 0.f;
        for (int d = l16 * 8; d < dim; d += 128) {
            float qv[8];
#pragma unroll
            for (int e = 0; e < 8; ++e) qv[e] = q[b * dim + d + e];
#pragma unroll
            for (int j = 0; j < J; ++j) {
                const int r = r0 + g + 16 * j;
                if (r >= rank) continue;
                const uint4 v = *reinterpret_cast<const uint4*>(wk + r * ldw + (int64_t)h * dim + d);
                const uint32_t vw[4] = {v.x, v.y, v.z, v.w};
#pragma unroll
                for (int e = 0; e < 4; ++e) { s[j] += qv[2 * e] * bf16lo(vw[e]); s[j] += qv[2 * e + 1] * bf16hi(vw[e]); }
            }
        }
#pragma unroll
        for (int j = 0; j < J; ++j) {
            const float tot = row16_sum(s[j]);
            const int r = r0 + g + 16 * j;
            if (l16 == 0 && r < rank) ql[((int64_t)b * H + h) * w + r] = f32_to_bf16(tot);
        }
    }
}

// Workgroup = slice of the positions x 16 heads x sequence.  Tiles of 64 cache rows in LDS; scores on the matrix cores (wave w:
// rows 16 w ..), softmax over the tile, weights split into a bf16 value and its remainder, weighted rows on the matrix cores
// (wave w: latent dimensions 16 (w + 4 i) ..).  part f32 [nseq][heads][nsplit][rank + 2]: sums, maximum, weight.
template <int RT>
__global__ __launch_bounds__(256) void latent_partial_kernel(LatentDecodeArgs a, const bf16_t* __restrict__ ql, float* __restrict__ part, int nsplit) {
    extern __shared__ __align__(16) unsigned char lat_smem[];
    const int rank = (int)a.rank, w = rank + (int)a.rot, H = (int)a.heads, ws = w + 8;   // LDS row stride
    bf16_t* rows = reinterpret_cast<bf16_t*>(lat_smem);               // [64][ws]
    bf16_t* qs = rows + kTileP * ws;                                  // [16][ws]
    constexpr int PS = kTileP + 8;
    bf16_t* ph = qs + kHeadTile * ws;                                 // [16][PS] weights
    bf16_t* pl = ph + kHeadTile * PS;                                 // [16][PS] their remainders
    float* sc = reinterpret_cast<float*>(pl + kHeadTile * PS);        // [16][64 + 1]
    float* corr = sc + kHeadTile * (kTileP + 1);                      // [16]
    const int t = threadIdx.x, lane = t & 63, wave = t >> 6, c = lane & 15, kg = lane >> 4;
    const int b = blockIdx.z, h0 = blockIdx.y * kHeadTile, sp = blockIdx.x;
    const int n = min(max(a.pos[b], 0) + 1, (int)a.capacity);
    const int per = ((n + nsplit - 1) / nsplit + 15) / 16 * 16;
    const int p0 = sp * per, p1 = min(p0 + per, n);
    const int hr = H - h0 < kHeadTile ? H - h0 : kHeadTile;           // heads that exist
    float* rec = part + (((int64_t)b * H + h0) * nsplit + sp) * (rank + 2);
    const int64_t rec_h = (int64_t)nsplit * (rank + 2);
    if (p0 >= p1) {   // nothing falls to this slice: an empty record
        for (int i = t; i < hr; i += 256) { rec[i * rec_h + rank] = -INFINITY; rec[i * rec_h + rank + 1] = 0.f; }
        return;
    }
    const int wv = w / 8;                                             // 16-byte words per row
    for (int i = t; i < kHeadTile * wv; i += 256) {
        const int r = i / wv, k = i % wv;
        const uint4 v = *reinterpret_cast<const uint4*>(ql + ((int64_t)b * H + h0 + (r < hr ? r : 0)) * w + 8 * k);
        *reinterpret_cast<uint4*>(qs + r * ws + 8 * k) = v;
    }
    f32x4_m acc[RT];
#pragma unroll
    for (int i = 0; i < RT; ++i) acc[i] = f32x4_m{0.f, 0.f, 0.f, 0.f};
    float m_run = -INFINITY, l_run = 0.f;                             // of head 4 * wave + kg, in all its 16 lanes
    const bf16_t* cache = (const bf16_t*)a.cache[b];
    for (int q0 = p0; q0 < p1; q0 += kTileP) {
        const int np = min(kTileP, p1 - q0);
        const int npad = (np + 31) / 32 * 32;                         // the matrix cores take 32 rows at a time
        __syncthreads();
        for (int i = t; i < npad * wv; i += 256) {
            const int r = i / wv, k = i % wv;
            uint4 v = make_uint4(0u, 0u, 0u, 0u);
            if (r < np) v = *reinterpret_cast<const uint4*>(cache + (int64_t)(q0 + r) * w + 8 * k);
            *reinterpret_cast<uint4*>(rows + r * ws + 8 * k) = v;
        }
        __syncthreads();
        if (wave * 16 < npad) {
            f32x4_m s = {0.f, 0.f, 0.f, 0.f};
            for (int k = 0; k < w; k += 32)
                s = mma16(*reinterpret_cast<const u32x4_m*>(qs + c * ws + k + 8 * kg), *reinterpret_cast<const u32x4_m*>(rows + (wave * 16 + c) * ws + k + 8 * kg), s);
#pragma unroll
            for (int i = 0; i < 4; ++i) sc[(4 * kg + i) * (kTileP + 1) + wave * 16 + c] = s[i] * a.scale;
        }
        __syncthreads();
        {   // head 4 * wave + kg: lanes c take rows c, c + 16, ..
            const int h = 4 * wave + kg;
            float v[4], mx = -INFINITY;
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                v[i] = c + 16 * i < np ? sc[h * (kTileP + 1) + c + 16 * i] : -INFINITY;
                mx = fmaxf(mx, v[i]);
            }
            const float mn = fmaxf(m_run, row16_max(mx));
            float sum = 0.f;
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const float p = expf(v[i] - mn);
                const bf16_t hi = f32_to_bf16(p);
                ph[h * PS + c + 16 * i] = hi;
                pl[h * PS + c + 16 * i] = f32_to_bf16(p - bf16_to_f32(hi));
                sum += p;
            }
            const float cr = expf(m_run - mn);
            l_run = l_run * cr + row16_sum(sum);
            m_run = mn;
            if (c == 0) corr[h] = cr;
        }
        __syncthreads();
        float cr[4];
#pragma unroll
        for (int i = 0; i < 4; ++i) cr[i] = corr[4 * kg + i];
#pragma unroll
        for (int i = 0; i < RT; ++i)
#pragma unroll
            for (int e = 0; e < 4; ++e) acc[i][e] *= cr[e];
        for (int k = 0; k < npad; k += 32) {
            const u32x4_m ah = *reinterpret_cast<const u32x4_m*>(ph + c * PS + k + 8 * kg), al = *reinterpret_cast<const u32x4_m*>(pl + c * PS + k + 8 * kg);
#pragma unroll
            for (int i = 0; i < RT; ++i) {
                const int r = (wave + 4 * i) * 16;
                if (r >= rank) break;
                const u32x4_m bv = lds_operand_t(rows + k * ws + r, ws, lane);
                acc[i] = mma16(ah, bv, acc[i]);
                acc[i] = mma16(al, bv, acc[i]);
            }
        }
    }
#pragma unroll
    for (int i = 0; i < RT; ++i) {
        const int r = (wave + 4 * i) * 16 + c;
        if (r >= rank) break;
#pragma unroll
        for (int e = 0; e < 4; ++e)
            if (4 * kg + e < hr) rec[(4 * kg + e) * rec_h + r] = acc[i][e];
    }
    if (c == 0 && 4 * wave + kg < hr) {
        rec[(4 * wave + kg) * rec_h + rank] = m_run;
        rec[(4 * wave + kg) * rec_h + rank + 1] = l_run;
    }
}

constexpr int kOutV = 32;        // values per workgroup of the output part
// Workgroup = head x 32 values x sequence: the slices' records merged into the weighted latent, times W_uv.
__global__ __launch_bounds__(256) void latent_combine_kernel(LatentDecodeArgs a, const float* __restrict__ part, int nsplit) {
    extern __shared__ float lat_lds[];
    const int rank = (int)a.rank, vdim = (int)a.vdim, H = (int)a.heads;
    float* lat = lat_lds;                        // [rank]
    float* wgt = lat + rank;                     // [nsplit]
    float* red = wgt + nsplit;                   // [256 / kOutV][kOutV]
    const int t = threadIdx.x, h = blockIdx.x, v0 = blockIdx.y * kOutV, b = blockIdx.z;
    const float* rec = part + ((int64_t)b * H + h) * nsplit * (rank + 2);
    float m = -INFINITY, l = 0.f;
    for (int s = 0; s < nsplit; ++s) m = fmaxf(m, rec[(int64_t)s * (rank + 2) + rank]);
    for (int s = 0; s < nsplit; ++s) l += expf(rec[(int64_t)s * (rank + 2) + rank] - m) * rec[(int64_t)s * (rank + 2) + rank + 1];
    if (t < nsplit) wgt[t] = expf(rec[(int64_t)t * (rank + 2) + rank] - m) / l;
    __syncthreads();
    for (int r = t; r < rank; r += 256) {
        float v = 0.f;
        for (int s = 0; s < nsplit; ++s)
            if (wgt[s] != 0.f) v += wgt[s] * rec[(int64_t)s * (rank + 2) + r];   // (an empty slice left its sums unset)
        lat[r] = v;
    }
    __syncthreads();
    const int v = t % kOutV, g = t / kOutV;
    const bf16_t* wv = (const bf16_t*)a.w_uv + (int64_t)h * vdim + v0 + v;
    float s = 0.f;
    if (v0 + v < vdim)
        for (int r = g; r < rank; r += 256 / kOutV) s += lat[r] * bf16_to_f32(wv[(int64_t)r * H * vdim]);
    red[g * kOutV + v] = s;
    __syncthreads();
    if (t < kOutV && v0 + t < vdim) {
        float o = 0.f;
        for (int q = 0; q < 256 / kOutV; ++q) o += red[q * kOutV + t];
        ((bf16_t*)a.ctx)[((int64_t)b * H + h) * vdim + v0 + t] = f32_to_bf16(o);
    }
}

// ---------------------------------------------------------------------------- prompts (bf16)
constexpr int kQTile = 128;      // queries per workgroup: 32 per wave, two 16-row operands that share every key operand
constexpr int kKTile = 64;       // keys per step

// Workgroup = 128 queries x head x sequence.  Keys [unrotated | shared rotated part] and values of 64 positions in LDS; scores,
// online softmax in f32, weights as a bf16 value and its remainder, so that the products with the values see the f32
// weights to 16 bits.  KS: dim + rot in steps of 32 (zero padded), VT: vdim in tiles of 16 (zero padded).
template <int KS, int VT>
__global__ __launch_bounds__(256, 1) void latent_prefill_kernel(LatentPrefillArgs a) {
    extern __shared__ __align__(16) unsigned char lat_smem[];
    constexpr int KSTR = KS * 32 + 8, VSTR = VT * 16 + 8, PSTR = kKTile + 8;
    bf16_t* kt = reinterpret_cast<bf16_t*>(lat_smem);      // [64][KSTR]
    bf16_t* vt = kt + kKTile * KSTR;                       // [64][VSTR]
    bf16_t* pw = vt + kKTile * VSTR;                       // per wave: [2][32][PSTR]
    const int t = threadIdx.x, lane = t & 63, wave = t >> 6, c = lane & 15, kg = lane >> 4;
    const int b = blockIdx.z, h = blockIdx.y, T = a.len[b], r0 = a.row0[b];
    const int q0 = ((int)gridDim.x - 1 - (int)blockIdx.x) * kQTile;   // the longest workgroups first
    if (q0 >= T) return;
    const int dim = (int)a.dim, rot = (int)a.rot, hd = dim + rot, vdim = (int)a.vdim, H = (int)a.heads, w = (int)(a.rank + a.rot);
    bf16_t* ph = pw + wave * 2 * 32 * PSTR;
    bf16_t* pl = ph + 32 * PSTR;

    // queries: rotated on the way in, rounded once; rows behind the prompt repeat its last row and are not stored
    u32x4_m q[2][KS];
#pragma unroll
    for (int i = 0; i < 2; ++i) {
        const int row = r0 + min(q0 + wave * 32 + i * 16 + c, T - 1);
        const bf16_t* src = (const bf16_t*)a.x + ((int64_t)row * H + h) * hd;
        const float* tab = a.table + (int64_t)row * rot;
#pragma unroll
        for (int k = 0; k < KS; ++k) {
            const int d = 32 * k + 8 * kg;
            u32x4_m v = {0u, 0u, 0u, 0u};
            if (d < hd) {
                v = *reinterpret_cast<const u32x4_m*>(src + d);
                if (d >= dim) {
#pragma unroll
                    for (int e = 0; e < 4; ++e) {
                        const float cs = tab[(d - dim) / 2 + e], sn = tab[rot / 2 + (d - dim) / 2 + e];
                        const float x0 = bf16lo(v[e]), x1 = bf16hi(v[e]);
                        v[e] = pack_bf16_hw(x0 * cs - x1 * sn, x1 * cs + x0 * sn);
                    }
                }
            }
            q[i][k] = v;
        }
    }
    f32x4_m o[2][VT];
    float m[2][4], l[2][4];
#pragma unroll
    for (int i = 0; i < 2; ++i) {
#pragma unroll
        for (int v = 0; v < VT; ++v) o[i][v] = f32x4_m{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int e = 0; e < 4; ++e) { m[i][e] = -INFINITY; l[i][e] = 0.f; }
    }
    const float scale2 = a.scale * 1.44269504f;            // weights as powers of two
    const int kend = min(q0 + kQTile, T);
    const int myq = q0 + wave * 32;                        // the wave's first query
    constexpr int KW = KS * 4, VW = VT * 2;                // 16-byte words per staged row
    for (int k0 = 0; k0 < kend; k0 += kKTile) {
        __syncthreads();
        for (int i = t; i < kKTile * KW; i += 256) {
            const int r = i / KW, d = (i % KW) * 8, pos = k0 + r;
            uint4 v = make_uint4(0u, 0u, 0u, 0u);
            if (pos < kend && d < hd)
                v = d < dim ? *reinterpret_cast<const uint4*>((const bf16_t*)a.k + ((int64_t)(r0 + pos) * H + h) * dim + d)
                            : *reinterpret_cast<const uint4*>((const bf16_t*)a.rows + (int64_t)(r0 + pos) * w + (int)a.rank + d - dim);
            *reinterpret_cast<uint4*>(kt + r * KSTR + d) = v;
        }
        for (int i = t; i < kKTile * VW; i += 256) {
            const int r = i / VW, d = (i % VW) * 8, pos = k0 + r;
            uint4 v = make_uint4(0u, 0u, 0u, 0u);
            if (pos < kend && d < vdim) v = *reinterpret_cast<const uint4*>((const bf16_t*)a.v + ((int64_t)(r0 + pos) * H + h) * vdim + d);
            *reinterpret_cast<uint4*>(vt + r * VSTR + d) = v;
        }
        __syncthreads();
        if (k0 > myq + 31) continue;                       // all keys of the step lie ahead of the wave's queries
        f32x4_m s[2][4];
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            s[0][j] = s[1][j] = f32x4_m{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int k = 0; k < KS; ++k) {
                const u32x4_m kv = *reinterpret_cast<const u32x4_m*>(kt + (16 * j + c) * KSTR + 32 * k + 8 * kg);
                s[0][j] = mma16(q[0][k], kv, s[0][j]);
                s[1][j] = mma16(q[1][k], kv, s[1][j]);
            }
        }
        const bool edge = k0 + kKTile - 1 > myq;           // some key lies ahead of some query (or behind the prompt)
#pragma unroll
        for (int i = 0; i < 2; ++i) {
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int qi = myq + i * 16 + 4 * kg + e;
                float x[4], mx = -INFINITY;
#pragma unroll
                for (int j = 0; j < 4; ++j) {
                    x[j] = s[i][j][e] * scale2;
                    if (edge && k0 + 16 * j + c > qi) x[j] = -INFINITY;
                    mx = fmaxf(mx, x[j]);
                }
                const float mn = fmaxf(m[i][e], row16_max(mx));   // finite: key k0 <= myq + 31 may lie ahead of qi only after key 0 was seen
                const float corr = __builtin_amdgcn_exp2f(m[i][e] - mn);
                float sum = 0.f;
#pragma unroll
                for (int j = 0; j < 4; ++j) {
                    const float p = __builtin_amdgcn_exp2f(x[j] - mn);
                    sum += p;
                    const uint32_t hi = pack_bf16_hw(p, 0.f) & 0xFFFFu;
                    ph[(i * 16 + 4 * kg + e) * PSTR + 16 * j + c] = (bf16_t)hi;
                    pl[(i * 16 + 4 * kg + e) * PSTR + 16 * j + c] = (bf16_t)(pack_bf16_hw(p - __uint_as_float(hi << 16), 0.f) & 0xFFFFu);
                }
                l[i][e] = l[i][e] * corr + row16_sum(sum);
                m[i][e] = mn;
#pragma unroll
                for (int v = 0; v < VT; ++v) o[i][v][e] *= corr;
            }
        }
        // (the weights are the wave's own: its LDS operations complete in order)
        asm volatile("" ::: "memory");
#pragma unroll
        for (int k = 0; k < kKTile / 32; ++k) {
            u32x4_m p0[2], p1[2];
#pragma unroll
            for (int i = 0; i < 2; ++i) {
                p0[i] = *reinterpret_cast<const u32x4_m*>(ph + (i * 16 + c) * PSTR + 32 * k + 8 * kg);
                p1[i] = *reinterpret_cast<const u32x4_m*>(pl + (i * 16 + c) * PSTR + 32 * k + 8 * kg);
            }
#pragma unroll
            for (int v = 0; v < VT; ++v) {
                const u32x4_m vv = lds_operand_t(vt + 32 * k * VSTR + 16 * v, VSTR, lane);
#pragma unroll
                for (int i = 0; i < 2; ++i) {
                    o[i][v] = mma16(p0[i], vv, o[i][v]);
                    o[i][v] = mma16(p1[i], vv, o[i][v]);
                }
            }
        }
        asm volatile("" ::: "memory");
    }
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const int qi = myq + i * 16 + 4 * kg + e;
            if (qi >= T) continue;
            const float inv = 1.0f / l[i][e];
            bf16_t* out = (bf16_t*)a.ctx + ((int64_t)(r0 + qi) * H + h) * vdim;
#pragma unroll
            for (int v = 0; v < VT; ++v)
                if (16 * v + c < vdim) out[16 * v + c] = f32_to_bf16(o[i][v][e] * inv);
        }
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
    if (dtype == 0) latent_rows_kernel<float><<<(unsigned)rows, 256, 0, s>>>(raw, gain, table, (float*)y, rank, half, eps, nullptr, 0);
    else latent_rows_kernel<bf16_t><<<(unsigned)rows, 256, 0, s>>>(raw, gain, table, (bf16_t*)y, rank, half, eps, nullptr, 0);
}
static void latent_append(hipStream_t s, int dtype, const float* raw, const float* gain, const float* table, const int32_t* starts, void* cache,
                          int64_t capacity, int64_t rank, int64_t half, float eps) {
    if (dtype == 0) latent_rows_kernel<float><<<1, 256, 0, s>>>(raw, gain, table, (float*)cache, rank, half, eps, starts, capacity);
    else latent_rows_kernel<bf16_t><<<1, 256, 0, s>>>(raw, gain, table, (bf16_t*)cache, rank, half, eps, starts, capacity);
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


static size_t lat_align(size_t n) { return (n + 255) / 256 * 256; }
// slices of the positions: 32 rows each up to 32 of them, fewer where the batch fills the chip by itself
static int latent_nsplit(int64_t nseq, int64_t capacity, int64_t heads) {
    const int64_t blocks = nseq * cdiv_l(heads, kHeadTile);
    int64_t n = std::min<int64_t>(cdiv_l(capacity, 32), 32);
    while (n > 4 && blocks * n > 1024) n = (n + 1) / 2;
    return (int)std::max<int64_t>(n, 1);
}
static size_t latent_partial_lds(int64_t w) {
    return (size_t)((kTileP + kHeadTile) * (w + 8) + 2 * kHeadTile * (kTileP + 8)) * 2 + (kHeadTile * (kTileP + 1) + kHeadTile) * 4;
}
static bool latent_fast(int dtype, int64_t heads, int64_t dim, int64_t rot, int64_t rank) {
    return dtype == 2 && heads >= 1 && dim % 8 == 0 && rot % 2 == 0 && rank % 16 == 0 && (rank + rot) % 32 == 0 && rank <= 1024 && dim <= 512 &&
           latent_partial_lds(rank + rot) <= 160 * 1024;
}
size_t latent_decode_scratch_bytes(int dtype, int64_t nseq, int64_t capacity, int64_t heads, int64_t dim, int64_t rot, int64_t rank) {
    if (latent_fast(dtype, heads, dim, rot, rank))
        return lat_align((size_t)(nseq * heads * (rank + rot)) * 2) + (size_t)(nseq * heads * (rank + 2)) * 32 * sizeof(float);
    const size_t es = dtype == 0 ? 4 : 2;
    return lat_align((size_t)(nseq * heads * (dim + rot)) * es);
}
int latent_decode(hipStream_t s, const LatentDecodeArgs& a) {
    const size_t es = a.dtype == 0 ? 4 : 2;
    const int64_t w = a.rank + a.rot;
    if (latent_fast(a.dtype, a.heads, a.dim, a.rot, a.rank)) {
        bf16_t* ql = (bf16_t*)a.scratch;
        float* part = (float*)((char*)a.scratch + lat_align((size_t)(a.nseq * a.heads * w) * 2));
        const int ns = latent_nsplit(a.nseq, a.capacity, a.heads);
        const int64_t rc = cdiv_l(a.rank, kPrepRows);
        latent_prep_kernel<<<(unsigned)(a.heads * rc + (a.raw ? a.nseq : 0)), 256, (size_t)std::max<int64_t>(a.nseq * a.dim, 16) * 4, s>>>(a, ql);
        const size_t lds = latent_partial_lds(w);
        const dim3 grid((unsigned)ns, (unsigned)cdiv_l(a.heads, kHeadTile), (unsigned)a.nseq);
        const int64_t rt = cdiv_l(a.rank / 16, 4);
#define GPTRS_PARTIAL(RT) do { with_lds(latent_partial_kernel<RT>, lds); latent_partial_kernel<RT><<<grid, 256, lds, s>>>(a, ql, part, ns); } while (0)
        if (rt <= 2) GPTRS_PARTIAL(2);
        else if (rt <= 4) GPTRS_PARTIAL(4);
        else if (rt <= 8) GPTRS_PARTIAL(8);
        else GPTRS_PARTIAL(16);
#undef GPTRS_PARTIAL
        latent_combine_kernel<<<dim3((unsigned)a.heads, (unsigned)cdiv_l(a.vdim, kOutV), (unsigned)a.nseq), 256, (size_t)(a.rank + ns + 256) * 4, s>>>(a, part, ns);
        return 3;
    }
    rope_pairs(s, a.dtype, a.x, a.table, a.scratch, a.nseq, a.heads, a.dim + a.rot, a.dim, a.rot / 2);
    int n = 1;
    for (int64_t b = 0; b < a.nseq; ++b) {
        if (a.raw) {
            latent_append(s, a.dtype, a.raw + b * w, a.gain, a.table + b * a.rot, a.starts + 3 * b, a.cache[b], a.capacity, a.rank, a.rot / 2, a.eps);
            ++n;
        }
        LatentAttnArgs q{};
        q.dtype = a.dtype;
        q.q = (const char*)a.scratch + (size_t)(b * a.heads * (a.dim + a.rot)) * es;
        q.rows = a.cache[b]; q.w_uk = a.w_uk; q.w_uv = a.w_uv; q.start = a.pos + b;
        q.ctx = (char*)a.ctx + (size_t)(b * a.heads * a.vdim) * es;
        q.t = 1; q.capacity = a.capacity; q.heads = a.heads; q.dim = a.dim; q.rot = a.rot; q.rank = a.rank; q.vdim = a.vdim; q.scale = a.scale;
        latent_attn(s, q);
        ++n;
    }
    return n;
}

size_t latent_prefill_scratch_bytes(int dtype, int64_t total, int64_t heads, int64_t dim, int64_t rot, int64_t vdim) {
    (void)vdim;
    return lat_align((size_t)(total * heads * (dim + rot)) * (dtype == 0 ? 4 : 2));
}
template <int KS, int VT>
static void launch_prefill(hipStream_t s, const LatentPrefillArgs& a, int64_t longest) {
    constexpr int lds = (kKTile * (KS * 32 + 8) + kKTile * (VT * 16 + 8) + 4 * 2 * 32 * (kKTile + 8)) * 2;
    static_assert(lds <= 160 * 1024, "LDS of one CU");
    with_lds(latent_prefill_kernel<KS, VT>, lds);
    latent_prefill_kernel<KS, VT><<<dim3((unsigned)cdiv_l(longest, kQTile), (unsigned)a.heads, (unsigned)a.nseq), 256, lds, s>>>(a);
}
template <int KS>
static void launch_prefill_v(hipStream_t s, const LatentPrefillArgs& a, int64_t longest) {
    if (a.vdim <= 64) launch_prefill<KS, 4>(s, a, longest);
    else if (a.vdim <= 128) launch_prefill<KS, 8>(s, a, longest);
    else launch_prefill<KS, 16>(s, a, longest);
}
int latent_prefill(hipStream_t s, const LatentPrefillArgs& a) {
    if (a.dtype == 2 && a.dim % 8 == 0 && a.rot % 8 == 0 && a.rank % 8 == 0 && a.vdim % 8 == 0 && a.dim + a.rot <= 256 && a.vdim <= 256) {
        int64_t longest = 0;
        for (int b = 0; b < a.nseq; ++b) longest = std::max<int64_t>(longest, a.len[b]);
        const int64_t ks = cdiv_l(a.dim + a.rot, 32);
        if (ks <= 2) launch_prefill_v<2>(s, a, longest);
        else if (ks <= 3) launch_prefill_v<3>(s, a, longest);
        else if (ks <= 4) launch_prefill_v<4>(s, a, longest);
        else if (ks <= 6) launch_prefill_v<6>(s, a, longest);
        else launch_prefill_v<8>(s, a, longest);
        return 1;
    }
    const size_t es = a.dtype == 0 ? 4 : 2;
    const int64_t hd = a.heads * (a.dim + a.rot), w = a.rank + a.rot;
    int n = 0;
    for (int b = 0; b < a.nseq; ++b) {
        const int64_t r = a.row0[b];
        char* q = (char*)a.scratch + (size_t)(r * hd) * es;
        rope_pairs(s, a.dtype, (const char*)a.x + (size_t)(r * hd) * es, a.table + r * a.rot, q, a.len[b], a.heads, a.dim + a.rot, a.dim, a.rot / 2);
        LatentAttnXArgs x{};
        x.dtype = a.dtype;
        x.q = q;
        x.k = (const char*)a.k + (size_t)(r * a.heads * a.dim) * es;
        x.v = (const char*)a.v + (size_t)(r * a.heads * a.vdim) * es;
        x.rows = (const char*)a.rows + (size_t)(r * w) * es;
        x.ctx = (char*)a.ctx + (size_t)(r * a.heads * a.vdim) * es;
        x.t = x.l = a.len[b];
        x.heads = a.heads; x.dim = a.dim; x.rot = a.rot; x.rank = a.rank; x.vdim = a.vdim; x.scale = a.scale;
        latent_attn_expanded(s, x);
        n += 2;
    }
    return n;
}

}  // namespace k
}  // namespace gptrs
