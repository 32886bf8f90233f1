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

// The same one element per thread, for heads of an odd size
template <typename T>
__global__ __launch_bounds__(256) void rope_pairs_any_kernel(const T* __restrict__ x, const float* __restrict__ table, T* __restrict__ y, int64_t n,
                                                             int64_t per_row, int64_t head_dim, int64_t offset, int64_t half) {
    const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (i >= n) return;
    const int64_t r = i / per_row, d = i % per_row % head_dim - offset;
    float v = Elem<T>::ld(x, i);
    if (d >= 0 && d < 2 * half) {
        const float c = table[r * 2 * half + d / 2], s = table[r * 2 * half + half + d / 2], w = Elem<T>::ld(x, d & 1 ? i - 1 : i + 1);
        v = d & 1 ? v * c + w * s : v * c - w * s;
    }
    Elem<T>::st(y, i, v);
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
    constexpr int J = kPrepRows / 16, BT = 8;    // a word of W_uk serves up to 8 sequences
    for (int b0 = 0; b0 < (int)a.nseq; b0 += BT) {
        float s[BT][J];
#pragma unroll
        for (int b = 0; b < BT; ++b)
#pragma unroll
            for (int j = 0; j < J; ++j) s[b][j] = 0.f;
        for (int d = l16 * 8; d < dim; d += 128) {
            u32x4_m x[J];
#pragma unroll
            for (int j = 0; j < J; ++j) x[j] = *reinterpret_cast<const u32x4_m*>(wk + (int64_t)min(r0 + g + 16 * j, rank - 1) * ldw + (int64_t)h * dim + d);
#pragma unroll
            for (int b = 0; b < BT; ++b) {
                if (b0 + b >= (int)a.nseq) break;
                const float4 qa = *reinterpret_cast<const float4*>(q + (b0 + b) * dim + d), qb = *reinterpret_cast<const float4*>(q + (b0 + b) * dim + d + 4);
#pragma unroll
                for (int j = 0; j < J; ++j) {
                    float v = s[b][j];
                    v += qa.x * bf16lo(x[j][0]); v += qa.y * bf16hi(x[j][0]);
                    v += qa.z * bf16lo(x[j][1]); v += qa.w * bf16hi(x[j][1]);
                    v += qb.x * bf16lo(x[j][2]); v += qb.y * bf16hi(x[j][2]);
                    v += qb.z * bf16lo(x[j][3]); v += qb.w * bf16hi(x[j][3]);
                    s[b][j] = v;
                }
            }
        }
#pragma unroll
        for (int b = 0; b < BT; ++b) {
            if (b0 + b >= (int)a.nseq) break;
#pragma unroll
            for (int j = 0; j < J; ++j) {
                const float tot = row16_sum(s[b][j]);
                const int r = r0 + g + 16 * j;
                if (l16 == 0 && r < rank) ql[((int64_t)(b0 + b) * H + h) * w + r] = f32_to_bf16(tot);
            }
        }
    }
}

// Workgroup = slice of the positions x sequence x up to 4 waves; a wave = 16 heads and 16 RT latent dimensions of their result, and
// all waves share the cache rows, 64 at a time in LDS.  Scores transposed (rows: positions, columns: heads), so a lane holds 16
// positions of one head: softmax in registers, and the weights (a bf16 value and its remainder) feed the product with the
// cached latents from there.  part f32 [nseq][heads][nsplit][rank + 2]: sums, maximum (base 2), weight.
template <int RT>
__global__ __launch_bounds__(256) void latent_partial_kernel(LatentDecodeArgs a, const bf16_t* __restrict__ ql, float* __restrict__ part, int nsplit) {
    extern __shared__ __align__(16) unsigned char lat_smem[];
    const int rank = (int)a.rank, w = rank + (int)a.rot, H = (int)a.heads, ws = w + 8;   // LDS row stride
    bf16_t* rows = reinterpret_cast<bf16_t*>(lat_smem);               // [32][ws]
    bf16_t* q0s = rows + kTileP * ws;                                 // queries of the workgroup's tiles of 16 heads, [16][ws] each
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, W = (int)blockDim.x >> 6, c = lane & 15, kg = lane >> 4;
    const int rparts = (rank + 16 * RT - 1) / (16 * RT), units = (H + kHeadTile - 1) / kHeadTile * rparts;
    const int unit = (int)blockIdx.y * W + wave;
    const bool live = unit < units;
    const int ht0 = (int)blockIdx.y * W / rparts, ht1 = min((int)blockIdx.y * W + W - 1, units - 1) / rparts;   // the workgroup's tiles of heads
    const int ht = live ? unit / rparts : ht0, rp0 = live ? (unit % rparts) * 16 * RT : 0;
    const int b = blockIdx.z, h0 = ht * kHeadTile, sp = blockIdx.x;
    const int n = min(max(a.pos[b], 0) + 1, (int)a.capacity);
    const int per = ((n + nsplit - 1) / nsplit + 15) / 16 * 16;
    const int p0 = sp * per, p1 = min(p0 + per, n);
    const int hr = !live ? 0 : (H - h0 < kHeadTile ? H - h0 : kHeadTile);   // heads that exist
    float* rec = part + (((int64_t)b * H + h0) * nsplit + sp) * (rank + 2);
    const int64_t rec_h = (int64_t)nsplit * (rank + 2);
    if (p0 >= p1) {   // nothing falls to this slice: its weight is zero, and whoever merges does not use its sums
        if (lane < hr && rp0 == 0) { rec[lane * rec_h + rank] = -INFINITY; rec[lane * rec_h + rank + 1] = 0.f; }
        return;
    }
    const int wv = w / 8;                                             // 16-byte words per row (a multiple of 4)
    const bf16_t* cache = (const bf16_t*)a.cache[b];
    // 8 threads to a row: a thread takes every eighth word of it
    auto stage = [&](const bf16_t* src, bf16_t* dst, int nrows, int last) {   // rows behind `last` repeat it
        constexpr int R = 2, U = 10;                                  // rows x words per thread requested before the first is stored
        for (int r0 = tid >> 3; r0 < nrows; r0 += 8 * W * R)
            for (int k0 = tid & 7; k0 < wv; k0 += 8 * U) {
                u32x4_m v[R][U];
#pragma unroll
                for (int i = 0; i < R; ++i) {
                    const u32x4_m* from = reinterpret_cast<const u32x4_m*>(src + (int64_t)min(r0 + 8 * W * i, last) * w);
#pragma unroll
                    for (int u = 0; u < U; ++u) v[i][u] = from[min(k0 + 8 * u, wv - 1)];
                }
#pragma unroll
                for (int i = 0; i < R; ++i) {
                    u32x4_m* to = reinterpret_cast<u32x4_m*>(dst + (r0 + 8 * W * i) * ws);
#pragma unroll
                    for (int u = 0; u < U; ++u)
                        if (r0 + 8 * W * i < nrows && k0 + 8 * u < wv) to[k0 + 8 * u] = v[i][u];
                }
            }
    };
    stage(ql + ((int64_t)b * H + ht0 * kHeadTile) * w, q0s, (ht1 - ht0 + 1) * kHeadTile, H - 1 - ht0 * kHeadTile);
    const bf16_t* qs = q0s + (ht - ht0) * kHeadTile * ws;
    f32x4_m acc[RT];                                                  // rows: latent dimensions, column: head c
#pragma unroll
    for (int i = 0; i < RT; ++i) acc[i] = f32x4_m{0.f, 0.f, 0.f, 0.f};
    float m_run = -INFINITY, l_run = 0.f;                             // of head c, in its four lanes
    const float scale2 = a.scale * 1.44269504f;
    for (int q0 = p0; q0 < p1; q0 += kTileP) {
        const int np = min(kTileP, p1 - q0);
        __syncthreads();
        stage(cache + (int64_t)q0 * w, rows, kTileP, np - 1);
        __syncthreads();
        constexpr int PT = kTileP / 16;
        f32x4_m sc[PT];
#pragma unroll
        for (int j = 0; j < PT; ++j) sc[j] = f32x4_m{0.f, 0.f, 0.f, 0.f};
        for (int k = 0; k < w; k += 32) {
            const u32x4_m qv = *reinterpret_cast<const u32x4_m*>(qs + c * ws + k + 8 * kg);
#pragma unroll
            for (int j = 0; j < PT; ++j) sc[j] = mma16(*reinterpret_cast<const u32x4_m*>(rows + (16 * j + c) * ws + k + 8 * kg), qv, sc[j]);
        }
        float mx = -INFINITY;
#pragma unroll
        for (int j = 0; j < PT; ++j)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                sc[j][e] = 16 * j + 4 * kg + e < np ? sc[j][e] * scale2 : -INFINITY;
                mx = fmaxf(mx, sc[j][e]);
            }
        const float mn = fmaxf(m_run, col4_max(mx)), corr = __builtin_amdgcn_exp2f(m_run - mn);
        float sum = 0.f;
        u32x4_m ph[PT / 2], pl[PT / 2];
#pragma unroll
        for (int j = 0; j < PT; ++j)
#pragma unroll
            for (int e = 0; e < 2; ++e) {
                const float u = __builtin_amdgcn_exp2f(sc[j][2 * e] - mn), v = __builtin_amdgcn_exp2f(sc[j][2 * e + 1] - mn);
                sum += u + v;
                uint32_t hi, lo;
                split_bf16_hw(u, v, hi, lo);
                ph[j / 2][2 * (j & 1) + e] = hi;
                pl[j / 2][2 * (j & 1) + e] = lo;
            }
        l_run = l_run * corr + col4_sum(sum);
        m_run = mn;
#pragma unroll
        for (int i = 0; i < RT; ++i) {
            if (rp0 + 16 * i >= rank) break;
#pragma unroll
            for (int e = 0; e < 4; ++e) acc[i][e] *= corr;
#pragma unroll
            for (int k = 0; k < PT / 2; ++k) {
                const u32x4_m rv = lds_operand_t2(rows + 32 * k * ws + rp0 + 16 * i, ws, lane);
                acc[i] = mma16(rv, ph[k], acc[i]);
                acc[i] = mma16(rv, pl[k], acc[i]);
            }
        }
    }
    if (c < hr) {
#pragma unroll
        for (int i = 0; i < RT; ++i) {
            if (rp0 + 16 * i >= rank) break;
#pragma unroll
            for (int e = 0; e < 2; ++e)   // (records are 8-byte aligned: rank is even)
                *reinterpret_cast<float2*>(rec + c * rec_h + rp0 + 16 * i + 4 * kg + 2 * e) = make_float2(acc[i][2 * e], acc[i][2 * e + 1]);
        }
        if (kg == 0 && rp0 == 0) {
            rec[c * rec_h + rank] = m_run;
            rec[c * rec_h + rank + 1] = l_run;
        }
    }
}

// Workgroup = head x OV values x sequence (narrow where there are few heads and sequences): the slices' records merged into the weighted latent, times W_uv.
template <int OV>
__global__ __launch_bounds__(256) void latent_combine_kernel(LatentDecodeArgs a, const float* __restrict__ part, int nsplit) {
    extern __shared__ float lat_lds[];
    const int rank = (int)a.rank, vdim = (int)a.vdim, H = (int)a.heads;
    float* lat = lat_lds;                        // [rank]
    float* wgt = lat + rank;                     // [32]
    float* red = wgt + 32;                       // [4][OV]
    constexpr int VL = OV / 8, GR = 256 / VL;    // lanes of 8 values, groups of latent dimensions
    const int t = threadIdx.x, lane = t & 63, wave = t >> 6, h = blockIdx.x, v0 = blockIdx.y * OV, b = blockIdx.z;
    const int rs = rank + 2;
    const float* rec = part + ((int64_t)b * H + h) * nsplit * rs;
    // the first words of W_uv and the first records are requested at once
    const int v8 = 8 * (t % VL), g = t / VL;
    const bool vlive = v0 + v8 < vdim;
    const int64_t ldw = (int64_t)H * vdim;
    const bf16_t* wv = (const bf16_t*)a.w_uv + (int64_t)h * vdim + (vlive ? v0 + v8 : 0);
    constexpr int U = 8;
    u32x4_m x[U];
    auto request = [&](int r0) {
#pragma unroll
        for (int u = 0; u < U; ++u) x[u] = *reinterpret_cast<const u32x4_m*>(wv + (int64_t)min(r0 + GR * u, rank - 1) * ldw);
    };
    request(g);
    const float mv = lane < nsplit ? rec[(int64_t)lane * rs + rank] : -INFINITY, lv = lane < nsplit ? rec[(int64_t)lane * rs + rank + 1] : 0.f;
    constexpr int SU = 16;
    float2 y[2][SU];
    auto records = [&](int r, int s0, float2* dst) __attribute__((always_inline)) {   // (clamped: what is not there is not used)
#pragma unroll
        for (int u = 0; u < SU; ++u) dst[u] = *reinterpret_cast<const float2*>(rec + (int64_t)min(s0 + u, nsplit - 1) * rs + min(r, rank - 2));
    };
    records(2 * t, 0, y[0]);
    records(2 * t, SU, y[1]);
    {   // every wave finds the weights of the (at most 32) slices; wave 0 leaves them in LDS
        const float m = wave_max(mv), e = __builtin_amdgcn_exp2f(mv - m);
        const float l = wave_sum(e * lv);
        if (wave == 0 && lane < 32) wgt[lane] = e / l;
    }
    __syncthreads();
    for (int r = 2 * t; r < rank; r += 512) {
        if (r != 2 * t) { records(r, 0, y[0]); records(r, SU, y[1]); }
        float2 v = make_float2(0.f, 0.f);
#pragma unroll
        for (int q = 0; q < 2; ++q)
#pragma unroll
            for (int u = 0; u < SU; ++u) {
                const float f = wgt[q * SU + u];   // zero behind the last slice, and for an empty one, whose sums are unset
                v.x += f != 0.f ? f * y[q][u].x : 0.f;
                v.y += f != 0.f ? f * y[q][u].y : 0.f;
            }
        lat[r] = v.x;
        lat[r + 1] = v.y;
    }
    __syncthreads();
    float o[8];
#pragma unroll
    for (int e = 0; e < 8; ++e) o[e] = 0.f;
    for (int r0 = g; r0 < rank; r0 += GR * U) {
        if (r0 != g) request(r0);
#pragma unroll
        for (int u = 0; u < U; ++u) {
            const float f = r0 + GR * u < rank ? lat[r0 + GR * u] : 0.f;
#pragma unroll
            for (int e = 0; e < 4; ++e) { o[2 * e] += f * bf16lo(x[u][e]); o[2 * e + 1] += f * bf16hi(x[u][e]); }
        }
    }
#pragma unroll
    for (int e = 0; e < 8; ++e) {   // over the groups of the wave: lanes VL apart
        float x = o[e];
        if (VL == 4) { x += __shfl_xor(x, 4, 64); x += __shfl_xor(x, 8, 64); }
        x = col4_sum(x);
        if (lane < VL) red[wave * OV + v8 + e] = x;
    }
    __syncthreads();
    static_assert(VL == 4 || VL == 16, "reduction above");
    if (t < OV && v0 + t < vdim)
        ((bf16_t*)a.ctx)[((int64_t)b * H + h) * vdim + v0 + t] = f32_to_bf16(red[t] + red[OV + t] + red[2 * OV + t] + red[3 * OV + t]);
}

// ---------------------------------------------------------------------------- prompts (bf16)
constexpr int kQTile = 128;      // queries per workgroup: 16 per wave
constexpr int kKTile = 64;       // keys per step

// Workgroup = 128 queries x head x sequence, 8 waves.  Keys [unrotated | shared rotated part] and values of a step in LDS, the
// next step's words in registers meanwhile.  Everything is transposed (scores: rows = keys, columns = queries; result:
// rows = values), so a lane works on one query: softmax in f32 registers, the weights go from there into the product with the
// values, as a bf16 value and its remainder.  KS: dim + rot in steps of 32, VT: vdim in tiles of 16 (both zero padded).
template <int KS, int VT>
__global__ __launch_bounds__(512) void latent_prefill_kernel(LatentPrefillArgs a) {
    extern __shared__ __align__(16) unsigned char lat_smem[];
    constexpr int KSTR = KS * 32 + 8, VSTR = VT * 16 + 8;
    bf16_t* kt = reinterpret_cast<bf16_t*>(lat_smem);                 // [64][KSTR]
    bf16_t* vt = kt + kKTile * KSTR;                                  // [64][VSTR]
    const int t = threadIdx.x, lane = t & 63, wave = t >> 6, c = lane & 15, kg = lane >> 4;
    const int b = blockIdx.z, h = blockIdx.y, T = a.len[b], r0 = a.row0[b];
    const int q0 = ((int)gridDim.x - 1 - (int)blockIdx.x) * kQTile;   // the longest workgroups first
    if (q0 >= T) return;
    const int dim = (int)a.dim, rot = (int)a.rot, hd = dim + rot, vdim = (int)a.vdim, H = (int)a.heads, w = (int)(a.rank + a.rot);
    const int kend = min(q0 + kQTile, T);
    const int myq = q0 + wave * 16, qi = myq + c;                     // the wave's first query, the lane's

    // A thread's words of a step, by 32-bit offsets from uniform bases.  Nothing is loaded conditionally: keys behind the last
    // one repeat it (their scores are masked), columns behind a row's end repeat its start (the queries are zero there, or the
    // result is not stored).
    constexpr int KW = KS * 4, VW = VT * 2;                           // 16-byte words per staged row
    constexpr int KU = kKTile * KW / 512, VU = (kKTile * VW + 511) / 512;   // ... per thread
    static_assert(kKTile * KW % 512 == 0 && kKTile * VW % 512 == 0, "whole rounds of the workgroup");
    u32x4_m rk[KU], rv[VU];
    const char* kbase = (const char*)a.k + ((int64_t)r0 * H + h) * dim * 2;
    const char* rbase = (const char*)a.rows + ((int64_t)r0 * w + a.rank) * 2;
    const char* vbase = (const char*)a.v + ((int64_t)r0 * H + h) * vdim * 2;
    auto fetch = [&](int k0) {
#pragma unroll
        for (int u = 0; u < KU; ++u) {
            const int i = t + 512 * u, d = (i % KW) * 8, pos = min(k0 + i / KW, kend - 1);
            const bool un = d < dim || d >= hd;                       // an unrotated column
            const char* base = un ? kbase : rbase;
            const unsigned off = un ? (unsigned)pos * (unsigned)(H * dim * 2) + (unsigned)((d < dim ? d : 0) * 2) : (unsigned)pos * (unsigned)(w * 2) + (unsigned)((d - dim) * 2);
            rk[u] = *reinterpret_cast<const u32x4_m*>(base + off);
        }
#pragma unroll
        for (int u = 0; u < VU; ++u) {
            const int i = t + 512 * u, d = (i % VW) * 8, pos = min(k0 + i / VW, kend - 1);
            rv[u] = *reinterpret_cast<const u32x4_m*>(vbase + ((unsigned)pos * (unsigned)(H * vdim * 2) + (unsigned)((d < vdim ? d : 0) * 2)));
        }
    };
    fetch(0);

    // queries: rotated on the way in, rounded once; columns behind the prompt repeat its last query and are not stored
    u32x4_m q[KS];
    {
        const int row = r0 + min(qi, T - 1);
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
            q[k] = v;
        }
    }
    f32x4_m o[VT];
    float m = -INFINITY, l = 0.f;
#pragma unroll
    for (int v = 0; v < VT; ++v) o[v] = f32x4_m{0.f, 0.f, 0.f, 0.f};
    const float scale2 = a.scale * 1.44269504f;                       // weights as powers of two
    for (int k0 = 0; k0 < kend; k0 += kKTile) {
        __syncthreads();
#pragma unroll
        for (int u = 0; u < KU; ++u) {
            const int i = t + 512 * u;
            *reinterpret_cast<u32x4_m*>(kt + (i / KW) * KSTR + (i % KW) * 8) = rk[u];
        }
#pragma unroll
        for (int u = 0; u < VU; ++u) {
            const int i = t + 512 * u;
            *reinterpret_cast<u32x4_m*>(vt + (i / VW) * VSTR + (i % VW) * 8) = rv[u];
        }
        __syncthreads();
        if (k0 + kKTile < kend) fetch(k0 + kKTile);
        if (k0 > myq + 15) continue;                                  // all keys of the step lie ahead of the wave's queries
        f32x4_m s[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            s[j] = f32x4_m{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int k = 0; k < KS; ++k) s[j] = mma16(*reinterpret_cast<const u32x4_m*>(kt + (16 * j + c) * KSTR + 32 * k + 8 * kg), q[k], s[j]);
        }
        const bool edge = k0 + kKTile - 1 > myq;                      // some key lies ahead of some query
        float mx = -INFINITY;
#pragma unroll
        for (int j = 0; j < 4; ++j)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                float x = s[j][e] * scale2;
                if (edge && k0 + 16 * j + 4 * kg + e > qi) x = -INFINITY;
                s[j][e] = x;
                mx = fmaxf(mx, x);
            }
        // k0 and myq are multiples of 16 and k0 <= myq + 15, so every query sees key k0: the maximum is finite
        const float mn = fmaxf(m, col4_max(mx));
        float sum = 0.f;
        u32x4_m ph[2], pl[2];
#pragma unroll
        for (int j = 0; j < 4; ++j)
#pragma unroll
            for (int e = 0; e < 2; ++e) {
                const float u = __builtin_amdgcn_exp2f(s[j][2 * e] - mn), v = __builtin_amdgcn_exp2f(s[j][2 * e + 1] - mn);
                sum += u + v;
                uint32_t hi, lo;
                split_bf16_hw(u, v, hi, lo);
                ph[j / 2][2 * (j & 1) + e] = hi;
                pl[j / 2][2 * (j & 1) + e] = lo;
            }
        sum = col4_sum(sum);
        if (__builtin_amdgcn_ballot_w64(mn > m) != 0) {               // some column's maximum has moved
            const float corr = __builtin_amdgcn_exp2f(m - mn);
            l *= corr;
#pragma unroll
            for (int v = 0; v < VT; ++v)
#pragma unroll
                for (int e = 0; e < 4; ++e) o[v][e] *= corr;
            m = mn;
        }
        l += sum;
#pragma unroll
        for (int k = 0; k < kKTile / 32; ++k)
#pragma unroll
            for (int v = 0; v < VT; ++v) {
                const u32x4_m vv = lds_operand_t2(vt + 32 * k * VSTR + 16 * v, VSTR, lane);
                o[v] = mma16(vv, ph[k], o[v]);
                o[v] = mma16(vv, pl[k], o[v]);
            }
    }
    if (qi >= T) return;
    const float inv = 1.0f / l;
    bf16_t* out = (bf16_t*)a.ctx + ((int64_t)(r0 + qi) * H + h) * vdim + 4 * kg;
#pragma unroll
    for (int v = 0; v < VT; ++v)
        if (16 * v + 4 * kg < vdim)
            *reinterpret_cast<uint2*>(out + 16 * v) = make_uint2(pack_bf16_hw(o[v][0] * inv, o[v][1] * inv), pack_bf16_hw(o[v][2] * inv, o[v][3] * inv));
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
    if (rows * per_row <= 0) return;
    if (head_dim % 2 || offset % 2) {
        const unsigned ge = (unsigned)cdiv_l(rows * per_row, 256);
        if (dtype == 0) rope_pairs_any_kernel<float><<<ge, 256, 0, s>>>((const float*)x, table, (float*)y, rows * per_row, per_row, head_dim, offset, half);
        else rope_pairs_any_kernel<bf16_t><<<ge, 256, 0, s>>>((const bf16_t*)x, table, (bf16_t*)y, rows * per_row, per_row, head_dim, offset, half);
        return;
    }
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
// slices of the positions: 64 rows each up to 32 of them, fewer where the batch fills the chip by itself
static int latent_nsplit(int64_t nseq, int64_t capacity, int64_t heads) {
    const int64_t blocks = nseq * cdiv_l(heads, kHeadTile);
    int64_t n = std::min<int64_t>(cdiv_l(capacity, kTileP), 32);
    while (n > 4 && blocks * n > 512) n = (n + 1) / 2;
    return (int)std::max<int64_t>(n, 1);
}
static size_t latent_partial_lds(int64_t w, int64_t head_tiles = 1) {
    return (size_t)(kTileP + head_tiles * kHeadTile) * (w + 8) * 2;
}
static bool latent_fast(int dtype, int64_t heads, int64_t dim, int64_t rot, int64_t rank, int64_t vdim) {
    return dtype == 2 && heads >= 1 && dim % 8 == 0 && vdim % 8 == 0 && rot % 2 == 0 && rank % 16 == 0 && (rank + rot) % 32 == 0 && rank <= 1024 && dim <= 512 &&
           latent_partial_lds(rank + rot) <= 160 * 1024;
}
size_t latent_decode_scratch_bytes(int dtype, int64_t nseq, int64_t capacity, int64_t heads, int64_t dim, int64_t rot, int64_t rank, int64_t vdim) {
    if (latent_fast(dtype, heads, dim, rot, rank, vdim))
        return lat_align((size_t)(nseq * heads * (rank + rot)) * 2) + (size_t)(nseq * heads * (rank + 2)) * 32 * sizeof(float);
    const size_t es = dtype == 0 ? 4 : 2;
    return lat_align((size_t)(nseq * heads * (dim + rot)) * es);
}
int latent_decode(hipStream_t s, const LatentDecodeArgs& a) {
    const size_t es = a.dtype == 0 ? 4 : 2;
    const int64_t w = a.rank + a.rot;
    if (latent_fast(a.dtype, a.heads, a.dim, a.rot, a.rank, a.vdim)) {
        bf16_t* ql = (bf16_t*)a.scratch;
        float* part = (float*)((char*)a.scratch + lat_align((size_t)(a.nseq * a.heads * w) * 2));
        const int ns = latent_nsplit(a.nseq, a.capacity, a.heads);
        const int64_t rc = cdiv_l(a.rank, kPrepRows);
        latent_prep_kernel<<<(unsigned)(a.heads * rc + (a.raw ? a.nseq : 0)), 256, (size_t)std::max<int64_t>(a.nseq * a.dim, 16) * 4, s>>>(a, ql);
        const int64_t rt = a.rank / 16, parts = cdiv_l(rt, 16), units = cdiv_l(a.heads, kHeadTile) * parts;
        // waves per workgroup, as many as have work and whose queries fit beside the rows (a workgroup of W consecutive units
        // meets at most (W - 2) / parts + 2 tiles of heads)
        int64_t W = std::min<int64_t>(units, 4);
        auto tiles = [&](int64_t n) { return n <= 1 ? 1 : std::min<int64_t>((n - 2) / parts + 2, n); };
        while (W > 1 && latent_partial_lds(w, tiles(W)) > 160 * 1024) --W;
        const size_t lds = latent_partial_lds(w, tiles(W));
        const dim3 grid((unsigned)ns, (unsigned)cdiv_l(units, W), (unsigned)a.nseq);
#define GPTRS_PARTIAL(RT) do { with_lds(latent_partial_kernel<RT>, lds); latent_partial_kernel<RT><<<grid, (unsigned)(64 * W), lds, s>>>(a, ql, part, ns); } while (0)
        if (rt <= 8) GPTRS_PARTIAL(8);
        else GPTRS_PARTIAL(16);
#undef GPTRS_PARTIAL
#define GPTRS_COMBINE(OV) latent_combine_kernel<OV><<<dim3((unsigned)a.heads, (unsigned)cdiv_l(a.vdim, OV), (unsigned)a.nseq), 256, (size_t)(a.rank + 32 + 4 * OV) * 4, s>>>(a, part, ns)
        if (a.vdim > 64 && a.heads * a.nseq >= 192) GPTRS_COMBINE(128);
        else GPTRS_COMBINE(32);
#undef GPTRS_COMBINE
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
    constexpr int lds = kKTile * (KS * 32 + 8 + VT * 16 + 8) * 2;
    static_assert(lds <= 160 * 1024, "LDS of one CU");
    with_lds(latent_prefill_kernel<KS, VT>, lds);
    latent_prefill_kernel<KS, VT><<<dim3((unsigned)cdiv_l(longest, kQTile), (unsigned)a.heads, (unsigned)a.nseq), 512, lds, s>>>(a);
}
template <int KS>
static void launch_prefill_v(hipStream_t s, const LatentPrefillArgs& a, int64_t longest) {
    if (a.vdim <= 64) launch_prefill<KS, 4>(s, a, longest);
    else if (a.vdim <= 128) launch_prefill<KS, 8>(s, a, longest);
    else launch_prefill<KS, 16>(s, a, longest);
}
int latent_prefill(hipStream_t s, const LatentPrefillArgs& a) {
    if (a.dtype == 2 && a.dim % 8 == 0 && a.rot % 8 == 0 && a.rank % 8 == 0 && a.vdim % 8 == 0 && a.dim + a.rot <= 256 && a.vdim <= 256 &&
        a.total * std::max(a.heads * std::max(a.dim, a.vdim), a.rank + a.rot) < (1ll << 30)) {   // 32-bit offsets
        int64_t longest = 0;
        for (int b = 0; b < a.nseq; ++b) longest = std::max<int64_t>(longest, a.len[b]);
        const int64_t ks = cdiv_l(a.dim + a.rot, 32);
        if (ks <= 2) launch_prefill_v<2>(s, a, longest);
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
