// Grouped-query attention whose positions see their own chunk of the sequence only, with unit-RMS queries and keys, a sink per
// head in the softmax denominator and a gate per head on the result.  Key and value sizes are independent of each other.
//
// A layer's input is one f32 projection per row, q | k | v | gate: `heads` queries and `kv_heads` keys of `dim` values, `kv_heads`
// values of `vdim`, one gate per head.  Caches hold the rows of the current chunk: position p's row is p % chunk (chunk 0: the
// whole sequence).
//
// The first part are the stand-alone kernels of the CustomCall targets and the row preparation, for any sizes and either element
// type; the second the bf16 launches of Mix::ChunkDecode and Mix::ChunkPrefill on the matrix cores.
#include <algorithm>

#include "kernels.hpp"
#include "device_utils.hpp"

namespace gptrs {
namespace k {

namespace {

inline int64_t cdiv_c(int64_t a, int64_t b) { return (a + b - 1) / b; }
inline size_t chunk_align(size_t n) { return (n + 255) / 256 * 256; }
// 16 bytes at any 4-byte boundary
typedef float f32x4_u __attribute__((ext_vector_type(4), aligned(4)));

__device__ __forceinline__ float sigmoid_f32(float x) { return 1.0f / (1.0f + expf(-x)); }
__device__ __forceinline__ int clamp_row(int v, int last) { return v < 0 ? 0 : (v > last ? last : v); }

// ---------------------------------------------------------------------------- stand-alone kernels
// A wave per head of a row.
template <typename TI, typename TO>
__global__ __launch_bounds__(256) void head_norm_kernel(const TI* __restrict__ x, TO* __restrict__ y, int64_t n, int64_t hd, float eps) {
    const int64_t i = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
    const int lane = threadIdx.x & 63;
    if (i >= n) return;
    float q = 0.f;
    for (int64_t d = lane; d < hd; d += 64) { const float v = Elem<TI>::ld(x, i * hd + d); q += v * v; }
    const float inv = 1.0f / sqrtf(wave_sum(q) / (float)hd + eps);
    for (int64_t d = lane; d < hd; d += 64) Elem<TO>::st(y, i * hd + d, Elem<TI>::ld(x, i * hd + d) * inv);
}

// gate: one value per head, rows `ld` apart
template <typename T>
__global__ __launch_bounds__(256) void head_gate_kernel(const T* __restrict__ x, const float* __restrict__ gate, T* __restrict__ y, int64_t n, int64_t heads,
                                                        int64_t vd, int64_t ld) {
    const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (i >= n) return;
    const int64_t r = i / (heads * vd), h = i / vd % heads;
    Elem<T>::st(y, i, Elem<T>::ld(x, i) * sigmoid_f32(gate[r * ld + h]));
}

// Workgroup = query x head.  Keys in tiles of 256, one per thread; online softmax that starts from the sink.
template <typename T>
__global__ __launch_bounds__(256) void chunk_attn_kernel(ChunkAttnArgs a) {
    extern __shared__ float chk_lds[];
    float* q = chk_lds;                          // [dim]
    float* acc = q + a.dim;                      // [vdim]
    float* pr = acc + a.vdim;                    // [256]
    float* red = pr + 256;                       // [16]
    const int t = threadIdx.x;
    const int64_t i = blockIdx.x, h = blockIdx.y, g = h / (a.heads / a.kv_heads);
    const T* qrow = (const T*)a.q + (i * a.heads + h) * a.dim;
    const T* kb = (const T*)a.k + g * a.k_head;
    const T* vb = (const T*)a.v + g * a.v_head;
    for (int64_t d = t; d < a.dim; d += 256) q[d] = Elem<T>::ld(qrow, d);
    for (int64_t v = t; v < a.vdim; v += 256) acc[v] = 0.f;
    __syncthreads();
    int64_t lo, end;                             // rows [lo, end) are seen
    if (a.position) {
        const int64_t p = a.position[0] < 0 ? 0 : a.position[0];
        lo = 0;
        end = (a.chunk > 0 ? p % a.chunk : p) + 1;
        if (end > a.rows) end = a.rows;
    } else {
        lo = a.chunk > 0 ? i / a.chunk * a.chunk : 0;
        end = i + 1;
    }
    float m = a.sink[h], l = 1.0f;
    for (int64_t j0 = lo; j0 < end; j0 += 256) {
        const int64_t j = j0 + t;
        float s = -INFINITY;
        if (j < end) {
            s = 0.f;
            for (int64_t d = 0; d < a.dim; ++d) s += q[d] * Elem<T>::ld(kb, j * a.k_row + d);
            s *= a.scale;
        }
        const float mn = fmaxf(m, block_max(s, red));
        const float corr = expf(m - mn), p = expf(s - mn);
        pr[t] = p;
        l = l * corr + block_sum(p, red);
        m = mn;
        const int nj = (int)(end - j0 < 256 ? end - j0 : 256);
        for (int64_t v = t; v < a.vdim; v += 256) {
            float o = acc[v] * corr;
            for (int jj = 0; jj < nj; ++jj) o += pr[jj] * Elem<T>::ld(vb, (j0 + jj) * a.v_row + v);
            acc[v] = o;
        }
        __syncthreads();
    }
    const float inv = 1.0f / l;
    for (int64_t v = t; v < a.vdim; v += 256) Elem<T>::st((T*)a.ctx, (i * a.heads + h) * a.vdim + v, acc[v] * inv);
}

// ---------------------------------------------------------------------------- rows of a layer
// A wave per (row of a sequence, head); heads in the order queries, keys, values, the first `skip` of them left out.  Queries
// and keys are rotated and divided by their root mean square, values only stored; rows that the sequence's cache takes (the last
// `keep` of it) go there as well, from row starts[3 b + 1] on.
template <typename T>
__global__ __launch_bounds__(256) void chunk_rows_kernel(ChunkSeqArgs a, int skip, T* __restrict__ qo, T* __restrict__ ko, T* __restrict__ vo) {
    const int b = blockIdx.z, lane = threadIdx.x & 63;
    const int H = (int)a.heads, G = (int)a.kv_heads, D = (int)a.dim, V = (int)a.vdim, rot = (int)a.rot;
    const int per = H + 2 * G - skip;
    const int64_t w = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
    if (w >= (int64_t)a.len[b] * per) return;
    const int lr = (int)(w / per), h = (int)(w % per) + skip;
    const int64_t row = a.row0[b] + lr;
    const float* p = a.proj + row * a.ld;
    const int cl = lr - (a.len[b] - a.keep[b]);                       // place among the rows the cache takes
    int64_t at = 0;
    if (cl >= 0) at = (int64_t)clamp_row(a.starts[3 * b + 1], (int)a.rows - a.keep[b]) + cl;
    if (h >= H + G) {
        const int g = h - H - G;
        const float* x = p + (int64_t)(H + G) * D + (int64_t)g * V;
        T* y = vo ? vo + (row * G + g) * V : nullptr;
        T* c = cl >= 0 ? (T*)a.vcache[b] + ((int64_t)g * a.rows + at) * V : nullptr;
        for (int d = lane; d < V; d += 64) {
            if (y) Elem<T>::st(y, d, x[d]);
            if (c) Elem<T>::st(c, d, x[d]);
        }
        return;
    }
    const float* x = p + (int64_t)h * D;
    const float* tab = a.table + row * rot;
    float q = 0.f;
    auto turned = [&](int d) {
        if (d >= rot) return x[d];
        const float u = x[d & ~1], v = x[d | 1], cs = tab[d >> 1], sn = tab[rot / 2 + (d >> 1)];
        return d & 1 ? v * cs + u * sn : u * cs - v * sn;
    };
    for (int d = lane; d < D; d += 64) { const float v = turned(d); q += v * v; }
    const float inv = 1.0f / sqrtf(wave_sum(q) / (float)D + a.eps);
    const int g = h - H;
    T* y = h < H ? qo + (row * H + h) * D : (ko ? ko + (row * G + g) * D : nullptr);
    T* c = h >= H && cl >= 0 ? (T*)a.kcache[b] + ((int64_t)g * a.rows + at) * D : nullptr;
    for (int d = lane; d < D; d += 64) {
        const float v = turned(d) * inv;
        if (y) Elem<T>::st(y, d, v);
        if (c) Elem<T>::st(c, d, v);
    }
}

// The keys and values of whole prompts in bf16, sizes of up to 8 * 16 * U values and multiples of 8: 16 lanes to a head, 8 values
// of it per lane and round, all of them requested before the first is used.
template <int U>
__global__ __launch_bounds__(256) void chunk_rows16_kernel(ChunkSeqArgs a, bf16_t* __restrict__ ko, bf16_t* __restrict__ vo) {
    const int b = blockIdx.z, l16 = threadIdx.x & 15;
    const int H = (int)a.heads, G = (int)a.kv_heads, D = (int)a.dim, V = (int)a.vdim, rot = (int)a.rot;
    const int w = (int)blockIdx.x * 16 + (int)(threadIdx.x >> 4);
    if (w >= a.len[b] * 2 * G) return;                                // (16 lanes at a time)
    const int lr = w / (2 * G), u = w % (2 * G), g = u % G;
    const bool key = u < G;
    const int n = key ? D : V;
    const int64_t row = a.row0[b] + lr;
    const float* x = a.proj + row * a.ld + (int64_t)H * D + (key ? (int64_t)g * D : (int64_t)G * D + (int64_t)g * V);
    const float* tab = a.table + row * rot;
    f32x4_m v[U][2];
    f32x4_m cs[U], sn[U];
#pragma unroll
    for (int i = 0; i < U; ++i) {
        const int d = 8 * (l16 + 16 * i);
        v[i][0] = v[i][1] = f32x4_m{0.f, 0.f, 0.f, 0.f};
        if (d < n) {
            v[i][0] = *reinterpret_cast<const f32x4_u*>(x + d);
            v[i][1] = *reinterpret_cast<const f32x4_u*>(x + d + 4);
        }
        cs[i] = f32x4_m{1.f, 1.f, 1.f, 1.f};
        sn[i] = f32x4_m{0.f, 0.f, 0.f, 0.f};
        if (key) {
#pragma unroll
            for (int e = 0; e < 4; ++e)
                if (d + 2 * e < rot) { cs[i][e] = tab[d / 2 + e]; sn[i][e] = tab[rot / 2 + d / 2 + e]; }
        }
    }
    float f = 1.0f;
    if (key) {
        float q = 0.f;
#pragma unroll
        for (int i = 0; i < U; ++i)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const float p = v[i][e >> 1][2 * (e & 1)], r = v[i][e >> 1][2 * (e & 1) + 1];
                const float y = p * cs[i][e] - r * sn[i][e], z = r * cs[i][e] + p * sn[i][e];
                v[i][e >> 1][2 * (e & 1)] = y;
                v[i][e >> 1][2 * (e & 1) + 1] = z;
                q += y * y + z * z;
            }
        f = 1.0f / sqrtf(row16_sum(q) / (float)D + a.eps);
    }
    const int cl = lr - (a.len[b] - a.keep[b]);
    bf16_t* y = (key ? ko : vo) + (row * G + g) * n;
    bf16_t* c = nullptr;
    if (cl >= 0) c = (bf16_t*)(key ? a.kcache[b] : a.vcache[b]) + ((int64_t)g * a.rows + clamp_row(a.starts[3 * b + 1], (int)a.rows - a.keep[b]) + cl) * n;
#pragma unroll
    for (int i = 0; i < U; ++i) {
        const int d = 8 * (l16 + 16 * i);
        if (d >= n) break;
        u32x4_m o;
#pragma unroll
        for (int e = 0; e < 4; ++e) o[e] = pack_bf16_hw(v[i][e >> 1][2 * (e & 1)] * f, v[i][e >> 1][2 * (e & 1) + 1] * f);
        *reinterpret_cast<u32x4_m*>(y + d) = o;
        if (c) *reinterpret_cast<u32x4_m*>(c + d) = o;
    }
}

// ---------------------------------------------------------------------------- decode (bf16)
constexpr int kDecTile = 32;     // cache rows per wave and step
constexpr int kDecHeads = 16;    // query heads per workgroup (of one key / value head)

// Workgroup = slice of the chunk's rows x up to 16 query heads of a key / value head x sequence; its four waves take 32 rows at a
// time, each on its own.  The queries and the step's new key are rotated and normed on the way in; the slice that holds the new
// row takes it from LDS, and the first workgroup of its key / value head writes it to the cache.  Scores transposed (rows:
// positions, columns: heads), so a lane holds 8 positions of one head: softmax in registers, the weights (a bf16 value and its
// remainder) feed the product with the values from there.  The slices' records (sums, maximum in base 2, weight) meet through
// `part`: the workgroup that draws the last ticket merges them, adds the sink to the denominator and applies the gate.  KS: dim
// in steps of 32, VT: vdim in tiles of 16 (both zero padded).
template <int KS, int VT>
__global__ __launch_bounds__(256) void chunk_decode_kernel(ChunkSeqArgs a, float* __restrict__ part, unsigned* __restrict__ tickets, int ns) {
    extern __shared__ __align__(16) unsigned char chk_smem[];
    constexpr int QS = KS * 32 + 8, VS = VT * 16 + 8, VW = VT * 2, VP = VT * 16;
    bf16_t* qs = reinterpret_cast<bf16_t*>(chk_smem);                 // [16][QS]
    bf16_t* knew = qs + kDecHeads * QS;                               // [QS]
    bf16_t* vnew = knew + QS;                                         // [VS]
    bf16_t* vt = vnew + VS;                                           // [4][32][VS]
    float* so = reinterpret_cast<float*>(vt);                         // [4][16][VP], once the rows have been used
    __shared__ float sm[4][kDecHeads], sl[4][kDecHeads];
    __shared__ unsigned drawn;
    const int t = threadIdx.x, lane = t & 63, wave = t >> 6, c = lane & 15, kg = lane >> 4;
    const int H = (int)a.heads, G = (int)a.kv_heads, D = (int)a.dim, V = (int)a.vdim, rot = (int)a.rot, per_kv = H / G;
    const int ht = (per_kv + kDecHeads - 1) / kDecHeads;
    const int b = blockIdx.z, g = (int)blockIdx.y / ht, h0 = g * per_kv + (int)blockIdx.y % ht * kDecHeads, sp = blockIdx.x;
    const int nh = min(kDecHeads, (g + 1) * per_kv - h0);             // heads that exist
    const int C = (int)a.rows, p = max(a.pos[b], 0), upd = clamp_row(a.starts[3 * b + 1], C - 1);
    const int n = min((a.chunk > 0 ? (int)(p % a.chunk) : p) + 1, C);
    const int per = ((n + ns - 1) / ns + kDecTile - 1) / kDecTile * kDecTile;
    const int p0 = sp * per, p1 = min(p0 + per, n);
    const bool owner = upd >= p0 && (upd < p0 + per || sp == ns - 1); // this slice holds the new row (or the row lies behind the last seen one)
    const float* prow = a.proj + (int64_t)(a.row0[b]) * a.ld;
    const float* tab = a.table + (int64_t)a.row0[b] * rot;
    bf16_t* kc = (bf16_t*)a.kcache[b] + (int64_t)g * C * D;
    bf16_t* vc = (bf16_t*)a.vcache[b] + (int64_t)g * C * V;

    // the first step's cache rows are requested ahead of everything else.  Rows behind the last one repeat it (weight zero),
    // columns behind a row's end repeat its start (the queries are zero there, or the sums are not used).
    u32x4_m kf[2][KS], vw[VT];
    auto fetch = [&](int r0) {
#pragma unroll
        for (int j = 0; j < 2; ++j) {
            const bf16_t* row = kc + (int64_t)min(r0 + 16 * j + c, p1 - 1) * D;
#pragma unroll
            for (int k = 0; k < KS; ++k) { const int d = 32 * k + 8 * kg; kf[j][k] = *reinterpret_cast<const u32x4_m*>(row + (d < D ? d : 0)); }
        }
#pragma unroll
        for (int u = 0; u < VT; ++u) {
            const int i = lane + 64 * u, d = (i % VW) * 8;
            vw[u] = *reinterpret_cast<const u32x4_m*>(vc + (int64_t)min(r0 + i / VW, p1 - 1) * V + (d < V ? d : 0));
        }
    };
    const int r_first = p0 + wave * kDecTile;
    if (r_first < p1) fetch(r_first);

    // queries: 16 lanes to a head, and once more for the new key
    auto prepare = [&](const float* x, bf16_t* to, bool live) {
        const int l16 = t & 15;
        float u[KS], v[KS], q = 0.f;
#pragma unroll
        for (int k = 0; k < KS; ++k) {
            const int d = 32 * k + 2 * l16;
            u[k] = v[k] = 0.f;
            if (live && d < D) {
                const float x0 = x[d], x1 = x[d + 1];
                u[k] = x0; v[k] = x1;
                if (d < rot) {
                    const float cs = tab[d >> 1], sn = tab[rot / 2 + (d >> 1)];
                    u[k] = x0 * cs - x1 * sn;
                    v[k] = x1 * cs + x0 * sn;
                }
            }
            q += u[k] * u[k] + v[k] * v[k];
        }
        const float inv = 1.0f / sqrtf(row16_sum(q) / (float)D + a.eps);
#pragma unroll
        for (int k = 0; k < KS; ++k) *reinterpret_cast<uint32_t*>(to + 32 * k + 2 * l16) = pack_bf16_hw(u[k] * inv, v[k] * inv);
    };
    prepare(prow + (int64_t)(h0 + min(t >> 4, nh - 1)) * D, qs + (t >> 4) * QS, (t >> 4) < nh);
    if (owner) {
        if (t < 16) prepare(prow + (int64_t)(H + g) * D, knew, true);
        const float* xv = prow + (int64_t)(H + G) * D + (int64_t)g * V;
        for (int d = t; d < VP; d += 256) vnew[d] = d < V ? f32_to_bf16(xv[d]) : (bf16_t)0;
    }
    __syncthreads();
    if (owner && (int)blockIdx.y % ht == 0) {
        for (int d = t; d < D; d += 256) kc[(int64_t)upd * D + d] = knew[d];
        for (int d = t; d < V; d += 256) vc[(int64_t)upd * V + d] = vnew[d];
    }

    f32x4_m o[VT];                                                    // rows: values, column: head c
#pragma unroll
    for (int i = 0; i < VT; ++i) o[i] = f32x4_m{0.f, 0.f, 0.f, 0.f};
    float m_run = -INFINITY, l_run = 0.f;                             // of head c, in its four lanes
    const float scale2 = a.scale * 1.44269504f;
    bf16_t* mine = vt + wave * kDecTile * VS;
    for (int r0 = r_first; r0 < p1; r0 += 4 * kDecTile) {
        if (r0 != r_first) fetch(r0);
        f32x4_m s[2];
#pragma unroll
        for (int j = 0; j < 2; ++j) {
            s[j] = f32x4_m{0.f, 0.f, 0.f, 0.f};
            const bool fresh = owner && r0 + 16 * j + c == upd;
#pragma unroll
            for (int k = 0; k < KS; ++k) {
                u32x4_m kv = kf[j][k];
                if (fresh) kv = *reinterpret_cast<const u32x4_m*>(knew + 32 * k + 8 * kg);
                s[j] = mma16(kv, *reinterpret_cast<const u32x4_m*>(qs + c * QS + 32 * k + 8 * kg), s[j]);
            }
        }
        __builtin_amdgcn_wave_barrier();                              // the wave's own area: its last step's reads come first
#pragma unroll
        for (int u = 0; u < VT; ++u) {
            const int i = lane + 64 * u, r = i / VW, d = (i % VW) * 8;
            u32x4_m v = vw[u];
            if (owner && r0 + r == upd) v = *reinterpret_cast<const u32x4_m*>(vnew + d);
            *reinterpret_cast<u32x4_m*>(mine + r * VS + d) = v;
        }
        float mx = -INFINITY;
#pragma unroll
        for (int j = 0; j < 2; ++j)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                s[j][e] = r0 + 16 * j + 4 * kg + e < p1 ? s[j][e] * scale2 : -INFINITY;
                mx = fmaxf(mx, s[j][e]);
            }
        const float mn = fmaxf(m_run, col4_max(mx)), corr = __builtin_amdgcn_exp2f(m_run - mn);   // (row r0 is seen: finite)
        float sum = 0.f;
        u32x4_m ph, pl;
#pragma unroll
        for (int j = 0; j < 2; ++j)
#pragma unroll
            for (int e = 0; e < 2; ++e) {
                const float u = __builtin_amdgcn_exp2f(s[j][2 * e] - mn), v = __builtin_amdgcn_exp2f(s[j][2 * e + 1] - mn);
                sum += u + v;
                uint32_t hi, lo;
                split_bf16_hw(u, v, hi, lo);
                ph[2 * j + e] = hi;
                pl[2 * j + e] = lo;
            }
        l_run = l_run * corr + col4_sum(sum);
        m_run = mn;
        __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
        __builtin_amdgcn_wave_barrier();
#pragma unroll
        for (int i = 0; i < VT; ++i) {
#pragma unroll
            for (int e = 0; e < 4; ++e) o[i][e] *= corr;
            const u32x4_m vv = lds_operand_t2(mine + 16 * i, VS, lane);
            o[i] = mma16(vv, ph, o[i]);
            o[i] = mma16(vv, pl, o[i]);
        }
    }
    __syncthreads();
#pragma unroll
    for (int i = 0; i < VT; ++i)
#pragma unroll
        for (int e = 0; e < 4; ++e) so[(wave * kDecHeads + c) * VP + 16 * i + 4 * kg + e] = o[i][e];
    if (kg == 0) { sm[wave][c] = m_run; sl[wave][c] = l_run; }
    __syncthreads();

    const float* gate = prow + (int64_t)(H + G) * D + (int64_t)G * V;
    bf16_t* ctx = (bf16_t*)a.ctx + (int64_t)a.row0[b] * H * V;
    const int rs = V + 2;
    float* rec = part + ((int64_t)b * H + h0) * ns * rs;              // of head h0: [ns][rs]
    for (int i = t; i < nh * V; i += 256) {
        const int h = i / V, d = i % V;
        const float mm = fmaxf(fmaxf(sm[0][h], sm[1][h]), fmaxf(sm[2][h], sm[3][h]));
        float L = 0.f, O = 0.f;
#pragma unroll
        for (int w = 0; w < 4; ++w) {
            const float f = sm[w][h] == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(sm[w][h] - mm);
            L += f * sl[w][h];
            O += f * so[(w * kDecHeads + h) * VP + d];
        }
        if (ns == 1) {
            const float s2 = a.sink[h0 + h] * 1.44269504f, mt = fmaxf(mm, s2);
            const float f = __builtin_amdgcn_exp2f(mm - mt), den = L * f + __builtin_amdgcn_exp2f(s2 - mt);
            ctx[(int64_t)(h0 + h) * V + d] = f32_to_bf16(O * f / den * sigmoid_f32(gate[h0 + h]));
        } else {
            float* r = rec + ((int64_t)h * ns + sp) * rs;
            __hip_atomic_store(r + d, O, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
            if (d == 0) {
                __hip_atomic_store(r + V, mm, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
                __hip_atomic_store(r + V + 1, L, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
            }
        }
    }
    if (ns == 1) return;
    // records and tickets cross workgroups through device-scope accesses only; stores acknowledged, then the ticket
    __builtin_amdgcn_s_waitcnt(0x0F70);  // vmcnt(0)
    asm volatile("" ::: "memory");
    __syncthreads();
    unsigned* ticket = tickets + (int64_t)b * gridDim.y + blockIdx.y;
    if (t == 0) drawn = __hip_atomic_fetch_add(ticket, 1u, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    __syncthreads();
    if (drawn + 1 != (unsigned)ns) return;
    asm volatile("" ::: "memory");
    if (t == 0) __hip_atomic_store(ticket, 0u, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);   // zero for the next launch
    float* wgt = so;                                                  // [16][ns], with the denominator and the gate in it
    for (int h = wave; h < nh; h += 4) {                              // ns <= 64: a lane per slice
        const float* r = rec + ((int64_t)h * ns + min(lane, ns - 1)) * rs + V;
        const float mv = __hip_atomic_load(r, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT), lv = __hip_atomic_load(r + 1, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
        const float s2 = a.sink[h0 + h] * 1.44269504f;
        const float mt = fmaxf(wave_max(lane < ns ? mv : -INFINITY), s2);
        const float f = lane < ns && mv != -INFINITY ? __builtin_amdgcn_exp2f(mv - mt) : 0.f;
        const float den = wave_sum(f * lv) + __builtin_amdgcn_exp2f(s2 - mt);
        if (lane < ns) wgt[h * ns + lane] = f / den * sigmoid_f32(gate[h0 + h]);
    }
    __syncthreads();
    for (int i = t; i < nh * V; i += 256) {
        const int h = i / V, d = i % V;
        const float* r = rec + (int64_t)h * ns * rs + d;
        float v = 0.f;
        constexpr int U = 8;
        for (int s0 = 0; s0 < ns; s0 += U) {
            float x[U];
#pragma unroll
            for (int u = 0; u < U; ++u) x[u] = __hip_atomic_load(r + (int64_t)min(s0 + u, ns - 1) * rs, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
#pragma unroll
            for (int u = 0; u < U; ++u) v += s0 + u < ns ? wgt[h * ns + s0 + u] * x[u] : 0.f;
        }
        ctx[(int64_t)(h0 + h) * V + d] = f32_to_bf16(v);
    }
}

// ---------------------------------------------------------------------------- prompts (bf16)
constexpr int kQTile = 128;      // queries per workgroup: 16 per wave
constexpr int kKTile = 64;       // keys per step

// Workgroup = 128 queries (16 per wave) x head x sequence; keys from the first query's chunk on.  Keys and values of a step in LDS,
// the next step's words in registers meanwhile.  Queries come from the projection, rotated and normed on the way in.  Everything is
// transposed (scores: rows = keys, columns = queries; result: rows = values), so a lane works on one query: softmax in f32
// registers, started from the sink (maximum = sink, weight 1: always finite, also for a step of which a query sees nothing); the
// weights go from there into the product with the values, as a bf16 value and its remainder.
template <int KS, int VT>
__global__ __launch_bounds__(512) void chunk_prefill_kernel(ChunkSeqArgs a, const bf16_t* __restrict__ kr, const bf16_t* __restrict__ vr) {
    extern __shared__ __align__(16) unsigned char chk_smem[];
    constexpr int KSTR = KS * 32 + 8, VSTR = VT * 16 + 8;
    bf16_t* kt = reinterpret_cast<bf16_t*>(chk_smem);                 // [64][KSTR]
    bf16_t* vt = kt + kKTile * KSTR;                                  // [64][VSTR]
    const int t = threadIdx.x, lane = t & 63, wave = t >> 6, c = lane & 15, kg = lane >> 4;
    const int b = blockIdx.z, h = blockIdx.y, T = a.len[b], r0 = a.row0[b];
    const int q0 = ((int)gridDim.x - 1 - (int)blockIdx.x) * kQTile;
    if (q0 >= T) return;
    const int H = (int)a.heads, G = (int)a.kv_heads, D = (int)a.dim, V = (int)a.vdim, rot = (int)a.rot, g = h / (H / G);
    const int chunk = a.chunk > 0 && a.chunk < T ? (int)a.chunk : T;
    const int kend = min(q0 + kQTile, T), kbeg = q0 / chunk * chunk;
    const int myq = q0 + wave * 16, qi = myq + c;                     // the wave's first query, the lane's
    const int wlo = myq / chunk * chunk, whi = (myq + 15) / chunk * chunk, qlo = qi / chunk * chunk;   // first keys seen: wave's first, last query, lane's

    constexpr int KW = KS * 4, VW = VT * 2;                           // 16-byte words per staged row
    constexpr int KU = kKTile * KW / 512, VU = kKTile * VW / 512;     // ... per thread
    static_assert(kKTile * KW % 512 == 0 && kKTile * VW % 512 == 0, "whole rounds of the workgroup");
    u32x4_m rk[KU], rv[VU];
    const char* kbase = (const char*)(kr + ((int64_t)r0 * G + g) * D);
    const char* vbase = (const char*)(vr + ((int64_t)r0 * G + g) * V);
    auto fetch = [&](int k0) {
#pragma unroll
        for (int u = 0; u < KU; ++u) {
            const int i = t + 512 * u, d = (i % KW) * 8, pos = min(k0 + i / KW, kend - 1);
            rk[u] = *reinterpret_cast<const u32x4_m*>(kbase + ((unsigned)pos * (unsigned)(G * D * 2) + (unsigned)((d < D ? d : 0) * 2)));
        }
#pragma unroll
        for (int u = 0; u < VU; ++u) {
            const int i = t + 512 * u, d = (i % VW) * 8, pos = min(k0 + i / VW, kend - 1);
            rv[u] = *reinterpret_cast<const u32x4_m*>(vbase + ((unsigned)pos * (unsigned)(G * V * 2) + (unsigned)((d < V ? d : 0) * 2)));
        }
    };
    fetch(kbeg);

    const int64_t row = r0 + min(qi, T - 1);                          // queries behind the prompt repeat its last one and are not stored
    u32x4_m q[KS];
    {
        const float* src = a.proj + row * a.ld + (int64_t)h * D;
        const float* tab = a.table + row * rot;
        f32x4_m x[KS][2];
        float ss = 0.f;
#pragma unroll
        for (int k = 0; k < KS; ++k) {
            const int d = 32 * k + 8 * kg;
            x[k][0] = x[k][1] = f32x4_m{0.f, 0.f, 0.f, 0.f};
            if (d < D) {
                x[k][0] = *reinterpret_cast<const f32x4_u*>(src + d);
                x[k][1] = *reinterpret_cast<const f32x4_u*>(src + d + 4);
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    const int dd = d + 2 * e;
                    if (dd < rot) {
                        const float cs = tab[dd >> 1], sn = tab[rot / 2 + (dd >> 1)];
                        const float u = x[k][e >> 1][2 * (e & 1)], v = x[k][e >> 1][2 * (e & 1) + 1];
                        x[k][e >> 1][2 * (e & 1)] = u * cs - v * sn;
                        x[k][e >> 1][2 * (e & 1) + 1] = v * cs + u * sn;
                    }
                }
            }
#pragma unroll
            for (int e = 0; e < 8; ++e) ss += x[k][e >> 2][e & 3] * x[k][e >> 2][e & 3];
        }
        const float inv = 1.0f / sqrtf(col4_sum(ss) / (float)D + a.eps);
#pragma unroll
        for (int k = 0; k < KS; ++k)
#pragma unroll
            for (int e = 0; e < 4; ++e) q[k][e] = pack_bf16_hw(x[k][e >> 1][2 * (e & 1)] * inv, x[k][e >> 1][2 * (e & 1) + 1] * inv);
    }
    f32x4_m o[VT];
    float m = a.sink[h] * 1.44269504f, l = 1.0f;                      // weights as powers of two
#pragma unroll
    for (int v = 0; v < VT; ++v) o[v] = f32x4_m{0.f, 0.f, 0.f, 0.f};
    const float scale2 = a.scale * 1.44269504f;
    for (int k0 = kbeg; k0 < kend; k0 += kKTile) {
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
        if (k0 > myq + 15 || k0 + kKTile <= wlo) continue;            // no query of the wave sees a key of the step
        f32x4_m s[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            s[j] = f32x4_m{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int k = 0; k < KS; ++k) s[j] = mma16(*reinterpret_cast<const u32x4_m*>(kt + (16 * j + c) * KSTR + 32 * k + 8 * kg), q[k], s[j]);
        }
        const bool edge = k0 + kKTile - 1 > myq || k0 < whi;          // some query does not see some key
        float mx = -INFINITY;
#pragma unroll
        for (int j = 0; j < 4; ++j)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int key = k0 + 16 * j + 4 * kg + e;
                float x = s[j][e] * scale2;
                if (edge && (key > qi || key < qlo)) x = -INFINITY;
                s[j][e] = x;
                mx = fmaxf(mx, x);
            }
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
    const float f = sigmoid_f32(a.proj[row * a.ld + (int64_t)(H + G) * D + (int64_t)G * V + h]) / l;
    bf16_t* out = (bf16_t*)a.ctx + (row * H + h) * V + 4 * kg;
#pragma unroll
    for (int v = 0; v < VT; ++v)
        if (16 * v + 4 * kg < V)
            *reinterpret_cast<uint2*>(out + 16 * v) = make_uint2(pack_bf16_hw(o[v][0] * f, o[v][1] * f), pack_bf16_hw(o[v][2] * f, o[v][3] * f));
}

template <typename F>
void with_lds(F kern, size_t bytes) { (void)hipFuncSetAttribute((const void*)kern, hipFuncAttributeMaxDynamicSharedMemorySize, (int)bytes); }

}  // namespace

void head_rms_norm(hipStream_t s, int in_dtype, int out_dtype, const void* x, void* y, int64_t n, int64_t head_dim, float eps) {
    if (n <= 0) return;
    const unsigned g = (unsigned)cdiv_c(n, 4);
    if (in_dtype == 0 && out_dtype == 0) head_norm_kernel<float, float><<<g, 256, 0, s>>>((const float*)x, (float*)y, n, head_dim, eps);
    else if (in_dtype == 0) head_norm_kernel<float, bf16_t><<<g, 256, 0, s>>>((const float*)x, (bf16_t*)y, n, head_dim, eps);
    else if (out_dtype == 0) head_norm_kernel<bf16_t, float><<<g, 256, 0, s>>>((const bf16_t*)x, (float*)y, n, head_dim, eps);
    else head_norm_kernel<bf16_t, bf16_t><<<g, 256, 0, s>>>((const bf16_t*)x, (bf16_t*)y, n, head_dim, eps);
}
void head_gate(hipStream_t s, int dtype, const void* x, const float* gate, void* y, int64_t rows, int64_t heads, int64_t vdim, int64_t ld) {
    const int64_t n = rows * heads * vdim;
    if (n <= 0) return;
    const unsigned g = (unsigned)cdiv_c(n, 256);
    if (dtype == 0) head_gate_kernel<float><<<g, 256, 0, s>>>((const float*)x, gate, (float*)y, n, heads, vdim, ld);
    else head_gate_kernel<bf16_t><<<g, 256, 0, s>>>((const bf16_t*)x, gate, (bf16_t*)y, n, heads, vdim, ld);
}
void chunk_attn(hipStream_t s, const ChunkAttnArgs& a) {
    if (a.t <= 0) return;
    const size_t lds = (size_t)(a.dim + a.vdim + 256 + 16) * sizeof(float);
    const dim3 grid((unsigned)a.t, (unsigned)a.heads);
    if (a.dtype == 0) { with_lds(chunk_attn_kernel<float>, lds); chunk_attn_kernel<float><<<grid, 256, lds, s>>>(a); }
    else { with_lds(chunk_attn_kernel<bf16_t>, lds); chunk_attn_kernel<bf16_t><<<grid, 256, lds, s>>>(a); }
}

static void chunk_rows(hipStream_t s, const ChunkSeqArgs& a, int64_t skip, void* q, void* k, void* v) {
    int64_t longest = 0;
    for (int b = 0; b < a.nseq; ++b) longest = std::max<int64_t>(longest, a.len[b]);
    const dim3 grid((unsigned)cdiv_c(longest * (a.heads + 2 * a.kv_heads - skip), 4), 1, (unsigned)a.nseq);
    if (a.dtype == 0) chunk_rows_kernel<float><<<grid, 256, 0, s>>>(a, (int)skip, (float*)q, (float*)k, (float*)v);
    else chunk_rows_kernel<bf16_t><<<grid, 256, 0, s>>>(a, (int)skip, (bf16_t*)q, (bf16_t*)k, (bf16_t*)v);
}
// the sizes that the matrix-core launches tile
static bool chunk_fast(int dtype, int64_t dim, int64_t vdim) {
    return dtype == 2 && dim % 8 == 0 && vdim % 8 == 0 && dim <= 256 && vdim <= 256;
}
// slices of a chunk's rows: one step of the four waves each, fewer where the batch fills the chip by itself or tickets run out
static int64_t chunk_nsplit(int64_t nseq, int64_t rows, int64_t heads, int64_t kv_heads) {
    const int64_t blocks = nseq * kv_heads * cdiv_c(heads / kv_heads, kDecHeads);
    if (blocks > (int64_t)kSkinnyTickets) return 1;
    int64_t n = std::min<int64_t>(cdiv_c(rows, 4 * kDecTile), 64);
    while (n > 1 && blocks * n > 1024) n = (n + 1) / 2;
    return n;
}
size_t chunk_decode_scratch_bytes(int dtype, int64_t nseq, int64_t rows, int64_t heads, int64_t kv_heads, int64_t dim, int64_t vdim) {
    if (chunk_fast(dtype, dim, vdim)) {   // any number of sequences of a launch may come up to nseq
        int64_t ns = 1;
        for (int64_t b = 1; b <= nseq; ++b) ns = std::max(ns, chunk_nsplit(b, rows, heads, kv_heads));
        return (size_t)(nseq * heads * ns * (vdim + 2)) * sizeof(float);
    }
    const size_t es = dtype == 0 ? 4 : 2;
    return chunk_align((size_t)(nseq * heads * dim) * es) + chunk_align((size_t)(nseq * heads * vdim) * es);
}
template <int KS, int VT>
static void launch_decode(hipStream_t s, const ChunkSeqArgs& a) {
    constexpr size_t rows = (size_t)4 * kDecTile * (VT * 16 + 8) * 2, sums = (size_t)4 * kDecHeads * VT * 16 * 4;
    constexpr size_t lds = (size_t)(kDecHeads * (KS * 32 + 8) + KS * 32 + 8 + VT * 16 + 8) * 2 + (rows > sums ? rows : sums);
    static_assert(lds + 1024 <= 160 * 1024, "LDS of one CU");
    static_assert(((KS * 32 + 8) * 2) % 16 == 0 && ((VT * 16 + 8) * 2) % 16 == 0, "16-byte rows");
    with_lds(chunk_decode_kernel<KS, VT>, lds);
    const int64_t ns = chunk_nsplit(a.nseq, a.rows, a.heads, a.kv_heads);
    const dim3 grid((unsigned)ns, (unsigned)(a.kv_heads * cdiv_c(a.heads / a.kv_heads, kDecHeads)), (unsigned)a.nseq);
    chunk_decode_kernel<KS, VT><<<grid, 256, lds, s>>>(a, (float*)a.scratch, a.tickets, (int)ns);
}
template <int KS>
static void launch_decode_v(hipStream_t s, const ChunkSeqArgs& a) {
    if (a.vdim <= 64) launch_decode<KS, 4>(s, a);
    else if (a.vdim <= 128) launch_decode<KS, 8>(s, a);
    else launch_decode<KS, 16>(s, a);
}
int chunk_decode(hipStream_t s, const ChunkSeqArgs& a) {
    if (chunk_fast(a.dtype, a.dim, a.vdim)) {
        const int64_t ks = cdiv_c(a.dim, 32);
        if (ks <= 2) launch_decode_v<2>(s, a);
        else if (ks <= 4) launch_decode_v<4>(s, a);
        else launch_decode_v<8>(s, a);
        return 1;
    }
    const size_t es = a.dtype == 0 ? 4 : 2;
    char* q = (char*)a.scratch;
    char* y = q + chunk_align((size_t)(a.nseq * a.heads * a.dim) * es);
    ChunkSeqArgs r = a;   // (the scratch holds this launch's rows from 0 on)
    const int64_t first = a.row0[0];
    r.proj += first * a.ld;
    r.table = a.table ? a.table + first * a.rot : nullptr;
    for (int b = 0; b < a.nseq; ++b) r.row0[b] -= (int)first;
    chunk_rows(s, r, 0, q, nullptr, nullptr);
    for (int b = 0; b < a.nseq; ++b) {
        ChunkAttnArgs x{};
        x.dtype = a.dtype;
        x.q = q + (size_t)(b * a.heads * a.dim) * es; x.k = a.kcache[b]; x.v = a.vcache[b]; x.sink = a.sink; x.position = a.pos + b;
        x.ctx = y + (size_t)(b * a.heads * a.vdim) * es;
        x.t = 1; x.heads = a.heads; x.kv_heads = a.kv_heads; x.dim = a.dim; x.vdim = a.vdim; x.chunk = a.chunk; x.rows = a.rows;
        x.k_row = a.dim; x.k_head = a.rows * a.dim; x.v_row = a.vdim; x.v_head = a.rows * a.vdim; x.scale = a.scale;
        chunk_attn(s, x);
    }
    head_gate(s, a.dtype, y, r.proj + (a.heads + a.kv_heads) * a.dim + a.kv_heads * a.vdim, (char*)a.ctx + (size_t)(first * a.heads * a.vdim) * es, a.nseq,
              a.heads, a.vdim, a.ld);
    return 2 + a.nseq;
}

static bool chunk_prefill_fast(int dtype, int64_t total, int64_t kv_heads, int64_t dim, int64_t vdim) {
    return chunk_fast(dtype, dim, vdim) && total * kv_heads * std::max(dim, vdim) < (1ll << 31);   // 32-bit byte offsets
}
size_t chunk_prefill_scratch_bytes(int dtype, int64_t total, int64_t heads, int64_t kv_heads, int64_t dim, int64_t vdim) {
    const size_t es = dtype == 0 ? 4 : 2;
    size_t n = chunk_align((size_t)(total * kv_heads * dim) * es) + chunk_align((size_t)(total * kv_heads * vdim) * es);
    if (!chunk_prefill_fast(dtype, total, kv_heads, dim, vdim)) n += chunk_align((size_t)(total * heads * dim) * es) + chunk_align((size_t)(total * heads * vdim) * es);
    return n;
}
template <int KS, int VT>
static void launch_prefill(hipStream_t s, const ChunkSeqArgs& a, const void* k, const void* v, int64_t longest) {
    constexpr int lds = kKTile * (KS * 32 + 8 + VT * 16 + 8) * 2;
    static_assert(lds <= 160 * 1024, "LDS of one CU");
    with_lds(chunk_prefill_kernel<KS, VT>, lds);
    chunk_prefill_kernel<KS, VT><<<dim3((unsigned)cdiv_c(longest, kQTile), (unsigned)a.heads, (unsigned)a.nseq), 512, lds, s>>>(a, (const bf16_t*)k, (const bf16_t*)v);
}
template <int KS>
static void launch_prefill_v(hipStream_t s, const ChunkSeqArgs& a, const void* k, const void* v, int64_t longest) {
    if (a.vdim <= 64) launch_prefill<KS, 4>(s, a, k, v, longest);
    else if (a.vdim <= 128) launch_prefill<KS, 8>(s, a, k, v, longest);
    else launch_prefill<KS, 16>(s, a, k, v, longest);
}
int chunk_prefill(hipStream_t s, const ChunkSeqArgs& a) {
    const size_t es = a.dtype == 0 ? 4 : 2;
    char* k = (char*)a.scratch;
    char* v = k + chunk_align((size_t)(a.total * a.kv_heads * a.dim) * es);
    if (chunk_prefill_fast(a.dtype, a.total, a.kv_heads, a.dim, a.vdim)) {
        int64_t longest = 0;
        for (int b = 0; b < a.nseq; ++b) longest = std::max<int64_t>(longest, a.len[b]);
        const dim3 rows((unsigned)cdiv_c(longest * 2 * a.kv_heads, 16), 1, (unsigned)a.nseq);
        if (std::max(a.dim, a.vdim) <= 128) chunk_rows16_kernel<1><<<rows, 256, 0, s>>>(a, (bf16_t*)k, (bf16_t*)v);
        else chunk_rows16_kernel<2><<<rows, 256, 0, s>>>(a, (bf16_t*)k, (bf16_t*)v);
        const int64_t ks = cdiv_c(a.dim, 32);
        if (ks <= 2) launch_prefill_v<2>(s, a, k, v, longest);
        else if (ks <= 4) launch_prefill_v<4>(s, a, k, v, longest);
        else launch_prefill_v<8>(s, a, k, v, longest);
        return 2;
    }
    char* q = v + chunk_align((size_t)(a.total * a.kv_heads * a.vdim) * es);
    char* y = q + chunk_align((size_t)(a.total * a.heads * a.dim) * es);
    chunk_rows(s, a, 0, q, k, v);
    int n = 1;
    for (int b = 0; b < a.nseq; ++b) {
        const int64_t r = a.row0[b];
        ChunkAttnArgs x{};
        x.dtype = a.dtype;
        x.q = q + (size_t)(r * a.heads * a.dim) * es; x.k = k + (size_t)(r * a.kv_heads * a.dim) * es; x.v = v + (size_t)(r * a.kv_heads * a.vdim) * es;
        x.sink = a.sink;
        x.ctx = y + (size_t)(r * a.heads * a.vdim) * es;
        x.t = a.len[b]; x.heads = a.heads; x.kv_heads = a.kv_heads; x.dim = a.dim; x.vdim = a.vdim; x.chunk = a.chunk; x.rows = a.len[b];
        x.k_row = a.kv_heads * a.dim; x.k_head = a.dim; x.v_row = a.kv_heads * a.vdim; x.v_head = a.vdim; x.scale = a.scale;
        chunk_attn(s, x);
        head_gate(s, a.dtype, x.ctx, a.proj + r * a.ld + (a.heads + a.kv_heads) * a.dim + a.kv_heads * a.vdim,
                  (char*)a.ctx + (size_t)(r * a.heads * a.vdim) * es, a.len[b], a.heads, a.vdim, a.ld);
        n += 2;
    }
    return n;
}

}  // namespace k
}  // namespace gptrs
