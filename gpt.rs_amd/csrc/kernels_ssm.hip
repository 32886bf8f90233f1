// State-space mixer (Mamba-2): short causal convolution, selective state recurrence, gated norm.
//
// The second part are the launches of Mix::SsmSeq, a layer's whole mixer for every sequence of a batch:
//   * one row per sequence (decode): a step kernel (convolution of the channels it needs, recurrence, un-gated rows) and a
//     finish kernel (gated norm, the convolution's new history); both read the old history, so the caller may donate it;
//   * prompts: convolution, then the recurrence in chunks of 64 tokens on the matrix cores (bf16; ssd_kernel), gated norm.
//     f32 (and sizes outside its tiling) runs the token-by-token kernel.
//
// This file's first part are the stand-alone kernels of the CustomCall targets, one per target, for any sizes and either
// element type.  Rows of the input projection stay f32 (step sizes enter the recurrence from them); the state is f32.
#include <algorithm>

#include "kernels.hpp"
#include "device_utils.hpp"

namespace gptrs {
namespace k {

namespace {

inline int64_t cdiv_m(int64_t a, int64_t b) { return (a + b - 1) / b; }

// ---------------------------------------------------------------------------- convolution
template <typename T>
__global__ __launch_bounds__(256) void conv_silu_kernel(ConvArgs a) {
    const int64_t c = (int64_t)blockIdx.y * 256 + threadIdx.x, t = blockIdx.x;
    if (c >= a.ch) return;
    float acc = a.bias[c];
    for (int64_t k = 0; k < a.ntaps; ++k) {
        const int64_t r = t + k - (a.ntaps - 1);   // row of the input that tap k meets; negative: before this call
        const float v = r >= 0 ? a.p[r * a.ld + a.col + c] : a.state[(r + a.ntaps - 1) * a.ch + c];
        acc += a.taps[k * a.ch + c] * v;
    }
    Elem<T>::st((T*)a.y, t * a.ch + c, silu_f32(acc));
}

// one thread per channel; ascending j reads ahead of what it writes, so state_out may be state
__global__ __launch_bounds__(256) void conv_state_kernel(const float* __restrict__ p, const float* state, float* state_out, int64_t rows,
                                                         int64_t ld, int64_t col, int64_t ch, int64_t keep) {
    const int64_t c = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (c >= ch) return;
    for (int64_t j = 0; j < keep; ++j) {
        const int64_t r = rows + j - keep;
        state_out[j * ch + c] = r >= 0 ? p[r * ld + col + c] : state[(r + keep) * ch + c];
    }
}

// ---------------------------------------------------------------------------- recurrence, token by token
// Workgroup = head x slice of VC values; the slice's state [n][VC] lives in LDS.  Thread (v, g) owns the states
// n = g, g + NG, ... of value v.
template <typename T, int VC>
__global__ __launch_bounds__(256) void ssm_scan_kernel(SsmArgs a) {
    constexpr int NG = 256 / VC;
    extern __shared__ float ssm_lds[];
    float* S = ssm_lds;                        // [n][VC]
    float* red = ssm_lds + a.n * VC;           // [NG][VC]
    const int h = blockIdx.x, v0 = blockIdx.y * VC, v = threadIdx.x % VC, g = threadIdx.x / VC;
    const bool live = v0 + v < a.vdim;
    const int64_t inner = a.heads * a.vdim, ch = inner + 2 * a.groups * a.n;
    const int64_t grp = h / (a.heads / a.groups);
    const int64_t so = (int64_t)h * a.n * a.vdim + v0 + v;
    for (int64_t n = g; n < a.n; n += NG) S[n * VC + v] = live ? a.state[so + n * a.vdim] : 0.f;
    const float rate = expf(a.a_log[h]), bias = a.dt_bias[h], dd = a.d ? a.d[h] : 0.f;
    const T* xbc = (const T*)a.xbc;
    for (int64_t t = 0; t < a.rows; ++t) {
        const float dt = softplus_f32(a.p[t * a.ld + a.dt_col + h] + bias);
        const float decay = expf(-rate * dt);
        const float x = live ? Elem<T>::ld(xbc, t * ch + (int64_t)h * a.vdim + v0 + v) : 0.f;
        const float dx = dt * x;
        const int64_t bo = t * ch + inner + grp * a.n, co = bo + a.groups * a.n;
        float acc = 0.f;
        for (int64_t n = g; n < a.n; n += NG) {
            const float s = decay * S[n * VC + v] + dx * Elem<T>::ld(xbc, bo + n);
            S[n * VC + v] = s;
            acc += s * Elem<T>::ld(xbc, co + n);
        }
        if (a.y) {
            red[g * VC + v] = acc;
            __syncthreads();
            if (g == 0) {
                float y = 0.f;
                for (int q = 0; q < NG; ++q) y += red[q * VC + v];
                if (live) Elem<T>::st((T*)a.y, t * inner + (int64_t)h * a.vdim + v0 + v, y + dd * x);
            }
            __syncthreads();
        }
    }
    if (a.state_out && live)
        for (int64_t n = g; n < a.n; n += NG) a.state_out[so + n * a.vdim] = S[n * VC + v];
}

// ---------------------------------------------------------------------------- gated norm
// Workgroup = row x part.
template <typename T>
__global__ __launch_bounds__(256) void gated_rms_norm_kernel(const T* __restrict__ y, const float* __restrict__ p, const float* __restrict__ gain,
                                                             T* __restrict__ out, int64_t n, int64_t ld, int64_t col, int64_t part, float eps) {
    __shared__ float red[16];
    const int64_t r = blockIdx.x, g0 = (int64_t)blockIdx.y * part;
    float q = 0.f;
    for (int64_t i = threadIdx.x; i < part; i += 256) {
        const float v = Elem<T>::ld(y, r * n + g0 + i) * silu_f32(p[r * ld + col + g0 + i]);
        q += v * v;
    }
    const float inv = 1.0f / sqrtf(block_sum(q, red) / (float)part + eps);
    for (int64_t i = threadIdx.x; i < part; i += 256) {
        const float v = Elem<T>::ld(y, r * n + g0 + i) * silu_f32(p[r * ld + col + g0 + i]);
        Elem<T>::st(out, r * n + g0 + i, (v * inv) * gain[g0 + i]);
    }
}

template <typename T>
__global__ __launch_bounds__(256) void clamped_glu_kernel(const T* __restrict__ g, const T* __restrict__ u, T* __restrict__ y, int64_t n, GluParams p) {
    for (int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x; i < n; i += (int64_t)gridDim.x * 256)
        Elem<T>::st(y, i, glu_combine(Elem<T>::ld(g, i), Elem<T>::ld(u, i), p.kind, p.limit, p.alpha, p.shift));
}

// ---------------------------------------------------------------------------- decode: one token per sequence
// Workgroup = head x slice of VC values x sequence, 256 threads as VC / VEC columns of VEC values by NG groups of states.
template <int VC, int VEC>
__global__ __launch_bounds__(256) void ssm_step_kernel(SsmSeqArgs a, float* __restrict__ yraw) {
    constexpr int CT = VC / VEC, NG = 256 / CT;
    extern __shared__ float ssm_lds[];
    float* Bs = ssm_lds;              // [n]
    float* Cs = Bs + a.n;             // [n]
    float* xs = Cs + a.n;             // [VC]
    float* red = xs + VC;             // [NG][VC]
    const int h = blockIdx.x, v0 = blockIdx.y * VC, b = blockIdx.z, t = threadIdx.x;
    const int c = t % CT, g = t / CT;
    const int n = (int)a.n, vdim = (int)a.vdim, keep = (int)a.ntaps - 1;
    const int inner = (int)(a.heads * a.vdim), grp = h / (int)(a.heads / a.groups);
    const float* p = a.p + (int64_t)a.row0[b] * a.ld;
    const float* hist = a.conv_in[b];
    const float* S = a.state_in[b] + (int64_t)h * n * vdim + v0 + c * VEC;
    float* So = a.state_out[b] + (int64_t)h * n * vdim + v0 + c * VEC;
    const bool live = v0 + c * VEC < vdim;   // (VEC > 1: vdim is a multiple of it)
    // the first states are requested ahead of everything else
    constexpr int AHEAD = 4;
    float s[AHEAD][VEC];
#pragma unroll
    for (int u = 0; u < AHEAD; ++u) {
        const int i = g + u * NG;
#pragma unroll
        for (int e = 0; e < VEC; ++e) s[u][e] = 0.f;
        if (live && i < n) {
            if (VEC == 4) *reinterpret_cast<float4*>(s[u]) = *reinterpret_cast<const float4*>(S + (int64_t)i * vdim);
            else s[u][0] = S[(int64_t)i * vdim];
        }
    }
    auto conv = [&](int64_t ci) {
        float acc = a.bias[ci];
        for (int k = 0; k < keep; ++k) acc += a.taps[k * a.ch + ci] * hist[k * a.ch + ci];
        acc += a.taps[keep * a.ch + ci] * p[a.col + ci];
        return silu_f32(acc);
    };
    for (int i = t; i < 2 * n + VC; i += 256) {
        if (i < n) Bs[i] = conv(inner + (int64_t)grp * n + i);
        else if (i < 2 * n) Cs[i - n] = conv(inner + (a.groups + grp) * (int64_t)n + (i - n));
        else xs[i - 2 * n] = v0 + i - 2 * n < vdim ? conv((int64_t)h * vdim + v0 + i - 2 * n) : 0.f;
    }
    const float dt = softplus_f32(p[a.dt_col + h] + a.dt_bias[h]);
    const float decay = expf(-expf(a.a_log[h]) * dt);
    __syncthreads();
    float dx[VEC], acc[VEC];
#pragma unroll
    for (int e = 0; e < VEC; ++e) { dx[e] = dt * xs[c * VEC + e]; acc[e] = 0.f; }
    for (int i0 = g; i0 < n; i0 += AHEAD * NG) {
#pragma unroll
        for (int u = 0; u < AHEAD; ++u) {
            const int i = i0 + u * NG;
            if (i >= n) break;
            if (i0 != g && live) {
                if (VEC == 4) *reinterpret_cast<float4*>(s[u]) = *reinterpret_cast<const float4*>(S + (int64_t)i * vdim);
                else s[u][0] = S[(int64_t)i * vdim];
            }
            const float bb = Bs[i], cc = Cs[i];
#pragma unroll
            for (int e = 0; e < VEC; ++e) {
                s[u][e] = decay * s[u][e] + dx[e] * bb;
                acc[e] += s[u][e] * cc;
            }
            if (live) {
                if (VEC == 4) *reinterpret_cast<float4*>(So + (int64_t)i * vdim) = *reinterpret_cast<const float4*>(s[u]);
                else So[(int64_t)i * vdim] = s[u][0];
            }
        }
    }
#pragma unroll
    for (int e = 0; e < VEC; ++e) red[g * VC + c * VEC + e] = acc[e];
    __syncthreads();
    if (t < VC && v0 + t < vdim) {
        float y = 0.f;
        for (int q = 0; q < NG; ++q) y += red[q * VC + t];
        yraw[(int64_t)b * inner + (int64_t)h * vdim + v0 + t] = y + a.d[h] * xs[t];
    }
}

// Blocks 0 .. norm_groups - 1 of a sequence: the gated norm of one part; the others: the convolution's new history.
template <typename T>
__global__ __launch_bounds__(256) void ssm_finish_kernel(SsmSeqArgs a, const float* __restrict__ yraw) {
    __shared__ float red[16];
    const int b = blockIdx.y, t = threadIdx.x;
    const float* p = a.p + (int64_t)a.row0[b] * a.ld;
    const int64_t inner = a.heads * a.vdim;
    if ((int64_t)blockIdx.x >= a.norm_groups) {
        const int64_t c = ((int64_t)blockIdx.x - a.norm_groups) * 256 + t;
        if (c >= a.ch) return;
        const int64_t keep = a.ntaps - 1;
        for (int64_t j = 0; j + 1 < keep; ++j) a.conv_out[b][j * a.ch + c] = a.conv_in[b][(j + 1) * a.ch + c];
        if (keep > 0) a.conv_out[b][(keep - 1) * a.ch + c] = p[a.col + c];
        return;
    }
    const int64_t part = inner / a.norm_groups, g0 = (int64_t)blockIdx.x * part;
    const float* y = yraw + (int64_t)b * inner + g0;
    const float* z = p + a.z_col + g0;
    constexpr int KEEP = 8;   // gated values held in registers; longer parts form the rest twice
    float v[KEEP];
    float q = 0.f;
    int64_t i = t;
#pragma unroll
    for (int u = 0; u < KEEP; ++u, i += 256) {
        v[u] = i < part ? y[i] * silu_f32(z[i]) : 0.f;
        q += v[u] * v[u];
    }
    for (; i < part; i += 256) { const float w = y[i] * silu_f32(z[i]); q += w * w; }
    const float inv = 1.0f / sqrtf(block_sum(q, red) / (float)part + a.eps);
    T* out = (T*)a.out + (int64_t)a.row0[b] * inner + g0;
    i = t;
#pragma unroll
    for (int u = 0; u < KEEP; ++u, i += 256)
        if (i < part) Elem<T>::st(out, i, (v[u] * inv) * a.gain[g0 + i]);
    for (; i < part; i += 256) Elem<T>::st(out, i, ((y[i] * silu_f32(z[i])) * inv) * a.gain[g0 + i]);
}

// ---------------------------------------------------------------------------- prompts
// The convolution over whole prompts: a thread takes 4 channels of kConvRows rows and slides its window of taps along them.
constexpr int kConvRows = 16;
template <typename T, int K>
__global__ __launch_bounds__(256) void conv_rows_kernel(SsmSeqArgs a, T* __restrict__ xbc) {
    const int b = blockIdx.z;
    const int64_t c = 4 * ((int64_t)blockIdx.x * 256 + threadIdx.x), t0 = (int64_t)blockIdx.y * kConvRows;
    if (c >= a.ch || t0 >= a.len[b]) return;
    const float* p = a.p + (int64_t)a.row0[b] * a.ld + a.col + c;
    T* out = xbc + ((int64_t)(a.row0[b] - a.row0[0])) * a.ch + c;
    float4 tap[K], win[K];
#pragma unroll
    for (int k = 0; k < K; ++k) tap[k] = *reinterpret_cast<const float4*>(a.taps + k * a.ch + c);
    const float4 bias = *reinterpret_cast<const float4*>(a.bias + c);
#pragma unroll
    for (int k = 0; k + 1 < K; ++k) {
        const int64_t r = t0 + k - (K - 1);
        win[k + 1] = r >= 0 ? *reinterpret_cast<const float4*>(p + r * a.ld) : *reinterpret_cast<const float4*>(a.conv_in[b] + (r + K - 1) * a.ch + c);
    }
    const int64_t t1 = t0 + kConvRows < a.len[b] ? t0 + kConvRows : a.len[b];
    float4 in[kConvRows];   // all rows requested before the first is used
#pragma unroll
    for (int u = 0; u < kConvRows; ++u) in[u] = *reinterpret_cast<const float4*>(p + (t0 + u < t1 ? t0 + u : t1 - 1) * a.ld);
#pragma unroll
    for (int u = 0; u < kConvRows; ++u) {
        const int64_t t = t0 + u;
        if (t >= t1) break;
#pragma unroll
        for (int k = 0; k + 1 < K; ++k) win[k] = win[k + 1];
        win[K - 1] = in[u];
        float4 v = bias;
#pragma unroll
        for (int k = 0; k < K; ++k) { v.x += tap[k].x * win[k].x; v.y += tap[k].y * win[k].y; v.z += tap[k].z * win[k].z; v.w += tap[k].w * win[k].w; }
        v.x = silu_f32(v.x); v.y = silu_f32(v.y); v.z = silu_f32(v.z); v.w = silu_f32(v.w);
        if (sizeof(T) == 2) *reinterpret_cast<uint2*>(out + t * a.ch) = make_uint2(pack_bf16_hw(v.x, v.y), pack_bf16_hw(v.z, v.w));
        else *reinterpret_cast<float4*>(out + t * a.ch) = v;
    }
}

// The recurrence in chunks of 64 tokens (state-space duality).  With cum_t the running sum of the log decays inside a chunk,
//     y_t = sum_{s <= t} (C_t . B_s) exp(cum_t - cum_s) dt_s x_s  +  exp(cum_t) S^T C_t  +  D x_t
//     S  <- exp(cum_end) S + sum_s exp(cum_end - cum_s) dt_s B_s x_s^T
// so a chunk is four small matrix products.  Workgroup = head x slice of 16 VT values x sequence, 4 waves; it walks the chunks of
// its sequence, the next chunk's words in registers while one is worked on.  Wave w owns the tokens t = 16 w .. of a chunk and
// the states n = 16 (w + 4 i) .., i < NPW, which it keeps in f32 accumulators (rows: states, columns: values) from the first
// chunk to the last.  Products are taken transposed (scores: rows = s, columns = t; result: rows = values, columns = t): the
// decayed scores feed the second product from registers.  Factors that are not bf16 already (the decayed scores, the
// weighted x, the state as an operand) enter the products as a bf16 value plus its remainder.  Logarithms are to base 2.
constexpr int kChunk = 64;
template <int NPW, int VT>
__global__ __launch_bounds__(256) void ssd_kernel(SsmSeqArgs a, const bf16_t* __restrict__ xbc, bf16_t* __restrict__ y) {
    constexpr int NP = 64 * NPW, NSTR = NP + 8, VS = 16 * VT, XSTR = VS + 8;
    extern __shared__ __align__(16) unsigned char ssd_smem[];
    bf16_t* Bm = reinterpret_cast<bf16_t*>(ssd_smem);   // [64][NSTR] token rows of B
    bf16_t* Cm = Bm + kChunk * NSTR;                    // [64][NSTR]
    bf16_t* xm = Cm + kChunk * NSTR;                    // [64][XSTR]
    bf16_t* sh = xm + kChunk * XSTR;                    // [VS][NSTR] S^T
    bf16_t* sl = sh + VS * NSTR;                        // [VS][NSTR] its remainder
    float* steps = reinterpret_cast<float*>(sl + VS * NSTR);   // two buffers of cum | dt | exp(cum_end - cum_s) dt_s, [64] each
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, c = lane & 15, kg = lane >> 4;
    const int h = blockIdx.x, v0 = blockIdx.y * VS, b = blockIdx.z, T = a.len[b];
    const int N = (int)a.n, vdim = (int)a.vdim, inner = (int)(a.heads * a.vdim), grp = h / (int)(a.heads / a.groups);
    const int64_t ch = a.ch;
    const bf16_t* rows = xbc + (int64_t)(a.row0[b] - a.row0[0]) * ch;
    bf16_t* yout = y + (int64_t)(a.row0[b] - a.row0[0]) * inner + (int64_t)h * vdim + v0;
    const float* p = a.p + (int64_t)a.row0[b] * a.ld + a.dt_col + h;
    const bf16_t* bsrc = rows + inner + (int64_t)grp * N;
    const bf16_t* csrc = bsrc + a.groups * (int64_t)N;
    const bf16_t* xsrc = rows + (int64_t)h * vdim + v0;
    const float rate2 = expf(a.a_log[h]) * 1.44269504f, dtb = a.dt_bias[h], dd = a.d[h];

    f32x4_m S[NPW][VT];                                 // rows n = 16 (wave + 4 j) + 4 kg + e, column v = 16 i + c
#pragma unroll
    for (int j = 0; j < NPW; ++j)
#pragma unroll
        for (int i = 0; i < VT; ++i)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int n = 16 * (wave + 4 * j) + 4 * kg + e, v = v0 + 16 * i + c;
                S[j][i][e] = n < N && v < vdim ? a.state_in[b][((int64_t)h * N + n) * vdim + v] : 0.f;
            }
    // columns that no token fills stay zero
    for (int i = tid; i < kChunk * (NP / 8); i += 256) {
        const int r = i / (NP / 8), n = (i % (NP / 8)) * 8;
        if (n >= N) {
            *reinterpret_cast<uint4*>(Bm + r * NSTR + n) = make_uint4(0u, 0u, 0u, 0u);
            *reinterpret_cast<uint4*>(Cm + r * NSTR + n) = make_uint4(0u, 0u, 0u, 0u);
        }
    }
    // a thread's words of a chunk: the same place of rows BR apart
    constexpr int NW = NP / 8, BR = 256 / NW, BU = kChunk / BR, XW = VS / 8, XU = (kChunk * XW + 255) / 256;
    const int br = tid / NW, bk = 8 * (tid % NW);
    const bool bl = bk < N;
    uint4 rb[BU], rc[BU], rx[XU];
    float rdt = 0.f;
    auto fetch = [&](int t0) {                          // tokens behind the prompt are zero
#pragma unroll
        for (int u = 0; u < BU; ++u) {
            const int r = t0 + br + BR * u;
            rb[u] = rc[u] = make_uint4(0u, 0u, 0u, 0u);
            if (bl && r < T) {
                rb[u] = *reinterpret_cast<const uint4*>(bsrc + (int64_t)r * ch + bk);
                rc[u] = *reinterpret_cast<const uint4*>(csrc + (int64_t)r * ch + bk);
            }
        }
#pragma unroll
        for (int u = 0; u < XU; ++u) {
            const int i = tid + 256 * u, r = i / XW, k = i % XW;
            rx[u] = make_uint4(0u, 0u, 0u, 0u);
            if (i < kChunk * XW && t0 + r < T && v0 + 8 * k < vdim) rx[u] = *reinterpret_cast<const uint4*>(xsrc + (int64_t)(t0 + r) * ch + 8 * k);
        }
        if (wave == 0) rdt = t0 + lane < T ? p[(int64_t)(t0 + lane) * a.ld] : 0.f;
    };
    auto decays = [&](int t0, float* st) {              // wave 0: step sizes and running decays of a chunk
        const bool live = t0 + lane < T;                // behind the prompt: no step, no decay
        const float dt = live ? softplus_f32(rdt + dtb) : 0.f;
        float s = -rate2 * dt;
#pragma unroll
        for (int off = 1; off < 64; off <<= 1) {
            const float o = __shfl_up(s, off, 64);
            if (lane >= off) s += o;
        }
        const float end = __shfl(s, 63, 64);
        st[lane] = s;
        st[kChunk + lane] = dt;
        st[2 * kChunk + lane] = __builtin_amdgcn_exp2f(end - s) * dt;
    };
    fetch(0);
    if (wave == 0) decays(0, steps);
    int buf = 0;
    for (int t0 = 0; t0 < T; t0 += kChunk, buf ^= 1) {
        const float* cum = steps + buf * 3 * kChunk;
        __syncthreads();                                // the previous chunk has been read
        if (bl) {
#pragma unroll
            for (int u = 0; u < BU; ++u) {
                *reinterpret_cast<uint4*>(Bm + (br + BR * u) * NSTR + bk) = rb[u];
                *reinterpret_cast<uint4*>(Cm + (br + BR * u) * NSTR + bk) = rc[u];
            }
        }
#pragma unroll
        for (int u = 0; u < XU; ++u) {
            const int i = tid + 256 * u, r = i / XW, k = i % XW;
            if (i < kChunk * XW) *reinterpret_cast<uint4*>(xm + r * XSTR + 8 * k) = rx[u];
        }
#pragma unroll
        for (int j = 0; j < NPW; ++j)
#pragma unroll
            for (int i = 0; i < VT; ++i) {
                const int at = (16 * i + c) * NSTR + 16 * (wave + 4 * j) + 4 * kg;
                uint2 hi, lo;
                split_bf16_hw(S[j][i][0], S[j][i][1], hi.x, lo.x);
                split_bf16_hw(S[j][i][2], S[j][i][3], hi.y, lo.y);
                *reinterpret_cast<uint2*>(sh + at) = hi;
                *reinterpret_cast<uint2*>(sl + at) = lo;
            }
        __syncthreads();
        const bool more = t0 + kChunk < T;
        if (more) fetch(t0 + kChunk);

        // columns: the wave's 16 tokens
        u32x4_m ca[2 * NPW];
#pragma unroll
        for (int k = 0; k < 2 * NPW; ++k) ca[k] = *reinterpret_cast<const u32x4_m*>(Cm + (16 * wave + c) * NSTR + 32 * k + 8 * kg);
        const float ct = cum[16 * wave + c];
        f32x4_m yt[VT];
        const float et = __builtin_amdgcn_exp2f(ct);
#pragma unroll
        for (int i = 0; i < VT; ++i) {
            yt[i] = f32x4_m{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int k = 0; k < 2 * NPW; ++k) {
                yt[i] = mma16(*reinterpret_cast<const u32x4_m*>(sh + (16 * i + c) * NSTR + 32 * k + 8 * kg), ca[k], yt[i]);
                yt[i] = mma16(*reinterpret_cast<const u32x4_m*>(sl + (16 * i + c) * NSTR + 32 * k + 8 * kg), ca[k], yt[i]);
            }
#pragma unroll
            for (int e = 0; e < 4; ++e) yt[i][e] *= et;
        }
#pragma unroll
        for (int k = 0; k < 2; ++k) {                   // steps of 32 tokens s
            if (k > wave / 2) break;
            u32x4_m mh, ml;
#pragma unroll
            for (int jj = 0; jj < 2; ++jj) {
                const int j = 2 * k + jj;
                f32x4_m g = {0.f, 0.f, 0.f, 0.f};
                if (j <= wave) {                        // later tokens do not reach the wave's
#pragma unroll
                    for (int q = 0; q < 2 * NPW; ++q)
                        g = mma16(*reinterpret_cast<const u32x4_m*>(Bm + (16 * j + c) * NSTR + 32 * q + 8 * kg), ca[q], g);
                }
                const f32x4_m cs = *reinterpret_cast<const f32x4_m*>(cum + 16 * j + 4 * kg), ds = *reinterpret_cast<const f32x4_m*>(cum + kChunk + 16 * j + 4 * kg);
                float f[4];
#pragma unroll
                for (int e = 0; e < 4; ++e)
                    f[e] = 16 * j + 4 * kg + e <= 16 * wave + c ? g[e] * (__builtin_amdgcn_exp2f(ct - cs[e]) * ds[e]) : 0.f;
                uint32_t hi, lo;
                split_bf16_hw(f[0], f[1], hi, lo);
                mh[2 * jj] = hi; ml[2 * jj] = lo;
                split_bf16_hw(f[2], f[3], hi, lo);
                mh[2 * jj + 1] = hi; ml[2 * jj + 1] = lo;
            }
#pragma unroll
            for (int i = 0; i < VT; ++i) {
                const u32x4_m xv = lds_operand_t2(xm + 32 * k * XSTR + 16 * i, XSTR, lane);
                yt[i] = mma16(xv, mh, yt[i]);
                yt[i] = mma16(xv, ml, yt[i]);
            }
        }
        {
            const int t = 16 * wave + c;
            if (t0 + t < T) {
#pragma unroll
                for (int i = 0; i < VT; ++i) {
                    if (v0 + 16 * i + 4 * kg >= vdim) continue;
                    const uint2 xw = *reinterpret_cast<const uint2*>(xm + t * XSTR + 16 * i + 4 * kg);
                    *reinterpret_cast<uint2*>(yout + (int64_t)(t0 + t) * inner + 16 * i + 4 * kg) =
                        make_uint2(pack_bf16_hw(yt[i][0] + dd * bf16lo(xw.x), yt[i][1] + dd * bf16hi(xw.x)),
                                   pack_bf16_hw(yt[i][2] + dd * bf16lo(xw.y), yt[i][3] + dd * bf16hi(xw.y)));
                }
            }
        }
        // the state after the chunk
        const float edecay = __builtin_amdgcn_exp2f(cum[kChunk - 1]);
#pragma unroll
        for (int j = 0; j < NPW; ++j)
#pragma unroll
            for (int i = 0; i < VT; ++i)
#pragma unroll
                for (int e = 0; e < 4; ++e) S[j][i][e] *= edecay;
#pragma unroll
        for (int k = 0; k < kChunk / 32; ++k) {
            u32x4_m bv[NPW];
#pragma unroll
            for (int j = 0; j < NPW; ++j) bv[j] = lds_operand_t(Bm + 32 * k * NSTR + 16 * (wave + 4 * j), NSTR, lane);
            const f32x4_m w0 = *reinterpret_cast<const f32x4_m*>(cum + 2 * kChunk + 32 * k + 8 * kg), w1 = *reinterpret_cast<const f32x4_m*>(cum + 2 * kChunk + 32 * k + 8 * kg + 4);
            const float ws[8] = {w0[0], w0[1], w0[2], w0[3], w1[0], w1[1], w1[2], w1[3]};
#pragma unroll
            for (int i = 0; i < VT; ++i) {
                const u32x4_m xv = lds_operand_t(xm + 32 * k * XSTR + 16 * i, XSTR, lane);
                u32x4_m xh, xl;
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    uint32_t hi, lo;
                    split_bf16_hw(bf16lo(xv[e]) * ws[2 * e], bf16hi(xv[e]) * ws[2 * e + 1], hi, lo);
                    xh[e] = hi; xl[e] = lo;
                }
#pragma unroll
                for (int j = 0; j < NPW; ++j) {
                    S[j][i] = mma16(bv[j], xh, S[j][i]);
                    S[j][i] = mma16(bv[j], xl, S[j][i]);
                }
            }
        }
        if (more && wave == 0) decays(t0 + kChunk, steps + (buf ^ 1) * 3 * kChunk);
    }
#pragma unroll
    for (int j = 0; j < NPW; ++j)
#pragma unroll
        for (int i = 0; i < VT; ++i)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int n = 16 * (wave + 4 * j) + 4 * kg + e, v = v0 + 16 * i + c;
                if (n < N && v < vdim) a.state_out[b][((int64_t)h * N + n) * vdim + v] = S[j][i][e];
            }
}

// Gated norm of bf16 rows whose parts are multiples of 8: a wave per row and part of up to 64 * 8 * KEEP values, each formed once.
constexpr int kNormKeep = 4;
__global__ __launch_bounds__(256) void gated_norm_wave_kernel(const bf16_t* __restrict__ y, const float* __restrict__ p, const float* __restrict__ gain,
                                                              bf16_t* __restrict__ out, int64_t rows, int64_t n, int64_t ld, int64_t col, int part,
                                                              int groups, float eps) {
    const int lane = threadIdx.x & 63;
    const int64_t job = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
    if (job >= rows * groups) return;
    const int64_t r = job / groups, g0 = (job % groups) * part;
    float v[kNormKeep][8];
    float q = 0.f;
#pragma unroll
    for (int u = 0; u < kNormKeep; ++u) {
        const int i = 8 * (lane + 64 * u);
#pragma unroll
        for (int e = 0; e < 8; ++e) v[u][e] = 0.f;
        if (i < part) {
            const uint4 yw = *reinterpret_cast<const uint4*>(y + r * n + g0 + i);
            const float* z = p + r * ld + col + g0 + i;
            const float4 z0 = *reinterpret_cast<const float4*>(z), z1 = *reinterpret_cast<const float4*>(z + 4);
            v[u][0] = bf16lo(yw.x) * silu_f32(z0.x); v[u][1] = bf16hi(yw.x) * silu_f32(z0.y);
            v[u][2] = bf16lo(yw.y) * silu_f32(z0.z); v[u][3] = bf16hi(yw.y) * silu_f32(z0.w);
            v[u][4] = bf16lo(yw.z) * silu_f32(z1.x); v[u][5] = bf16hi(yw.z) * silu_f32(z1.y);
            v[u][6] = bf16lo(yw.w) * silu_f32(z1.z); v[u][7] = bf16hi(yw.w) * silu_f32(z1.w);
        }
#pragma unroll
        for (int e = 0; e < 8; ++e) q += v[u][e] * v[u][e];
    }
    const float inv = 1.0f / sqrtf(wave_sum(q) / (float)part + eps);
#pragma unroll
    for (int u = 0; u < kNormKeep; ++u) {
        const int i = 8 * (lane + 64 * u);
        if (i >= part) continue;
        const float4 a = *reinterpret_cast<const float4*>(gain + g0 + i), b = *reinterpret_cast<const float4*>(gain + g0 + i + 4);
        *reinterpret_cast<uint4*>(out + r * n + g0 + i) =
            make_uint4(pack_bf16_hw((v[u][0] * inv) * a.x, (v[u][1] * inv) * a.y), pack_bf16_hw((v[u][2] * inv) * a.z, (v[u][3] * inv) * a.w),
                       pack_bf16_hw((v[u][4] * inv) * b.x, (v[u][5] * inv) * b.y), pack_bf16_hw((v[u][6] * inv) * b.z, (v[u][7] * inv) * b.w));
    }
}

}  // namespace

void conv_silu(hipStream_t s, const ConvArgs& a) {
    if (a.rows <= 0 || a.ch <= 0) return;
    const dim3 grid((unsigned)a.rows, (unsigned)cdiv_m(a.ch, 256));
    if (a.dtype == 0) conv_silu_kernel<float><<<grid, 256, 0, s>>>(a);
    else conv_silu_kernel<bf16_t><<<grid, 256, 0, s>>>(a);
}
void conv_state(hipStream_t s, const float* p, const float* state, float* state_out, int64_t rows, int64_t ld, int64_t col, int64_t ch, int64_t ntaps) {
    if (ch <= 0 || ntaps <= 1) return;
    conv_state_kernel<<<(unsigned)cdiv_m(ch, 256), 256, 0, s>>>(p, state, state_out, rows, ld, col, ch, ntaps - 1);
}
template <typename T>
static void ssm_scan_t(hipStream_t s, const SsmArgs& a) {
    const int64_t budget = 96 * 1024;   // bytes of LDS for the state slice
#define GPTRS_SSM(VC)                                                                                                          \
    do {                                                                                                                       \
        const size_t lds = (size_t)(a.n * VC + 256) * sizeof(float);                                                           \
        (void)hipFuncSetAttribute((const void*)ssm_scan_kernel<T, VC>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds); \
        ssm_scan_kernel<T, VC><<<dim3((unsigned)a.heads, (unsigned)cdiv_m(a.vdim, VC)), 256, lds, s>>>(a);                     \
    } while (0)
    if (a.vdim > 32 && a.n * 64 * 4 <= budget) GPTRS_SSM(64);
    else if (a.vdim > 16 && a.n * 32 * 4 <= budget) GPTRS_SSM(32);
    else GPTRS_SSM(16);
#undef GPTRS_SSM
}
void ssm_scan(hipStream_t s, const SsmArgs& a) {
    if (a.rows <= 0 || a.heads <= 0 || a.vdim <= 0) return;
    if (a.dtype == 0) ssm_scan_t<float>(s, a);
    else ssm_scan_t<bf16_t>(s, a);
}
void gated_rms_norm(hipStream_t s, int dtype, const void* y, const float* p, const float* gain, void* out, int64_t rows, int64_t n, int64_t ld,
                    int64_t col, int64_t groups, float eps) {
    if (rows <= 0 || n <= 0) return;
    const int64_t part = n / groups;
    if (dtype == 2 && part % 8 == 0 && part <= 64 * 8 * kNormKeep && ld % 4 == 0 && col % 4 == 0 && rows * groups < (1ll << 31)) {
        gated_norm_wave_kernel<<<(unsigned)cdiv_m(rows * groups, 4), 256, 0, s>>>((const bf16_t*)y, p, gain, (bf16_t*)out, rows, n, ld, col, (int)part,
                                                                                 (int)groups, eps);
        return;
    }
    const dim3 grid((unsigned)rows, (unsigned)groups);
    if (dtype == 0) gated_rms_norm_kernel<float><<<grid, 256, 0, s>>>((const float*)y, p, gain, (float*)out, n, ld, col, n / groups, eps);
    else gated_rms_norm_kernel<bf16_t><<<grid, 256, 0, s>>>((const bf16_t*)y, p, gain, (bf16_t*)out, n, ld, col, n / groups, eps);
}
void clamped_glu(hipStream_t s, int dtype, const void* gate, const void* up, void* y, int64_t n, const GluParams& p) {
    if (n <= 0) return;
    const unsigned g = (unsigned)(cdiv_m(n, 256) > 4096 ? 4096 : cdiv_m(n, 256));
    if (dtype == 0) clamped_glu_kernel<float><<<g, 256, 0, s>>>((const float*)gate, (const float*)up, (float*)y, n, p);
    else clamped_glu_kernel<bf16_t><<<g, 256, 0, s>>>((const bf16_t*)gate, (const bf16_t*)up, (bf16_t*)y, n, p);
}


static size_t ssm_align(size_t n) { return (n + 255) / 256 * 256; }
// decode: un-gated f32 rows; prompts: convolved rows and un-gated rows in T
size_t ssm_seq_scratch_bytes(int dtype, int64_t rows, int64_t heads, int64_t groups, int64_t n, int64_t vdim) {
    const size_t es = dtype == 0 ? 4 : 2, inner = (size_t)(heads * vdim), ch = inner + 2 * (size_t)(groups * n);
    return std::max(ssm_align((size_t)rows * inner * 4), ssm_align((size_t)rows * ch * es) + ssm_align((size_t)rows * inner * es));
}

static int ssm_decode(hipStream_t s, const SsmSeqArgs& a) {
    float* yraw = (float*)a.scratch + (int64_t)a.row0[0] * a.heads * a.vdim;
    // slices of 16 values while that is what fills the chip, whole heads when there are many of them
    const bool vec = a.vdim % 4 == 0;
    const bool wide = vec && a.vdim >= 64 && a.heads * a.nseq >= 512;
#define GPTRS_STEP(VC, VEC)                                                                                                         \
    ssm_step_kernel<VC, VEC><<<dim3((unsigned)a.heads, (unsigned)cdiv_m(a.vdim, VC), (unsigned)a.nseq), 256,                        \
                               (2 * a.n + VC + 256 * VEC) * sizeof(float), s>>>(a, yraw)
    if (wide) GPTRS_STEP(64, 4);
    else if (vec) GPTRS_STEP(16, 4);
    else GPTRS_STEP(16, 1);
#undef GPTRS_STEP
    const dim3 grid((unsigned)(a.norm_groups + cdiv_m(a.ch, 256)), (unsigned)a.nseq);
    if (a.dtype == 0) ssm_finish_kernel<float><<<grid, 256, 0, s>>>(a, yraw);
    else ssm_finish_kernel<bf16_t><<<grid, 256, 0, s>>>(a, yraw);
    return 2;
}

int ssm_seq(hipStream_t s, const SsmSeqArgs& a) {
    bool one = true;
    for (int b = 0; b < a.nseq; ++b) one = one && a.len[b] == 1;
    if (one) return ssm_decode(s, a);
    const size_t es = a.dtype == 0 ? 4 : 2;
    const int64_t inner = a.heads * a.vdim;
    char* xbc = (char*)a.scratch;
    char* y = xbc + ssm_align((size_t)a.rows * a.ch * es);   // behind the convolved rows of this launch series
    int n = 0, longest = 0;
    for (int b = 0; b < a.nseq; ++b) longest = std::max(longest, a.len[b]);
    auto row = [&](int b) { return (int64_t)(a.row0[b] - a.row0[0]); };
    // convolution of all prompts in one launch where 4 channels go together, else prompt by prompt
    if (a.ch % 4 == 0 && a.ld % 4 == 0 && a.col % 4 == 0 && a.ntaps >= 2 && a.ntaps <= 4) {
        const dim3 grid((unsigned)cdiv_m(a.ch / 4, 256), (unsigned)cdiv_m(longest, kConvRows), (unsigned)a.nseq);
#define GPTRS_CONV(T) do { if (a.ntaps == 2) conv_rows_kernel<T, 2><<<grid, 256, 0, s>>>(a, (T*)xbc); \
                           else if (a.ntaps == 3) conv_rows_kernel<T, 3><<<grid, 256, 0, s>>>(a, (T*)xbc); \
                           else conv_rows_kernel<T, 4><<<grid, 256, 0, s>>>(a, (T*)xbc); } while (0)
        if (a.dtype == 0) GPTRS_CONV(float);
        else GPTRS_CONV(bf16_t);
#undef GPTRS_CONV
        ++n;
    } else {
        for (int b = 0; b < a.nseq; ++b) {
            ConvArgs c{};
            c.dtype = a.dtype;
            c.p = a.p + (int64_t)a.row0[b] * a.ld; c.taps = a.taps; c.bias = a.bias; c.state = a.conv_in[b];
            c.y = xbc + (size_t)(row(b) * a.ch) * es;
            c.rows = a.len[b]; c.ld = a.ld; c.col = a.col; c.ch = a.ch; c.ntaps = a.ntaps;
            conv_silu(s, c);
            ++n;
        }
    }
    for (int b = 0; b < a.nseq; ++b) {
        conv_state(s, a.p + (int64_t)a.row0[b] * a.ld, a.conv_in[b], a.conv_out[b], a.len[b], a.ld, a.col, a.ch, a.ntaps);
        ++n;
    }
    if (a.dtype == 2 && a.n % 8 == 0 && a.n <= 256 && a.vdim % 8 == 0) {
        // slices of 32 values, or of 16 where the slices are too few for the chip
#define GPTRS_SSD(NPW, VT)                                                                                                       \
        do {                                                                                                                     \
            constexpr int NS = 64 * NPW + 8, VS = 16 * VT;                                                                       \
            constexpr int lds = (2 * kChunk * NS + kChunk * (VS + 8) + 2 * VS * NS) * 2 + 6 * kChunk * 4;                        \
            static_assert(lds <= 160 * 1024, "LDS of one CU");                                                                   \
            (void)hipFuncSetAttribute((const void*)ssd_kernel<NPW, VT>, hipFuncAttributeMaxDynamicSharedMemorySize, lds);        \
            ssd_kernel<NPW, VT><<<dim3((unsigned)a.heads, (unsigned)cdiv_m(a.vdim, VS), (unsigned)a.nseq), 256, lds, s>>>(a, (const bf16_t*)xbc, (bf16_t*)y); \
        } while (0)
        const bool wide = a.vdim > 16 && a.heads * cdiv_m(a.vdim, 32) * a.nseq >= 160;
        if (a.n <= 64) { if (wide) GPTRS_SSD(1, 2); else GPTRS_SSD(1, 1); }
        else if (a.n <= 128) { if (wide) GPTRS_SSD(2, 2); else GPTRS_SSD(2, 1); }
        else { if (wide) GPTRS_SSD(4, 2); else GPTRS_SSD(4, 1); }
#undef GPTRS_SSD
        ++n;
    } else {
        for (int b = 0; b < a.nseq; ++b) {
            SsmArgs m{};
            m.dtype = a.dtype;
            m.xbc = xbc + (size_t)(row(b) * a.ch) * es; m.p = a.p + (int64_t)a.row0[b] * a.ld; m.dt_bias = a.dt_bias; m.a_log = a.a_log; m.d = a.d;
            m.state = a.state_in[b]; m.state_out = a.state_out[b]; m.y = y + (size_t)(row(b) * inner) * es;
            m.rows = a.len[b]; m.ld = a.ld; m.dt_col = a.dt_col; m.heads = a.heads; m.groups = a.groups; m.n = a.n; m.vdim = a.vdim;
            ssm_scan(s, m);
            ++n;
        }
    }
    gated_rms_norm(s, a.dtype, y, a.p + (int64_t)a.row0[0] * a.ld, a.gain, (char*)a.out + (size_t)a.row0[0] * inner * es, a.rows, inner, a.ld, a.z_col,
                   a.norm_groups, a.eps);
    return n + 1;
}

}  // namespace k
}  // namespace gptrs
