// State-space mixer (Mamba-2): short causal convolution, selective state recurrence, gated norm.
//
// The second part are the launches of Mix::SsmSeq, a layer's whole mixer for every sequence of a batch:
//   * one row per sequence (decode): a step kernel (convolution of the channels it needs, recurrence, un-gated rows) and a
//     finish kernel (gated norm, the convolution's new history); both read the old history, so the caller may donate it;
//   * prompts: convolution, then the recurrence in chunks of 64 tokens on the matrix cores (bf16; ssd_kernel), gated norm.
//     f32 runs the token-by-token kernel.
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
    char* y = xbc;   // behind the convolved rows of this launch series
    y += ssm_align((size_t)a.rows * a.ch * es);
    int n = 0;
    for (int b = 0; b < a.nseq; ++b) {
        const int64_t r = a.row0[b] - a.row0[0];
        ConvArgs c{};
        c.dtype = a.dtype;
        c.p = a.p + (int64_t)a.row0[b] * a.ld; c.taps = a.taps; c.bias = a.bias; c.state = a.conv_in[b];
        c.y = xbc + (size_t)(r * a.ch) * es;
        c.rows = a.len[b]; c.ld = a.ld; c.col = a.col; c.ch = a.ch; c.ntaps = a.ntaps;
        conv_silu(s, c);
        conv_state(s, c.p, a.conv_in[b], a.conv_out[b], a.len[b], a.ld, a.col, a.ch, a.ntaps);
        SsmArgs m{};
        m.dtype = a.dtype;
        m.xbc = c.y; m.p = c.p; m.dt_bias = a.dt_bias; m.a_log = a.a_log; m.d = a.d;
        m.state = a.state_in[b]; m.state_out = a.state_out[b]; m.y = y + (size_t)(r * inner) * es;
        m.rows = a.len[b]; m.ld = a.ld; m.dt_col = a.dt_col; m.heads = a.heads; m.groups = a.groups; m.n = a.n; m.vdim = a.vdim;
        ssm_scan(s, m);
        n += 3;
    }
    gated_rms_norm(s, a.dtype, y, a.p + (int64_t)a.row0[0] * a.ld, a.gain, (char*)a.out + (size_t)a.row0[0] * inner * es, a.rows, inner, a.ld, a.z_col,
                   a.norm_groups, a.eps);
    return n + 1;
}

}  // namespace k
}  // namespace gptrs
