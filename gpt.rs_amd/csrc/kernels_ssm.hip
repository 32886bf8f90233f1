// State-space mixer (Mamba-2): short causal convolution, selective state recurrence, gated norm.
//
// This file's first part are the stand-alone kernels of the CustomCall targets, one per target, for any sizes and either
// element type.  Rows of the input projection stay f32 (step sizes enter the recurrence from them); the state is f32.
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

}  // namespace k
}  // namespace gptrs
