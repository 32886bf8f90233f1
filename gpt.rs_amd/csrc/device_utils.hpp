// Device helpers shared by the HIP kernels: bf16 <-> f32, wave64 reductions, 128-bit loads.
#pragma once
#include <hip/hip_runtime.h>

#include <cstdint>

namespace gptrs {
namespace k {

typedef uint16_t bf16_t;  // raw bf16 bit pattern

__device__ __forceinline__ float bf16_to_f32(bf16_t v) { return __uint_as_float((uint32_t)v << 16); }
// round-to-nearest-even (docs/backend.md:99); NaN stays a quiet NaN
__device__ __forceinline__ bf16_t f32_to_bf16(float f) {
    uint32_t u = __float_as_uint(f);
    if ((u & 0x7fffffffu) > 0x7f800000u) return (bf16_t)((u >> 16) | 0x0040u);
    u += 0x7fffu + ((u >> 16) & 1u);
    return (bf16_t)(u >> 16);
}
__device__ __forceinline__ float bf16lo(uint32_t w) { return __uint_as_float(w << 16); }
__device__ __forceinline__ float bf16hi(uint32_t w) { return __uint_as_float(w & 0xffff0000u); }
__device__ __forceinline__ uint32_t pack_bf16x2(float lo, float hi) {
    return (uint32_t)f32_to_bf16(lo) | ((uint32_t)f32_to_bf16(hi) << 16);
}

// A gate / up pair of a feed-forward layer.  kind 0: silu(g) * u (ops/functional/activation.rs:141-162).  kind 1, the
// clamped unit: g <- min(g, limit), u <- clamp(u, +-limit), g * sigmoid(alpha g) * (u + shift).
__device__ __forceinline__ float glu_combine(float g, float u, int kind, float limit, float alpha, float shift) {
    if (kind == 1) {
        g = fminf(g, limit);
        u = fminf(fmaxf(u, -limit), limit);
        return (g / (1.0f + expf(g * -alpha))) * (u + shift);
    }
    return (g / (1.0f + expf(g * -1.0f))) * u;
}
__device__ __forceinline__ float silu_f32(float x) { return x / (1.0f + expf(-x)); }
__device__ __forceinline__ float softcap_f32(float x, float cap) { return cap * tanhf(x / cap); }
// log(1 + e^x) without overflow and without losing small values
__device__ __forceinline__ float softplus_f32(float x) { return fmaxf(x, 0.0f) + log1pf(expf(-fabsf(x))); }

// Loads / stores as f32 whatever the element type
template <typename T> struct Elem;
template <> struct Elem<float> {
    static __device__ __forceinline__ float ld(const float* p, int64_t i) { return p[i]; }
    static __device__ __forceinline__ void st(float* p, int64_t i, float v) { p[i] = v; }
    static __device__ __forceinline__ float round(float v) { return v; }
};
template <> struct Elem<bf16_t> {
    static __device__ __forceinline__ float ld(const bf16_t* p, int64_t i) { return bf16_to_f32(p[i]); }
    static __device__ __forceinline__ void st(bf16_t* p, int64_t i, float v) { p[i] = f32_to_bf16(v); }
    static __device__ __forceinline__ float round(float v) { return bf16_to_f32(f32_to_bf16(v)); }
};

// ---- 16 x 16 x 32 bf16 matrix-core tiles.  Operand: lane = 16 * k-group + row (A) or column (B) holds 8 consecutive k;
// result: lane = 16 * kg + column holds rows 4 kg .. 4 kg + 3.
typedef __bf16 bf16x8_m __attribute__((ext_vector_type(8)));
typedef float f32x4_m __attribute__((ext_vector_type(4)));
typedef uint32_t u32x4_m __attribute__((ext_vector_type(4)));
typedef uint32_t u32x2_m __attribute__((ext_vector_type(2)));
__device__ __forceinline__ f32x4_m mma16(const u32x4_m& a, const u32x4_m& b, f32x4_m c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_m, a), __builtin_bit_cast(bf16x8_m, b), c, 0, 0, 0);
}
// Operand whose k runs DOWN the rows of an LDS matrix m[k][..] (stride in elements, a multiple of 4; m 8-byte aligned): the
// lane's row / column is m's column.  ds_read_b64_tr_b16 hands lane i of 16 the column i of 4 rows; lane 4 e + j of the 16 names
// columns 4 j .. 4 j + 3 of row e.
__device__ __forceinline__ u32x4_m lds_operand_t(const bf16_t* m, int stride, int lane) {
    typedef short s16x4 __attribute__((ext_vector_type(4)));
    typedef __attribute__((address_space(3))) s16x4* lds_p;
    const int c = lane & 15, kg = lane >> 4;
    const bf16_t* p = m + (8 * kg + (c >> 2)) * stride + 4 * (c & 3);
    const u32x2_m lo = __builtin_bit_cast(u32x2_m, __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_p)(p)));
    const u32x2_m hi = __builtin_bit_cast(u32x2_m, __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_p)(p + 4 * stride)));
    u32x4_m r;
    r.x = lo.x; r.y = lo.y; r.z = hi.x; r.w = hi.y;
    return r;
}
// The same for an operand whose k slots are the rows 4 kg .. 4 kg + 3 and 16 + 4 kg .. 16 + 4 kg + 3 of m: what the results of
// two stacked 16 x 16 tiles hold per lane, so that such results feed the next product from registers.
__device__ __forceinline__ u32x4_m lds_operand_t2(const bf16_t* m, int stride, int lane) {
    typedef short s16x4 __attribute__((ext_vector_type(4)));
    typedef __attribute__((address_space(3))) s16x4* lds_p;
    const int c = lane & 15, kg = lane >> 4;
    const bf16_t* p = m + (4 * kg + (c >> 2)) * stride + 4 * (c & 3);
    const u32x2_m lo = __builtin_bit_cast(u32x2_m, __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_p)(p)));
    const u32x2_m hi = __builtin_bit_cast(u32x2_m, __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_p)(p + 16 * stride)));
    u32x4_m r;
    r.x = lo.x; r.y = lo.y; r.z = hi.x; r.w = hi.y;
    return r;
}
// Sum / maximum over the four lanes that share a column (lane, lane ^ 16, lane ^ 32, lane ^ 48)
__device__ __forceinline__ float col4_sum(float v) {
    const u32x2_m a = __builtin_bit_cast(u32x2_m, __builtin_amdgcn_permlane16_swap(__float_as_uint(v), __float_as_uint(v), false, false));
    v = __uint_as_float(a.x) + __uint_as_float(a.y);
    const u32x2_m b = __builtin_bit_cast(u32x2_m, __builtin_amdgcn_permlane32_swap(__float_as_uint(v), __float_as_uint(v), false, false));
    return __uint_as_float(b.x) + __uint_as_float(b.y);
}
__device__ __forceinline__ float col4_max(float v) {
    const u32x2_m a = __builtin_bit_cast(u32x2_m, __builtin_amdgcn_permlane16_swap(__float_as_uint(v), __float_as_uint(v), false, false));
    v = fmaxf(__uint_as_float(a.x), __uint_as_float(a.y));
    const u32x2_m b = __builtin_bit_cast(u32x2_m, __builtin_amdgcn_permlane32_swap(__float_as_uint(v), __float_as_uint(v), false, false));
    return fmaxf(__uint_as_float(b.x), __uint_as_float(b.y));
}
// bf16 pair by the hardware converter (round to nearest even)
__device__ __forceinline__ uint32_t pack_bf16_hw(float lo, float hi) {
    typedef float f32x2_p __attribute__((ext_vector_type(2)));
    typedef __bf16 bf16x2_p __attribute__((ext_vector_type(2)));
    f32x2_p f;
    f.x = lo; f.y = hi;
    return __builtin_bit_cast(uint32_t, __builtin_convertvector(f, bf16x2_p));
}
// (a, b) as a pair of bf16 values plus the pair of their remainders: together 16 bits of each
__device__ __forceinline__ void split_bf16_hw(float a, float b, uint32_t& hi, uint32_t& lo) {
    hi = pack_bf16_hw(a, b);
    lo = pack_bf16_hw(a - bf16lo(hi), b - bf16hi(hi));
}
// Sum / maximum over the 16 lanes of a row, in every lane of it
__device__ __forceinline__ float row16_sum(float v) {
    int x = __float_as_int(v);
#define GPTRS_DPP_ADD(ctrl) x = __float_as_int(__int_as_float(x) + __int_as_float(__builtin_amdgcn_update_dpp(0, x, (ctrl), 0xf, 0xf, false)))
    GPTRS_DPP_ADD(0xB1);    // quad_perm [1,0,3,2]
    GPTRS_DPP_ADD(0x4E);    // quad_perm [2,3,0,1]
    GPTRS_DPP_ADD(0x141);   // row_half_mirror
    GPTRS_DPP_ADD(0x140);   // row_mirror
#undef GPTRS_DPP_ADD
    return __int_as_float(x);
}
__device__ __forceinline__ float row16_max(float v) {
    int x = __float_as_int(v);
#define GPTRS_DPP_MAX(ctrl) x = __float_as_int(fmaxf(__int_as_float(x), __int_as_float(__builtin_amdgcn_update_dpp(0, x, (ctrl), 0xf, 0xf, false))))
    GPTRS_DPP_MAX(0xB1);
    GPTRS_DPP_MAX(0x4E);
    GPTRS_DPP_MAX(0x141);
    GPTRS_DPP_MAX(0x140);
#undef GPTRS_DPP_MAX
    return __int_as_float(x);
}

// Sum over the 64 lanes of a wave, result in every lane.  Cross-lane moves use DPP modifiers
// (register-to-register, VALU rate) instead of ds_bpermute: 16 x 6 bpermutes per thread at the end of
// a GEMV block kept the LDS pipe busy for ~4 us.  Steps: xor 1 and xor 2 inside quads, mirrored
// halves of 8 and 16 lanes, then lane 15 / lane 31 of the previous rows broadcast into rows 1,3 /
// 2,3; lane 63 then holds the total and is read back as a scalar.
__device__ __forceinline__ float wave_sum(float v) {
    int x = __float_as_int(v);
#define GPTRS_DPP_ADD(ctrl, row_mask)                                                                         \
    x = __float_as_int(__int_as_float(x) +                                                                     \
                       __int_as_float(__builtin_amdgcn_update_dpp(0, x, (ctrl), (row_mask), 0xf, false)))
    GPTRS_DPP_ADD(0xB1, 0xf);   // quad_perm [1,0,3,2]
    GPTRS_DPP_ADD(0x4E, 0xf);   // quad_perm [2,3,0,1]
    GPTRS_DPP_ADD(0x141, 0xf);  // row_half_mirror
    GPTRS_DPP_ADD(0x140, 0xf);  // row_mirror
    GPTRS_DPP_ADD(0x142, 0xa);  // row_bcast:15 into rows 1 and 3
    GPTRS_DPP_ADD(0x143, 0xc);  // row_bcast:31 into rows 2 and 3
#undef GPTRS_DPP_ADD
    return __int_as_float(__builtin_amdgcn_readlane(x, 63));
}
__device__ __forceinline__ float wave_max(float v) {
#pragma unroll
    for (int off = 32; off > 0; off >>= 1) v = fmaxf(v, __shfl_xor(v, off, 64));
    return v;
}

// Block-wide sum / max for blocks of up to 1024 threads (16 waves); every thread gets the result.
__device__ __forceinline__ float block_sum(float v, float* smem16) {
    v = wave_sum(v);
    const int w = threadIdx.x >> 6, nw = (blockDim.x + 63) >> 6;
    __syncthreads();
    if ((threadIdx.x & 63) == 0) smem16[w] = v;
    __syncthreads();
    float r = 0.f;
    for (int i = 0; i < nw; ++i) r += smem16[i];
    return r;
}
__device__ __forceinline__ float block_max(float v, float* smem16) {
    v = wave_max(v);
    const int w = threadIdx.x >> 6, nw = (blockDim.x + 63) >> 6;
    __syncthreads();
    if ((threadIdx.x & 63) == 0) smem16[w] = v;
    __syncthreads();
    float r = -INFINITY;
    for (int i = 0; i < nw; ++i) r = fmaxf(r, smem16[i]);
    return r;
}

}  // namespace k
}  // namespace gptrs
