// Launchers for the HIP kernels (gfx950).  Plain-pointer interfaces; all launches are
// asynchronous on the given stream.  Shapes are validated by the executor before any call.
#pragma once
#include <hip/hip_runtime.h>

#include <cstdint>

namespace gptrs {
namespace k {

constexpr int kMaxRank = 6;

// dst[dst_off + sum c_i*dst_stride_i] = src[src_off + sum c_i*src_stride_i] over `dims`.
// Strides in elements.  dyn: 0 static; 1 = add clamp(starts[i],0,dyn_max[i])*dyn_stride[i] to the
// SOURCE offset (DynamicSlice, cpu.rs:804-820); 2 = to the DEST offset (DynamicUpdateSlice).
struct CopyDesc {
    int rank = 0;
    int dyn = 0;
    int64_t total = 0;
    int64_t dst_off = 0, src_off = 0;
    int64_t dims[kMaxRank] = {};
    int64_t dst_stride[kMaxRank] = {};
    int64_t src_stride[kMaxRank] = {};
    int dyn_rank = 0;
    int64_t dyn_max[kMaxRank] = {};
    int64_t dyn_stride[kMaxRank] = {};
};
void copy_strided(hipStream_t s, void* dst, const void* src, int elem_size, const CopyDesc& d, const int32_t* starts);

// Up to 256 payload bytes travel as kernel arguments: an upload with no staging buffer and
// no host synchronisation (token ids, positions, update_starts, RoPE rows).
struct SmallPayload { uint32_t w[64]; };
void store_small(hipStream_t s, void* dst, const SmallPayload& p, int nbytes);
void fill_zero(hipStream_t s, void* dst, size_t nbytes);

// dtype: 0 f32, 2 bf16 (tags of include/gptrs_hip.h).  Math in f32, output rounded to dtype.
void unary(hipStream_t s, int dtype, int op, const void* x, void* y, int64_t n);
void binary(hipStream_t s, int dtype, int op, const void* a, const void* b, void* y, int64_t n);
// b is a scalar (broadcast literal) -- used when the rhs is BroadcastTo(scalar literal)
void binary_scalar(hipStream_t s, int dtype, int op, const void* a, float b, void* y, int64_t n);
void compare(hipStream_t s, int dtype, int op, const void* a, const void* b, uint8_t* y, int64_t n);
void select(hipStream_t s, int elem_size, const uint8_t* p, const void* t, const void* f, void* y, int64_t n);
void cast(hipStream_t s, int src_dtype, int dst_dtype, const void* x, void* y, int64_t n);
void iota(hipStream_t s, int32_t* y, int64_t outer, int64_t axis_len, int64_t inner);
// x viewed as [outer][axis_len][inner]; kind 0 sum 1 max 2 min; f32 accumulation
void reduce(hipStream_t s, int dtype, int kind, const void* x, void* y, int64_t outer, int64_t axis_len, int64_t inner);
// rows of `table` ([vocab][inner] elements of elem_size) by si32 index; an out-of-range index
// zero-fills the row and raises *err_flag (checked at the next synchronising call)
void take(hipStream_t s, int elem_size, const void* table, const int32_t* idx, void* y, int64_t n_idx,
          int64_t vocab, int64_t inner, int* err_flag);

// C[b][m][n] = sum_k A[b][m][k] * B[b][k][n]; element strides given per operand; f32 accumulate.
struct DotDesc {
    int64_t batch, m, n, k;
    int64_t a_sb, a_sm, a_sk;
    int64_t b_sb, b_sk, b_sn;
    int64_t c_sb, c_sm;  // C is [b][m][n] with n contiguous
};
// dtype: of A and B; out_f32: bf16 operands, the f32 accumulator is stored as f32 (DotGeneralSpec.out_dtype)
void dot_generic(hipStream_t s, int dtype, const void* a, const void* b, void* c, const DotDesc& d, bool out_f32 = false);

// last row of [rows][vocab] logits; ties -> smallest index; result (int64) written to *out
// greedy token of every row (rows * partial blocks <= scratch_cap), ties to the smallest index; out: si32[rows]
void argmax_rows(hipStream_t s, int dtype, const void* logits, int64_t rows, int64_t vocab, int32_t* out, float* scratch_val,
                 int32_t* scratch_idx, int scratch_cap);
void argmax_last_row(hipStream_t s, int dtype, const void* logits, int64_t rows, int64_t vocab, int64_t* out,
                     float* scratch_val, int32_t* scratch_idx, int scratch_cap);
// argmax_rows over a fixed device array of the library instead of caller scratch: no allocation anywhere.
// argmax_noalloc_init: once per device, with that device current (resolves the array's address on that GPU).
// argmax_rows_noalloc: false when the device was not initialised or rows is outside [1, argmax_noalloc_max_rows()].
hipError_t argmax_noalloc_init(int device);
int argmax_noalloc_max_rows();
bool argmax_rows_noalloc(hipStream_t s, int device, int dtype, const void* logits, int64_t rows, int64_t vocab, int32_t* out);
// temperature sampling with a caller-supplied uniform u (inverse-CDF over softmax(logits/T))
void sample_temperature_last_row(hipStream_t s, int dtype, const void* logits, int64_t rows, int64_t vocab,
                                 float temperature, float u, int64_t* out);

// How a gate / up pair is combined (see glu_combine in device_utils.hpp)
struct GluParams { int kind = 0; float limit = 0.f, alpha = 1.f, shift = 0.f; };
// What the unquantised linear kernels apply besides bias, GELU and residual: factors per output column (f32, between bias and
// residual), the kind of pair, and c * tanh(y / c) of the result (softcap c > 0; the weight-streaming kernels only)
struct EpiExtra { const float* colscale = nullptr; GluParams glu; float softcap = 0.f; };

// ---- fused kernels (kernels_fused.hip) --------------------------------------------------
// y[r] = LN(x[r]) * gamma + beta over the last axis, two-pass (mean, then centred variance):
// ops/functional/normalization.rs:123-174.  inv_n is the f32-rounded 1/N multiplier.
void layer_norm(hipStream_t s, int dtype, const void* x, const void* gamma, const void* beta, void* y,
                int64_t rows, int64_t n, float inv_n, float eps);
// the same over f32 rows, gains and offsets with a bf16 result (the f32 value rounded once)
void layer_norm_f32_to_bf16(hipStream_t s, const void* x, const void* gamma, const void* beta, void* y, int64_t rows, int64_t n,
                            float inv_n, float eps);
// y = x * rsqrt(mean(x^2)+eps) * gamma: normalization.rs:183-217
void rms_norm(hipStream_t s, int dtype, const void* x, const void* gamma, void* y, int64_t rows, int64_t n,
              float inv_n, float eps);
// the same over f32 rows and gains with a bf16 result (the f32 value rounded once)
void rms_norm_f32_to_bf16(hipStream_t s, const void* x, const void* gamma, void* y, int64_t rows, int64_t n, float inv_n,
                          float eps);
// out = x + mult * (y * rsqrt(mean(y^2) + eps) * gain) over f32 rows; out16 (may be null): the same rounded to bf16
void post_norm_add(hipStream_t s, const float* x, const float* y, const float* gain, float* out, void* out16, int64_t rows, int64_t n, float mult,
                   float inv_n, float eps);
void softcap(hipStream_t s, const float* x, float* y, int64_t n, float cap);
// rows of `table` [vocab, n] by index, as f32 times scale; out16 (may be null): the same rounded to bf16.  Indices as in take().
void embed_rows(hipStream_t s, int dtype, const void* table, const int32_t* idx, float* out, void* out16, int64_t n_idx, int64_t vocab, int64_t n,
                float scale, int* err_flag);
void softmax_rows(hipStream_t s, int dtype, const void* x, void* y, int64_t rows, int64_t n);
void gelu(hipStream_t s, int dtype, const void* x, void* y, int64_t n, float half, float inv_div, float one);
void swiglu(hipStream_t s, int dtype, const void* gate, const void* up, void* y, int64_t n);  // up==nullptr: silu

// Linear layer y[M,N] = act(x[M,K] . W[K,N] + bias) (+ residual), W row-major [in,out]
// (nn/layers/linear.rs:50-71).  act: 0 none, 1 exact-erf gelu.  w2 != nullptr: SwiGLU pair,
// y = silu(x.W) * (x.W2).  Picks a bandwidth-bound GEMV kernel for small M and an MFMA tile
// kernel for large M.  `ws` is a scratch buffer of at least linear_workspace_bytes().
struct LinearArgs {
    int dtype;
    const void* x; const void* w; const void* w2; const void* bias; const void* residual;
    void* y;
    int64_t m, k, n;
    int act;
    void* ws; size_t ws_bytes;
    int* counters;  // >= kLinearCounters zero-initialised ints, left zero by every launch
};
constexpr int kLinearCounters = 4096;
size_t linear_workspace_bytes(int dtype, int64_t m, int64_t k, int64_t n, bool dual);
void linear(hipStream_t s, const LinearArgs& a);
// Decode GEMV (M <= 16) over a column-tiled copy of the weights, Wt[tile][k][v] with
// v = column % (16 bytes / element size): no split-K, one launch per linear layer.  gamma != nullptr
// fuses a preceding RMSNorm (x is then the un-normalised row; inv_n, eps as in rms_norm()).
struct TiledLinearArgs {
    int dtype;
    const void* x; const void* wt; const void* wt2; const void* gamma; const void* bias; const void* residual;
    void* y;
    int64_t m, k, n;
    int act;
    float inv_n, eps;
    const void* beta;   // with gamma: LayerNorm (normalization.rs:123-174) instead of RMSNorm
    // bf16 weights only.  out_f32: y and residual are f32 (the accumulator leaves unrounded).  x_f32 (with gamma, RMSNorm):
    // x and gamma are f32, the normalised row is rounded to bf16 once as it is staged.
    int out_f32 = 0, x_f32 = 0;   // (x_f32 with beta: the f32 LayerNorm, beta f32)
    EpiExtra extra;
};
size_t tiled_weight_bytes(int dtype, int64_t k, int64_t n);
void tile_weights(hipStream_t s, int dtype, const void* w, void* wt, int64_t k, int64_t n);
bool gemv_tiled_supported(int dtype, int64_t m, int64_t k, int64_t n);
void gemv_tiled(hipStream_t s, const TiledLinearArgs& a);

// Batched-decode linear layers (2 <= M <= 16, bf16 or f32) on the matrix cores over a 16-column tiled, k-grouped copy
// of the weights, Ws[tile][K/KPC][16][KPC] with KPC = 8 (bf16) or 4 (f32) k per 16 bytes (kernels_skinny.hip).  ws2 != nullptr: SwiGLU pair.  act: 0 none, 1 gelu.
struct SkinnyLinearArgs {
    int dtype;   // 0 f32, 2 bf16
    const void* x; const void* ws; const void* ws2; const void* bias; const void* residual;
    void* y;
    int64_t m, k, n;
    int act;
    // split-K over workgroups (layers with few tiles): part = skinny_workspace_bytes() of scratch, tickets =
    // kSkinnyTickets counters zeroed once (every launch leaves them zero); without them the layer runs unsplit
    void* part; size_t part_bytes; unsigned* tickets;
    // weight-only quantised: quant 1 = int8 (scale [N]), 2 = int4 groups of 128 (scale [K/128, N]); ws / ws2 are then
    // the code copies of skinny_pack_codes, scale / scale2 the scale tensors as the program holds them (bf16)
    int quant; const void* scale; const void* scale2;
    int out_f32 = 0;   // bf16 only: y and residual are f32
    EpiExtra extra;    // unquantised only
};
bool skinny_quant_supported(int dtype, int64_t m, int64_t k, int64_t n, int qf);
size_t skinny_codes_bytes(int64_t k, int64_t n, int qf);
void skinny_pack_codes(hipStream_t s, const void* codes, void* out, int64_t k, int64_t n, int qf);
constexpr size_t kSkinnyTickets = 1024;
int skinny_ksplit(int64_t k, int64_t n);
size_t skinny_workspace_bytes(int64_t k, int64_t n, bool dual);
bool skinny_gemm_supported(int dtype, int64_t m, int64_t k, int64_t n);
size_t skinny_weight_bytes(int dtype, int64_t k, int64_t n);
void skinny_pack_weights(hipStream_t s, int dtype, const void* w, void* out, int64_t k, int64_t n);
void skinny_gemm(hipStream_t s, const SkinnyLinearArgs& a);

// ---- weight-only quantisation (kernels_quant.hip) ------------------------------------------
// Build-defined extension (the reference has no quantisation scheme, docs/backend.md:620-632):
//   int8: symmetric, one scale per output column of W[K,N]: s_n = bf16(max_k |W[k,n]| / 127) (1 when 0),
//         q = clamp(rint(W / s_n), -127, 127)
//   int4: symmetric, groups of 128 along K per column: s[g,n] = bf16(max |w| / 7) (1 when 0), q in [-7,7],
//         two per byte along K: byte[k/2, n] = (q[k] & 0xF) | ((q[k+1] & 0xF) << 4)
// All arithmetic in f32 with IEEE division and round-half-even, so the results are bit-identical to
// the numpy closed form.  dtype tags: 0 f32, 2 bf16 (of w / scales / dequantised output).
void quant_w8_scales(hipStream_t s, int dtype, const void* w, void* scales, int64_t k, int64_t n);
void quant_w8(hipStream_t s, int dtype, const void* w, const void* scales, int8_t* q, int64_t k, int64_t n);
void quant_w4g128_scales(hipStream_t s, int dtype, const void* w, void* scales, int64_t k, int64_t n);
void quant_w4g128(hipStream_t s, int dtype, const void* w, const void* scales, uint8_t* packed, int64_t k, int64_t n);
// out[k,n] = dtype(f32(q) * f32(scale))
void dequant_w8(hipStream_t s, int dtype, const int8_t* q, const void* scales, void* out, int64_t k, int64_t n);
void dequant_w4g128(hipStream_t s, int dtype, const uint8_t* packed, const void* scales, void* out, int64_t k, int64_t n);

// Persistent decode chain (kernels_chain.hip): a run of consecutive M = 1 bf16 linear layers in
// ONE launch of one workgroup per CU, phases separated by a grid barrier, weights read from a
// 4-column / k-pair tiled copy, Wc[tile][k/2][4][2].  `flags` of a phase: RMSNorm prologue
// (gamma, inv_n, eps), SwiGLU pair (weights of gate and up interleaved column by column in one
// copy), bias, exact-erf GELU, residual.  x, residual and y may be produced by earlier phases of
// the same launch.
constexpr int kChainCounters = 16;        // striped arrival counters of the grid barrier
constexpr int kChainMaxPhases = 192;
constexpr int kChainMaxXsWords = 12288;   // staged activation words (48 KiB): K <= 24576 for bf16 weights
constexpr size_t kChainBarrierBytes = (kChainCounters * 64 + 64) * sizeof(unsigned);  // zero-initialised once
// kChainOutF32: y and the residual are f32.  kChainXF32 (with kChainNorm): x and gamma are f32, the normalised row is
// rounded to bf16 once as it is staged.
// kChainLayerNorm (with kChainNorm, f32 phases or kChainXF32): LayerNorm with gains `gamma` and offsets `beta` instead of RMSNorm.
enum : int { kChainNorm = 1, kChainDual = 2, kChainGelu = 4, kChainResidual = 8, kChainBias = 16, kChainOutF32 = 32, kChainXF32 = 64,
             kChainLayerNorm = 128, kChainAttnFinal = 256, kChainColScale = 512, kChainClampedGlu = 1024, kChainPostNorm = 2048, kChainSoftcap = 4096 };
// kChainPostNorm (bf16 weights, with kChainXF32): x is a sublayer's f32 output, the phase's input is r = post_res + post_mult *
// rms_norm(x) * post_gain, left in post_y as well when that is given; with kChainNorm the RMS norm of r (gains `gamma`).
// kChainSoftcap: y <- softcap * tanh(y / softcap), a layer without bias, residual and factors.
// weight format of a linear phase; kChainW32: f32 weights (16-byte word = 4 columns x 1 k) with f32 activations,
// bias, residual and output (the launch's attention phases then read f32 rows and caches as well)
enum : int { kChainW16 = 0, kChainW8 = 1, kChainW4 = 2, kChainW32 = 3 };
enum : int { kChainLinear = 0, kChainAttnPartial = 1, kChainAttnCombine = 2 };
// One phase of a chain.  Linear: y = act(norm?(x) . W + bias) (+ residual).  Decode attention
// (attention.rs:657-779, T = 1) takes two phases: "partial" appends this step's K/V row and leaves
// one online-softmax record (max, sum, weighted V) per query head and position chunk in `part`;
// "combine" merges the records of a head into the context row y.
struct ChainPhase {
    int kind, flags;
    const void* w; const void* x; const void* gamma; const void* bias; const void* residual;
    void* y;
    int K, N, Kw, ntiles, wpt, units, upb, lds_bytes;
    float inv_n, eps;
    // quantised weights: wfmt 1 = int8 (16-byte word = 4 columns x 4 k, biased by 128; `scale`/`scale2` = the
    // per-column scale tensors of W and of the SwiGLU partner, as wscale/wscale2), wfmt 2 = int4 groups of 128 (word = 4 columns x 8 k,
    // biased by 8; `wscale` = derived copy sc[tile][group][4] bf16, staged into LDS behind the activations)
    int wfmt, lds_total;   // lds_total: lds_bytes plus what the phase stages behind the activations
    const void* wscale; const void* wscale2;
    // attention: x = packed qkv row [(n_q + 2 n_kv) * head_dim], y = context row [n_q * head_dim]
    union { void* k_cache; void* post_y; };    // [n_kv, capacity, head_dim], updated in place
    void* v_cache;
    const int32_t* update_starts;              // si32[3]
    const int32_t* query_start;                // si32[1]
    union { const void* cos; const void* post_gain; };   // RoPE rows of this position, or null (qkv already rotated)
    union { const void* sin; const void* post_res; };    // (post_*: kChainPostNorm, linear phases)
    float* part;                               // [n_q][nch][head_dim + 2] f32
    int n_q, n_kv, head_dim;
    union { int capacity; float post_eps; };
    int rot_half, nch;
    union { float scale; float post_mult; };
    union { float glu_limit; float softcap; }; // kChainClampedGlu (with kChainDual): see glu_combine; kChainSoftcap
    const void* beta;                          // LayerNorm offsets (kChainLayerNorm)
    const void* colscale;                      // kChainColScale: f32 factor per output column, between bias and residual
    float glu_alpha, glu_shift;
};
int chain_grid();  // workgroups per launch (one per CU), 0 when no device is current
bool chain_supported(int dtype, int64_t m, int64_t k, int64_t n, bool dual, bool norm, int wfmt = kChainW16, bool x_f32 = false, bool plain = false);
size_t chain_weight_bytes(int64_t k, int64_t n, bool dual, int wfmt = kChainW16);
// w2 != nullptr: SwiGLU pair, columns of w (gate) and w2 (up) interleaved.  wfmt 0: w is bf16 [k,n];
// 1: si8 [k,n]; 2: packed int4, ui8 [k/2,n]; 3: f32 [k,n] (no pair)
void chain_pack_weights(hipStream_t s, const void* w, const void* w2, void* out, int64_t k, int64_t n, int wfmt = kChainW16);
// bf16 copies only: the row-major matrix (of a pair: whichever of w / w2 is non-null) back out of the packed copy, exactly
void chain_unpack_weights(hipStream_t s, const void* packed, void* w, void* w2, int64_t k, int64_t n, bool dual);
// int4 only: derived scale copy sc[tile][group][4] (bf16) from s [k/128, n] (and the partner's s2)
size_t chain_scale_bytes(int64_t k, int64_t n, bool dual);
void chain_pack_scales_w4(hipStream_t s, int dtype, const void* sc, const void* sc2, void* out, int64_t k, int64_t n);
// fills K, N, Kw, ntiles, wpt, units, upb, lds_bytes, wfmt (and the dual flag); false when one workgroup would
// own more bias/residual columns than the kernel stages
bool chain_fill_phase(ChainPhase& p, int64_t k, int64_t n, bool dual, int wfmt = kChainW16);
// Decode attention inside a chain: supported shapes, scratch for the per-chunk records, and the
// two phases (shape fields filled; the caller sets the pointers of both).
bool chain_attn_supported(int dtype, int64_t t, int64_t n_q, int64_t n_kv, int64_t head_dim, int64_t rot_half);
size_t chain_attn_part_bytes(int64_t n_q, int64_t n_kv, int64_t head_dim);
// phases a decode attention takes: 2, or 1 for a cache of at most 128 positions (one chunk per kv head; the "partial"
// phase then writes the context row itself, kChainAttnFinal, and `combine` is left untouched)
int chain_attn_phases(int64_t capacity);
void chain_fill_attn(ChainPhase& partial, ChainPhase& combine, int64_t n_q, int64_t n_kv, int64_t head_dim, int64_t capacity,
                     int64_t rot_half, float scale);
// bar: kChainBarrierBytes of device memory zeroed once; abort_flag: raised when a barrier wait
// gives up (every wave then leaves the kernel).  false: launch not possible (caller falls back).
// stall_phase >= 0 (tests of the give-up path): every workgroup expects one arrival too many at that phase's barrier.
bool chain_launch(hipStream_t s, const ChainPhase* dev_table, int nphases, int lds_bytes, unsigned* bar, int* abort_flag,
                  int wfmt = kChainW16, int stall_phase = -1);   // wfmt: the weight format of EVERY linear phase of the table

// Prefill GEMM (M > 16, bf16) on the matrix cores over a k-grouped copy of the weights,
// Wk8[K/8][Npad][8] (kernels_mfma.hip).  wk2 != nullptr: SwiGLU pair.
struct MfmaLinearArgs {
    int dtype;   // 0 f32, 2 bf16
    const void* x; const void* wk; const void* wk2; const void* bias; const void* residual;
    void* y;
    int64_t m, k, n;
    int act;
    // weight-only quantised (bf16 activations): quant 1 = int8 per column, 2 = int4 groups of 128; wk / wk2 are then
    // the k-grouped CODE copies (mfma_pack_codes) and scale / scale2 the matrices' scale tensors
    int quant;
    const void* scale; const void* scale2;
    // tail split: when the last round of 128 x 128 tiles would leave most CUs idle, those tiles are split over k between
    // 2 or 4 workgroups that meet through `part` (mfma_workspace_bytes() of scratch) and `tickets` (kSkinnyTickets
    // counters, zero before and after every launch); without them every tile runs whole
    void* part = nullptr; size_t part_bytes = 0; unsigned* tickets = nullptr;
    int out_f32 = 0;   // bf16 only: y and residual are f32
    EpiExtra extra;    // unquantised only
    int lds_direct = 1;   // unquantised bf16: the LDS-direct kernel where it applies (0: the register-staged one)
};
size_t mfma_workspace_bytes(int dtype, int64_t m, int64_t k, int64_t n, bool dual, int quant);
size_t mfma_weight_bytes(int dtype, int64_t k, int64_t n);
void mfma_pack_weights(hipStream_t s, int dtype, const void* w, void* out, int64_t k, int64_t n);
size_t mfma_codes_bytes(int64_t k, int64_t n, int quant);
void mfma_pack_codes(hipStream_t s, const void* q, void* out, int64_t k, int64_t n, int quant);
bool mfma_gemm_supported(int dtype, int64_t m, int64_t k, int64_t n, int quant = 0);
void mfma_gemm(hipStream_t s, const MfmaLinearArgs& a);

// Rotate-half RoPE on packed [T, Q|K|V] rows (ops/functional/rotary.rs:430-536).
void rope_packed(hipStream_t s, int dtype, const void* qkv, const void* cos, const void* sin, void* out,
                 int64_t t, int64_t n_q, int64_t n_kv, int64_t head_dim, int64_t half);

// Decode attention over a fixed-capacity cache (ops/functional/attention.rs:657-779), T = 1.
// Appends this step's K/V rows at clamp(update_starts[1]) into k_out/v_out (which already hold
// the previous cache contents: either the donated buffers or a copy) and attends over positions
// 0..=query_start[0].
struct AttnDecodeArgs {
    int dtype;
    const void* qkv;            // [1, (n_q + 2 n_kv) * head_dim]
    void* k_cache; void* v_cache;  // [n_kv, capacity, head_dim], updated in place
    const int32_t* update_starts;  // si32[3]
    const int32_t* query_start;    // si32[1]
    void* ctx;                  // [1, n_q * head_dim]
    int64_t n_q, n_kv, head_dim, capacity;
    float scale;
    void* ws; size_t ws_bytes;
    // optional fused RoPE of Q and of the appended K row (qkv is then the pre-RoPE projection):
    // cos/sin rows [rot_half] of this position; requires rot_half % (16 / element size) == 0
    const void* cos; const void* sin; int64_t rot_half;
    // batch > 1: `batch` independent sequences in one launch: qkv is [batch, P], ctx [batch, n_q * head_dim], the caches
    // of sequence b are k_caches[b] / v_caches[b] (k_cache / v_cache are ignored), ws holds batch x the single size
    int batch;
    void* k_caches[16]; void* v_caches[16];
};
size_t attn_decode_workspace_bytes(int64_t n_q, int64_t head_dim, int64_t capacity);
int attn_decode(hipStream_t s, const AttnDecodeArgs& a);   // returns the number of launches it made

// Prefill causal attention (ops/functional/attention.rs:443-522): packed qkv [T, P] ->
// ctx [T, n_q*head_dim], and K/V in cache layout [n_kv, T, head_dim].
struct AttnPrefillArgs {
    int dtype;
    const void* qkv;
    void* ctx; void* k_out; void* v_out;
    int64_t t, n_q, n_kv, head_dim;
    float scale;
};
void attn_prefill(hipStream_t s, const AttnPrefillArgs& a);

// Causal attention over a growing cache (ops/functional/attention.rs:359-437, the `cache = Some` branch): T new rows of
// packed qkv [T, P] behind caches [n_kv, C, head_dim]: k_all / v_all [n_kv, C + T, head_dim] = the caches with the new
// rows appended, ctx [T, n_q*head_dim] = row i attends keys 0 .. C + i.  Two launches.
struct AttnConcatArgs {
    int dtype;
    const void* qkv; const void* k_cache; const void* v_cache;
    void* ctx; void* k_all; void* v_all;
    int64_t t, cache_len, n_q, n_kv, head_dim;
    float scale;
};
void attn_concat(hipStream_t s, const AttnConcatArgs& a);

// ---- sequence mixers (kernels_ssm.hip, kernels_latent.hip) ------------------------------------------------------------
// dtype: 0 f32, 2 bf16, of the tensors called "T" below; everything else is f32.

// cos | sin of positions[r] * freqs[i], times `magnitude`: out f32 [rows, 2 * half]
void rope_table(hipStream_t s, const int32_t* positions, const float* freqs, float magnitude, float* out, int64_t rows, int64_t half);
// rotates the pairs (offset + 2i, offset + 2i + 1), i < half, of every head of x T [rows, heads * head_dim]; the rest is copied
void rope_pairs(hipStream_t s, int dtype, const void* x, const float* table, void* y, int64_t rows, int64_t heads, int64_t head_dim,
                int64_t offset, int64_t half);
// raw f32 [rows, rank + 2 * half] -> T: RMS norm with gains over the first `rank` values, pair rotation of the rest
void latent_rows(hipStream_t s, int dtype, const float* raw, const float* gain, const float* table, void* y, int64_t rows, int64_t rank,
                 int64_t half, float eps);

// Latent attention over cached rows [latent: rank | rotated key part: rot] (one row per position, shared by all heads).
// Query t (position start + t) sees rows 0 .. start + t.  Scores q_n . (W_uk c) + q_r . k_r are taken as
// (W_uk^T q_n) . c + q_r . k_r and the values as W_uv (sum_j p_j c_j): the cache is read as it is.
struct LatentAttnArgs {
    int dtype;
    const void* q;                 // T [t, heads * (dim + rot)], rotated
    const void* rows;              // T [capacity, rank + rot]
    const void* w_uk; const void* w_uv;   // T [rank, heads * dim], T [rank, heads * vdim]
    const int32_t* start;          // si32[1]
    void* ctx;                     // T [t, heads * vdim]
    int64_t t, capacity, heads, dim, rot, rank, vdim;
    float scale;
};
void latent_attn(hipStream_t s, const LatentAttnArgs& a);
// The same with keys and values spelled out per head, k T [l, heads * dim], v T [l, heads * vdim] and the shared part read
// from rows T [l, ld_rows] at column rank; query t sees keys 0 .. l - t_rows + t.
struct LatentAttnXArgs {
    int dtype;
    const void* q; const void* k; const void* v; const void* rows;
    void* ctx;
    int64_t t, l, heads, dim, rot, rank, vdim;
    float scale;
};
void latent_attn_expanded(hipStream_t s, const LatentAttnXArgs& a);

// Depthwise causal convolution with bias and silu over `ch` columns of p f32 [rows, ld] from column `col`; taps f32
// [taps, ch] (last row meets the current token), state f32 [taps - 1, ch]: the inputs before the first row.  y T [rows, ch].
struct ConvArgs {
    int dtype;
    const float* p; const float* taps; const float* bias; const float* state;
    void* y;
    int64_t rows, ld, col, ch, ntaps;
};
void conv_silu(hipStream_t s, const ConvArgs& a);
// the last taps - 1 inputs after `rows` more rows; state_out may be state
void conv_state(hipStream_t s, const float* p, const float* state, float* state_out, int64_t rows, int64_t ld, int64_t col, int64_t ch, int64_t ntaps);

// Mamba-2 recurrence, head h of group h / (heads / groups): dt = softplus(p[t, dt_col + h] + dt_bias[h]),
// S <- exp(-exp(A_log[h]) dt) S + dt B x^T, y = S^T C + D[h] x.  xbc T [rows, heads * vdim + 2 groups * n] = x | B | C.
// y null: only the state; state_out null: only the rows.  state_out may be state.
struct SsmArgs {
    int dtype;
    const void* xbc; const float* p; const float* dt_bias; const float* a_log; const float* d;
    const float* state; float* state_out; void* y;
    int64_t rows, ld, dt_col, heads, groups, n, vdim;
};
void ssm_scan(hipStream_t s, const SsmArgs& a);
// y T [rows, n] = rms-normed in `groups` equal parts of (y * silu(p[:, col ..])), times gain[n]
void gated_rms_norm(hipStream_t s, int dtype, const void* y, const float* p, const float* gain, void* out, int64_t rows, int64_t n, int64_t ld,
                    int64_t col, int64_t groups, float eps);
// The whole mixer for up to kMixerBatch sequences of one launch series (Mix::SsmSeq): sequence b owns the rows [row0[b],
// row0[b] + len[b]) of p and y.  out T [rows, inner].  scratch: ssm_seq_scratch_bytes().  Returns the number of launches.
constexpr int kMixerBatch = 16;
struct SsmSeqArgs {
    int dtype;
    const float* p; const float* taps; const float* bias; const float* dt_bias; const float* a_log; const float* d; const float* gain;
    void* out;
    int64_t rows, ld, col, ch, ntaps, dt_col, z_col, heads, groups, n, vdim, norm_groups;
    float eps;
    int nseq;
    int row0[kMixerBatch], len[kMixerBatch];
    const float* conv_in[kMixerBatch]; float* conv_out[kMixerBatch];
    const float* state_in[kMixerBatch]; float* state_out[kMixerBatch];
    void* scratch;
};
size_t ssm_seq_scratch_bytes(int dtype, int64_t rows, int64_t heads, int64_t groups, int64_t n, int64_t vdim);
int ssm_seq(hipStream_t s, const SsmSeqArgs& a);

// One decode step of latent attention for up to kMixerBatch sequences (Mix::LatentDecode): x T [nseq, heads * (dim + rot)]
// unrotated queries, table f32 [nseq, rot]; with raw the step's row is formed (latent_rows) and written at row
// starts[3 b + 1] of cache b first.  Sequence b attends rows 0 .. pos[b].
struct LatentDecodeArgs {
    int dtype;
    const void* x; const float* table; const void* w_uk; const void* w_uv; const int32_t* pos;
    const float* raw; const float* gain; const int32_t* starts;
    void* cache[kMixerBatch];
    void* ctx;
    int64_t nseq, capacity, heads, dim, rot, rank, vdim;
    float scale, eps;
    void* scratch;
};
size_t latent_decode_scratch_bytes(int dtype, int64_t nseq, int64_t capacity, int64_t heads, int64_t dim, int64_t rot, int64_t rank, int64_t vdim);
int latent_decode(hipStream_t s, const LatentDecodeArgs& a);

// Causal latent attention of whole prompts (Mix::LatentPrefill), nseq sequences stacked: x T [rows, heads * (dim + rot)]
// unrotated queries, k / v / rows as in LatentAttnXArgs.
struct LatentPrefillArgs {
    int dtype;
    const void* x; const float* table; const void* k; const void* v; const void* rows;
    void* ctx;
    int64_t total, heads, dim, rot, rank, vdim;
    float scale;
    int nseq;
    int row0[kMixerBatch], len[kMixerBatch];
    void* scratch;
};
size_t latent_prefill_scratch_bytes(int dtype, int64_t total, int64_t heads, int64_t dim, int64_t rot, int64_t vdim);
int latent_prefill(hipStream_t s, const LatentPrefillArgs& a);

// ---- chunked attention (kernels_chunked.hip) --------------------------------------------------------------------------
// n heads of head_dim values, each divided by its root mean square
void head_rms_norm(hipStream_t s, int in_dtype, int out_dtype, const void* x, void* y, int64_t n, int64_t head_dim, float eps);
// y = x * sigmoid(gate): x T [rows, heads * vdim], gate f32 with one value per head, rows `ld` apart
void head_gate(hipStream_t s, int dtype, const void* x, const float* gate, void* y, int64_t rows, int64_t heads, int64_t vdim, int64_t ld);
// Grouped-query attention inside chunks with a sink per head: q T [t, heads * dim], keys and values of kv head g in row j at
// k + g * k_head + j * k_row and v + g * v_head + j * v_row.  Without `position` query i (position i) sees the rows from its
// chunk's first up to i; with it (t = 1) the rows 0 .. position % chunk of `rows` cached ones.  chunk 0: one chunk.
struct ChunkAttnArgs {
    int dtype;
    const void* q; const void* k; const void* v; const float* sink; const int32_t* position;
    void* ctx;                     // T [t, heads * vdim]
    int64_t t, heads, kv_heads, dim, vdim, chunk, rows, k_row, k_head, v_row, v_head;
    float scale;
};
void chunk_attn(hipStream_t s, const ChunkAttnArgs& a);
// The whole mixer between its projections for up to kMixerBatch sequences (Mix::ChunkDecode, Mix::ChunkPrefill): proj f32
// [total, ld] = q | k | v | gate per row, table f32 [total, rot] or null, ctx T [total, heads * vdim] gated.  Sequence b owns the
// rows [row0[b], row0[b] + len[b]); its last keep[b] keys and values go to rows starts[3 b + 1] .. of its caches T [kv_heads,
// rows, dim] and [kv_heads, rows, vdim].  Decode: one row each at position pos[b].  tickets: kSkinnyTickets zeroed counters.
struct ChunkSeqArgs {
    int dtype;
    const float* proj; const float* table; const float* sink; const int32_t* pos; const int32_t* starts;
    void* ctx;
    int64_t total, ld, heads, kv_heads, dim, vdim, rot, rows, chunk;
    float scale, eps;
    int nseq;
    int row0[kMixerBatch], len[kMixerBatch], keep[kMixerBatch];
    void* kcache[kMixerBatch]; void* vcache[kMixerBatch];
    void* scratch; unsigned* tickets;
};
size_t chunk_decode_scratch_bytes(int dtype, int64_t nseq, int64_t rows, int64_t heads, int64_t kv_heads, int64_t dim, int64_t vdim);
int chunk_decode(hipStream_t s, const ChunkSeqArgs& a);
size_t chunk_prefill_scratch_bytes(int dtype, int64_t total, int64_t heads, int64_t kv_heads, int64_t dim, int64_t vdim);
int chunk_prefill(hipStream_t s, const ChunkSeqArgs& a);
void clamped_glu(hipStream_t s, int dtype, const void* gate, const void* up, void* y, int64_t n, const GluParams& p);

}  // namespace k
}  // namespace gptrs
