// Sequence-mixer CustomCall targets of this backend (build-defined; the reference has no counterpart): validation, launch
// descriptors and launches.  Operands per target (T: f32 or bf16, the model's dtype; everything else f32 unless said):
//
//   rope_table(positions si32[R], freqs[half]) {magnitude}                              -> [R, 2 half]   cos | sin
//   rope_pairs(x T[R, heads * hd], table[R, 2 half]) {heads, offset}                    -> T, x's shape
//   latent_rows(raw[R, rank + 2 half], gain[rank], table) {eps}                         -> T[R, rank + 2 half]
//   latent_attention(q T[R, heads * (dim + rot)], cache T[1, C, rank + rot], w_uk T[rank, heads * dim],
//                    w_uv T[rank, heads * vdim], start si32[1]) {heads, rot, scale}      -> T[R, heads * vdim]
//   latent_attention_expanded(q T[R, ..], k T[L, heads * dim], v T[L, heads * vdim], rows T[L, rank + rot])
//                    {heads, rot, scale}                                                -> T[R, heads * vdim]
//   causal_conv_silu(p[R, W], taps[K, ch], bias[ch], state[K - 1, ch]) {col}            -> T[R, ch]
//   causal_conv_state(p, state) {col}                                                   -> state's shape
//   ssm_scan(xbc T[R, ch], p, dt_bias[H], a_log[H], d[H], state[H, N, V]) {groups, dt_col} -> T[R, H * V]
//   ssm_state(xbc, p, dt_bias, a_log, state) {groups, dt_col}                           -> state's shape
//   gated_rms_norm(y T[R, n], p[R, W], gain[n]) {groups, col, eps}                      -> T[R, n]
//   clamped_glu(gate T, up T) {limit, alpha, shift}                                     -> T, gate's shape
//   head_rms_norm(x T[R, heads * hd]) {heads, eps}                                      -> T' [R, heads * hd]
//   head_gate(x T[R, heads * vd], gate[R, heads]) {heads}                               -> T, x's shape
//   chunk_attention(q T[R, heads * D], k T[R, G * D], v T[R, G * V], sink[heads])
//                    {heads, kv_heads = G, chunk, scale}                                -> T[R, heads * V]
//   chunk_attention_cache(q T[1, heads * D], keys T[G, C, D], values T[G, C, V], sink[heads], position si32[1])
//                    {heads, chunk, scale}                                              -> T[1, heads * V]
//
// latent_attention: query i stands at position start + i.  latent_attention_expanded: the queries are the last R of the L
// positions.  p is the f32 result of an input projection whose columns hold several inputs of the mixer.
#include <algorithm>
#include <cmath>
#include <cstring>

#include "runtime.hpp"

namespace gptrs {

namespace {
const Json* attr(const Instr& in, const char* name) {
    auto it = in.attrs.find(name);
    return it == in.attrs.end() ? nullptr : it->second.find("value");
}
int64_t attr_int(const Instr& in, const char* name) {
    const Json* v = attr(in, name);
    try {
        if (v) return v->as_int();
    } catch (const JsonError&) {
    }
    fail_spec(in.target + ": attribute `" + name + "` (I64) is missing");
}
float attr_float(const Instr& in, const char* name) {
    const Json* v = attr(in, name);
    try {
        if (v) {
            const double d = v->as_double();
            if (std::isfinite(d)) return (float)d;
        }
    } catch (const JsonError&) {
    }
    fail_spec(in.target + ": attribute `" + name + "` (F64) is missing or not finite");
}
}  // namespace

void lower_mixer_calls(Function& fn) {
    bool any = false;
    for (const Instr& in : fn.body) any = any || (in.op == OpKind::CustomCall && mixer_call_target(in.target) != Mix::None);
    if (!any) return;
    std::vector<const Spec*> spec(fn.max_value_id + 1, nullptr);
    for (size_t i = 0; i < fn.param_ids.size(); ++i) spec[fn.param_ids[i]] = &fn.param_specs[i];
    for (const Instr& in : fn.body)
        for (size_t o = 0; o < in.out_ids.size(); ++o) spec[in.out_ids[o]] = &in.out_specs[o];

    for (Instr& in : fn.body) {
        if (in.op != OpKind::CustomCall) continue;
        const Mix mix = mixer_call_target(in.target);
        if (mix == Mix::None) continue;
        auto need = [&](bool ok, const char* what) { if (!ok) fail_spec(in.target + ": " + what); };
        static const std::map<Mix, size_t> kArity = {{Mix::RopeTable, 2}, {Mix::RopePairs, 2}, {Mix::LatentRows, 3}, {Mix::LatentAttn, 5},
                                                     {Mix::LatentAttnX, 4}, {Mix::ConvSilu, 4}, {Mix::ConvState, 2}, {Mix::SsmScan, 6},
                                                     {Mix::SsmState, 5}, {Mix::GatedNorm, 3}, {Mix::Glu, 2}, {Mix::HeadNorm, 1},
                                                     {Mix::HeadGate, 2}, {Mix::ChunkAttn, 4}, {Mix::ChunkAttnCache, 5}};
        need(in.operands.size() == kArity.at(mix), "wrong number of operands");
        std::vector<const Spec*> s;
        for (const Operand& o : in.operands) {
            need(o.value >= 0 && o.value <= fn.max_value_id && spec[o.value], "operands must be values");
            s.push_back(spec[o.value]);
        }
        const Spec& out = in.out_specs[0];
        auto is = [](const Spec& x, DType d, std::vector<int64_t> dims) { return x.dtype == d && x.dims == dims; };
        auto f32 = [&](const Spec& x, std::vector<int64_t> dims) { return is(x, DType::F32, std::move(dims)); };
        auto rows2 = [&](const Spec& x) { return x.rank() == 2 && x.dims[0] >= 1 && x.dims[1] >= 1; };
        Instr::MixAttrs& m = in.mx;
        switch (mix) {
            case Mix::RopeTable:
                need(s[0]->dtype == DType::SI32 && s[0]->rank() == 1, "positions must be si32[R]");
                need(s[1]->rank() == 1 && f32(*s[1], s[1]->dims), "freqs must be f32[half]");
                need(f32(out, {s[0]->dims[0], 2 * s[1]->dims[0]}), "output must be f32[R, 2 half]");
                in.scale = attr_float(in, "magnitude");
                break;
            case Mix::RopePairs: {
                m.heads = attr_int(in, "heads");
                m.col = attr_int(in, "offset");
                need(rows2(*s[0]) && dtype_is_float(s[0]->dtype) && out == *s[0], "x must be a float matrix, the output has its type");
                need(m.heads > 0 && s[0]->dims[1] % m.heads == 0, "row length must be heads * head_dim");
                m.dim = s[0]->dims[1] / m.heads;
                need(s[1]->rank() == 2 && f32(*s[1], {s[0]->dims[0], s[1]->dims[1]}) && s[1]->dims[1] % 2 == 0, "table must be f32[R, 2 half]");
                m.rot = s[1]->dims[1];
                need(m.col >= 0 && m.col + m.rot <= m.dim, "the rotated part must lie in the head");
                break;
            }
            case Mix::LatentRows:
                need(rows2(*s[0]) && f32(*s[0], s[0]->dims), "raw must be an f32 matrix");
                need(s[1]->rank() == 1 && s[1]->dims[0] >= 1 && f32(*s[1], s[1]->dims), "gain must be f32[rank]");
                m.rank = s[1]->dims[0];
                m.rot = s[0]->dims[1] - m.rank;
                need(m.rot >= 0 && m.rot % 2 == 0 && f32(*s[2], {s[0]->dims[0], m.rot}), "table must be f32[R, width - rank]");
                need(dtype_is_float(out.dtype) && out.dims == s[0]->dims, "output must have raw's shape");
                in.eps = attr_float(in, "eps");
                break;
            case Mix::LatentAttn:
            case Mix::LatentAttnX: {
                const bool x = mix == Mix::LatentAttnX;
                m.heads = attr_int(in, "heads");
                m.rot = attr_int(in, "rot");
                in.scale = attr_float(in, "scale");
                need(m.heads > 0 && m.rot >= 0 && m.rot % 2 == 0, "heads must be positive, rot even");
                const DType dt = s[0]->dtype;
                need(dtype_is_float(dt) && rows2(*s[0]), "q must be a float matrix");
                const Spec& kk = *s[x ? 1 : 2];
                const Spec& vv = *s[x ? 2 : 3];
                need(rows2(kk) && rows2(vv) && kk.dtype == dt && vv.dtype == dt && kk.dims[0] == vv.dims[0], "key / value operands must be matrices of q's dtype");
                need(kk.dims[1] % m.heads == 0 && vv.dims[1] % m.heads == 0, "key / value widths must be multiples of heads");
                m.dim = kk.dims[1] / m.heads;
                m.vdim = vv.dims[1] / m.heads;
                need(s[0]->dims[1] == m.heads * (m.dim + m.rot), "q must be [R, heads * (dim + rot)]");
                const Spec& rr = *s[x ? 3 : 1];
                if (x) {
                    need(rr.dtype == dt && rr.rank() == 2 && rr.dims[0] == kk.dims[0] && rr.dims[1] > m.rot, "rows must be T[L, rank + rot]");
                    need(kk.dims[0] >= s[0]->dims[0], "at least as many keys as queries");
                    m.rank = rr.dims[1] - m.rot;
                } else {
                    m.rank = kk.dims[0];
                    need(rr.dtype == dt && rr.rank() == 3 && rr.dims[0] == 1 && rr.dims[1] >= 1 && rr.dims[2] == m.rank + m.rot, "cache must be T[1, C, rank + rot]");
                    need(is(*s[4], DType::SI32, {1}), "start must be si32[1]");
                }
                need(is(out, dt, {s[0]->dims[0], m.heads * m.vdim}), "output must be T[R, heads * vdim]");
                break;
            }
            case Mix::ConvSilu:
                m.col = attr_int(in, "col");
                need(rows2(*s[0]) && f32(*s[0], s[0]->dims), "p must be an f32 matrix");
                need(s[1]->rank() == 2 && s[1]->dims[0] >= 1 && f32(*s[1], s[1]->dims), "taps must be f32[K, ch]");
                m.taps = s[1]->dims[0];
                m.dim = s[1]->dims[1];
                need(f32(*s[2], {m.dim}) && f32(*s[3], {m.taps - 1, m.dim}), "bias must be f32[ch], state f32[K - 1, ch]");
                need(m.col >= 0 && m.col + m.dim <= s[0]->dims[1], "channels must lie in p's columns");
                need(dtype_is_float(out.dtype) && out.dims == std::vector<int64_t>{s[0]->dims[0], m.dim}, "output must be T[R, ch]");
                break;
            case Mix::ConvState:
                m.col = attr_int(in, "col");
                need(rows2(*s[0]) && f32(*s[0], s[0]->dims) && s[1]->rank() == 2 && f32(*s[1], s[1]->dims), "p and state must be f32 matrices");
                m.taps = s[1]->dims[0] + 1;
                m.dim = s[1]->dims[1];
                need(m.col >= 0 && m.col + m.dim <= s[0]->dims[1] && out == *s[1], "channels must lie in p's columns, the output has state's type");
                break;
            case Mix::SsmScan:
            case Mix::SsmState: {
                const bool scan = mix == Mix::SsmScan;
                const Spec& st = *s[scan ? 5 : 4];
                m.groups = attr_int(in, "groups");
                m.dt_col = attr_int(in, "dt_col");
                need(st.rank() == 3 && f32(st, st.dims), "state must be f32[H, N, V]");
                m.heads = st.dims[0]; m.state = st.dims[1]; m.vdim = st.dims[2];
                need(m.heads >= 1 && m.state >= 1 && m.vdim >= 1 && m.state <= 1024, "state sizes out of range");
                need(m.groups >= 1 && m.heads % m.groups == 0, "heads must be a multiple of groups");
                need(dtype_is_float(s[0]->dtype) && s[0]->rank() == 2 && s[0]->dims[0] >= 1 && s[0]->dims[1] == m.heads * m.vdim + 2 * m.groups * m.state,
                     "xbc must be T[R, H * V + 2 groups * N]");
                need(rows2(*s[1]) && f32(*s[1], {s[0]->dims[0], s[1]->dims[1]}) && m.dt_col >= 0 && m.dt_col + m.heads <= s[1]->dims[1], "step sizes must lie in p's columns");
                for (size_t i = 2; i < (scan ? 5u : 4u); ++i) need(f32(*s[i], {m.heads}), "per-head vectors must be f32[H]");
                if (scan) need(is(out, s[0]->dtype, {s[0]->dims[0], m.heads * m.vdim}), "output must be T[R, H * V]");
                else need(out == st, "the output has state's type");
                break;
            }
            case Mix::GatedNorm:
                m.groups = attr_int(in, "groups");
                m.col = attr_int(in, "col");
                in.eps = attr_float(in, "eps");
                need(rows2(*s[0]) && dtype_is_float(s[0]->dtype) && out == *s[0], "y must be a float matrix, the output has its type");
                m.dim = s[0]->dims[1];
                need(m.groups >= 1 && m.dim % m.groups == 0, "row length must be a multiple of groups");
                need(s[1]->rank() == 2 && f32(*s[1], {s[0]->dims[0], s[1]->dims[1]}) && m.col >= 0 && m.col + m.dim <= s[1]->dims[1], "the gate must lie in p's columns");
                need(f32(*s[2], {m.dim}), "gain must be f32[n]");
                break;
            case Mix::Glu:
                need(*s[0] == *s[1] && *s[0] == out && dtype_is_float(out.dtype), "gate, up and output must be of one float type");
                in.fparam[0] = attr_float(in, "limit");
                in.fparam[1] = attr_float(in, "alpha");
                in.fparam[2] = attr_float(in, "shift");
                break;
            case Mix::HeadNorm:
                m.heads = attr_int(in, "heads");
                in.eps = attr_float(in, "eps");
                need(rows2(*s[0]) && dtype_is_float(s[0]->dtype) && dtype_is_float(out.dtype) && out.dims == s[0]->dims, "x must be a float matrix, the output has its shape");
                need(m.heads > 0 && s[0]->dims[1] % m.heads == 0, "row length must be heads * head_dim");
                m.dim = s[0]->dims[1] / m.heads;
                break;
            case Mix::HeadGate:
                m.heads = attr_int(in, "heads");
                need(rows2(*s[0]) && dtype_is_float(s[0]->dtype) && out == *s[0], "x must be a float matrix, the output has its type");
                need(m.heads > 0 && s[0]->dims[1] % m.heads == 0, "row length must be heads * vdim");
                m.vdim = s[0]->dims[1] / m.heads;
                need(f32(*s[1], {s[0]->dims[0], m.heads}), "gate must be f32[R, heads]");
                break;
            case Mix::ChunkAttn:
            case Mix::ChunkAttnCache: {
                const bool cached = mix == Mix::ChunkAttnCache;
                m.heads = attr_int(in, "heads");
                m.chunk = attr_int(in, "chunk");
                in.scale = attr_float(in, "scale");
                need(m.heads > 0 && m.chunk >= 0, "heads must be positive, chunk not negative");
                const DType dt = s[0]->dtype;
                need(dtype_is_float(dt) && rows2(*s[0]) && s[0]->dims[1] % m.heads == 0, "q must be a float matrix [R, heads * D]");
                m.dim = s[0]->dims[1] / m.heads;
                if (cached) {
                    need(s[1]->rank() == 3 && s[2]->rank() == 3 && s[1]->dims[0] >= 1 && s[1]->dims[1] >= 1 && s[2]->dims[2] >= 1, "caches must be of rank 3");
                    m.groups = s[1]->dims[0];
                    m.vdim = s[2]->dims[2];
                    need(is(*s[1], dt, {m.groups, s[1]->dims[1], m.dim}) && is(*s[2], dt, {m.groups, s[1]->dims[1], m.vdim}), "caches must be T[G, C, D] and T[G, C, V]");
                    need(s[0]->dims[0] == 1 && is(*s[4], DType::SI32, {1}), "one query at position si32[1]");
                } else {
                    m.groups = attr_int(in, "kv_heads");
                    need(m.groups > 0 && rows2(*s[1]) && rows2(*s[2]) && s[2]->dims[1] % m.groups == 0, "keys and values must be matrices of kv_heads parts");
                    m.vdim = s[2]->dims[1] / m.groups;
                    need(is(*s[1], dt, {s[0]->dims[0], m.groups * m.dim}) && is(*s[2], dt, {s[0]->dims[0], m.groups * m.vdim}), "k must be T[R, G * D], v T[R, G * V]");
                }
                need(m.heads % m.groups == 0, "heads must be a multiple of the key / value heads");
                need(f32(*s[3], {m.heads}), "sink must be f32[heads]");
                need(is(out, dt, {s[0]->dims[0], m.heads * m.vdim}), "output must be T[R, heads * V]");
                break;
            }
            default:
                fail_spec(in.target + ": not a call target");
        }
        in.op = OpKind::FMixer;
        in.mix = mix;
        in.op_name = "mixer." + in.target.substr(strlen("gpt_rs.hip."));
    }
}

// operands of Mix::ChunkDecode / ChunkPrefill: proj, sink, pos, starts, [table,] keys_0, values_0, keys_1, ..
static size_t chunk_cache_operand(const Instr& in, int64_t b) { return (size_t)(4 + (in.mx.rot > 0 ? 1 : 0) + 2 * b); }

size_t mixer_scratch_bytes(const Instr& in, const std::vector<const Spec*>& operands) {
    const Instr::MixAttrs& m = in.mx;
    const int dt = (int)in.out_specs[0].dtype;
    const int64_t rows = in.out_specs[0].rank() == 2 ? in.out_specs[0].dims[0] : 0;
    if (in.mix == Mix::SsmSeq) return k::ssm_seq_scratch_bytes(dt, rows, m.heads, m.groups, m.state, m.vdim);
    if (in.mix == Mix::LatentDecode)
        return k::latent_decode_scratch_bytes(dt, std::min<int64_t>(rows, k::kMixerBatch), operands[in.append ? 8 : 5]->dims[1], m.heads, m.dim, m.rot, m.rank, m.vdim);
    if (in.mix == Mix::LatentPrefill) return k::latent_prefill_scratch_bytes(dt, rows, m.heads, m.dim, m.rot, m.vdim);
    if (in.mix == Mix::ChunkDecode)
        return k::chunk_decode_scratch_bytes(dt, std::min<int64_t>(rows, k::kMixerBatch), operands[chunk_cache_operand(in, 0)]->dims[1], m.heads, m.groups, m.dim, m.vdim);
    if (in.mix == Mix::ChunkPrefill) return k::chunk_prefill_scratch_bytes(dt, rows, m.heads, m.groups, m.dim, m.vdim);
    return 0;
}

std::vector<std::pair<int, int>> mixer_inplace_pairs(const Instr& in) {
    std::vector<std::pair<int, int>> out;
    if (in.mix == Mix::SsmSeq)
        for (int b = 0; b < (int)in.lens.size(); ++b) { out.push_back({7 + 2 * b, 1 + 2 * b}); out.push_back({8 + 2 * b, 2 + 2 * b}); }
    if (in.mix == Mix::LatentDecode && in.append)
        for (int b = 0; b < (int)in.lens.size(); ++b) out.push_back({8 + b, 1 + b});
    if (in.mix == Mix::ChunkDecode || in.mix == Mix::ChunkPrefill)
        for (int i = 0; i < 2 * (int)in.lens.size(); ++i) out.push_back({(int)chunk_cache_operand(in, 0) + i, 1 + i});
    return out;
}

void run_mixer(const Plan& plan, const Step& st, ExecCtx& cx) {
    const Instr& in = st.in;
    const Instr::MixAttrs& m = in.mx;
    const Spec& out = in.out_specs[0];
    hipStream_t s = cx.stream;
    auto ptr = [&](size_t i) -> const void* { return cx.ptr[st.src[i]]; };
    auto f = [&](size_t i) { return (const float*)ptr(i); };
    auto spec = [&](size_t i) -> const Spec& { return plan.values[st.src[i]].spec; };
    void* dst = cx.ptr[st.dst[0]];
    const int dt = (int)out.dtype;
    switch (in.mix) {
        case Mix::RopeTable:
            k::rope_table(s, (const int32_t*)ptr(0), f(1), in.scale, (float*)dst, out.dims[0], out.dims[1] / 2);
            ++cx.launches;
            break;
        case Mix::RopePairs:
            k::rope_pairs(s, dt, ptr(0), f(1), dst, out.dims[0], m.heads, m.dim, m.col, m.rot / 2);
            ++cx.launches;
            break;
        case Mix::LatentRows:
            k::latent_rows(s, dt, f(0), f(1), f(2), dst, out.dims[0], m.rank, m.rot / 2, in.eps);
            ++cx.launches;
            break;
        case Mix::LatentAttn: {
            k::LatentAttnArgs a{};
            a.dtype = dt;
            a.q = ptr(0); a.rows = ptr(1); a.w_uk = ptr(2); a.w_uv = ptr(3); a.start = (const int32_t*)ptr(4); a.ctx = dst;
            a.t = out.dims[0]; a.capacity = spec(1).dims[1];
            a.heads = m.heads; a.dim = m.dim; a.rot = m.rot; a.rank = m.rank; a.vdim = m.vdim; a.scale = in.scale;
            k::latent_attn(s, a);
            ++cx.launches;
            break;
        }
        case Mix::LatentAttnX: {
            k::LatentAttnXArgs a{};
            a.dtype = dt;
            a.q = ptr(0); a.k = ptr(1); a.v = ptr(2); a.rows = ptr(3); a.ctx = dst;
            a.t = out.dims[0]; a.l = spec(1).dims[0];
            a.heads = m.heads; a.dim = m.dim; a.rot = m.rot; a.rank = m.rank; a.vdim = m.vdim; a.scale = in.scale;
            k::latent_attn_expanded(s, a);
            ++cx.launches;
            break;
        }
        case Mix::ConvSilu: {
            k::ConvArgs a{};
            a.dtype = dt;
            a.p = f(0); a.taps = f(1); a.bias = f(2); a.state = f(3); a.y = dst;
            a.rows = out.dims[0]; a.ld = spec(0).dims[1]; a.col = m.col; a.ch = m.dim; a.ntaps = m.taps;
            k::conv_silu(s, a);
            ++cx.launches;
            break;
        }
        case Mix::ConvState:
            k::conv_state(s, f(0), f(1), (float*)dst, spec(0).dims[0], spec(0).dims[1], m.col, m.dim, m.taps);
            ++cx.launches;
            break;
        case Mix::SsmScan:
        case Mix::SsmState: {
            const bool scan = in.mix == Mix::SsmScan;
            k::SsmArgs a{};
            a.dtype = (int)spec(0).dtype;
            a.xbc = ptr(0); a.p = f(1); a.dt_bias = f(2); a.a_log = f(3);
            if (scan) { a.d = f(4); a.state = f(5); a.y = dst; }
            else { a.state = f(4); a.state_out = (float*)dst; }
            a.rows = spec(0).dims[0]; a.ld = spec(1).dims[1]; a.dt_col = m.dt_col;
            a.heads = m.heads; a.groups = m.groups; a.n = m.state; a.vdim = m.vdim;
            k::ssm_scan(s, a);
            ++cx.launches;
            break;
        }
        case Mix::GatedNorm:
            k::gated_rms_norm(s, dt, ptr(0), f(1), f(2), dst, out.dims[0], m.dim, spec(1).dims[1], m.col, m.groups, in.eps);
            ++cx.launches;
            break;
        case Mix::Glu: {
            k::GluParams p;
            p.kind = 1; p.limit = in.fparam[0]; p.alpha = in.fparam[1]; p.shift = in.fparam[2];
            k::clamped_glu(s, dt, ptr(0), ptr(1), dst, out.count(), p);
            ++cx.launches;
            break;
        }
        case Mix::SsmSeq: {
            int64_t row = 0;
            for (size_t b0 = 0; b0 < in.lens.size(); b0 += k::kMixerBatch) {   // rows of the scratch are the rows of the batch
                k::SsmSeqArgs a{};
                a.dtype = dt;
                a.p = f(0); a.taps = f(1); a.bias = f(2); a.dt_bias = f(3); a.a_log = f(4); a.d = f(5); a.gain = f(6);
                a.out = dst;
                a.ld = spec(0).dims[1]; a.col = m.col; a.ch = m.dim; a.ntaps = m.taps; a.dt_col = m.dt_col; a.z_col = m.z_col;
                a.heads = m.heads; a.groups = m.groups; a.n = m.state; a.vdim = m.vdim; a.norm_groups = m.rank;
                a.eps = in.eps;
                a.nseq = (int)std::min<size_t>(in.lens.size() - b0, k::kMixerBatch);
                for (int b = 0; b < a.nseq; ++b) {
                    const int q = (int)b0 + b;
                    a.row0[b] = (int)row;
                    a.len[b] = (int)in.lens[q];
                    row += in.lens[q];
                    a.conv_in[b] = f(7 + 2 * q); a.state_in[b] = f(8 + 2 * q);
                    a.conv_out[b] = (float*)cx.ptr[st.dst[1 + 2 * q]]; a.state_out[b] = (float*)cx.ptr[st.dst[2 + 2 * q]];
                }
                a.rows = row - a.row0[0];
                a.scratch = cx.ws + st.scratch_off;
                cx.launches += k::ssm_seq(s, a);
            }
            break;
        }
        case Mix::LatentDecode: {
            const size_t c0 = in.append ? 8 : 5;
            for (size_t b0 = 0; b0 < in.lens.size(); b0 += k::kMixerBatch) {
                k::LatentDecodeArgs a{};
                a.dtype = dt;
                a.heads = m.heads; a.dim = m.dim; a.rot = m.rot; a.rank = m.rank; a.vdim = m.vdim; a.scale = in.scale; a.eps = in.eps;
                a.nseq = (int64_t)std::min<size_t>(in.lens.size() - b0, k::kMixerBatch);
                a.capacity = spec(c0).dims[1];
                const size_t es = dtype_size(out.dtype);
                a.x = (const char*)ptr(0) + b0 * (size_t)spec(0).dims[1] * es;
                a.table = f(1) + b0 * m.rot;
                a.w_uk = ptr(2); a.w_uv = ptr(3);
                a.pos = (const int32_t*)ptr(4) + b0;
                a.ctx = (char*)dst + b0 * (size_t)out.dims[1] * es;
                if (in.append) { a.raw = f(5) + b0 * (m.rank + m.rot); a.gain = f(6); a.starts = (const int32_t*)ptr(7) + 3 * b0; }
                for (int64_t b = 0; b < a.nseq; ++b) {
                    const void* from = ptr(c0 + b0 + b);
                    void* to = in.append ? cx.ptr[st.dst[1 + b0 + b]] : const_cast<void*>(from);
                    if (to != from) {   // a cache that was not donated is copied first
                        GPTRS_HIP_CHECK(hipMemcpyAsync(to, from, spec(c0).bytes(), hipMemcpyDeviceToDevice, s));
                        ++cx.launches;
                    }
                    a.cache[b] = to;
                }
                a.scratch = cx.ws + st.scratch_off;
                cx.launches += k::latent_decode(s, a);
            }
            break;
        }
        case Mix::LatentPrefill: {
            int64_t row = 0;
            for (size_t b0 = 0; b0 < in.lens.size(); b0 += k::kMixerBatch) {
                k::LatentPrefillArgs a{};
                a.dtype = dt;
                a.x = ptr(0); a.table = f(1); a.k = ptr(2); a.v = ptr(3); a.rows = ptr(4); a.ctx = dst;
                a.heads = m.heads; a.dim = m.dim; a.rot = m.rot; a.rank = m.rank; a.vdim = m.vdim; a.scale = in.scale;
                a.total = out.dims[0];
                a.nseq = (int)std::min<size_t>(in.lens.size() - b0, k::kMixerBatch);
                for (int b = 0; b < a.nseq; ++b) { a.row0[b] = (int)row; a.len[b] = (int)in.lens[b0 + b]; row += in.lens[b0 + b]; }
                a.scratch = cx.ws + st.scratch_off;
                cx.launches += k::latent_prefill(s, a);
            }
            break;
        }
        case Mix::HeadNorm:
            k::head_rms_norm(s, (int)spec(0).dtype, dt, ptr(0), dst, out.dims[0] * m.heads, m.dim, in.eps);
            ++cx.launches;
            break;
        case Mix::HeadGate:
            k::head_gate(s, dt, ptr(0), f(1), dst, out.dims[0], m.heads, m.vdim, m.heads);
            ++cx.launches;
            break;
        case Mix::ChunkAttn:
        case Mix::ChunkAttnCache: {
            k::ChunkAttnArgs a{};
            a.dtype = dt;
            a.q = ptr(0); a.k = ptr(1); a.v = ptr(2); a.sink = f(3); a.ctx = dst;
            a.t = out.dims[0]; a.heads = m.heads; a.kv_heads = m.groups; a.dim = m.dim; a.vdim = m.vdim; a.chunk = m.chunk; a.scale = in.scale;
            if (in.mix == Mix::ChunkAttnCache) {
                a.position = (const int32_t*)ptr(4);
                a.rows = spec(1).dims[1];
                a.k_row = m.dim; a.k_head = a.rows * m.dim; a.v_row = m.vdim; a.v_head = a.rows * m.vdim;
            } else {
                a.rows = a.t;
                a.k_row = m.groups * m.dim; a.k_head = m.dim; a.v_row = m.groups * m.vdim; a.v_head = m.vdim;
            }
            k::chunk_attn(s, a);
            ++cx.launches;
            break;
        }
        case Mix::ChunkDecode:
        case Mix::ChunkPrefill: {
            int64_t row = 0;
            for (size_t b0 = 0; b0 < in.lens.size(); b0 += k::kMixerBatch) {
                k::ChunkSeqArgs a{};
                a.dtype = dt;
                a.proj = f(0); a.sink = f(1); a.pos = (const int32_t*)ptr(2) + b0; a.starts = (const int32_t*)ptr(3) + 3 * b0;
                if (m.rot > 0) a.table = f(4);
                a.ctx = dst;
                a.total = out.dims[0]; a.ld = spec(0).dims[1];
                a.heads = m.heads; a.kv_heads = m.groups; a.dim = m.dim; a.vdim = m.vdim; a.rot = m.rot; a.chunk = m.chunk; a.scale = in.scale; a.eps = in.eps;
                a.rows = spec(chunk_cache_operand(in, 0)).dims[1];
                a.nseq = (int)std::min<size_t>(in.lens.size() - b0, k::kMixerBatch);
                for (int b = 0; b < a.nseq; ++b) {
                    const size_t q = b0 + b;
                    a.row0[b] = (int)row;
                    a.len[b] = (int)in.lens[q];
                    a.keep[b] = m.chunk > 0 ? (int)((in.lens[q] - 1) % m.chunk + 1) : (int)in.lens[q];
                    row += in.lens[q];
                    for (int kv = 0; kv < 2; ++kv) {
                        const size_t ci = chunk_cache_operand(in, q) + kv;
                        const void* from = ptr(ci);
                        void* to = cx.ptr[st.dst[1 + 2 * q + kv]];
                        if (to != from) {   // a cache that was not donated is copied first
                            GPTRS_HIP_CHECK(hipMemcpyAsync(to, from, spec(ci).bytes(), hipMemcpyDeviceToDevice, s));
                            ++cx.launches;
                        }
                        (kv ? a.vcache : a.kcache)[b] = to;
                    }
                }
                a.scratch = cx.ws + st.scratch_off;
                a.tickets = cx.be->skinny_tickets();
                cx.launches += in.mix == Mix::ChunkDecode ? k::chunk_decode(s, a) : k::chunk_prefill(s, a);
            }
            break;
        }
        case Mix::PostNorm:
            k::post_norm_add(s, f(0), f(1), f(2), (float*)dst, st.dst.size() > 1 ? cx.ptr[st.dst[1]] : nullptr, out.dims[0], out.dims[1], in.post_mult, in.scale, in.eps);
            ++cx.launches;
            break;
        case Mix::EmbedRows:
            k::embed_rows(s, (int)spec(0).dtype, ptr(0), (const int32_t*)ptr(1), (float*)dst, st.dst.size() > 1 ? cx.ptr[st.dst[1]] : nullptr, out.dims[0],
                          spec(0).dims[0], out.dims[1], in.scale, cx.err_flag);
            ++cx.launches;
            break;
        case Mix::Softcap:
            k::softcap(s, f(0), (float*)dst, out.count(), in.softcap);
            ++cx.launches;
            break;
        default:
            fail_unimpl(in.op_name, "no kernel bound to this operation");
    }
}

}  // namespace gptrs
