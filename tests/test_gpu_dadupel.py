"""The Dadupel design on the device: every mixer call against the oracle, the fused launches against the calls they replace, and
whole models against the plain implementation (tests/dadupel_util.py makes configurations and weights)."""
import numpy as np
import pytest

import dadupel_util as U
import __graft_entry__ as entry
from oracle.dadupel_reference import Reference
from gptrs_amd import functional as F, loader, models
from gptrs_amd.ptir import FunctionBuilder, Program, TensorSpec, f32_to_bf16_bits

pytestmark = pytest.mark.gpu
po = entry.load_oracle()


def upload(be, a, dtype):
    if dtype == "Si32":
        return be.materialize(TensorSpec("Si32", a.shape), np.ascontiguousarray(a, "<i4").tobytes())
    data = np.ascontiguousarray(a, "<f4") if dtype == "F32" else f32_to_bf16_bits(np.asarray(a, np.float32)).astype("<u2")
    return be.materialize(TensorSpec(dtype, a.shape), data.tobytes())


def both(be, emit, args, fusion=True):
    """The program's results on the device and on the oracle; args = [(array, dtype)]."""
    fb = FunctionBuilder("main", "F32")
    outs = emit(fb, *[fb.param(dt, a.shape) for a, dt in args])
    fb.set_results(list(outs) if isinstance(outs, (list, tuple)) else [outs])
    prog = Program(fb)
    be.set_option("fusion", 1 if fusion else 0)
    try:
        got = [be.to_numpy(h) for h in be.run_program(prog, [upload(be, a, dt) for a, dt in args])]
    finally:
        be.set_option("fusion", 1)
    import json
    ins = [po.OTensor(dt, np.asarray(a, np.int32) if dt == "Si32" else (U.bf16(a).reshape(a.shape) if dt == "Bf16" else np.asarray(a, np.float32))) for a, dt in args]
    return got, [o.a for o in po.run_program(json.loads(prog.json_bytes), ins)]


def check(got, want, tol, what=""):
    got, want = np.asarray(got, np.float64), np.asarray(want, np.float64)
    assert got.shape == want.shape and np.all(np.isfinite(got)), what
    err = np.max(np.abs(got - want)) / (np.max(np.abs(want)) + 1e-30)
    assert err < tol, (what, err)


TOL = {"F32": 3e-5, "Bf16": 1.2e-2}   # Bf16: a couple of roundings of a result


def rn(seed, *shape):
    return np.random.default_rng(seed).standard_normal(shape).astype(np.float32)


# ------------------------------------------------------------------------------------------ mechanisms, alone
@pytest.mark.parametrize("dt", ["F32", "Bf16"])
@pytest.mark.parametrize("heads,hd,off,rot", [(3, 24, 16, 8), (1, 16, 4, 6), (5, 8, 0, 8)])
def test_pair_rotation_far_out(hip, dt, heads, hd, off, rot):
    pos = np.array([0, 1, 2, 1023, 40000, 131071], np.int32)
    f = F.pair_frequencies(rot, 100.0)
    got, want = both(hip, lambda fb, x, p, fr: F.rope_pairs(x, F.rope_table(p, fr, 1.3), heads, off), [(rn(1, 6, heads * hd), dt), (pos, "Si32"), (f, "F32")])
    check(got[0], want[0], TOL[dt])


@pytest.mark.parametrize("dt", ["F32", "Bf16"])
@pytest.mark.parametrize("rank,rot,rows", [(24, 8, 5), (512, 64, 3), (7, 2, 1)])
def test_latent_rows(hip, dt, rank, rot, rows):
    pos = np.arange(rows, dtype=np.int32) + 11
    got, want = both(hip, lambda fb, raw, g, p, fr: F.latent_rows(raw, g, F.rope_table(p, fr), 1e-5, dt),
                     [(rn(1, rows, rank + rot), "F32"), (1 + 0.1 * rn(2, rank), "F32"), (pos, "Si32"), (F.pair_frequencies(rot, 50.0), "F32")])
    check(got[0], want[0], TOL[dt])


@pytest.mark.parametrize("dt", ["F32", "Bf16"])
def test_clamped_unit(hip, dt):
    got, want = both(hip, lambda fb, g, u: F.clamped_glu(g, u, 1.25), [(3 * rn(1, 7, 33), dt), (3 * rn(2, 7, 33), dt)])
    check(got[0], want[0], TOL[dt])


@pytest.mark.parametrize("dt", ["F32", "Bf16"])
@pytest.mark.parametrize("rows,ch,K", [(1, 10, 4), (2, 10, 4), (5, 12, 2), (9, 300, 3), (4, 8, 1), (3, 8, 7)])
def test_convolution_and_its_history(hip, dt, rows, ch, K):
    got, want = both(hip, lambda fb, p, t, b, s: F.causal_conv_silu(p, t, b, s, 3, dt),
                     [(rn(1, rows, ch + 5), "F32"), (rn(2, K, ch), "F32"), (rn(3, ch), "F32"), (rn(4, K - 1, ch), "F32")])
    check(got[0], want[0], TOL[dt])
    if K > 1:
        assert np.array_equal(got[1], want[1])


@pytest.mark.parametrize("dt", ["F32", "Bf16"])
@pytest.mark.parametrize("rows,H,G,N,V", [(1, 4, 2, 16, 16), (9, 3, 1, 12, 20), (70, 6, 3, 8, 70), (5, 2, 2, 130, 40)])
def test_recurrence(hip, dt, rows, H, G, N, V):
    got, want = both(hip, lambda fb, x, p, b, a, d, s: F.ssm_scan(x, p, b, a, d, s, G, 2),
                     [(rn(1, rows, H * V + 2 * G * N), dt), (rn(2, rows, H + 3), "F32"), (rn(3, H) - 2, "F32"), (rn(4, H) * 0.5, "F32"), (rn(5, H), "F32"), (rn(6, H, N, V), "F32")])
    check(got[0], want[0], TOL[dt])
    check(got[1], want[1], 3e-5)


@pytest.mark.parametrize("dt", ["F32", "Bf16"])
@pytest.mark.parametrize("n,groups", [(48, 3), (40, 1), (20, 4), (4096, 2), (24, 24)])
def test_gated_norm(hip, dt, n, groups):
    got, want = both(hip, lambda fb, y, p, g: F.gated_rms_norm(y, p, g, groups, 4, 1e-3), [(rn(1, 5, n), dt), (rn(2, 5, n + 8), "F32"), (rn(3, n), "F32")])
    check(got[0], want[0], TOL[dt])


@pytest.mark.parametrize("dt", ["F32", "Bf16"])
@pytest.mark.parametrize("heads,dim,rot,rank,vdim,L,start,T", [(3, 16, 8, 24, 24, 40, 17, 1), (1, 10, 6, 11, 7, 300, 290, 2), (4, 32, 32, 64, 32, 530, 513, 3)])
def test_attention_over_cached_rows(hip, dt, heads, dim, rot, rank, vdim, L, start, T):
    args = [(rn(1, T, heads * (dim + rot)), dt), (rn(2, 1, L, rank + rot), dt), (rn(3, rank, heads * dim) * rank ** -0.5, dt), (rn(4, rank, heads * vdim) * rank ** -0.5, dt),
            (np.array([start], np.int32), "Si32")]
    got, want = both(hip, lambda fb, *a: F.latent_attention(*a, heads, rot, 0.3), args)
    check(got[0], want[0], TOL[dt])


# ------------------------------------------------------------------------------------------ one key or token among many
def latent_args(seed, T, heads, dim, rot, rank, vdim, dt, n=None):
    """Operands of a prompt's attention (unrotated queries, keys, values, cached rows) with small scores."""
    pos = np.arange(T if n is None else n, dtype=np.int32)
    return [(0.02 * rn(seed, len(pos), heads * (dim + rot)), dt), (pos, "Si32"), (F.pair_frequencies(rot, 30.0), "F32"), (0.1 * rn(seed + 1, len(pos), heads * dim), dt),
            (rn(seed + 2, len(pos), heads * vdim), dt), (0.1 * rn(seed + 3, len(pos), rank + rot), dt)]


SHAPES = [(2, 16, 8, 24, 24), (1, 32, 32, 64, 32), (3, 128, 64, 32, 128), (2, 64, 24, 16, 136), (1, 200, 56, 32, 256), (1, 10, 6, 11, 7)]


@pytest.mark.parametrize("dt", ["F32", "Bf16"])
@pytest.mark.parametrize("shape", SHAPES)
@pytest.mark.parametrize("T", [1, 2, 63, 64, 65, 130, 200])
def test_prompt_attention_and_single_keys(hip, dt, shape, T):
    """Query i's score with key i (its own: the last it may see) and with one far key stands out, the next key's would stand
    out more and must not be seen."""
    heads, dim, rot, rank, vdim = shape
    args = latent_args(5, T, heads, dim, rot, rank, vdim, dt)
    q, k = args[0][0].reshape(T, heads, dim + rot), args[3][0].reshape(T, heads, dim)
    dirs = np.linalg.qr(rn(9, max(dim, T), dim))[0][:T] if T > dim else np.eye(T, dim, dtype=np.float32)
    dirs = dirs / np.linalg.norm(dirs, axis=1, keepdims=True)
    for i in range(T):
        k[i] = 6 * dirs[i]
        q[i, :, :dim] = 4 * dirs[i] + 5 * dirs[min(i + 1, T - 1)] + (4 * dirs[i // 3] if i % 7 == 0 else 0)
    emit = lambda fb, x, p, fr, kk, v, r: F.latent_attention_expanded(F.rope_pairs(x, F.rope_table(p, fr), heads, dim), kk, v, r, heads, rot, 0.9)
    got, want = both(hip, emit, args)
    check(got[0], want[0], TOL[dt], (shape, T))


@pytest.mark.parametrize("dt", ["F32", "Bf16"])
@pytest.mark.parametrize("shape", [(3, 16, 8, 24, 24), (5, 32, 32, 64, 32), (24, 16, 32, 96, 8), (32, 128, 64, 512, 128), (2, 40, 24, 360, 40), (1, 10, 6, 11, 7)])
@pytest.mark.parametrize("lens", [[1], [2, 63, 64, 65], [500, 1, 257], [4000, 2049, 66], list(range(1, 19))])
def test_decode_attention_of_a_batch(hip, dt, shape, lens):
    """One step of unequal sequences (more than one launch's worth in the last case), caches written in place of nothing but the
    new row; one far row, the row before and the new row itself stand out in turn."""
    heads, dim, rot, rank, vdim = shape
    B, C = len(lens), 512 if max(lens) <= 512 else 4096
    if (len(lens) > 4 and rank > 96) or (C > 512 and (rank == 512 or heads < 2)):
        pytest.skip("a few sizes of long batches and long caches are enough")
    pos = np.array([n - 1 for n in lens], np.int32)
    starts = np.array([v for n in lens for v in (0, n - 1, 0)], np.int32)
    caches = [0.3 * rn(20 + b, 1, C, rank + rot) for b in range(B)]
    w_uk, w_uv = rn(1, rank, heads * dim) * rank ** -0.5, rn(2, rank, heads * vdim) * rank ** -0.5
    x = 0.5 * rn(3, B, heads * (dim + rot))
    for b, n in enumerate(lens):
        j = [0, n - 1, max(n - 2, 0), n // 2][b % 4]   # a cached row along W_uk^T q of head 0
        caches[b][0, j, :rank] += 2.0 * (w_uk[:, :dim] @ x[b, :dim]) / max(1e-3, np.linalg.norm(w_uk[:, :dim] @ x[b, :dim]))
        if n < C:
            caches[b][0, n:] += 50.0                    # rows that nobody has written yet
    raw, gain = rn(4, B, rank + rot), 1 + 0.1 * rn(5, rank)
    args = [(x, dt), (pos, "Si32"), (starts, "Si32"), (F.pair_frequencies(rot, 30.0), "F32"), (w_uk, dt), (w_uv, dt), (raw, "F32"), (gain, "F32")] + [(c, dt) for c in caches]

    def emit(fb, x, p, st, fr, wk, wv, raw, g, *cs):
        tab = F.rope_table(p, fr)
        q, rows = F.rope_pairs(x, tab, heads, dim), F.latent_rows(raw, g, tab, 1e-5, dt)
        part = lambda t, b: t if B == 1 else t.slice([b, 0], [1, t.dims[1]])
        new = [F.dynamic_update_slice_into(c, part(rows, b).reshape([1, 1, rank + rot]), st if B == 1 else st.slice([3 * b], [3])) for b, c in enumerate(cs)]
        own = [F.latent_attention(part(q, b), new[b], wk, wv, p if B == 1 else p.slice([b], [1]), heads, rot, 1.1) for b in range(B)]
        # a second layer reads the caches the first has written
        sec = [F.latent_attention(part(q, b), new[b], wk, wv, p if B == 1 else p.slice([b], [1]), heads, rot, 0.4) for b in range(B)]
        st2 = lambda t: t[0] if B == 1 else type(t[0]).concat(0, t)
        return [st2(own), st2(sec)] + new
    for fusion in (True, False):
        got, want = both(hip, emit, args, fusion)
        check(got[0], want[0], TOL[dt], "own")
        check(got[1], want[1], TOL[dt], "shared")
        for b in range(B):
            check(got[2 + b], want[2 + b], TOL[dt], "cache")


@pytest.mark.parametrize("dt", ["F32", "Bf16"])
@pytest.mark.parametrize("H,G,N,V,K,ng", [(4, 2, 16, 16, 4, 2), (3, 1, 12, 20, 2, 3), (8, 4, 64, 48, 4, 4), (2, 1, 128, 64, 3, 1), (2, 2, 200, 24, 4, 1), (6, 3, 8, 40, 5, 1)])
@pytest.mark.parametrize("lens", [[1], [1, 1, 1], [2], [63], [64], [65, 1, 129], [16, 17]])
def test_state_space_mixer(hip, dt, H, G, N, V, K, ng, lens):
    """The whole mixer over ragged prompts or one token each, from states that are not zero; one early token's B and x stand
    out, so that a lost state or a decay that is off by a token shows at the end."""
    B, rows, inner = len(lens), sum(lens), H * V
    ch = inner + 2 * G * N
    Wd = inner + ch + H
    p = rn(1, rows, Wd) * 0.7
    r0 = 0
    for n in lens:
        p[r0, inner:inner + ch] *= 6.0
        r0 += n
    args = [(p, "F32"), (rn(2, K, ch), "F32"), (rn(3, ch), "F32"), (rn(4, H) * 0.3 - 4, "F32"), (rn(5, H) * 0.3 - 1, "F32"), (rn(6, H), "F32"), (1 + 0.1 * rn(7, inner), "F32")]
    for b in range(B):
        args += [(rn(30 + b, K - 1, ch), "F32"), (0.3 * rn(50 + b, H, N, V), "F32")]

    def emit(fb, p, taps, bias, dtb, al, d, gain, *st):
        ys, new, r0 = [], [], 0
        for b, n in enumerate(lens):
            pr = p if B == 1 else p.slice([r0, 0], [n, Wd])
            r0 += n
            xbc, c2 = F.causal_conv_silu(pr, taps, bias, st[2 * b], inner, dt)
            y, s2 = F.ssm_scan(xbc, pr, dtb, al, d, st[2 * b + 1], G, inner + ch)
            ys.append(y)
            new += [c2, s2]
        y = ys[0] if B == 1 else type(ys[0]).concat(0, ys)
        return [F.gated_rms_norm(y, p, gain, ng, 0, 1e-5)] + new
    fused, want = both(hip, emit, args)
    plain, _ = both(hip, emit, args, fusion=False)
    for got, what in ((fused, "fused"), (plain, "plain")):
        check(got[0], want[0], {"F32": 1e-4, "Bf16": 2.5e-2}[dt], what)
        for b in range(B):
            assert np.array_equal(got[1 + 2 * b], want[1 + 2 * b]), what
            check(got[2 + 2 * b], want[2 + 2 * b], {"F32": 1e-4, "Bf16": 1.5e-2}[dt], what)


# ------------------------------------------------------------------------------------------ linear steps
@pytest.mark.parametrize("dt", ["F32", "Bf16"])
@pytest.mark.parametrize("M", [1, 3, 16, 17, 130])
@pytest.mark.parametrize("K,N", [(64, 96), (256, 1000), (128, 37), (100, 50)])
def test_layer_norm_pair_and_column_factors(hip, dt, M, K, N):
    """layer norm of the f32 stream -> clamped pair -> down projection times a factor per column plus the stream."""
    def emit(fb, x, g, b, wg, wu, wd, ls):
        h, *_ = F.layer_norm(x, g, b, 1e-5)
        h = h if dt == "F32" else h.cast(dt)
        a = F.clamped_glu(F.linear(h, wg), F.linear(h, wu), 0.9)
        return F.scale_columns(F.linear(a, wd, out_dtype="F32"), ls) + x
    args = [(3 * rn(1, M, K) + 1, "F32"), (1 + 0.2 * rn(2, K), "F32"), (0.3 * rn(3, K), "F32"), (rn(4, K, N) * K ** -0.5, dt), (rn(5, K, N) * K ** -0.5, dt),
            (rn(6, N, K) * N ** -0.5, dt), (rn(7, K), "F32")]
    for fusion in (True, False):
        got, want = both(hip, emit, args, fusion)
        check(got[0], want[0], {"F32": 3e-5, "Bf16": 4e-3}[dt], fusion)


# ------------------------------------------------------------------------------------------ whole models
def load(hip, tmp_path, name, dt, seed=0, **kw):
    cfg = U.STACKS[name]
    W = U.weights(cfg, seed)
    return loader.load_model(hip, U.write_folder(str(tmp_path / name), cfg, W), dtype=dt, **kw), Reference(cfg, W), cfg


def tokens(cfg, n, seed=1):
    return np.random.default_rng(seed).integers(0, cfg["vocab"], n).tolist()


def rms(got, want, dt, what=""):
    """Root mean square of the logits' difference in units of their spread: every position within a few roundings."""
    got, want = np.asarray(got, np.float64), np.asarray(want, np.float64)
    assert got.shape == want.shape and np.all(np.isfinite(got)), what
    err = np.sqrt(((got - want) ** 2).mean(axis=-1)) / want.std()
    assert err.max() < {"F32": 3e-5, "Bf16": 6e-2}[dt] and np.median(err) < {"F32": 1e-5, "Bf16": 2.5e-2}[dt], (what, err.max(), np.median(err), int(err.argmax()))


@pytest.mark.parametrize("dt", ["F32", "Bf16"])
@pytest.mark.parametrize("name", sorted(U.STACKS))
def test_prompt_decode_and_batches(hip, tmp_path, name, dt):
    m, ref, cfg = load(hip, tmp_path, name, dt)
    n = 150
    toks = tokens(cfg, n)
    want, _ = ref.forward(toks)
    fresh = lambda: [None] * m.num_layers
    rms(hip.to_numpy(m.forward_with_decode_cache(toks, 0, fresh())), want, dt, "whole")
    for cut in (1, 63, 127):   # a prompt of `cut` tokens, the rest one by one; capacities grow on the way
        c = fresh()
        rows = [hip.to_numpy(m.forward_with_decode_cache(toks[:cut], 0, c))]
        stop = min(n, cut + (40 if cut > 1 else 70))
        for i in range(cut, stop):
            rows.append(hip.to_numpy(m.forward_with_decode_cache([toks[i]], i, c)))
        rms(np.concatenate(rows), want[:stop], dt, f"cut {cut}")
    # unequal requests together, one of them ending early, then others in their place
    for round_, lens in enumerate(((1, 70, 33, 5), (40, 2))):
        seqs = [tokens(cfg, k, 20 + 10 * round_ + b) for b, k in enumerate(lens)]
        full = [s + tokens(cfg, 6, 60 + b) for b, s in enumerate(seqs)]
        wants = [ref.forward(s)[0] for s in full]
        cs = [fresh() for _ in lens]
        got = hip.to_numpy(m.forward_batch(seqs, 0, cs))
        rms(got, np.concatenate([w[:len(s)] for w, s in zip(wants, seqs)]), dt, "batch prompt")
        live = list(range(len(lens)))
        for step in range(6):
            if step == 3:
                cs[live[0]] = None
                live = live[1:]
            got = hip.to_numpy(m.forward_batch([[full[b][lens[b] + step]] for b in live], [lens[b] + step for b in live], [cs[b] for b in live]))
            rms(got, np.stack([wants[b][lens[b] + step] for b in live]), dt, f"batch step {step}")


@pytest.mark.parametrize("dt", ["F32", "Bf16"])
def test_long_decoding_with_replayed_graphs(hip, tmp_path, dt):
    """400 single steps in a fixed capacity (the steps are replayed as one graph): state and cache stay right to the end, and the
    eager launches say the same."""
    m, ref, cfg = load(hip, tmp_path, "tiled", dt)
    toks = tokens(cfg, 420)
    want, _ = ref.forward(toks)
    outs = []
    for graphs in (1, 0):
        hip.set_option("graphs", graphs)
        try:
            before = hip.counter("graph_launches")
            c = [None] * m.num_layers
            m.forward_with_decode_cache(toks[:20], 0, c, 512)
            outs.append(np.concatenate([hip.to_numpy(m.forward_with_decode_cache([toks[i]], i, c, 512)) for i in range(20, 420)]))
            if graphs:
                assert hip.counter("graph_launches") > before + 300
        finally:
            hip.set_option("graphs", 1)
    rms(outs[0], want[20:], dt)
    assert np.array_equal(outs[0], outs[1])


@pytest.mark.parametrize("dt", ["F32", "Bf16"])
def test_fused_and_plain_programs_agree(hip, tmp_path, dt):
    m, ref, cfg = load(hip, tmp_path, "mixed", dt)
    toks = tokens(cfg, 40)
    res = []
    for fusion in (1, 0):
        hip.set_option("fusion", fusion)
        try:
            c = [None] * m.num_layers
            rows = [hip.to_numpy(m.forward_with_decode_cache(toks[:33], 0, c))]
            rows += [hip.to_numpy(m.forward_with_decode_cache([toks[i]], i, c)) for i in range(33, 40)]
            res.append(np.concatenate(rows))
        finally:
            hip.set_option("fusion", 1)
    want = ref.forward(toks)[0]
    rms(res[0], want, dt)
    rms(res[1], want, dt)


def test_inputs_are_kept_unless_donated(hip, tmp_path):
    """Running the same step twice from one set of caches: nothing that was not given away has changed."""
    m, ref, cfg = load(hip, tmp_path, "mixed", "Bf16")
    toks = tokens(cfg, 12)
    c = [None] * m.num_layers
    m.forward_with_decode_cache(toks[:11], 0, c, 16)
    prog, _ = m._build((1,), 16, True)
    args = [m._upload_i32([toks[11]]), m._upload_i32([11]), m._upload_i32([0, 11, 0])]
    held = [h for s in c for h in ((s.conv, s.state) if isinstance(s, models.DecodeSsmState) else (s.rows,) if isinstance(s, models.DecodeLatentCache) else ())]
    before = [hip.to_numpy(h) for h in held]
    a = hip.to_numpy(m._run(prog, args + held)[-1])
    b = hip.to_numpy(m._run(prog, args + held)[-1])
    assert np.array_equal(a, b)
    for x, h in zip(before, held):
        assert np.array_equal(x, hip.to_numpy(h))


def test_greedy_generation(hip, tmp_path):
    """Generator (pipelined, device sampling) and BatchGenerator over unequal prompts write the plain implementation's tokens."""
    m, ref, cfg = load(hip, tmp_path, "tiled", "F32")
    prompts = [tokens(cfg, n, s) for s, n in ((1, 20), (2, 1), (3, 67))]
    want = []
    for p in prompts:
        logits, st = ref.forward(p)
        out = []
        for _ in range(24):
            out.append(int(np.argmax(logits[-1])))
            logits, st = ref.forward(out[-1:], st)
        want.append(out)
    assert models.Generator(m, prompts[0]).generate(24) == want[0]
    assert models.Generator(m, prompts[2], pipelined=False).generate(24) == want[2]
    assert models.BatchGenerator(m, prompts).generate(24) == want
    top = models.Generator(m, prompts[1], temperature=0.7, top_k=3, seed=5).generate(8)
    assert len(top) == 8 and all(0 <= t < cfg["vocab"] for t in top)


def test_trace_replay(hip, tmp_path):
    import json
    from gptrs_amd import trace
    m, ref, cfg = load(hip, tmp_path, "mixed", "F32")
    a, b = tokens(cfg, 12, 1), tokens(cfg, 7, 2)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:10], "want": [0, 9]}, {"id": "b", "tokens": b[:5], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": [b[5]], "want": [0]}, {"id": "a", "tokens": [a[10]], "want": []}], "end": ["b"]},
             {"step": 2, "entries": [{"id": "a", "tokens": [a[11]], "want": []}], "end": ["a"]},
             {"step": 3, "entries": [{"id": "b", "tokens": b, "want": [6]}], "end": ["b"]}]
    said = []
    trace.replay(m, iter(json.dumps(s) + "\n" for s in steps), str(tmp_path), said.append)
    assert said == [f"done {i}" for i in range(4)]
    read = lambda i: np.fromfile(tmp_path / f"{i}.f32", "<f4").reshape(-1, cfg["vocab"])
    wa, wb = ref.forward(a)[0], ref.forward(b)[0]
    rms(read(0), wa[[0, 9]], "F32")
    rms(read(1), wb[[5]], "F32")
    rms(read(3), wb[[6]], "F32")
    assert not (tmp_path / "2.f32").exists()
