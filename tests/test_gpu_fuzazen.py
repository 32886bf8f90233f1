"""The Fuzazen design on the device: every call against the oracle, the fused launches against the calls they replace, and whole
models against the plain implementation (tests/fuzazen_util.py makes configurations and weights)."""
import json

import numpy as np
import pytest

import fuzazen_util as U
import __graft_entry__ as entry
from oracle.fuzazen_reference import Reference
from gptrs_amd import functional as F, loader, models, trace
from gptrs_amd.ptir import FunctionBuilder, Program, TensorSpec, f32_to_bf16_bits

pytestmark = pytest.mark.gpu
po = entry.load_oracle()


def upload(be, a, dtype):
    if dtype == "Si32":
        return be.materialize(TensorSpec("Si32", a.shape), np.ascontiguousarray(a, "<i4").tobytes())
    data = np.ascontiguousarray(a, "<f4") if dtype == "F32" else f32_to_bf16_bits(np.asarray(a, np.float32)).astype("<u2")
    return be.materialize(TensorSpec(dtype, a.shape), data.tobytes())


def build(emit, args):
    fb = FunctionBuilder("main", "F32")
    outs = emit(fb, *[fb.param(dt, a.shape) for a, dt in args])
    fb.set_results(list(outs) if isinstance(outs, (list, tuple)) else [outs])
    return Program(fb)


def on_device(be, prog, args, **options):
    for k, v in options.items():
        be.set_option(k, v)
    try:
        return [be.to_numpy(h) for h in be.run_program(prog, [upload(be, a, dt) for a, dt in args])]
    finally:
        for k in options:
            be.set_option(k, 1)


def on_oracle(prog, args):
    ins = [po.OTensor(dt, np.asarray(a, np.int32) if dt == "Si32" else (U.bf16(a).reshape(a.shape) if dt == "Bf16" else np.asarray(a, np.float32))) for a, dt in args]
    return [o.a for o in po.run_program(json.loads(prog.json_bytes), ins)]


def both(be, emit, args, **options):
    prog = build(emit, args)
    return on_device(be, prog, args, **options), on_oracle(prog, args)


def check(got, want, tol, what=""):
    got, want = np.asarray(got, np.float64), np.asarray(want, np.float64)
    assert got.shape == want.shape and np.all(np.isfinite(got)), what
    err = np.max(np.abs(got - want)) / (np.max(np.abs(want)) + 1e-30)
    assert err < tol, (what, err)


TOL = {"F32": 3e-5, "Bf16": 1.2e-2}   # Bf16: a couple of roundings of a result


def rn(seed, *shape):
    return np.random.default_rng(seed).standard_normal(shape).astype(np.float32)


# ------------------------------------------------------------------------------------------ calls, alone
@pytest.mark.parametrize("dt", ["F32", "Bf16"])
@pytest.mark.parametrize("heads,hd,off,rot", [(3, 9, 0, 8), (1, 7, 1, 6), (2, 12, 3, 4)])
def test_rotation_in_heads_of_odd_size(hip, dt, heads, hd, off, rot):
    pos = np.array([0, 1, 2, 1023, 40000], np.int32)
    got, want = both(hip, lambda fb, x, p, fr: F.rope_pairs(x, F.rope_table(p, fr), heads, off), [(rn(1, 5, heads * hd), dt), (pos, "Si32"), (F.pair_frequencies(rot, 100.0), "F32")])
    check(got[0], want[0], TOL[dt])


@pytest.mark.parametrize("dt,out", [("F32", "F32"), ("F32", "Bf16"), ("Bf16", "Bf16"), ("Bf16", "F32")])
@pytest.mark.parametrize("rows,heads,hd", [(1, 1, 4), (5, 3, 7), (130, 2, 64), (3, 5, 200)])
def test_head_norm(hip, dt, out, rows, heads, hd):
    x = rn(1, rows, heads * hd) * (10.0 ** np.arange(-2, 3))[np.arange(rows) % 5, None].astype(np.float32)   # small rows: eps shows
    got, want = both(hip, lambda fb, x: F.head_rms_norm(x, heads, 1e-3, out), [(x, dt)])
    check(got[0], want[0], TOL[out])


@pytest.mark.parametrize("dt", ["F32", "Bf16"])
@pytest.mark.parametrize("rows,heads,vd", [(1, 1, 1), (7, 3, 5), (40, 8, 64)])
def test_head_gate(hip, dt, rows, heads, vd):
    got, want = both(hip, lambda fb, x, g: F.head_gate(x, g, heads), [(rn(1, rows, heads * vd), dt), (3 * rn(2, rows, heads), "F32")])
    check(got[0], want[0], TOL[dt])


@pytest.mark.parametrize("dt", ["F32", "Bf16"])
@pytest.mark.parametrize("T,H,G,D,V,chunk", [(1, 1, 1, 4, 4, 3), (9, 6, 2, 10, 7, 4), (300, 2, 1, 16, 24, 1), (300, 2, 2, 16, 8, 270), (70, 4, 1, 24, 16, 0), (20, 3, 1, 8, 8, 1000)])
def test_attention_in_chunks(hip, dt, T, H, G, D, V, chunk):
    sink = rn(4, H)
    sink[0] = 5.0
    args = [(rn(1, T, H * D), dt), (rn(2, T, G * D), dt), (rn(3, T, G * V), dt), (sink, "F32")]
    got, want = both(hip, lambda fb, *a: F.chunk_attention(*a, H, G, chunk, 0.5), args)
    check(got[0], want[0], TOL[dt])


@pytest.mark.parametrize("dt", ["F32", "Bf16"])
@pytest.mark.parametrize("pos,C,chunk", [(0, 8, 8), (7, 8, 8), (8, 8, 8), (1000, 300, 300), (899, 300, 300), (5, 6, 0), (37, 64, 1000)])
def test_attention_over_a_cached_chunk(hip, dt, pos, C, chunk):
    H, G, D, V = 6, 2, 12, 10
    args = [(rn(1, 1, H * D), dt), (rn(2, G, C, D), dt), (rn(3, G, C, V), dt), (rn(4, H), "F32"), (np.array([pos], np.int32), "Si32")]
    n = pos % chunk if chunk else pos
    args[1][0][:, n + 1:] += 9.0
    args[2][0][:, n + 1:] += 90.0   # rows of the chunk that nobody has written yet
    got, want = both(hip, lambda fb, *a: F.chunk_attention_cache(*a, H, chunk, 0.5), args)
    check(got[0], want[0], TOL[dt])


# ------------------------------------------------------------------------------------------ residual updates, soft cap
@pytest.mark.parametrize("fusion", [1, 0])
@pytest.mark.parametrize("mult", [0.35, 1.0])
@pytest.mark.parametrize("rows,n", [(1, 64), (5, 100), (3, 37), (2, 8200), (130, 1024)])
def test_post_norm_add(hip, rows, n, mult, fusion):
    y = rn(2, rows, n) * (10.0 ** np.arange(-3, 2))[np.arange(rows) % 5, None].astype(np.float32)

    def emit(fb, x, y, g):
        r = F.post_norm_add(x, y, g, mult, 1e-4)
        return [r, r.cast("Bf16")]
    got, want = both(hip, emit, [(rn(1, rows, n), "F32"), (y, "F32"), (1 + 0.2 * rn(3, n), "F32")], fusion=fusion)
    check(got[0], want[0], 1e-6)
    check(got[1], want[1], 8e-3)
    assert np.array_equal(U.bf16(got[0]).reshape(rows, n), got[1])


@pytest.mark.parametrize("fusion", [1, 0])
@pytest.mark.parametrize("dt", ["F32", "Bf16"])
@pytest.mark.parametrize("rows,n,scale", [(1, 64, 0.37), (7, 37, 0.37), (40, 3000, 5.0), (3, 64, 1.0)])
def test_scaled_embedding(hip, dt, rows, n, scale, fusion):
    idx = np.random.default_rng(0).integers(0, 19, rows).astype(np.int32)

    def emit(fb, t, i):
        x = F.embedding_lookup(t, i)
        x = x if dt == "F32" else x.cast("F32")
        x = x if scale == 1.0 else x * scale
        return [x, x.cast("Bf16")]
    got, want = both(hip, emit, [(rn(1, 19, n), dt), (idx, "Si32")], fusion=fusion)
    assert np.array_equal(got[0], want[0]) and np.array_equal(got[1], want[1])


@pytest.mark.parametrize("dt", ["F32", "Bf16"])
@pytest.mark.parametrize("M", [1, 3, 16, 17, 130])
@pytest.mark.parametrize("K,N", [(64, 96), (128, 37), (100, 50)])
def test_soft_cap_of_a_linear_layer(hip, dt, M, K, N):
    for fusion in (1, 0):
        got, want = both(hip, lambda fb, x, w: F.softcap(F.linear(x, w, out_dtype="F32"), 2.5), [(rn(1, M, K), dt), (3 * rn(2, K, N) * K ** -0.5, dt)], fusion=fusion)
        check(got[0], want[0], 1e-5 if dt == "F32" else 1e-4, fusion)
        assert np.abs(got[0]).max() <= 2.5 and np.abs(want[0]).max() > 2.4


@pytest.mark.parametrize("K,F_,N", [(64, 96, 40), (256, 1000, 37), (128, 48, 512), (3072, 320, 64), (4608, 64, 4096)])
def test_residual_prologue_of_the_decode_linears(hip, K, F_, N):
    """y1 -> x + m rms(y1) -> gate / up pair -> down -> x' + m rms(y2) -> another layer, and -> rms norm -> capped head; the sums are
    asked for as well, with the persistent launch and without."""
    def emit(fb, x, y, g1, g2, g3, wg, wu, wd, wq, wh):
        x1 = F.post_norm_add(x, y, g1, 0.4, 1e-5)
        h = x1.cast("Bf16")
        y2 = F.linear(F.swiglu(F.linear(h, wg), F.linear(h, wu)), wd, out_dtype="F32")
        x2 = F.post_norm_add(x1, y2, g2, 0.4, 1e-5)
        q = F.linear(x2.cast("Bf16"), wq, out_dtype="F32")
        x3 = F.post_norm_add(x2, F.linear(q.cast("Bf16"), wh, out_dtype="F32"), g1, 1.0, 1e-5)
        n, *_ = F.rms_norm(x3, g3, 1e-5)
        return [F.softcap(F.linear(n.cast("Bf16"), wq, out_dtype="F32"), 4.0), q, x1, x2]
    args = [(rn(1, 1, K), "F32"), (0.01 * rn(2, 1, K), "F32"), (1 + 0.2 * rn(3, K), "F32"), (1 + 0.2 * rn(4, K), "F32"), (1 + 0.2 * rn(5, K), "F32"),
            (rn(6, K, F_) * K ** -0.5, "Bf16"), (rn(7, K, F_) * K ** -0.5, "Bf16"), (rn(8, F_, K) * F_ ** -0.5, "Bf16"), (rn(9, K, N) * K ** -0.5, "Bf16"),
            (rn(10, N, K) * N ** -0.5, "Bf16")]
    prog = build(emit, args)
    want = on_oracle(prog, args)
    for opts in ({}, {"chain": 0}, {"fusion": 0}):
        got = on_device(hip, prog, args, **opts)
        for g, w, tol in zip(got, want, (2e-2, 2e-2, 2e-6, 1e-2)):
            check(g, w, tol, opts)
    first = on_device(hip, prog, args)
    for _ in range(3):
        for a, b in zip(first, on_device(hip, prog, args)):
            assert np.array_equal(a, b)


# ------------------------------------------------------------------------------------------ the whole mixer, single keys
def unrotate(x, pos, rot, base):
    """What the pair rotation at `pos` turns into x[.., D] (f64)."""
    y = np.array(x, np.float64)
    a = np.asarray(pos, np.float64)[:, None] * float(base) ** (-2.0 * np.arange(rot // 2) / max(rot, 1))
    a = a.reshape(a.shape[:1] + (1,) * (x.ndim - 2) + a.shape[1:])
    u, v = y[..., 0:rot:2].copy(), y[..., 1:rot:2].copy()
    y[..., 0:rot:2], y[..., 1:rot:2] = u * np.cos(a) + v * np.sin(a), v * np.cos(a) - u * np.sin(a)
    return y


def projection(seed, pos, H, G, D, V, rot, base, q, k):
    """q | k | v | gate rows whose rotated queries and keys point along q[R, H, D] and k[R, G, D]."""
    R = len(pos)
    p = rn(seed, R, H * D + G * (D + V) + H)
    p[:, :H * D] = unrotate(q, pos, rot, base).reshape(R, -1)
    p[:, H * D:H * D + G * D] = unrotate(k, pos, rot, base).reshape(R, -1)
    return p


def emit_mixer(dt, lens, H, G, D, V, rot, chunk, scale, decode):
    """The calls of a layer between its projections, as the model emits them."""
    B, rows = len(lens), sum(lens)
    cols = [0, H * D, G * D, G * V, H]

    def emit(fb, proj, sink, pos, starts, freqs, *caches):
        qs, ks, vs, gate = (proj.slice([0, sum(cols[:j + 1])], [rows, cols[j + 1]]) for j in range(4))
        table = F.rope_table(pos, freqs) if rot else None
        qs, ks = (F.rope_pairs(t, table, n, 0) if rot else t for t, n in ((qs, H), (ks, G)))
        qs, ks = F.head_rms_norm(qs, H, 1e-5, dt), F.head_rms_norm(ks, G, 1e-5, dt)
        vs = vs if dt == "F32" else vs.cast(dt)
        part = lambda t, b: t if B == 1 else t.slice([sum(lens[:b]), 0], [lens[b], t.dims[1]])
        ctx, new = [], []
        for b in range(B):
            kb, vb, n0 = part(ks, b), part(vs, b), 0 if decode else (lens[b] - 1) // chunk * chunk
            at, n = starts if B == 1 else starts.slice([3 * b], [3]), lens[b] - n0
            slot = [F.dynamic_update_slice_into(c, (t if n0 == 0 else t.slice([n0, 0], [n, t.dims[1]])).reshape([n, G, w]).transpose([1, 0, 2]), at)
                    for t, w, c in ((kb, D, caches[2 * b]), (vb, V, caches[2 * b + 1]))]
            new += slot
            ctx.append(F.chunk_attention_cache(part(qs, b), *slot, sink, pos if B == 1 else pos.slice([b], [1]), H, chunk, scale) if decode
                       else F.chunk_attention(part(qs, b), kb, vb, sink, H, G, chunk, scale))
        return [F.head_gate(ctx[0] if B == 1 else type(ctx[0]).concat(0, ctx), gate, H)] + new
    return emit


def unit(x):
    return x / np.linalg.norm(x, axis=-1, keepdims=True)


# heads, key / value heads, key size, value size, rotated part
SHAPES = [(4, 2, 16, 24, 8), (2, 1, 64, 64, 64), (8, 1, 128, 72, 32), (3, 3, 40, 136, 0), (34, 2, 24, 16, 24), (2, 2, 200, 256, 100), (3, 1, 7, 5, 4)]


@pytest.mark.parametrize("dt", ["F32", "Bf16"])
@pytest.mark.parametrize("shape", SHAPES)
@pytest.mark.parametrize("lens,chunk", [([1], 5), ([2, 64, 65], 64), ([130, 1, 63], 16), ([300], 128), ([257], 100), ([200], 1), ([150, 40], 1000), (list(range(1, 19)), 6)])
def test_prompt_and_single_keys(hip, dt, shape, lens, chunk):
    """Query i's scores with its own key, with its chunk's first key and with one on the way stand out; those with the key before
    the chunk and with the next key would stand out more and must not be seen.  The caches take the last chunk's rows."""
    H, G, D, V, rot = shape
    if len(lens) > 4 and D > 64:
        pytest.skip("a few sizes of many prompts are enough")
    T, cap = sum(lens), min(max(lens) + 3, chunk)
    local = np.concatenate([np.arange(n) for n in lens])
    dirs = unit(rn(9, T, G, D).astype(np.float64))
    q = 0.2 * rn(10, T, H, D).astype(np.float64)
    r0 = 0
    for n in lens:
        for i in range(n):
            lo, own = i // chunk * chunk, np.repeat(dirs[r0 + i], H // G, axis=0)
            at = lambda j: np.repeat(dirs[r0 + j], H // G, axis=0)
            q[r0 + i] += 2 * own + 2 * at(lo) + 2 * at((lo + i) // 2)
            if lo > 0:
                q[r0 + i] += 4 * at(lo - 1)
            if i + 1 < n:
                q[r0 + i] += 4 * at(i + 1)
        r0 += n
    proj = projection(1, local, H, G, D, V, rot, 30.0, q, dirs)
    sink = rn(2, H)
    sink[0] = 6.0   # as much as the keys that stand out
    starts = np.zeros(3 * len(lens), np.int32)
    args = [(proj, "F32"), (sink, "F32"), (local.astype(np.int32), "Si32"), (starts, "Si32"), (F.pair_frequencies(rot, 30.0) if rot else np.zeros(1, np.float32), "F32")]
    for b in range(len(lens)):
        args += [(rn(20 + b, G, cap, D), dt), (rn(40 + b, G, cap, V), dt)]
    prog = build(emit_mixer(dt, lens, H, G, D, V, rot, chunk, 9.0 / D, False), args)
    want = on_oracle(prog, args)
    for fusion in (1, 0):
        got = on_device(hip, prog, args, fusion=fusion)
        check(got[0], want[0], {"F32": 1e-4, "Bf16": 3e-2}[dt], (shape, lens, chunk, fusion))
        for g, w in zip(got[1:], want[1:]):
            check(g, w, TOL[dt], (shape, lens, chunk, fusion, "cache"))


@pytest.mark.parametrize("dt", ["F32", "Bf16"])
@pytest.mark.parametrize("shape", SHAPES)
@pytest.mark.parametrize("pos,cap,chunk", [([0], 4, 9), ([63, 64, 65], 128, 1000), ([127, 128, 255, 0], 128, 128), ([2000, 2047, 2048, 5], 1024, 1024),
                                           ([700, 1, 30], 30, 30), (list(range(90, 108)), 64, 100), ([9], 1, 1)])
def test_decode_of_a_batch_and_single_rows(hip, dt, shape, pos, cap, chunk):
    """One step of sequences at unequal places of their chunks (more than one launch's worth in a case).  A row of the chunk stands
    out, another one each time; rows behind the current place hold what a previous chunk left, which would stand out more."""
    H, G, D, V, rot = shape
    B = len(pos)
    if (cap > 512 and D > 128) or (B > 4 and D > 64):
        pytest.skip("a few sizes of long caches and of many sequences are enough")
    place = np.array([min(p % chunk, cap - 1) for p in pos])
    q = rn(3, B, H, D).astype(np.float64)
    k = 0.5 * rn(4, B, G, D).astype(np.float64)
    kc = [0.3 * rn(60 + b, G, cap, D) for b in range(B)]
    vc = [rn(80 + b, G, cap, V) for b in range(B)]
    lead = unit(q.reshape(B, G, H // G, D)[:, :, 0])
    for b in range(B):
        n = int(place[b])
        j = [0, max(n - 1, 0), n // 2, n][b % 4]
        if j == n:
            k[b] = lead[b]
        kc[b][:, j] = lead[b] * D ** 0.5
        kc[b][:, n + 1:] = 2 * lead[b][:, None] * D ** 0.5
        vc[b][:, n + 1:] += 50.0
    proj = projection(1, np.array(pos), H, G, D, V, rot, 30.0, q, k)
    starts = np.array([v for n in place for v in (0, n, 0)], np.int32)
    sink = rn(2, H)
    sink[0] = 6.0   # as much as the row that stands out
    args = [(proj, "F32"), (sink, "F32"), (np.array(pos, np.int32), "Si32"), (starts, "Si32"), (F.pair_frequencies(rot, 30.0) if rot else np.zeros(1, np.float32), "F32")]
    for b in range(B):
        args += [(kc[b], dt), (vc[b], dt)]
    if any(p % chunk >= cap for p in pos):
        pytest.skip("a place outside the cache")
    prog = build(emit_mixer(dt, [1] * B, H, G, D, V, rot, chunk, 9.0 / D, True), args)
    want = on_oracle(prog, args)
    for fusion in (1, 0):
        got = on_device(hip, prog, args, fusion=fusion)
        check(got[0], want[0], {"F32": 1e-4, "Bf16": 3e-2}[dt], (shape, pos, fusion))
        for g, w in zip(got[1:], want[1:]):
            check(g, w, TOL[dt], (shape, pos, fusion, "cache"))


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
    for cut in (1, 2, 63, 96, 127):   # a prompt of `cut` tokens, the rest one by one; capacities grow and rows are used again on the way
        c = fresh()
        rows = [hip.to_numpy(m.forward_with_decode_cache(toks[:cut], 0, c))]
        stop = min(n, cut + (40 if cut > 2 else 70))
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
    """400 single steps in a fixed capacity (the steps are replayed as one graph): caches are filled over and over, and the eager
    launches say the same."""
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
@pytest.mark.parametrize("name", ["mixed", "tiled"])
def test_fused_and_plain_programs_agree(hip, tmp_path, dt, name):
    m, ref, cfg = load(hip, tmp_path, name, dt)
    toks = tokens(cfg, 40)
    want = ref.forward(toks)[0]
    for opts in ({}, {"fusion": 0}, {"chain": 0}):
        for k, v in opts.items():
            hip.set_option(k, v)
        try:
            c = [None] * m.num_layers
            rows = [hip.to_numpy(m.forward_with_decode_cache(toks[:29], 0, c))]
            rows += [hip.to_numpy(m.forward_with_decode_cache([toks[i]], i, c)) for i in range(29, 40)]
            rms(np.concatenate(rows), want, dt, opts)
        finally:
            for k in opts:
                hip.set_option(k, 1)


def test_inputs_are_kept_unless_donated(hip, tmp_path):
    """Running the same step twice from one set of caches: nothing that was not given away has changed."""
    m, ref, cfg = load(hip, tmp_path, "mixed", "Bf16")
    toks = tokens(cfg, 12)
    c = [None] * m.num_layers
    m.forward_with_decode_cache(toks[:11], 0, c, 16)
    prog, _ = m._build((1,), 16, True)
    args = [m._upload_i32([toks[11]]), m._upload_i32([11])] + m._position_args([11])
    held = [h for s in c for h in (s.keys, s.values)]
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
        for _ in range(40):
            out.append(int(np.argmax(logits[-1])))
            logits, st = ref.forward(out[-1:], st)
        want.append(out)
    assert models.Generator(m, prompts[0]).generate(40) == want[0]
    assert models.Generator(m, prompts[2], pipelined=False).generate(40) == want[2]
    assert models.BatchGenerator(m, prompts).generate(40) == want
    top = models.Generator(m, prompts[1], temperature=0.7, top_k=3, seed=5).generate(8)
    assert len(top) == 8 and all(0 <= t < cfg["vocab"] for t in top)


def test_trace_replay(hip, tmp_path):
    m, ref, cfg = load(hip, tmp_path, "shared", "F32")
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
