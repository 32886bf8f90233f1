"""The Fuzazen design on the CPU: the plain implementation against closed forms, and the model driver (programs, caches, loader,
generators) through the oracle backend against the plain implementation."""
import numpy as np
import pytest

import fuzazen_util as U
from oracle.fuzazen_reference import Reference, chunk_attend, over_rms, post_norm_add, rotate_leading_pairs, sink_softmax, softcap
from oracle_backend import OracleBackend
from gptrs_amd import loader, models
from gptrs_amd.checkpoint import CheckpointError

RTOL = 2e-4


def close(got, want, tol=RTOL):
    got, want = np.asarray(got, np.float64), np.asarray(want, np.float64)
    assert got.shape == want.shape
    err = np.max(np.abs(got - want)) / (np.max(np.abs(want)) + 1e-30)
    assert err < tol, err


def load(tmp_path, name, dtype="F32", seed=0, backend=None, **kw):
    cfg = U.STACKS[name]
    W = U.weights(cfg, seed)
    path = U.write_folder(str(tmp_path / name), cfg, W)
    return loader.load_model(backend or OracleBackend(), path, dtype=dtype, **kw), Reference(cfg, W), cfg


def tokens(cfg, n, seed=1):
    return np.random.default_rng(seed).integers(0, cfg["vocab"], n).tolist()


# ------------------------------------------------------------------------------------------ the plain implementation
def test_chunks_are_blocks_of_the_causal_mask():
    rng = np.random.default_rng(0)
    T, H, G, D, V, chunk = 11, 4, 2, 6, 5, 4
    q, k, v, sink = rng.standard_normal((T, H, D)), rng.standard_normal((T, G, D)), rng.standard_normal((T, G, V)), rng.standard_normal(H)
    got = chunk_attend(q, k, v, sink, 0.7, chunk, 0)
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    seen = (j <= i) & (i // chunk == j // chunk)
    for h in range(H):
        s = np.where(seen, q[:, h] @ k[:, h // 2].T * 0.7, -np.inf)
        e = np.exp(s)
        close(got[:, h], e @ v[:, h // 2] / (e.sum(axis=1, keepdims=True) + np.exp(sink[h])), 1e-12)
    # a later start sees the same keys
    close(chunk_attend(q[7:], k, v, sink, 0.7, chunk, 7), got[7:], 1e-12)


def test_sink_counts_once_and_unscaled():
    w = sink_softmax(np.array([0.0, 0.0]), np.log(2.0))
    close(w, [0.25, 0.25], 1e-12)
    assert sink_softmax(np.array([3.0]), 800.0)[0] < 1e-300 and np.isfinite(sink_softmax(np.array([900.0, 3.0]), -5.0)).all()


def test_rotation_turns_leading_pairs_only():
    x = np.arange(1.0, 8.0)[None, None]          # seven values: three leading pairs could turn, two do
    y = rotate_leading_pairs(x, [3], 4, 100.0)
    for i in range(2):
        z = (x[0, 0, 2 * i] + 1j * x[0, 0, 2 * i + 1]) * np.exp(1j * 3 * 100.0 ** (-2 * i / 4))
        close([y[0, 0, 2 * i], y[0, 0, 2 * i + 1]], [z.real, z.imag], 1e-12)
    assert np.array_equal(y[..., 4:], x[..., 4:])


def test_row_functions():
    x = np.array([[3.0, 4.0]])
    close(over_rms(x, 0.0), x / np.sqrt(12.5), 1e-12)
    close(over_rms(x, 12.5), x / 5.0, 1e-12)     # eps inside the root
    close(post_norm_add(np.array([[1.0, 1.0]]), x, np.array([2.0, 1.0]), 0.5, 0.0), 1 + 0.5 * np.array([[6.0, 4.0]]) / np.sqrt(12.5), 1e-12)
    close(softcap(np.array([0.01, 1e6, -1e6]), 5.0), [5 * np.tanh(0.002), 5.0, -5.0], 1e-12)


@pytest.mark.parametrize("name", sorted(U.STACKS))
def test_plain_decoding_equals_the_prompt(name):
    cfg = U.STACKS[name]
    ref = Reference(cfg, U.weights(cfg))
    toks = tokens(cfg, 23)
    want, _ = ref.forward(toks)
    st, rows = None, []
    for cut in (toks[:2], toks[2:7], toks[7:8], toks[8:10], toks[10:]):
        r, st = ref.forward(cut, st)
        rows.append(r)
    close(np.concatenate(rows), want, 1e-10)


# ------------------------------------------------------------------------------------------ the driver
@pytest.mark.parametrize("name", sorted(U.STACKS))
def test_prompt_then_decode_on_the_oracle(tmp_path, name):
    m, ref, cfg = load(tmp_path, name)
    toks = tokens(cfg, 27)
    want, _ = ref.forward(toks)
    be = m.backend
    for cut in (1, 7, 13):   # cuts inside, at and behind chunks' edges; caches grow, and rows are used again
        caches = [None] * m.num_layers
        close(be.to_numpy(m.forward_with_decode_cache(toks[:cut], 0, caches)), want[:cut])
        for i in range(cut, 27):
            close(be.to_numpy(m.forward_with_decode_cache([toks[i]], i, caches)), want[i:i + 1])
        for L, slot in zip(cfg["layers"], caches):
            assert slot.capacity == min(32, L["mixer"]["mask"]["size"]) and slot.len == 27


@pytest.mark.parametrize("name", ["mixed", "shared"])
def test_unequal_batch_equals_each_alone(tmp_path, name):
    m, ref, cfg = load(tmp_path, name)
    be, seqs = m.backend, [tokens(cfg, n, s) for s, n in enumerate((1, 15, 4))]
    more = [tokens(cfg, 5, 10 + s) for s in range(3)]
    want = [ref.forward(a + b)[0] for a, b in zip(seqs, more)]
    caches = [[None] * m.num_layers for _ in seqs]
    got = be.to_numpy(m.forward_batch(seqs, 0, caches))
    close(got, np.concatenate([w[:len(a)] for w, a in zip(want, seqs)]))
    live = [0, 1, 2]
    for step in range(5):
        if step == 2:
            live = [0, 2]   # one request has ended
        got = be.to_numpy(m.forward_batch([[more[b][step]] for b in live], [len(seqs[b]) + step for b in live], [caches[b] for b in live]))
        close(got, np.stack([want[b][len(seqs[b]) + step] for b in live]))


def test_rows_whose_logits_are_wanted(tmp_path):
    m, ref, cfg = load(tmp_path, "mixed")
    seqs = [tokens(cfg, 5, 1), tokens(cfg, 8, 2)]
    want = np.concatenate([ref.forward(s)[0] for s in seqs])
    run = lambda **kw: m.backend.to_numpy(m.forward_batch(seqs, 0, [[None] * m.num_layers for _ in seqs], **kw))
    close(run(logit_rows=[0, 7, 12]), want[[0, 7, 12]])
    close(run(last_logits_only=True), want[[4, 12]])
    close(run(logit_rows=list(range(13))), want)


def test_generators_write_the_plain_greedy_tokens(tmp_path):
    m, ref, cfg = load(tmp_path, "mixed")
    prompts = [tokens(cfg, n, s) for s, n in ((1, 6), (2, 3))]
    want = []
    for p in prompts:
        t = list(p)
        for _ in range(9):
            t.append(int(np.argmax(ref.forward(t)[0][-1])))
        want.append(t[len(p):])
    assert models.Generator(m, prompts[0]).generate(9) == want[0]
    assert models.BatchGenerator(m, prompts).generate(9) == want


def test_calls_that_make_no_sense_are_refused(tmp_path):
    m, _, cfg = load(tmp_path, "mixed", context_length=16)
    fresh = lambda: [None] * m.num_layers
    c = fresh()
    m.forward_with_decode_cache([1, 2], 0, c)
    for bad in (lambda: m.forward_batch([[1], [2]], [2, 0], [c, fresh()]),             # a batch that starts and goes on
                lambda: m.forward_with_decode_cache([1, 2], 2, c),                     # two tokens on a cache
                lambda: m.forward_with_decode_cache([1], 3, c),                        # a position that is not the next
                lambda: m.forward_with_decode_cache([1], 5, fresh()),                  # a start that is not the first
                lambda: m.forward_with_decode_cache([cfg["vocab"]], 2, c),
                lambda: m.forward_with_decode_cache([1] * 17, 0, fresh()),
                lambda: m.forward_with_decode_cache([], 0, fresh())):
        with pytest.raises(ValueError):
            bad()


# ------------------------------------------------------------------------------------------ files
def test_model_folder_errors(tmp_path):
    cfg = U.STACKS["mixed"]
    W = U.weights(cfg)
    with pytest.raises(CheckpointError, match="not found"):
        loader.load_model(OracleBackend(), U.write_folder(str(tmp_path / "b"), cfg, {k: v for k, v in W.items() if k != "l0.mix.v"}))
    with pytest.raises(CheckpointError, match="shape"):
        loader.load_model(OracleBackend(), U.write_folder(str(tmp_path / "c"), cfg, dict(W, **{"l0.mix.v": W["l0.mix.v"][:-1]})))
    with pytest.raises(CheckpointError, match="stacked"):
        loader.load_model(OracleBackend(), U.write_folder(str(tmp_path / "d"), cfg, dict(W, **{"l0.mix.v": W["l0.mix.v"][:, :-1]})))
    base = U.layer()
    for layers in ([U.layer(heads=4, kv_heads=3)], [U.layer(rot=18)], [U.layer(rot=5)], [U.layer(chunk=0)],
                   [U.layer(weights_of=0)], [base, U.layer(weights_of=5)], [base, U.layer(weights_of=2), U.layer(weights_of=1)],   # nobody owns the weights
                   [base, U.layer(chunk=9, weights_of=0)], [base, U.layer(ff=None, weights_of=0)]):                               # other sizes than the owner's
        with pytest.raises(ValueError):
            models.Fuzazen(models.Fuzazen.config_from_json(U.config(layers)), OracleBackend(), "F32")
    with pytest.raises(ValueError, match="layer type"):
        models.Fuzazen.config_from_json(U.config([dict(base, type="convolution")]))


def test_checkpoint_round_trip_and_streaming(tmp_path):
    m, ref, cfg = load(tmp_path, "shared")
    toks = tokens(cfg, 19)
    want, _ = ref.forward(toks)
    p = str(tmp_path / "m.gptrs")
    m.save_checkpoint(p, "fuzazen", m.checkpoint_config())
    again = loader.load_model(OracleBackend(), p, dtype="F32")
    assert again.config == m.config
    close(again.backend.to_numpy(again.forward_with_decode_cache(toks, 0, [None] * again.num_layers)), want)
    m.save_checkpoint(p, "fuzazen", m.checkpoint_config(), runtime={"weight_streaming": {"enabled": True, "device_budget_bytes": 4096}})
    lazy = loader.load_model(OracleBackend(), p, dtype="F32")
    close(lazy.backend.to_numpy(lazy.forward_with_decode_cache(toks, 0, [None] * lazy.num_layers)), want)


def test_random_model_has_the_declared_shapes():
    cfg = models.Fuzazen.config_from_json(U.STACKS["tiled"])
    m = models.Fuzazen.random(cfg, OracleBackend(), seed=3)
    assert {n: tuple(m.param_specs[n].dims) for n in m.param_names} == {n: tuple(d) for n, d in m.expected_params().items()}
    assert m.param_specs["blocks.1.mixer.sink"].dtype == "F32" and m.param_specs["blocks.0.mixer.w_qkvg"].dtype == "Bf16"
    assert not any(n.startswith("blocks.2.") for n in m.param_names)   # it has no weights of its own
    out = m.backend.to_numpy(m.forward_with_decode_cache([1, 2, 3], 0, [None] * m.num_layers))
    assert np.all(np.isfinite(out)) and np.std(out) > 0.1


@pytest.mark.parametrize("dtype", ["Bf16", "F32"])
@pytest.mark.parametrize("lens,decode", [((1,), True), ((1, 1, 1), True), ((20, 33, 40), False), ((97,), False)])
def test_a_layer_is_a_handful_of_fused_steps(tmp_path, lens, decode, dtype):
    """What the backend's fusion pass leaves of a program (no device needed)."""
    from gptrs_amd import backend, front_end as FE
    m, _, _ = load(tmp_path, "tiled", dtype=dtype)
    prog, lay = m._build(lens, 128, decode, True)
    n = lay["n_args"]
    roles = [FE.ARG] * n + [FE.PARAM] * len(m.param_names)
    ids = [None] * n + [int.from_bytes(models.param_id(m.namespace, x), "little") for x in m.param_names]
    opt = FE.optimize(prog, roles, ids, m.backend, m.backend.param_resolver())
    rep = backend.fusion_report(opt.program, [p.type["Tensor"]["shape"]["dims"][-1]["Static"] if s is None else 0 for p, s in zip(opt.inputs, opt.source_index)])
    assert rep.count("fused.chunk_decode" if decode else "fused.chunk_prefill") == 3
    assert not any(r.startswith("mixer.") and r != "mixer.rope_table.v1" for r in rep) and not any(r in rep for r in ("DynamicUpdateSlice", "CustomCall", "ElementwiseUnary"))
    assert sum("softcap" in r for r in rep) == 1
    if dtype == "Bf16":
        assert sum("swiglu" in r for r in rep) == 3
        # one row: every residual update is some layer's prologue; more rows: an instruction that leaves the bf16 copy as well
        assert sum("+post_norm_add" in r for r in rep) == (6 if lens == (1,) else 0) and rep.count("fused.post_norm_add") == (0 if lens == (1,) else 6)
        assert rep.count("fused.embed_rows") == 1 and "Cast" not in rep
