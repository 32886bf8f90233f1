"""The Dadupel design on the CPU: the plain implementation against closed forms, and the model driver (programs, caches, loader,
generators) through the oracle backend against the plain implementation."""
import numpy as np
import pytest

import dadupel_util as U
from oracle.dadupel_reference import (Reference, causal_conv_silu, clamped_glu, grouped_rms_norm, latent_attend, rotary_tables, rotate_pairs,
                                      selective_state_scan, silu)
from oracle_backend import OracleBackend
from gptrs_amd import functional as F, loader, models
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
def test_scan_is_the_sum_over_earlier_tokens():
    rng = np.random.default_rng(0)
    T, H, V, N, G = 7, 4, 3, 5, 2
    x, B, C = rng.standard_normal((T, H, V)), rng.standard_normal((T, G, N)), rng.standard_normal((T, G, N))
    dt, a, D, S0 = rng.uniform(0.1, 1, (T, H)), rng.standard_normal(H), rng.standard_normal(H), rng.standard_normal((H, N, V))
    y, S = selective_state_scan(x, B, C, dt, a, D, S0)
    for h in range(H):
        g = h // 2
        lam = np.cumsum(-np.exp(a[h]) * dt[:, h])
        for t in range(T):
            want = np.exp(lam[t]) * (S0[h].T @ C[t, g]) + D[h] * x[t, h]
            for s in range(t + 1):
                want = want + np.exp(lam[t] - lam[s]) * dt[s, h] * (B[s, g] @ C[t, g]) * x[s, h]
            close(y[t, h], want, 1e-12)
    # cut anywhere, the state carries everything
    y1, S1 = selective_state_scan(x[:3], B[:3], C[:3], dt[:3], a, D, S0)
    y2, S2 = selective_state_scan(x[3:], B[3:], C[3:], dt[3:], a, D, S1)
    close(np.concatenate([y1, y2]), y, 1e-12)
    close(S2, S, 1e-12)


def test_convolution_last_tap_meets_the_current_row():
    x = np.zeros((4, 1))
    x[1] = 1.0
    taps = np.array([[4.0, 3.0, 2.0, 1.0]])
    y, st = causal_conv_silu(x, taps, np.zeros(1), np.zeros((3, 1)))
    close(y[:, 0], silu(np.array([0.0, 1.0, 2.0, 3.0])), 1e-12)
    close(st[:, 0], x[1:, 0], 1e-12)


def test_rotation_pairs_and_scaled_frequencies():
    rot = {"dims": 8, "base": 100.0}
    c, s = rotary_tables(rot, [3])
    x = np.arange(1.0, 9.0)[None]
    y = rotate_pairs(x, c, s)
    for i in range(4):
        z = (x[0, 2 * i] + 1j * x[0, 2 * i + 1]) * np.exp(1j * 3 * 100.0 ** (-2 * i / 8))
        close([y[0, 2 * i], y[0, 2 * i + 1]], [z.real, z.imag], 1e-12)
    # many turns inside the original length: unscaled; less than one turn: divided by the factor
    rot["scaling"] = {"factor": 8.0, "original": 60, "fast": 8.0, "slow": 1.0}
    f, mag = F.yarn_pair_frequencies(8, 100.0, 8.0, 60, 8.0, 1.0)
    assert f[0] == 1.0 and abs(f[3] - 100.0 ** (-6 / 8) / 8.0) < 1e-8 and abs(mag - (0.1 * np.log(8.0) + 1)) < 1e-12
    c, s = rotary_tables(rot, [5])
    close(c[0], np.cos(5 * f.astype(np.float64)) * mag, 1e-6)
    close(s[0], np.sin(5 * f.astype(np.float64)) * mag, 1e-6)


def test_absorbed_and_spelled_out_attention_agree():
    rng = np.random.default_rng(3)
    m = {"dim": 6, "vdim": 5, "scale": 0.7}
    H, R, rot, L = 3, 8, 4, 9
    Wuk, Wuv = rng.standard_normal((H * 6, R)), rng.standard_normal((H * 5, R))
    c, kr, qn, qr = rng.standard_normal((L, R)), rng.standard_normal((L, rot)), rng.standard_normal((2, H, 6)), rng.standard_normal((2, H, rot))
    got = latent_attend(qn, qr, c, kr, Wuk, Wuv, m, 7)
    for t in range(2):
        for h in range(H):
            ql = Wuk[h * 6:(h + 1) * 6].T @ qn[t, h]
            s = (c[:8 + t] @ ql + kr[:8 + t] @ qr[t, h]) * 0.7
            w = np.exp(s) / np.exp(s).sum()
            close(got[t, h * 5:(h + 1) * 5], Wuv[h * 5:(h + 1) * 5] @ (w @ c[:8 + t]), 1e-12)


def test_clamped_unit_and_grouped_norm():
    g, u = np.array([-9.0, 0.5, 3.0, 9.0]), np.array([5.0, -5.0, 0.5, 2.0])
    gc, uc = np.array([-9.0, 0.5, 2.0, 2.0]), np.array([2.0, -2.0, 0.5, 2.0])
    close(clamped_glu(g, u, 2.0), gc / (1 + np.exp(-1.702 * gc)) * (uc + 1), 1e-12)
    x = np.array([[3.0, 4.0, 30.0, 40.0]])
    close(grouped_rms_norm(x, np.ones(4), 2, 0.0), np.array([[3, 4, 3, 4]]) / np.sqrt(12.5), 1e-12)


# ------------------------------------------------------------------------------------------ the driver
@pytest.mark.parametrize("name", sorted(U.STACKS))
def test_prompt_then_decode_on_the_oracle(tmp_path, name):
    m, ref, cfg = load(tmp_path, name)
    toks = tokens(cfg, 21)
    want, _ = ref.forward(toks)
    caches = [None] * m.num_layers
    be = m.backend
    close(be.to_numpy(m.forward_with_decode_cache(toks[:13], 0, caches)), want[:13])
    for i in range(13, 21):   # the cache grows from 16 to 32 rows on the way
        close(be.to_numpy(m.forward_with_decode_cache([toks[i]], i, caches)), want[i:i + 1])


@pytest.mark.parametrize("name", ["mixed", "deep_share"])
def test_unequal_batch_equals_each_alone(tmp_path, name):
    m, ref, cfg = load(tmp_path, name)
    be, seqs = m.backend, [tokens(cfg, n, s) for s, n in enumerate((1, 9, 4))]
    more = [tokens(cfg, 3, 10 + s) for s in range(3)]
    want = [ref.forward(a + b)[0] for a, b in zip(seqs, more)]
    caches = [[None] * m.num_layers for _ in seqs]
    got = be.to_numpy(m.forward_batch(seqs, 0, caches))
    close(got, np.concatenate([w[:len(a)] for w, a in zip(want, seqs)]))
    live = [0, 1, 2]
    for step in range(3):
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


def test_generators_write_the_plain_greedy_tokens(tmp_path):
    m, ref, cfg = load(tmp_path, "mixed")
    prompts = [tokens(cfg, n, s) for s, n in ((1, 6), (2, 3))]
    want = []
    for p in prompts:
        t = list(p)
        for _ in range(7):
            t.append(int(np.argmax(ref.forward(t)[0][-1])))
        want.append(t[len(p):])
    assert models.Generator(m, prompts[0]).generate(7) == want[0]
    assert models.BatchGenerator(m, prompts).generate(7) == want
    # a window shorter than the sequence slides, as it does for the other models
    short, _, _ = load(tmp_path, "mixed", context_length=8)
    got = models.Generator(short, prompts[0]).generate(7)
    t = list(prompts[0])
    state, logits, n = None, None, 0
    logits, state = ref.forward(t)
    n = len(t)
    for _ in range(7):
        t.append(int(np.argmax(logits[-1])))
        if n >= 8:
            logits, state = ref.forward(t[len(t) - 8:])
            n = 8
        else:
            logits, state = ref.forward(t[-1:], state)
            n += 1
    assert got == t[len(prompts[0]):]


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
    with pytest.raises(CheckpointError, match="architecture"):
        loader.load_model(OracleBackend(), U.write_folder(str(tmp_path / "a"), dict(cfg, architecture="Nobody"), W))
    with pytest.raises(CheckpointError, match="not found"):
        loader.load_model(OracleBackend(), U.write_folder(str(tmp_path / "b"), cfg, {k: v for k, v in W.items() if k != "l0.ls1"}))
    with pytest.raises(CheckpointError, match="shape"):
        loader.load_model(OracleBackend(), U.write_folder(str(tmp_path / "c"), cfg, dict(W, **{"l0.ls1": W["l0.ls1"][:-1]})))
    p = U.write_folder(str(tmp_path / "d"), cfg, W)
    with open(p + "/model.safetensors", "r+b") as f:
        f.truncate(4000)
    with pytest.raises(CheckpointError):
        loader.load_model(OracleBackend(), p)
    for L in (U.ssm(heads=4, groups=3), U.ssm(norm_groups=5), U.latent(kv_from=3)):
        with pytest.raises(ValueError):
            models.Dadupel(models.Dadupel.config_from_json(U.config([L])), OracleBackend(), "F32")
    with pytest.raises(ValueError):   # a shared cache of other sizes
        models.Dadupel(models.Dadupel.config_from_json(U.config([U.latent(), U.latent(kv_rank=16, kv_from=0)])), OracleBackend(), "F32")


def test_checkpoint_round_trip_and_streaming(tmp_path):
    m, ref, cfg = load(tmp_path, "mixed")
    toks = tokens(cfg, 9)
    want, _ = ref.forward(toks)
    p = str(tmp_path / "m.gptrs")
    m.save_checkpoint(p, "dadupel", m.checkpoint_config())
    again = loader.load_model(OracleBackend(), p, dtype="F32")
    assert models.Dadupel.config_from_json(m.checkpoint_config()).layers == again.config.layers
    close(again.backend.to_numpy(again.forward_with_decode_cache(toks, 0, [None] * again.num_layers)), want)
    m.save_checkpoint(p, "dadupel", m.checkpoint_config(), runtime={"weight_streaming": {"enabled": True, "device_budget_bytes": 4096}})
    lazy = loader.load_model(OracleBackend(), p, dtype="F32")
    close(lazy.backend.to_numpy(lazy.forward_with_decode_cache(toks, 0, [None] * lazy.num_layers)), want)


def test_random_model_has_the_declared_shapes():
    cfg = models.Dadupel.config_from_json(U.STACKS["tiled"])
    m = models.Dadupel.random(cfg, OracleBackend(), seed=3)
    assert {n: tuple(m.param_specs[n].dims) for n in m.param_names} == {n: tuple(d) for n, d in m.expected_params().items()}
    assert m.param_specs["blocks.1.mixer.conv"].dtype == "F32" and m.param_specs["blocks.0.mixer.w_uk"].dtype == "Bf16"
    out = m.backend.to_numpy(m.forward_with_decode_cache([1, 2, 3], 0, [None] * m.num_layers))
    assert np.all(np.isfinite(out)) and np.std(out) > 0.1


@pytest.mark.parametrize("decode", [True, False])
def test_a_layer_is_a_handful_of_fused_steps(tmp_path, decode):
    """What the backend's fusion pass leaves of a three-sequence program (no device needed)."""
    from gptrs_amd import backend, front_end as FE
    m, _, _ = load(tmp_path, "tiled", dtype="Bf16")
    prog, lay = m._build((1, 1, 1) if decode else (20, 33, 40), 64, decode, True)
    n = lay["n_args"]
    roles = [FE.ARG] * n + [FE.PARAM] * len(m.param_names)
    ids = [None] * n + [int.from_bytes(models.param_id(m.namespace, x), "little") for x in m.param_names]
    opt = FE.optimize(prog, roles, ids, m.backend, m.backend.param_resolver())
    rep = backend.fusion_report(opt.program, [p.type["Tensor"]["shape"]["dims"][-1]["Static"] if s is None else 0 for p, s in zip(opt.inputs, opt.source_index)])
    assert rep.count("fused.ssm_mixer") == 1 and not any(r.startswith("mixer.") and r not in ("mixer.rope_table.v1", "mixer.latent_rows.v1") for r in rep)
    assert rep.count("fused.latent_decode" if decode else "fused.latent_prefill") == 2
    assert sum("clamped_glu" in r for r in rep) == 3 and sum("colscale+residual" in r for r in rep) == 6
    if decode:
        assert sum("layer_norm" in r for r in rep) == 3 * 2 + 1 + 1 and "mixer.latent_rows.v1" not in rep and "DynamicUpdateSlice" not in rep
