"""GPT-2 and Ministral model drivers and the greedy Generator, generic over a backend.

Host-side mirror of crates/gpt-rs/src/model/{gpt,ministral}.rs, nn/layers/*.rs and
inference/{generate,sampler}.rs: each forward call captures the whole model into ONE
PTIR program (as the reference's lazy GraphArena does, ops/graph/arena.rs:340-375),
caches it by shape (plan cache, ops/graph/plan.rs:20-29) and hands it to
`backend.run_program`.  Weights are program inputs fed from the backend's parameter
memo; per-step scalars (token ids, positions, update_starts, query_start, RoPE rows)
are tiny uploads, exactly the reference's calling convention.

`backend` is any object with the PortableBackend surface (spec.rs:1287-1349):
materialize / to_literal / run_program / param_resolver / sample_decode_token.
"""
from __future__ import annotations

import itertools
import os
from dataclasses import dataclass
from typing import Dict, List, Optional, Sequence, Tuple

import numpy as np

from . import functional as F
from .blake3 import blake3
from .ptir import FunctionBuilder, Program, Tensor, TensorSpec, bf16_bits_to_f32, f32_to_bf16_bits


def decode_cache_capacity(required_len: int, max_len: int) -> int:
    """model/gpt.rs:940-943: next power of two, capped at the context length."""
    bucket = 1
    while bucket < max(required_len, 1):
        bucket *= 2
    return min(bucket, max_len)


@dataclass
class DecodeKvCache:
    """ops/functional/attention.rs:100-126: fixed-capacity [Hkv, capacity, Dh] + active len."""

    keys: object
    values: object
    len: int
    capacity: int


@dataclass
class DecodeLatentCache:
    """One row [latent | rotated key part] per position, shared by all heads: [1, capacity, rank + rot]."""

    rows: object
    len: int
    capacity: int


@dataclass
class DecodeSsmState:
    """What a state-space layer carries from token to token: the convolution's last inputs f32 [taps - 1, channels] and the
    recurrent state f32 [heads, N, vdim].  Its size does not depend on the position."""

    conv: object
    state: object
    len: int


@dataclass
class SharedLayerCache:
    """A layer that reads the cache of layer `layer` and holds nothing itself."""

    layer: int
    len: int


def _np_to_bytes(arr: np.ndarray, dtype: str) -> bytes:
    if dtype == "Bf16":
        return f32_to_bf16_bits(np.asarray(arr, np.float32)).astype("<u2").tobytes()
    if dtype == "F32":
        return np.ascontiguousarray(arr, dtype="<f4").tobytes()
    if dtype == "Si32":
        return np.ascontiguousarray(arr, dtype="<i4").tobytes()
    raise ValueError(dtype)


def base_param_id(name: str) -> int:
    """crates/gpt-rs/src/params.rs:29-37: the first 16 bytes of blake3(name) as a little-endian u128."""
    if not name.isascii():
        raise ValueError(f"param name must be ASCII, got '{name}'")
    return int.from_bytes(blake3(name.encode("ascii"))[:16], "little")


def namespace_id(namespace: str) -> int:
    """The u128 a model instance is bound under.  The reference takes it from the model handle that `load_model` hands
    out (runtime/loader.rs: a counter per loaded model); here it is derived from the instance's label the same way a
    base id is derived from a name."""
    return int.from_bytes(blake3(b"gpt-rs:model-namespace:" + namespace.encode())[:16], "little")


def param_id(namespace: str, name: str) -> bytes:
    """Stable 16-byte parameter key, the reference's derivation (crates/gpt-rs/src/params.rs:39-48): the first 16 bytes of
    blake3("gpt-rs:param-key:v1" || namespace u128 LE || base id u128 LE), which read as a little-endian u128 are
    `ParamKey`; the memo of the C ABI is keyed by those 16 bytes."""
    msg = b"gpt-rs:param-key:v1" + namespace_id(namespace).to_bytes(16, "little") + base_param_id(name).to_bytes(16, "little")
    return blake3(msg)[:16]


class _ModelBase:
    """Shared plumbing: parameter registration, program cache, tiny uploads."""

    namespace = "model"

    _instances = itertools.count()

    def __init__(self, backend, dtype: str):
        self.backend = backend
        self.dtype = dtype
        # one memo namespace per model instance (the reference namespaces by model handle)
        self.namespace = f"{type(self).namespace}#{next(_ModelBase._instances)}"
        self.param_names: List[str] = []
        self.param_specs: Dict[str, TensorSpec] = {}
        self._programs: Dict[tuple, Tuple[Program, dict]] = {}
        self._param_handles: Optional[list] = None
        self._source = None                 # loader.CheckpointParamSource of a model opened by loader.load_model
        self._base_ids: Dict[str, int] = {}
        self._lazy = False                  # weight streaming: parameters are resolved through the source at every run
        # programs go through the reference's optimizer pipeline (front_end.py) before the backend sees them; False hands
        # the backend the emitters' instruction stream as it is captured
        self.front_end = True
        # with the front end on: also run the hip backend's own pipeline passes (front_end.hip_backend_pipeline: norms
        # become CustomCalls ahead of the parameter-only fold), the second route through the reference's optimizer
        self.backend_pipeline = False
        self._optimized: Dict[int, tuple] = {}

    # -- parameters ------------------------------------------------------------------
    def param_dtype(self, name: str) -> str:
        """Storage dtype of the parameter `name`."""
        return self.dtype

    def bind_param_source(self, source, base_ids: Dict[str, int], specs: Dict[str, TensorSpec], lazy: bool):
        """runtime/loader.rs:264-297: parameters come from `source` by base id.  Not lazy: each is loaded once and
        stored in the backend's memo under its stable id; lazy (`runtime.weight_streaming.enabled`): nothing is
        loaded here, every run asks the memo and then the source (`DeviceTensor::lazy_param`)."""
        self._source, self._lazy = source, bool(lazy)
        for name, spec in specs.items():
            if name not in self.param_specs:
                self.param_names.append(name)
            self.param_specs[name] = spec
            self._base_ids[name] = base_ids[name]
            if not lazy:
                self.backend.param_resolver().set(param_id(self.namespace, name), source.load(base_ids[name]))
        self._param_handles = None
        self._optimized.clear()

    def set_param(self, name: str, array: np.ndarray, dtype: Optional[str] = None):
        """runtime/loader.rs:234-239: materialize once, store under the stable id."""
        dtype = dtype or self.dtype
        spec = TensorSpec(dtype, array.shape)
        handle = self.backend.materialize(spec, _np_to_bytes(array, dtype))
        self.backend.param_resolver().set(param_id(self.namespace, name), handle)
        if name not in self.param_specs:
            self.param_names.append(name)
        self.param_specs[name] = spec
        self._param_handles = None
        self._optimized.clear()

    def set_param_bytes(self, name: str, spec: TensorSpec, data: bytes):
        handle = self.backend.materialize(spec, data)
        self.backend.param_resolver().set(param_id(self.namespace, name), handle)
        if name not in self.param_specs:
            self.param_names.append(name)
        self.param_specs[name] = spec
        self._param_handles = None
        self._optimized.clear()

    def set_param_handle(self, name: str, handle):
        """Register a tensor that already lives on the device."""
        self.backend.param_resolver().set(param_id(self.namespace, name), handle)
        if name not in self.param_specs:
            self.param_names.append(name)
        self.param_specs[name] = handle.spec
        self._param_handles = None
        self._optimized.clear()
        self._programs.clear()

    def drop_param(self, name: str):
        """Forget a parameter and release its device memory (the memo keeps a 1-element stand-in)."""
        spec = self.param_specs.pop(name)
        self.param_names.remove(name)
        stub = self.backend.materialize(TensorSpec(spec.dtype, [1]), None)
        self.backend.param_resolver().set(param_id(self.namespace, name), stub)
        self._param_handles = None
        self._optimized.clear()
        self._programs.clear()

    _quant_programs: Dict[tuple, Program] = {}

    def quantize_param(self, name: str, scheme: str):
        """Replace the matrix `name` by `name.q` (codes) and `name.s` (scales), quantised on the device
        (functional.quantize_weight); layers that find `name.q` read the codes directly."""
        spec = self.param_specs[name]
        key = (scheme, spec.dtype, tuple(spec.dims))
        prog = _ModelBase._quant_programs.get(key)
        if prog is None:
            fb = FunctionBuilder("main", spec.dtype)
            q, s = F.quantize_weight(fb.param(spec.dtype, spec.dims), scheme)
            fb.set_results([q, s])
            prog = _ModelBase._quant_programs[key] = Program(fb)
        q, s = self.backend.run_program(prog, [self.param_handle(name)])
        self.drop_param(name)
        self.set_param_handle(name + ".q", q)
        self.set_param_handle(name + ".s", s)

    # -- checkpoints -----------------------------------------------------------------
    def _load_tensors(self, ck, expected: Dict[str, tuple], dtype: Optional[str] = None):
        """Upload every expected tensor from an open checkpoint (checkpoint/loader.rs: by name, shape checked),
        one at a time out of the file mapping; `dtype` overrides the model's storage dtype."""
        from .checkpoint import CheckpointError
        for name, dims in expected.items():
            e = ck.entry(name)
            if tuple(e.dims) != tuple(dims):
                raise CheckpointError(f"tensor `{name}` has shape {list(e.dims)}, the model expects {list(dims)}")
            arr = ck.array(name)
            if e.dtype == "F32":
                host = np.asarray(arr, np.float32)
            elif e.dtype == "Bf16":
                host = bf16_bits_to_f32(np.asarray(arr))
            else:
                raise CheckpointError(f"tensor `{name}`: dtype {e.dtype} cannot feed a model parameter")
            self.set_param(name, host, dtype)

    def save_checkpoint(self, path: str, kind: str, config: Dict[str, object], runtime: Optional[Dict[str, object]] = None):
        """Write the parameters back as a GPTRSCHK v2 file (checkpoint/saver.rs), in their storage dtype."""
        from .checkpoint import write_checkpoint
        tensors, dtypes = {}, {}
        for name in self.param_names:
            spec = self.param_specs[name]
            if spec.dtype not in ("F32", "Bf16"):
                raise ValueError(f"parameter {name} of dtype {spec.dtype} has no checkpoint representation")
            raw = self.backend.to_literal(self.param_handle(name))
            if spec.dtype == "F32":
                tensors[name] = np.frombuffer(raw, "<f4").reshape(spec.dims)
            else:
                tensors[name] = np.frombuffer(raw, "<u2").reshape(spec.dims)
                dtypes[name] = "Bf16"
        write_checkpoint(path, kind, config, tensors, dtypes, runtime=runtime)

    def param_handle(self, name: str):
        h = self.backend.param_resolver().get(param_id(self.namespace, name))
        if h is None and self._source is not None and name in self._base_ids:
            h = self._source.load(self._base_ids[name])
        if h is None:
            raise KeyError(f"parameter {name} not materialized")
        return h

    def _declare_params(self, fb: FunctionBuilder) -> Dict[str, Tensor]:
        return {n: fb.param(self.param_specs[n].dtype, self.param_specs[n].dims) for n in self.param_names}

    def _upload_i32(self, values: Sequence[int]):
        arr = np.asarray(values, dtype=np.int32)
        return self.backend.materialize(TensorSpec("Si32", arr.shape), arr.tobytes())

    def _zeros(self, dims, dtype: Optional[str] = None):
        return self.backend.materialize(TensorSpec(dtype or self.dtype, dims), None)

    def _grow_rows(self, handle, dims, capacity: int):
        """A cache tensor of shape `dims` = [heads, old capacity, width] copied into a zero tensor of `capacity` rows
        (model/gpt.rs:626-657)."""
        heads, old_cap, width = dims
        key = ("grow", heads, old_cap, width, capacity)
        if key not in self._programs:
            fb = FunctionBuilder("main", self.dtype)
            base = fb.param(self.dtype, [heads, capacity, width])
            old = fb.param(self.dtype, [heads, old_cap, width])
            st = fb.param("Si32", [3])
            fb.set_results([F.dynamic_update_slice_into(base, old, st)])
            self._programs[key] = (Program(fb), {})
        return self.backend.run_program(self._programs[key][0], [self._zeros([heads, capacity, width]), handle, self._upload_i32([0, 0, 0])],
                                        [True, False, False])[0]

    def _run(self, program: Program, args: list, donate: Optional[list] = None):
        if self.front_end:
            return self._run_optimized(program, args, donate)
        if self._lazy:                    # streamed weights: resolved anew for every run, kept only by the source's cache
            params = [self.param_handle(n) for n in self.param_names]
        else:
            if self._param_handles is None:   # Param inputs are fed by stable id (arena.rs:1163-1168)
                self._param_handles = [self.param_handle(n) for n in self.param_names]
            params = self._param_handles
        don = None
        if donate is not None:
            don = list(donate) + [False] * len(params)
        return self.backend.run_program(program, list(args) + params, don)

    def _run_optimized(self, program: Program, args: list, donate: Optional[list] = None):
        """The reference's path from a captured graph to the backend: the program goes through the optimizer once
        (front_end.optimize: canonicalisers, parameter-only folds executed through the backend and stored in its memo
        under derived ids, CSE, DCE; ops/graph/arena.rs:744-922), the optimised program and its input roles are kept
        with the plan, and every run feeds Args positionally and Params by stable id (arena.rs:1116-1170)."""
        from . import front_end as FE
        n_args, names = len(args), self.param_names
        entry = self._optimized.get(program.key)
        if entry is None or entry[2] != tuple(names) or entry[3] != self.backend_pipeline:
            roles = [FE.ARG] * n_args + [FE.PARAM] * len(names)
            stable = [None] * n_args + [int.from_bytes(param_id(self.namespace, n), "little") for n in names]
            hooks = FE.hip_backend_pipeline() if self.backend_pipeline else {}
            opt = FE.optimize(program, roles, stable, self.backend, self.backend.param_resolver(), **hooks)
            entry = self._optimized[program.key] = (opt, {}, tuple(names), self.backend_pipeline)
        opt, held = entry[0], entry[1]
        inputs, don = [], []
        resolver = self.backend.param_resolver()
        for pos, (p, src) in enumerate(zip(opt.inputs, opt.source_index)):
            if p.role == FE.ARG:
                inputs.append(args[src])
                don.append(bool(donate[src]) if donate is not None else False)
                continue
            h = None if self._lazy and src is not None else held.get(pos)
            if h is None:
                if src is not None:
                    h = self.param_handle(names[src - n_args])
                else:
                    h = resolver.get(FE.stable_id_bytes(p.stable_id))
                    if h is None:
                        raise KeyError(f"derived parameter {p.stable_id:#x} is not in the backend's memo")
                held[pos] = h
            inputs.append(h)
            don.append(False)
        return self.backend.run_program(opt.program, inputs, don if donate is not None else None)


def _last_rows(hidden: Tensor, seq: int, batch: int) -> Tensor:
    """Row seq - 1 of each of the `batch` stacked sequences."""
    d = hidden.dims[1]
    rows = [hidden.slice([b * seq + seq - 1, 0], [1, d]) for b in range(batch)]
    return rows[0] if batch == 1 else Tensor.concat(0, rows)


# ================================================================================ GPT-2
@dataclass
class GptConfig:
    """model/gpt.rs GptConfig."""

    vocab_size: int = 50257
    context_length: int = 1024
    embed_dim: int = 768
    num_layers: int = 12
    num_heads: int = 12
    mlp_ratio: int = 4
    eps: float = 1e-5

    def attention_config(self) -> F.AttentionConfig:
        return F.AttentionConfig(self.embed_dim, self.num_heads, self.num_heads, self.embed_dim // self.num_heads)


class Gpt(_ModelBase):
    """model/gpt.rs: learned positions, pre-LN blocks with biases, final LN, lm_head[d,V]."""

    namespace = "gpt"

    def __init__(self, config: GptConfig, backend, dtype: str = "F32"):
        super().__init__(backend, dtype)
        self.config = config
        self.attn = config.attention_config()

    @classmethod
    def random(cls, config: GptConfig, backend, seed: int = 0, dtype: str = "F32", std: float = 0.02) -> "Gpt":
        """Shapes and constant inits of Gpt::random (model/gpt.rs:128-208); the random
        stream is numpy's PCG64, not Rust's StdRng."""
        m = cls(config, backend, dtype)
        rng = np.random.default_rng(seed)
        d, hid = config.embed_dim, config.embed_dim * config.mlp_ratio

        def rn(*shape):
            return (rng.standard_normal(shape, dtype=np.float32) * np.float32(std)).astype(np.float32)

        m.set_param("tok_embeddings.weight", rn(config.vocab_size, d))
        m.set_param("pos_embeddings", rn(config.context_length, d))
        for i in range(config.num_layers):
            p = f"blocks.{i}."
            m.set_param(p + "ln_1.gamma", np.ones(d, np.float32))
            m.set_param(p + "ln_1.beta", np.zeros(d, np.float32))
            m.set_param(p + "attention.w_qkv", rn(d, 3 * d))
            m.set_param(p + "attention.b_qkv", np.zeros(3 * d, np.float32))
            m.set_param(p + "attention.w_out", rn(d, d))
            m.set_param(p + "attention.b_out", np.zeros(d, np.float32))
            m.set_param(p + "ln_2.gamma", np.ones(d, np.float32))
            m.set_param(p + "ln_2.beta", np.zeros(d, np.float32))
            m.set_param(p + "feed_forward.w_in", rn(d, hid))
            m.set_param(p + "feed_forward.b_in", np.zeros(hid, np.float32))
            m.set_param(p + "feed_forward.w_out", rn(hid, d))
            m.set_param(p + "feed_forward.b_out", np.zeros(d, np.float32))
        m.set_param("final_ln.gamma", np.ones(d, np.float32))
        m.set_param("final_ln.beta", np.zeros(d, np.float32))
        m.set_param("lm_head", rn(d, config.vocab_size))
        return m

    def expected_params(self) -> Dict[str, tuple]:
        """Names and shapes as Gpt::build_from_params reads them (model/gpt.rs:300-370)."""
        c = self.config
        d, hid = c.embed_dim, c.embed_dim * c.mlp_ratio
        out = {"tok_embeddings.weight": (c.vocab_size, d), "pos_embeddings": (c.context_length, d)}
        for i in range(c.num_layers):
            p = f"blocks.{i}."
            out.update({p + "ln_1.gamma": (d,), p + "ln_1.beta": (d,), p + "attention.w_qkv": (d, 3 * d),
                        p + "attention.b_qkv": (3 * d,), p + "attention.w_out": (d, d), p + "attention.b_out": (d,),
                        p + "ln_2.gamma": (d,), p + "ln_2.beta": (d,), p + "feed_forward.w_in": (d, hid),
                        p + "feed_forward.b_in": (hid,), p + "feed_forward.w_out": (hid, d), p + "feed_forward.b_out": (d,)})
        out.update({"final_ln.gamma": (d,), "final_ln.beta": (d,), "lm_head": (d, c.vocab_size)})
        return out

    @staticmethod
    def config_from_json(c) -> GptConfig:
        """GptConfig's serde form (model/gpt.rs)."""
        return GptConfig(vocab_size=int(c["vocab_size"]), context_length=int(c["context_length"]), embed_dim=int(c["embed_dim"]),
                         num_layers=int(c["num_layers"]), num_heads=int(c["num_heads"]), mlp_ratio=int(c.get("mlp_ratio", 4)))

    @classmethod
    def from_checkpoint(cls, path: str, backend, dtype: str = "F32") -> "Gpt":
        """runtime/loader.rs:19-241 for kind "gpt": config from the file, tensors streamed by name."""
        from .checkpoint import Checkpoint, CheckpointError
        with Checkpoint(path) as ck:
            if ck.kind != "gpt":
                raise CheckpointError(f"checkpoint holds a `{ck.kind}` model, not `gpt`")
            m = cls(cls.config_from_json(ck.config), backend, dtype)
            m._load_tensors(ck, m.expected_params())
        return m

    def checkpoint_config(self) -> Dict[str, object]:
        c = self.config
        return {"vocab_size": c.vocab_size, "context_length": c.context_length, "embed_dim": c.embed_dim,
                "num_layers": c.num_layers, "num_heads": c.num_heads, "mlp_ratio": c.mlp_ratio, "dropout": 0.0}

    @property
    def num_layers(self): return self.config.num_layers
    @property
    def context_length(self): return self.config.context_length

    # -- graph pieces ----------------------------------------------------------------
    def _block_tail(self, P, i, x, attn_ctx):
        p = f"blocks.{i}."
        eps = self.config.eps
        attn_out = F.linear(attn_ctx, P[p + "attention.w_out"], P[p + "attention.b_out"])
        residual = attn_out + x                               # model/gpt.rs:81-97: attn_output.add(x)
        normed2, *_ = F.layer_norm(residual, P[p + "ln_2.gamma"], P[p + "ln_2.beta"], eps)
        hidden = F.linear(normed2, P[p + "feed_forward.w_in"], P[p + "feed_forward.b_in"])
        act = F.gelu(hidden)
        ff = F.linear(act, P[p + "feed_forward.w_out"], P[p + "feed_forward.b_out"])
        return ff + residual

    def _build(self, seq: int, capacity: int, decode: bool, batch: int = 1, last_only: bool = False) -> Tuple[Program, dict]:
        """One program for the whole forward (model/gpt.rs:585-751).  last_only: the head runs on the last row of
        each sequence only (logits [batch, V] instead of [batch * seq, V])."""
        last_only = last_only and seq > 1
        key = (seq, capacity, decode, batch, last_only)
        if key in self._programs:
            return self._programs[key]
        cfg, L = self.config, self.config.num_layers
        hkv, dh = self.attn.num_key_value_heads, self.attn.kv_head_dim
        fb = FunctionBuilder("main", self.dtype)
        rows = seq * batch
        tok = fb.param("Si32", [rows])
        pos = fb.param("Si32", [rows])
        layout = {"args": ["tokens", "positions"]}
        if decode:
            upd = fb.param("Si32", [3])
            qst = fb.param("Si32", [1])
            layout["args"] += ["update_starts", "query_start"]
            caches = [[(fb.param(self.dtype, [hkv, capacity, dh]), fb.param(self.dtype, [hkv, capacity, dh]))
                       for _ in range(L)] for _ in range(batch)]
        else:
            start_zeros = fb.param("Si32", [3])
            layout["args"] += ["start_zeros"]
            bases = [[(fb.param(self.dtype, [hkv, capacity, dh]), fb.param(self.dtype, [hkv, capacity, dh]))
                      for _ in range(L)] for _ in range(batch)]
        layout["n_args"] = len(fb.params)
        P = self._declare_params(fb)

        tok_emb = F.embedding_lookup(P["tok_embeddings.weight"], tok)
        pos_emb = F.embedding_lookup(P["pos_embeddings"], pos)
        hidden = tok_emb + pos_emb
        new_caches = [[None] * L for _ in range(batch)]
        for i in range(L):
            p = f"blocks.{i}."
            normed, *_ = F.layer_norm(hidden, P[p + "ln_1.gamma"], P[p + "ln_1.beta"], cfg.eps)
            qkv = F.linear(normed, P[p + "attention.w_qkv"], P[p + "attention.b_qkv"])
            ctxs = []
            for b in range(batch):
                qkv_b = qkv if batch == 1 else qkv.slice([b * seq, 0], [seq, qkv.dims[1]])
                if decode:
                    ck, cv = caches[b][i]
                    ctx, k2, v2 = F.attention_decode_cache(self.attn, qkv_b, ck, cv, upd, qst)
                else:
                    ctx, k, v = F.attention(self.attn, qkv_b, None)
                    kb, vb = bases[b][i]
                    k2 = F.dynamic_update_slice_into(kb, k, start_zeros)   # model/gpt.rs:712-730
                    v2 = F.dynamic_update_slice_into(vb, v, start_zeros)
                new_caches[b][i] = (k2, v2)
                ctxs.append(ctx)
            ctx_all = ctxs[0] if batch == 1 else Tensor.concat(0, ctxs)
            hidden = self._block_tail(P, i, hidden, ctx_all)
        if last_only:
            hidden = _last_rows(hidden, seq, batch)
        normalized, *_ = F.layer_norm(hidden, P["final_ln.gamma"], P["final_ln.beta"], cfg.eps)
        logits = normalized.matmul(P["lm_head"])
        results = []
        for b in range(batch):
            for i in range(L):
                results += list(new_caches[b][i])
        results.append(logits)
        fb.set_results(results)
        prog = Program(fb)
        self._programs[key] = (prog, layout)
        return prog, layout

    # -- forward -----------------------------------------------------------------------
    def forward_with_decode_cache(self, tokens: Sequence[int], position_offset: int,
                                  caches: List[Optional[DecodeKvCache]], fixed_capacity: Optional[int] = None,
                                  last_logits_only: bool = False):
        """model/gpt.rs:585-751.  Returns the logits handle [T, V]; `caches` is updated in place.
        last_logits_only: the final norm and the lm_head run on the last position only and the handle is [1, V] (the
        reference computes every row, gpt.rs:735-736, and its generation loop reads the last)."""
        return self.forward_batch([list(tokens)], position_offset, [caches], fixed_capacity, last_logits_only=last_logits_only)

    def forward_decode_device_token(self, token_handle, position_offset: int, caches: List[Optional[DecodeKvCache]],
                                    fixed_capacity: Optional[int] = None):
        """One decode step whose token id is already on the device (a si32[1] handle, e.g.
        backend.decode_token_tensor()): the same program as forward_with_decode_cache([token], ...), without the
        host having to know the token yet.  An id outside the vocabulary raises at the next synchronising call."""
        return self.forward_batch([[None]], position_offset, [caches], fixed_capacity, token_handle=token_handle)

    def forward_batch(self, token_rows: List[List[int]], position_offset: int,
                      caches: List[List[Optional[DecodeKvCache]]], fixed_capacity: Optional[int] = None,
                      token_handle=None, last_logits_only: bool = False):
        """Independent sequences sharing the weights: row-stacked hidden states, one M=B*T
        GEMM per linear, per-sequence attention.  The reference has no batch dimension
        (ops/functional/attention.rs:189-203); with one row this is exactly its path."""
        cfg = self.config
        batch, seq = len(token_rows), len(token_rows[0])
        if seq == 0:
            raise ValueError("token sequence must contain at least one element")
        if any(len(r) != seq for r in token_rows):
            raise ValueError("all sequences of a batch must have equal length")
        total = position_offset + seq
        if total > cfg.context_length:
            raise ValueError(f"token sequence length {total} exceeds model context length {cfg.context_length}")
        if token_handle is None:
            for row in token_rows:
                for t in row:
                    if not 0 <= t < cfg.vocab_size:
                        raise ValueError(f"token index {t} out of range")
        elif seq != 1:
            raise ValueError("device tokens feed one step (one token per sequence)")
        if any(len(c) != cfg.num_layers for c in caches):
            raise ValueError(f"expected {cfg.num_layers} cache slots (one per layer)")
        if fixed_capacity is not None:
            if not 0 < fixed_capacity <= cfg.context_length or fixed_capacity < total:
                raise ValueError(f"decode cache capacity {fixed_capacity} invalid for sequence length {total}")
            capacity = fixed_capacity
        else:
            capacity = decode_cache_capacity(total, cfg.context_length)
        have = caches[0][0] is not None
        if have and caches[0][0].capacity < capacity:
            self._grow_caches(caches, capacity)
        if have and (seq != 1):
            raise ValueError("decode with an existing cache supports one token per sequence")
        L = cfg.num_layers
        prog, _ = self._build(seq, capacity, have, batch, last_logits_only)
        poss = [position_offset + j for _ in range(batch) for j in range(seq)]
        tok_arg = token_handle if token_handle is not None else self._upload_i32([t for row in token_rows for t in row])
        args = [tok_arg, self._upload_i32(poss)]
        if have:
            for c in caches:
                for slot in c:
                    if slot.len != position_offset:
                        raise ValueError(f"decode cache length {slot.len} must match position offset {position_offset}")
            args += [self._upload_i32([0, position_offset, 0]), self._upload_i32([position_offset])]
            kv = [h for c in caches for slot in c for h in (slot.keys, slot.values)]
        else:
            hkv, dh = self.attn.num_key_value_heads, self.attn.kv_head_dim
            args.append(self._upload_i32([0, 0, 0]))
            kv = [self._zeros([hkv, capacity, dh]) for _ in range(2 * L * batch)]
        donate = [False] * len(args) + [True] * len(kv)       # old caches are dropped (gpt.rs:738-747)
        outs = self._run(prog, args + kv, donate)
        it = iter(outs[:-1])
        for b in range(batch):
            for i in range(L):
                k, v = next(it), next(it)
                caches[b][i] = DecodeKvCache(k, v, total, capacity)
        return outs[-1]

    def _grow_caches(self, caches, capacity: int):
        """model/gpt.rs:626-657: copy each layer's cache into a larger zero buffer."""
        dims = (self.attn.num_key_value_heads, caches[0][0].capacity, self.attn.kv_head_dim)
        for c in caches:
            for i, slot in enumerate(c):
                c[i] = DecodeKvCache(self._grow_rows(slot.keys, dims, capacity), self._grow_rows(slot.values, dims, capacity), slot.len, capacity)


# ================================================================================ Ministral
@dataclass
class MinistralConfig:
    """model/ministral.rs MinistralConfig."""

    vocab_size: int = 131072
    context_length: int = 4096
    embed_dim: int = 3072
    num_layers: int = 26
    num_heads: int = 32
    num_kv_heads: int = 8
    head_dim: int = 128
    ffn_dim: int = 9216
    rotary_dim: int = 128
    rope_theta: float = 1e6
    eps: float = 1e-5
    rope_scaling: Optional[object] = None   # None | ("linear", factor) | functional.YarnScaling (rotary.rs:20-43)

    def attention_config(self) -> F.AttentionConfig:
        return F.AttentionConfig(self.embed_dim, self.num_heads, self.num_kv_heads, self.head_dim)


class Ministral(_ModelBase):
    """model/ministral.rs: RMSNorm, packed-QKV RoPE from host tables, GQA, SwiGLU, no biases,
    untied lm_head."""

    namespace = "ministral"

    def __init__(self, config: MinistralConfig, backend, dtype: str = "Bf16", residual_dtype: Optional[str] = None):
        """`residual_dtype="F32"` on a bf16 model keeps the residual stream, the norms and the logits in f32: the
        embedding rows are cast up, RMSNorm runs on f32 (what the reference's rms_norm requires,
        ops/functional/normalization.rs:183-217) and is cast to bf16 for the projection that follows, the two
        projections that feed a residual add (attention out, feed-forward down) and the lm_head leave their f32
        accumulator as f32 (DotGeneralSpec.out_dtype, spec.rs:354-361; docs/backend.md:104-115).  Matmul operands,
        RoPE, attention and the KV cache stay bf16.  Norm gains are then stored as f32."""
        super().__init__(backend, dtype)
        self.config = config
        self.attn = config.attention_config()
        self.rope = F.RopeConfig(config.rotary_dim, config.rope_theta, config.rope_scaling)
        if residual_dtype is not None and residual_dtype not in ("F32",):
            raise ValueError("residual_dtype must be None or 'F32'")
        self.residual_dtype = residual_dtype if (residual_dtype and residual_dtype != dtype) else None

    @property
    def norm_dtype(self) -> str:
        return self.residual_dtype or self.dtype

    @classmethod
    def random(cls, config: MinistralConfig, backend, seed: int = 0, dtype: str = "Bf16", std: float = 0.02,
               bf16_values: bool = False, quant: Optional[str] = None, residual_dtype: Optional[str] = None):
        """Shapes and constant inits of Ministral::random (model/ministral.rs:262-330).  Every
        tensor draws from its own numpy stream SeedSequence([seed, index]), so the weights do not
        depend on the order or the number of worker threads that generate them.  `bf16_values`
        rounds the draws to bf16-representable values whatever the storage dtype, so an f32
        model can be given exactly the weights of a bf16 one.  `quant` ("w8" / "w4g128") quantises
        every linear weight (projections, feed-forward, lm_head) as it arrives on the device."""
        from concurrent.futures import ThreadPoolExecutor
        m = cls(config, backend, dtype, residual_dtype)
        d, a = config.embed_dim, config.attention_config()
        plan = [("tok_embeddings.weight", (config.vocab_size, d), "randn")]
        for i in range(config.num_layers):
            p = f"blocks.{i}."
            plan += [(p + "norm_1.gamma", (d,), "ones"),
                     (p + "attention.w_qkv", (d, a.total_projection_dim), "randn"),
                     (p + "attention.w_out", (a.query_projection_dim, d), "randn"),
                     (p + "norm_2.gamma", (d,), "ones"),
                     (p + "feed_forward.w_gate", (d, config.ffn_dim), "randn"),
                     (p + "feed_forward.w_up", (d, config.ffn_dim), "randn"),
                     (p + "feed_forward.w_down", (config.ffn_dim, d), "randn")]
        plan += [("final_norm.gamma", (d,), "ones"), ("lm_head", (d, config.vocab_size), "randn")]

        def make(idx):
            name, shape, kind = plan[idx]
            if kind == "ones":
                return name, shape, m.norm_dtype, _np_to_bytes(np.ones(shape, np.float32), m.norm_dtype)
            else:
                arr = np.random.default_rng(np.random.SeedSequence([seed, idx])).standard_normal(shape, dtype=np.float32)
                arr *= np.float32(std)
                if bf16_values and dtype != "Bf16":
                    arr = bf16_bits_to_f32(f32_to_bf16_bits(arr))
            return name, shape, dtype, _np_to_bytes(arr, dtype)

        workers = max(1, min(16, (os.cpu_count() or 1)))
        with ThreadPoolExecutor(max_workers=workers) as ex:
            # bounded look-ahead keeps at most a few tensors of host memory in flight
            pending, nxt = [], 0
            while nxt < len(plan) or pending:
                while nxt < len(plan) and len(pending) < 2 * workers:
                    pending.append(ex.submit(make, nxt))
                    nxt += 1
                name, shape, dt, data = pending.pop(0).result()
                m.set_param_bytes(name, TensorSpec(dt, shape), data)
                if quant and len(shape) == 2 and name != "tok_embeddings.weight":
                    m.quantize_param(name, quant)
        return m

    def expected_params(self) -> Dict[str, tuple]:
        """Names and shapes as Ministral::build_from_params reads them (model/ministral.rs:360-425)."""
        c, a = self.config, self.attn
        d = c.embed_dim
        out = {"tok_embeddings.weight": (c.vocab_size, d)}
        for i in range(c.num_layers):
            p = f"blocks.{i}."
            out.update({p + "norm_1.gamma": (d,), p + "attention.w_qkv": (d, a.total_projection_dim),
                        p + "attention.w_out": (a.query_projection_dim, d), p + "norm_2.gamma": (d,),
                        p + "feed_forward.w_gate": (d, c.ffn_dim), p + "feed_forward.w_up": (d, c.ffn_dim),
                        p + "feed_forward.w_down": (c.ffn_dim, d)})
        out.update({"final_norm.gamma": (d,), "lm_head": (d, c.vocab_size)})
        return out

    @staticmethod
    def _scaling_from_json(js) -> Optional[object]:
        """RopeScaling's serde form: {"kind": "none" | "linear" | "yarn", ...} (ops/functional/rotary.rs:20-43)."""
        if not js or js.get("kind", "none") == "none":
            return None
        if js["kind"] == "linear":
            return ("linear", float(js["factor"]))
        if js["kind"] == "yarn":
            return F.YarnScaling(factor=float(js["factor"]), original_max_position_embeddings=js.get("original_max_position_embeddings"),
                                 mscale=js.get("mscale"), mscale_all_dim=js.get("mscale_all_dim"), beta_fast=js.get("beta_fast"),
                                 beta_slow=js.get("beta_slow"), truncate=bool(js.get("truncate", True)))
        raise ValueError(f"unknown rope scaling kind {js['kind']!r}")

    @classmethod
    def config_from_json(cls, c) -> MinistralConfig:
        """MinistralConfig's serde form (model/ministral.rs:13-30)."""
        from .checkpoint import CheckpointError
        head_dim = int(c["head_dim"]) if c.get("head_dim") else int(c["embed_dim"]) // int(c["num_heads"])
        if c.get("kv_head_dim") and int(c["kv_head_dim"]) != head_dim:
            raise CheckpointError("kv_head_dim different from head_dim is not supported")
        return MinistralConfig(vocab_size=int(c["vocab_size"]), context_length=int(c["context_length"]), embed_dim=int(c["embed_dim"]),
                               num_layers=int(c["num_layers"]), num_heads=int(c["num_heads"]), num_kv_heads=int(c["num_kv_heads"]),
                               head_dim=head_dim, ffn_dim=int(c["mlp_hidden_dim"]), rotary_dim=int(c["rotary_dim"]),
                               rope_theta=float(c["rope_theta"]), eps=float(c["rms_norm_eps"]),
                               rope_scaling=cls._scaling_from_json(c.get("rope_scaling")))

    def param_dtype(self, name: str) -> str:
        return self.norm_dtype if name.endswith(".gamma") else self.dtype

    @classmethod
    def from_checkpoint(cls, path: str, backend, dtype: str = "Bf16", quant: Optional[str] = None,
                        residual_dtype: Optional[str] = None) -> "Ministral":
        """runtime/loader.rs:19-241 for kind "ministral" (MinistralConfig, model/ministral.rs:13-30)."""
        from .checkpoint import Checkpoint, CheckpointError
        with Checkpoint(path) as ck:
            if ck.kind != "ministral":
                raise CheckpointError(f"checkpoint holds a `{ck.kind}` model, not `ministral`")
            m = cls(cls.config_from_json(ck.config), backend, dtype, residual_dtype)
            for name, dims in m.expected_params().items():
                m._load_tensors(ck, {name: dims}, m.norm_dtype if name.endswith(".gamma") else None)
                if quant and len(dims) == 2 and name != "tok_embeddings.weight":
                    m.quantize_param(name, quant)
        return m

    def checkpoint_config(self) -> Dict[str, object]:
        c = self.config
        out = {"vocab_size": c.vocab_size, "context_length": c.context_length, "embed_dim": c.embed_dim, "num_layers": c.num_layers,
               "num_heads": c.num_heads, "num_kv_heads": c.num_kv_heads, "head_dim": c.head_dim, "mlp_hidden_dim": c.ffn_dim,
               "rms_norm_eps": c.eps, "rope_theta": c.rope_theta, "rotary_dim": c.rotary_dim}
        sc = c.rope_scaling
        if sc is None:
            out["rope_scaling"] = {"kind": "none"}
        elif isinstance(sc, F.YarnScaling):
            out["rope_scaling"] = {k: v for k, v in dict(kind="yarn", factor=sc.factor, mscale=sc.mscale, mscale_all_dim=sc.mscale_all_dim,
                                                         beta_fast=sc.beta_fast, beta_slow=sc.beta_slow,
                                                         original_max_position_embeddings=sc.original_max_position_embeddings,
                                                         truncate=sc.truncate).items() if v is not None}
        else:
            out["rope_scaling"] = {"kind": "linear", "factor": sc[1]}
        return out

    QUANTIZABLE = ("attention.w_qkv", "attention.w_out", "feed_forward.w_gate", "feed_forward.w_up",
                   "feed_forward.w_down", "lm_head")

    def quantize(self, scheme: str):
        """Weight-only quantisation of every linear weight of a loaded model, in place."""
        for name in list(self.param_names):
            if name.endswith(self.QUANTIZABLE) and len(self.param_specs[name].dims) == 2:
                self.quantize_param(name, scheme)
        return self

    @property
    def num_layers(self): return self.config.num_layers
    @property
    def context_length(self): return self.config.context_length

    def _linear(self, P, name: str, x: Tensor, out_dtype: Optional[str] = None) -> Tensor:
        """nn/layers/linear.rs:50-71 without bias; quantised weights are read as codes and scales."""
        if name + ".q" in P:
            return F.linear_quantized(x, P[name + ".q"], P[name + ".s"], out_dtype=out_dtype)
        return F.linear(x, P[name], out_dtype=out_dtype)

    def _norm(self, x: Tensor, gamma: Tensor) -> Tensor:
        """RMSNorm in the residual stream's dtype, handed on in the matmul dtype."""
        out, *_ = F.rms_norm(x, gamma, self.config.eps)
        return out.cast(self.dtype) if self.residual_dtype else out

    def _build(self, seq: int, capacity: int, decode: bool, batch: int = 1, last_only: bool = False) -> Tuple[Program, dict]:
        last_only = last_only and seq > 1
        key = (seq, capacity, decode, batch, last_only)
        if key in self._programs:
            return self._programs[key]
        cfg, L = self.config, self.config.num_layers
        hkv, dh = self.attn.num_key_value_heads, self.attn.kv_head_dim
        half = cfg.rotary_dim // 2
        fb = FunctionBuilder("main", self.dtype)
        rows = seq * batch
        tok = fb.param("Si32", [rows])
        cos = fb.param(self.dtype, [seq, half])
        sin = fb.param(self.dtype, [seq, half])
        layout = {"args": ["tokens", "cos", "sin"]}
        if decode:
            upd = fb.param("Si32", [3])
            qst = fb.param("Si32", [1])
            caches = [[(fb.param(self.dtype, [hkv, capacity, dh]), fb.param(self.dtype, [hkv, capacity, dh]))
                       for _ in range(L)] for _ in range(batch)]
        else:
            start_zeros = fb.param("Si32", [3])
            bases = [[(fb.param(self.dtype, [hkv, capacity, dh]), fb.param(self.dtype, [hkv, capacity, dh]))
                      for _ in range(L)] for _ in range(batch)]
        layout["n_args"] = len(fb.params)
        P = self._declare_params(fb)

        rdt = self.residual_dtype   # None: every tensor in the model dtype
        hidden = F.embedding_lookup(P["tok_embeddings.weight"], tok)
        if rdt:
            hidden = hidden.cast(rdt)
        new_caches = [[None] * L for _ in range(batch)]
        for i in range(L):
            p = f"blocks.{i}."
            normed = self._norm(hidden, P[p + "norm_1.gamma"])
            qkv = self._linear(P, p + "attention.w_qkv", normed)
            ctxs = []
            for b in range(batch):
                qkv_b = qkv if batch == 1 else qkv.slice([b * seq, 0], [seq, qkv.dims[1]])
                qkv_b = F.apply_rope_qkv_packed(self.attn, qkv_b, cos, sin)   # ministral.rs:166-201
                if decode:
                    ck, cv = caches[b][i]
                    ctx, k2, v2 = F.attention_decode_cache(self.attn, qkv_b, ck, cv, upd, qst)
                else:
                    ctx, k, v = F.attention(self.attn, qkv_b, None)
                    kb, vb = bases[b][i]
                    k2 = F.dynamic_update_slice_into(kb, k, start_zeros)
                    v2 = F.dynamic_update_slice_into(vb, v, start_zeros)
                new_caches[b][i] = (k2, v2)
                ctxs.append(ctx)
            ctx_all = ctxs[0] if batch == 1 else Tensor.concat(0, ctxs)
            attn_out = self._linear(P, p + "attention.w_out", ctx_all, rdt)
            residual = attn_out + hidden
            normed2 = self._norm(residual, P[p + "norm_2.gamma"])
            gate = self._linear(P, p + "feed_forward.w_gate", normed2)     # nn/layers/feed_forward.rs GatedFeedForward
            up = self._linear(P, p + "feed_forward.w_up", normed2)
            act = F.swiglu(gate, up)
            ff = self._linear(P, p + "feed_forward.w_down", act, rdt)
            hidden = ff + residual
        if last_only:
            hidden = _last_rows(hidden, seq, batch)
        normalized = self._norm(hidden, P["final_norm.gamma"])
        logits = self._linear(P, "lm_head", normalized, rdt)
        results = []
        for b in range(batch):
            for i in range(L):
                results += list(new_caches[b][i])
        results.append(logits)
        fb.set_results(results)
        prog = Program(fb)
        self._programs[key] = (prog, layout)
        return prog, layout

    def forward_with_decode_cache(self, tokens, position_offset, caches, fixed_capacity=None, last_logits_only=False):
        """model/ministral.rs:613-766.  last_logits_only: see Gpt.forward_with_decode_cache."""
        return self.forward_batch([list(tokens)], position_offset, [caches], fixed_capacity, last_logits_only=last_logits_only)

    def forward_decode_device_token(self, token_handle, position_offset, caches, fixed_capacity=None):
        """See Gpt.forward_decode_device_token."""
        return self.forward_batch([[None]], position_offset, [caches], fixed_capacity, token_handle=token_handle)

    def forward_batch(self, token_rows, position_offset, caches, fixed_capacity=None, token_handle=None, last_logits_only=False):
        cfg = self.config
        batch, seq = len(token_rows), len(token_rows[0])
        if token_handle is not None and seq != 1:
            raise ValueError("device tokens feed one step (one token per sequence)")
        if seq == 0:
            raise ValueError("token sequence must contain at least one element")
        if any(len(r) != seq for r in token_rows):
            raise ValueError("all sequences of a batch must have equal length")
        total = position_offset + seq
        if total > cfg.context_length:
            raise ValueError(f"token sequence length {total} exceeds model context length {cfg.context_length}")
        if fixed_capacity is not None:
            if not 0 < fixed_capacity <= cfg.context_length or fixed_capacity < total:
                raise ValueError(f"decode cache capacity {fixed_capacity} invalid for sequence length {total}")
            capacity = fixed_capacity
        else:
            capacity = decode_cache_capacity(total, cfg.context_length)
        have = caches[0][0] is not None
        if have and caches[0][0].capacity < capacity:
            Gpt._grow_caches(self, caches, capacity)
        if have and seq != 1:
            raise ValueError("decode with an existing cache supports one token per sequence")
        L = cfg.num_layers
        prog, _ = self._build(seq, capacity, have, batch, last_logits_only)
        cos, sin = F.rotary_cos_sin_cache_slice(position_offset, seq, self.rope)   # ministral.rs:253-261
        half = cfg.rotary_dim // 2
        tok_arg = token_handle if token_handle is not None else self._upload_i32([t for row in token_rows for t in row])
        args = [tok_arg,
                self.backend.materialize(TensorSpec(self.dtype, [seq, half]), _np_to_bytes(cos, self.dtype)),
                self.backend.materialize(TensorSpec(self.dtype, [seq, half]), _np_to_bytes(sin, self.dtype))]
        if have:
            args += [self._upload_i32([0, position_offset, 0]), self._upload_i32([position_offset])]
            kv = [h for c in caches for slot in c for h in (slot.keys, slot.values)]
        else:
            hkv, dh = self.attn.num_key_value_heads, self.attn.kv_head_dim
            args.append(self._upload_i32([0, 0, 0]))
            kv = [self._zeros([hkv, capacity, dh]) for _ in range(2 * L * batch)]
        donate = [False] * len(args) + [True] * len(kv)
        outs = self._run(prog, args + kv, donate)
        it = iter(outs[:-1])
        for b in range(batch):
            for i in range(L):
                k, v = next(it), next(it)
                caches[b][i] = DecodeKvCache(k, v, total, capacity)
        return outs[-1]


# ================================================================================ ragged batches
class _RaggedModel(_ModelBase):
    """Forward passes over batches of sequences of different lengths.  The rows of a batch are stacked without padding: linear
    layers run over all of them, mixers sequence by sequence (decode steps: all sequences in one launch).  A model says what a
    layer keeps per sequence (`_fresh_slot`, `_slot_handles`, `_grown_slot`, `_new_slot`), which arguments its programs take
    beside tokens and positions (`_position_args`) and builds the program (`_build`)."""

    ragged_batches = True

    @property
    def num_layers(self): return self.config.num_layers
    @property
    def context_length(self): return self.config.context_length

    def _stack(self, parts: List[Tensor]) -> Tensor:
        return parts[0] if len(parts) == 1 else Tensor.concat(0, parts)

    def expected_params(self) -> Dict[str, tuple]:
        return {n: e[0] for n, e in self._param_plan(self.config).items()}

    @classmethod
    def tensor_layout(cls, config) -> Dict[str, Tuple[object, bool]]:
        return {n: (e[1], e[2]) for n, e in cls._param_plan(config).items()}

    def param_dtype(self, name: str) -> str:
        """Matrices that feed products are in the model dtype; gains, scales, taps and per-head constants are f32."""
        leaf = name.rsplit(".", 1)[-1]
        return self.dtype if leaf.startswith("w_") or leaf in ("weight", "lm_head") else "F32"

    def _fill_random(self, names: Sequence[str], seed: int, draw, keep: Sequence[str] = ()) -> Dict[str, np.ndarray]:
        """Sets the parameters `names` to draw(rng, name, dims), one numpy stream per tensor; returns those in `keep`."""
        from concurrent.futures import ThreadPoolExecutor
        dims_of, names, kept = self.expected_params(), list(names), {}

        def make(idx):
            name = names[idx]
            arr = draw(np.random.default_rng(np.random.SeedSequence([seed, idx])), name, dims_of[name])
            dt = self.param_dtype(name)
            return name, dt, _np_to_bytes(arr, dt), arr if name in keep else None

        workers = max(1, min(16, os.cpu_count() or 1))
        with ThreadPoolExecutor(max_workers=workers) as ex:
            pending, nxt = [], 0
            while nxt < len(names) or pending:   # bounded look-ahead: a few tensors of host memory in flight
                while nxt < len(names) and len(pending) < 2 * workers:
                    pending.append(ex.submit(make, nxt))
                    nxt += 1
                name, dt, data, arr = pending.pop(0).result()
                self.set_param_bytes(name, TensorSpec(dt, dims_of[name]), data)
                if arr is not None:
                    kept[name] = arr
        return kept

    # -- forward -----------------------------------------------------------------------
    def forward_with_decode_cache(self, tokens, position_offset, caches, fixed_capacity=None, last_logits_only=False):
        """See Gpt.forward_with_decode_cache."""
        return self.forward_batch([list(tokens)], position_offset, [caches], fixed_capacity, last_logits_only=last_logits_only)

    def forward_decode_device_token(self, token_handle, position_offset, caches, fixed_capacity=None):
        """See Gpt.forward_decode_device_token."""
        return self.forward_batch([[None]], position_offset, [caches], fixed_capacity, token_handle=token_handle)

    def forward_batch(self, token_rows, position_offset, caches, fixed_capacity=None, token_handle=None, last_logits_only=False,
                      logit_rows: Optional[Sequence[int]] = None):
        """Independent sequences of any lengths.  `position_offset`: one for all or one per sequence.  The batch either starts
        (empty caches, offset 0) or goes on by one token each; `caches[b]` is updated in place.  `logit_rows`: the stacked rows
        whose logits are wanted (default: all, or each sequence's last with `last_logits_only`)."""
        cfg, B = self.config, len(token_rows)
        lens = tuple(len(r) for r in token_rows)
        if B == 0 or min(lens) == 0:
            raise ValueError("token sequence must contain at least one element")
        offs = [int(position_offset)] * B if isinstance(position_offset, (int, np.integer)) else [int(o) for o in position_offset]
        if len(offs) != B or len(caches) != B or any(len(c) != cfg.num_layers for c in caches):
            raise ValueError(f"expected an offset and {cfg.num_layers} cache slots (one per layer) for every sequence")
        have = caches[0][0] is not None
        if any((slot is not None) != have for c in caches for slot in c):
            raise ValueError("the sequences of a batch either all start or all go on")
        if have and max(lens) != 1:
            raise ValueError("decode with an existing cache supports one token per sequence")
        if not have and any(offs):
            raise ValueError("a sequence without a cache starts at position 0")
        if token_handle is not None and max(lens) != 1:
            raise ValueError("device tokens feed one step (one token per sequence)")
        if token_handle is None:
            for row in token_rows:
                for t in row:
                    if not 0 <= t < cfg.vocab_size:
                        raise ValueError(f"token index {t} out of range")
        totals = [o + n for o, n in zip(offs, lens)]
        need = max(totals)
        if need > cfg.context_length:
            raise ValueError(f"token sequence length {need} exceeds model context length {cfg.context_length}")
        if fixed_capacity is not None:
            if not 0 < fixed_capacity <= cfg.context_length or fixed_capacity < need:
                raise ValueError(f"decode cache capacity {fixed_capacity} invalid for sequence length {need}")
            capacity = fixed_capacity
        else:
            capacity = decode_cache_capacity(need, cfg.context_length)
        if have:
            for c, o in zip(caches, offs):
                for slot in c:
                    if slot.len != o:
                        raise ValueError(f"decode cache length {slot.len} must match position offset {o}")
            # the sequences of a step share one capacity: the largest any of them has or needs
            capacity = max([capacity] + [getattr(s, "capacity", 0) for c in caches for s in c])
            for c in caches:
                for i, s in enumerate(c):
                    c[i] = self._grown_slot(i, s, capacity)
        if logit_rows is not None and list(logit_rows) == list(range(sum(lens))):
            logit_rows = None
        prog, _ = self._build(lens, capacity, have, last_logits_only and logit_rows is None, None if logit_rows is None else len(logit_rows))
        tok_arg = token_handle if token_handle is not None else self._upload_i32([t for row in token_rows for t in row])
        args = [tok_arg, self._upload_i32([o + j for o, n in zip(offs, lens) for j in range(n)])] + self._position_args(offs)
        if logit_rows is not None:
            args.append(self._upload_i32(logit_rows))
        held = [h for c in caches for i, slot in enumerate(c) for h in (self._slot_handles(slot) if have else self._fresh_slot(i, capacity))]
        outs = self._run(prog, args + held, [False] * len(args) + [True] * len(held))
        it = iter(outs[:-1])
        for b in range(B):
            for i in range(cfg.num_layers):
                caches[b][i] = self._new_slot(i, it, totals[b], capacity)
        return outs[-1]


# ================================================================================ Dadupel
@dataclass
class SsmMixerConfig:
    """A Mamba-2 mixer (state-space duality)."""

    heads: int
    vdim: int
    state: int
    groups: int
    conv: int
    norm_groups: int

    @property
    def inner(self): return self.heads * self.vdim
    @property
    def channels(self): return self.inner + 2 * self.groups * self.state       # x | B | C
    @property
    def projection(self): return self.inner + self.channels + self.heads       # z | x | B | C | dt


@dataclass
class LatentMixerConfig:
    """A latent-attention mixer.  `kv_from`: the layer whose cached rows it attends to (None: its own)."""

    heads: int
    dim: int
    rot_dim: int
    vdim: int
    q_rank: int
    kv_rank: int
    scale: float
    rope_base: float
    rope_scaling: Optional[Tuple[float, float, float, float]] = None   # YaRN: (factor, original, fast, slow)
    kv_from: Optional[int] = None

    @property
    def row_width(self): return self.kv_rank + self.rot_dim

    def frequencies(self) -> Tuple[np.ndarray, float]:
        if self.rope_scaling is None:
            return F.pair_frequencies(self.rot_dim, self.rope_base), 1.0
        return F.yarn_pair_frequencies(self.rot_dim, self.rope_base, *self.rope_scaling)


@dataclass
class DadupelLayer:
    mixer: object                     # SsmMixerConfig | LatentMixerConfig
    ffn_dim: Optional[int] = None     # None: no feed-forward
    glu_limit: float = 0.0


@dataclass
class DadupelConfig:
    vocab_size: int
    embed_dim: int
    eps: float
    layers: List[DadupelLayer]
    context_length: int = 1 << 20     # the design states no limit; this one bounds the caches

    @property
    def num_layers(self): return len(self.layers)


class Dadupel(_RaggedModel):
    """Hybrid decoder: Mamba-2 and latent-attention mixers in any order, each beside a clamped gated feed-forward under ONE
    layer norm (x + scale_1 * mixer(h) + scale_2 * ff(h)), tied embedding and head.

    The residual stream, the norms, the input projections of the mixers' f32 parts and the logits are f32; matmul operands
    and the latent cache are in the model dtype; recurrent states are f32.  A batch may hold sequences of different lengths:
    their rows are stacked without padding, the linear layers run over all of them, the mixers sequence by sequence (decode
    steps: all sequences in one launch)."""

    namespace = "dadupel"

    def __init__(self, config: DadupelConfig, backend, dtype: str = "Bf16", context_length: Optional[int] = None):
        super().__init__(backend, dtype)
        self.config = config
        if context_length is not None:
            config.context_length = int(context_length)
        for i, L in enumerate(config.layers):
            m = L.mixer
            if isinstance(m, SsmMixerConfig):
                if m.heads % m.groups or m.inner % m.norm_groups:
                    raise ValueError(f"layer {i}: heads must be a multiple of groups, heads * vdim of norm_groups")
            elif m.kv_from is not None:
                src = config.layers[m.kv_from].mixer if 0 <= m.kv_from < i else None
                if not isinstance(src, LatentMixerConfig) or src.kv_from is not None or (src.kv_rank, src.rot_dim) != (m.kv_rank, m.rot_dim):
                    raise ValueError(f"layer {i}: kv_from must name an earlier latent-attention layer with a cache of the same sizes")

    # -- configuration and parameters ---------------------------------------------------
    @staticmethod
    def config_from_json(c) -> DadupelConfig:
        layers = []
        for L in c["layers"]:
            m = L["mixer"]
            if L["type"] == "mamba2":
                mixer = SsmMixerConfig(heads=int(m["heads"]), vdim=int(m["vdim"]), state=int(m["state"]), groups=int(m["groups"]),
                                       conv=int(m["conv"]), norm_groups=int(m["norm_groups"]))
            elif L["type"] == "latent_attention":
                rot, sc = m["rot"], m["rot"].get("scaling")
                if int(rot["dims"]) != int(m["rot_dim"]):
                    raise ValueError("latent attention rotates its whole rot_dim part: rot.dims must equal rot_dim")
                mixer = LatentMixerConfig(heads=int(m["heads"]), dim=int(m["dim"]), rot_dim=int(m["rot_dim"]), vdim=int(m["vdim"]),
                                          q_rank=int(m["q_rank"]), kv_rank=int(m["kv_rank"]), scale=float(m["scale"]), rope_base=float(rot["base"]),
                                          rope_scaling=None if not sc else tuple(float(sc[k]) for k in ("factor", "original", "fast", "slow")),
                                          kv_from=None if m.get("kv_from") is None else int(m["kv_from"]))
            else:
                raise ValueError(f"unknown layer type {L['type']!r}")
            mlp = L.get("mlp")
            if mlp is not None and mlp["kind"] != "dense":
                raise ValueError(f"unknown feed-forward kind {mlp['kind']!r}")
            layers.append(DadupelLayer(mixer, None if mlp is None else int(mlp["ff"]), 0.0 if mlp is None else float(mlp["limit"])))
        return DadupelConfig(vocab_size=int(c["vocab"]), embed_dim=int(c["width"]), eps=float(c["norm"]["eps"]), layers=layers,
                             context_length=int(c.get("context_length", 1 << 20)))

    def checkpoint_config(self) -> Dict[str, object]:
        c, layers = self.config, []
        for L in c.layers:
            m = L.mixer
            if isinstance(m, SsmMixerConfig):
                e = {"type": "mamba2", "mixer": dict(heads=m.heads, vdim=m.vdim, state=m.state, groups=m.groups, conv=m.conv, norm_groups=m.norm_groups)}
            else:
                rot = {"dims": m.rot_dim, "base": m.rope_base}
                if m.rope_scaling is not None:
                    rot["scaling"] = dict(zip(("factor", "original", "fast", "slow"), m.rope_scaling))
                mix = dict(heads=m.heads, dim=m.dim, rot_dim=m.rot_dim, vdim=m.vdim, q_rank=m.q_rank, kv_rank=m.kv_rank, scale=m.scale, rot=rot)
                if m.kv_from is not None:
                    mix["kv_from"] = m.kv_from
                e = {"type": "latent_attention", "mixer": mix}
            e["mlp"] = None if L.ffn_dim is None else {"kind": "dense", "ff": L.ffn_dim, "limit": L.glu_limit}
            layers.append(e)
        return {"architecture": "Dadupel", "vocab": c.vocab_size, "width": c.embed_dim, "norm": {"eps": c.eps}, "layers": layers}

    @staticmethod
    def _param_plan(c: DadupelConfig) -> Dict[str, Tuple[tuple, str, bool]]:
        """parameter -> (shape, tensor of a model folder, transposed there)."""
        d = c.embed_dim
        out = {"tok_embeddings.weight": ((c.vocab_size, d), "embed", False)}
        for i, L in enumerate(c.layers):
            p, t, m = f"blocks.{i}.", f"l{i}.", L.mixer
            out[p + "norm_1.gamma"] = ((d,), t + "norm1", False)
            out[p + "norm_1.beta"] = ((d,), t + "norm1.b", False)
            q, u = p + "mixer.", t + "mix."
            if isinstance(m, SsmMixerConfig):
                out[q + "w_in"] = ((d, m.projection), u + "in", True)
                out[q + "conv"] = ((m.conv, m.channels), u + "conv", True)
                out[q + "conv_bias"] = ((m.channels,), u + "conv.b", False)
                out[q + "dt_bias"] = ((m.heads,), u + "dt_bias", False)
                out[q + "a_log"] = ((m.heads,), u + "A_log", False)
                out[q + "d"] = ((m.heads,), u + "D", False)
                out[q + "norm.gamma"] = ((m.inner,), u + "norm", False)
                out[q + "w_out"] = ((m.inner, d), u + "o", True)
            else:
                out[q + "w_dq"] = ((d, m.q_rank), u + "dq", True)
                out[q + "q_norm.gamma"] = ((m.q_rank,), u + "dq.norm", False)
                out[q + "w_uq"] = ((m.q_rank, m.heads * (m.dim + m.rot_dim)), u + "uq", True)
                if m.kv_from is None:
                    out[q + "w_dkv"] = ((d, m.row_width), u + "dkv", True)
                    out[q + "kv_norm.gamma"] = ((m.kv_rank,), u + "dkv.norm", False)
                out[q + "w_uk"] = ((m.kv_rank, m.heads * m.dim), u + "uk", True)
                out[q + "w_uv"] = ((m.kv_rank, m.heads * m.vdim), u + "uv", True)
                out[q + "w_out"] = ((m.heads * m.vdim, d), u + "o", True)
            out[p + "scale_1"] = ((d,), t + "ls1", False)
            if L.ffn_dim is not None:
                out[p + "feed_forward.w_gate"] = ((d, L.ffn_dim), t + "mlp.gate", True)
                out[p + "feed_forward.w_up"] = ((d, L.ffn_dim), t + "mlp.up", True)
                out[p + "feed_forward.w_down"] = ((L.ffn_dim, d), t + "mlp.down", True)
                out[p + "scale_2"] = ((d,), t + "ls2", False)
        out["final_norm.gamma"] = ((d,), "final.norm", False)
        out["final_norm.beta"] = ((d,), "final.norm.b", False)
        out["lm_head"] = ((d, c.vocab_size), "embed", True)     # the tied table once more, as a linear layer reads it
        return out

    @classmethod
    def random(cls, config: DadupelConfig, backend, seed: int = 0, dtype: str = "Bf16", context_length: Optional[int] = None) -> "Dadupel":
        """Random weights of the right shapes and of sensible sizes, one numpy stream per tensor."""
        m = cls(config, backend, dtype, context_length)

        def draw(rng, name, dims):
            leaf = name.rsplit(".", 1)[-1]
            if leaf == "dt_bias":
                return np.log(np.expm1(np.exp(rng.uniform(np.log(1e-3), np.log(1e-1), dims)))).astype(np.float32)
            if leaf == "a_log":
                return np.log(rng.uniform(1.0, 16.0, dims)).astype(np.float32)
            if leaf in ("gamma", "d"):
                return (1.0 + 0.1 * rng.standard_normal(dims)).astype(np.float32)
            if leaf in ("beta", "conv_bias"):
                return (0.1 * rng.standard_normal(dims)).astype(np.float32)
            if leaf in ("scale_1", "scale_2"):
                return rng.uniform(0.3, 1.0, dims).astype(np.float32)
            arr = rng.standard_normal(dims, dtype=np.float32)
            arr *= np.float32((dims[1] if leaf == "weight" else dims[0]) ** -0.5)
            return arr

        table = m._fill_random([n for n in m.expected_params() if n != "lm_head"], seed, draw, ["tok_embeddings.weight"])["tok_embeddings.weight"]
        m.set_param("lm_head", np.ascontiguousarray(table.T), m.param_dtype("lm_head"))
        return m

    # -- graph pieces ----------------------------------------------------------------
    def _norm(self, x: Tensor, P, name: str) -> Tensor:
        """Layer norm of the f32 stream, handed on in the matmul dtype."""
        out, *_ = F.layer_norm(x, P[name + ".gamma"], P[name + ".beta"], self.config.eps)
        return out if self.dtype == "F32" else out.cast(self.dtype)

    def _ssm_mixer(self, P, p: str, m: SsmMixerConfig, proj: Tensor, lens, states):
        """proj f32 [rows, z | x | B | C | dt] of all sequences; returns (rows in the matmul dtype, new (conv, state) per sequence)."""
        ys, new, r0 = [], [], 0
        dt_col = m.inner + m.channels
        for n, (conv, state) in zip(lens, states):
            pr = proj if len(lens) == 1 else proj.slice([r0, 0], [n, m.projection])
            r0 += n
            xbc, conv2 = F.causal_conv_silu(pr, P[p + "conv"], P[p + "conv_bias"], conv, m.inner, self.dtype)
            y, state2 = F.ssm_scan(xbc, pr, P[p + "dt_bias"], P[p + "a_log"], P[p + "d"], state, m.groups, dt_col)
            ys.append(y)
            new.append((conv2, state2))
        return F.gated_rms_norm(self._stack(ys), proj, P[p + "norm.gamma"], m.norm_groups, 0, self.config.eps), new

    def _build(self, lens: Tuple[int, ...], capacity: int, decode: bool, last_only: bool = False, n_logit_rows: Optional[int] = None):
        """One program for a forward of len(lens) sequences, sequence b bringing lens[b] rows (decode: one each).
        last_only: the head runs on every sequence's last row; n_logit_rows: on that many rows, named by an argument."""
        last_only = last_only and not decode
        key = (lens, capacity, decode, last_only, n_logit_rows)
        if key in self._programs:
            return self._programs[key]
        cfg, dt, B, rows = self.config, self.dtype, len(lens), sum(lens)
        fb = FunctionBuilder("main", dt)
        tok = fb.param("Si32", [rows])
        pos = fb.param("Si32", [rows])
        starts = fb.param("Si32", [3 * B])       # [0, position, 0] of every sequence: where its new cache rows go
        layout = {"args": ["tokens", "positions", "starts"]}
        pick = None
        if n_logit_rows is not None:
            pick = fb.param("Si32", [n_logit_rows])
            layout["args"].append("logit_rows")
        held = []                                # per sequence and layer: the tensors of its slot
        for _ in range(B):
            per = []
            for L in cfg.layers:
                m = L.mixer
                if isinstance(m, SsmMixerConfig):
                    per.append((fb.param("F32", [m.conv - 1, m.channels]), fb.param("F32", [m.heads, m.state, m.vdim])))
                elif m.kv_from is None:
                    per.append((fb.param(dt, [1, capacity, m.row_width]),))
                else:
                    per.append(())
            held.append(per)
        layout["n_args"] = len(fb.params)
        P = self._declare_params(fb)
        tables: Dict[tuple, Tensor] = {}
        new_rows: Dict[int, Tensor] = {}

        def table_of(m: LatentMixerConfig) -> Tensor:
            f, mag = m.frequencies()
            k = (f.tobytes(), mag)
            if k not in tables:
                tables[k] = F.rope_table(pos, fb.constant(TensorSpec("F32", f.shape), f.astype("<f4").tobytes()), mag)
            return tables[k]

        def part(t: Tensor, b: int) -> Tensor:   # the rows of sequence b
            return t if B == 1 else t.slice([sum(lens[:b]), 0], [lens[b], t.dims[1]])

        for L in cfg.layers:
            if isinstance(L.mixer, LatentMixerConfig):
                table_of(L.mixer)
        hidden = F.embedding_lookup(P["tok_embeddings.weight"], tok)
        if dt != "F32":
            hidden = hidden.cast("F32")
        new = [[()] * cfg.num_layers for _ in range(B)]
        for i, L in enumerate(cfg.layers):
            p, m = f"blocks.{i}.", L.mixer
            q = p + "mixer."
            h = self._norm(hidden, P, p + "norm_1")
            ssm = isinstance(m, SsmMixerConfig)
            # everything that reads the normed row comes first, so that a decode step's launches stay together
            if ssm:
                proj = F.linear(h, P[q + "w_in"], out_dtype="F32")
            else:
                cq = F.linear(h, P[q + "w_dq"], out_dtype="F32")
                raw = F.linear(h, P[q + "w_dkv"], out_dtype="F32") if m.kv_from is None else None
            act = None
            if L.ffn_dim is not None:
                f = p + "feed_forward."
                act = F.clamped_glu(F.linear(h, P[f + "w_gate"]), F.linear(h, P[f + "w_up"]), L.glu_limit)
            if ssm:
                mixed, states = self._ssm_mixer(P, q, m, proj, lens, [held[b][i] for b in range(B)])
                for b in range(B):
                    new[b][i] = states[b]
            else:
                table, half = table_of(m), m.rot_dim // 2
                cqn, *_ = F.rms_norm(cq, P[q + "q_norm.gamma"], cfg.eps)
                qh = F.linear(cqn if dt == "F32" else cqn.cast(dt), P[q + "w_uq"])
                qh = F.rope_pairs(qh, table, m.heads, m.dim)
                src = i if m.kv_from is None else m.kv_from
                if m.kv_from is None:
                    new_rows[i] = F.latent_rows(raw, P[q + "kv_norm.gamma"], table, cfg.eps, dt)
                    for b in range(B):
                        upd = part(new_rows[i], b).reshape([1, lens[b], m.row_width])
                        at = starts if B == 1 else starts.slice([3 * b], [3])
                        new[b][i] = (F.dynamic_update_slice_into(held[b][i][0], upd, at),)
                ctxs = []
                if decode:
                    for b in range(B):
                        ctxs.append(F.latent_attention(part(qh, b), new[b][src][0], P[q + "w_uk"], P[q + "w_uv"], pos if B == 1 else pos.slice([b], [1]),
                                                       m.heads, m.rot_dim, m.scale))
                else:   # a prompt starts at its first token: its keys and values are the rows at hand
                    lat = new_rows[src].slice([0, 0], [rows, m.kv_rank])
                    kn, vv = F.linear(lat, P[q + "w_uk"]), F.linear(lat, P[q + "w_uv"])
                    for b in range(B):
                        ctxs.append(F.latent_attention_expanded(part(qh, b), part(kn, b), part(vv, b), part(new_rows[src], b), m.heads, m.rot_dim, m.scale))
                mixed = self._stack(ctxs)
            hidden = F.scale_columns(F.linear(mixed, P[q + "w_out"], out_dtype="F32"), P[p + "scale_1"]) + hidden
            if act is not None:
                hidden = F.scale_columns(F.linear(act, P[p + "feed_forward.w_down"], out_dtype="F32"), P[p + "scale_2"]) + hidden
        if pick is not None:
            hidden = hidden.take(pick)
        elif last_only:
            hidden = self._stack([hidden.slice([sum(lens[:b + 1]) - 1, 0], [1, cfg.embed_dim]) for b in range(B)])
        logits = F.linear(self._norm(hidden, P, "final_norm"), P["lm_head"], out_dtype="F32")
        fb.set_results([t for b in range(B) for slot in new[b] for t in slot] + [logits])
        prog = Program(fb)
        self._programs[key] = (prog, layout)
        return prog, layout

    # -- what a layer keeps per sequence -------------------------------------------------
    def _position_args(self, offs):
        return [self._upload_i32([v for o in offs for v in (0, o, 0)])]

    def _fresh_slot(self, i, capacity):
        m = self.config.layers[i].mixer
        if isinstance(m, SsmMixerConfig):
            return [self._zeros([m.conv - 1, m.channels], "F32"), self._zeros([m.heads, m.state, m.vdim], "F32")]
        return [self._zeros([1, capacity, m.row_width])] if m.kv_from is None else []

    def _slot_handles(self, slot):
        return [slot.conv, slot.state] if isinstance(slot, DecodeSsmState) else [slot.rows] if isinstance(slot, DecodeLatentCache) else []

    def _grown_slot(self, i, slot, capacity):
        if not isinstance(slot, DecodeLatentCache) or slot.capacity >= capacity:
            return slot
        return DecodeLatentCache(self._grow_rows(slot.rows, (1, slot.capacity, self.config.layers[i].mixer.row_width), capacity), slot.len, capacity)

    def _new_slot(self, i, handles, length, capacity):
        m = self.config.layers[i].mixer
        if isinstance(m, SsmMixerConfig):
            return DecodeSsmState(next(handles), next(handles), length)
        return DecodeLatentCache(next(handles), length, capacity) if m.kv_from is None else SharedLayerCache(m.kv_from, length)


# ================================================================================ Fuzazen
@dataclass
class ChunkedMixerConfig:
    """A grouped-query attention mixer whose positions see their own chunk of `chunk` positions only."""

    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot_dims: int
    rope_base: float
    chunk: int

    @property
    def keys(self): return self.kv_heads * self.dim
    @property
    def values(self): return self.kv_heads * self.vdim
    @property
    def projection(self): return self.heads * self.dim + self.keys + self.values + self.heads    # q | k | v | gate

    def rows(self, capacity: int) -> int:
        """Cache rows of a sequence of at most `capacity` positions: a position's row is its place in its chunk."""
        return min(capacity, self.chunk)


@dataclass
class FuzazenLayer:
    mixer: ChunkedMixerConfig
    ffn_dim: Optional[int] = None       # None: no feed-forward
    weights_of: Optional[int] = None    # the layer whose tensors this one uses (None: its own)


@dataclass
class FuzazenConfig:
    vocab_size: int
    embed_dim: int
    eps: float
    layers: List[FuzazenLayer]
    embedding_scale: float = 1.0
    residual_mult: float = 1.0
    logit_softcap: Optional[float] = None
    context_length: int = 1 << 20       # the design states no limit; this one bounds the caches

    @property
    def num_layers(self): return len(self.layers)

    def owner(self, i: int) -> int:
        """The layer whose tensors layer i uses."""
        seen = set()
        while self.layers[i].weights_of is not None:
            if i in seen or not 0 <= self.layers[i].weights_of < len(self.layers):
                raise ValueError(f"layer {i}: weights_of must lead to a layer with weights of its own")
            seen.add(i)
            i = self.layers[i].weights_of
        return i


class Fuzazen(_RaggedModel):
    """Decoder of chunked grouped-query attention (pairwise rotation, unit-RMS queries and keys, a sink and an output gate per
    head) and SwiGLU layers that read the residual stream itself; the norm stands on a sublayer's output: x + m * rms_norm(f(x)).
    Layers may share their weights.  Soft-capped logits.

    The residual stream, the norms, the packed projection q | k | v | gate and the logits are f32; matmul operands and the caches
    are in the model dtype.  A cache holds the rows of the current chunk only: position p's row is p % chunk."""

    namespace = "fuzazen"

    def __init__(self, config: FuzazenConfig, backend, dtype: str = "Bf16", context_length: Optional[int] = None):
        super().__init__(backend, dtype)
        self.config = config
        if context_length is not None:
            config.context_length = int(context_length)
        for i, L in enumerate(config.layers):
            m, own = L.mixer, config.layers[config.owner(i)]
            if m.kv_heads < 1 or m.heads % m.kv_heads or m.rot_dims % 2 or not 0 <= m.rot_dims <= m.dim or m.chunk < 1:
                raise ValueError(f"layer {i}: heads must be a multiple of kv_heads, rot.dims even and at most dim, the chunk at least 1")
            if (m, L.ffn_dim) != (own.mixer, own.ffn_dim):
                raise ValueError(f"layer {i}: a layer that uses another's weights has its sizes")
        self.chunks = sorted({L.mixer.chunk for L in config.layers})

    # -- configuration and parameters ---------------------------------------------------
    @staticmethod
    def config_from_json(c) -> FuzazenConfig:
        layers = []
        for L in c["layers"]:
            if L["type"] != "attention":
                raise ValueError(f"unknown layer type {L['type']!r}")
            m, mlp = L["mixer"], L.get("mlp")
            if mlp is not None and mlp["kind"] != "dense":
                raise ValueError(f"unknown feed-forward kind {mlp['kind']!r}")
            mixer = ChunkedMixerConfig(heads=int(m["heads"]), kv_heads=int(m["kv_heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]), scale=float(m["scale"]),
                                       rot_dims=int(m["rot"]["dims"]), rope_base=float(m["rot"]["base"]), chunk=int(m["mask"]["size"]))
            layers.append(FuzazenLayer(mixer, None if mlp is None else int(mlp["ff"]), None if L.get("weights_of") is None else int(L["weights_of"])))
        cap = c.get("logit_softcap")
        return FuzazenConfig(vocab_size=int(c["vocab"]), embed_dim=int(c["width"]), eps=float(c["norm"]["eps"]), layers=layers,
                             embedding_scale=float(c["embedding"]["scale"]), residual_mult=float(c["residual_mult"]),
                             logit_softcap=None if cap is None else float(cap), context_length=int(c.get("context_length", 1 << 20)))

    def checkpoint_config(self) -> Dict[str, object]:
        c, layers = self.config, []
        for L in c.layers:
            m = L.mixer
            e = {"type": "attention", "mlp": None if L.ffn_dim is None else {"kind": "dense", "ff": L.ffn_dim},
                 "mixer": dict(heads=m.heads, kv_heads=m.kv_heads, dim=m.dim, vdim=m.vdim, scale=m.scale, rot={"dims": m.rot_dims, "base": m.rope_base},
                               mask={"size": m.chunk})}
            if L.weights_of is not None:
                e["weights_of"] = L.weights_of
            layers.append(e)
        return {"architecture": "Fuzazen", "vocab": c.vocab_size, "width": c.embed_dim, "norm": {"eps": c.eps}, "embedding": {"scale": c.embedding_scale},
                "residual_mult": c.residual_mult, "logit_softcap": c.logit_softcap, "layers": layers}

    @staticmethod
    def _param_plan(c: FuzazenConfig) -> Dict[str, Tuple[tuple, object, bool]]:
        """parameter -> (shape, tensor of a model folder or the tensors stacked in it, transposed there)."""
        d = c.embed_dim
        out = {"tok_embeddings.weight": ((c.vocab_size, d), "embed", False)}
        for i, L in enumerate(c.layers):
            if L.weights_of is not None:
                continue
            p, t, m = f"blocks.{i}.", f"l{i}.", L.mixer
            out[p + "mixer.w_qkvg"] = ((d, m.projection), tuple(t + "mix." + n for n in "qkvg"), True)
            out[p + "mixer.sink"] = ((m.heads,), t + "mix.sink", False)
            out[p + "mixer.w_out"] = ((m.heads * m.vdim, d), t + "mix.o", True)
            out[p + "norm_1.gamma"] = ((d,), t + "norm1", False)
            if L.ffn_dim is not None:
                out[p + "feed_forward.w_gate"] = ((d, L.ffn_dim), t + "mlp.gate", True)
                out[p + "feed_forward.w_up"] = ((d, L.ffn_dim), t + "mlp.up", True)
                out[p + "feed_forward.w_down"] = ((L.ffn_dim, d), t + "mlp.down", True)
                out[p + "norm_2.gamma"] = ((d,), t + "norm2", False)
        out["final_norm.gamma"] = ((d,), "final.norm", False)
        out["lm_head"] = ((d, c.vocab_size), "head", True)
        return out

    @classmethod
    def random(cls, config: FuzazenConfig, backend, seed: int = 0, dtype: str = "Bf16", context_length: Optional[int] = None) -> "Fuzazen":
        """Random weights of the right shapes and of sensible sizes, one numpy stream per tensor."""
        m = cls(config, backend, dtype, context_length)

        def draw(rng, name, dims):
            leaf = name.rsplit(".", 1)[-1]
            if leaf == "gamma":
                return (1.0 + 0.1 * rng.standard_normal(dims)).astype(np.float32)
            if leaf == "sink":
                return rng.standard_normal(dims).astype(np.float32)
            arr = rng.standard_normal(dims, dtype=np.float32)
            if leaf != "weight":
                arr *= np.float32(dims[0] ** -0.5)
            return arr

        m._fill_random(m.expected_params(), seed, draw)
        return m

    # -- graph ---------------------------------------------------------------------------
    def _operand(self, x: Tensor) -> Tensor:
        """The f32 stream as an operand of matrix products."""
        return x if self.dtype == "F32" else x.cast(self.dtype)

    def _build(self, lens: Tuple[int, ...], capacity: int, decode: bool, last_only: bool = False, n_logit_rows: Optional[int] = None):
        """One program for a forward of len(lens) sequences, sequence b bringing lens[b] rows (decode: one each).
        last_only: the head runs on every sequence's last row; n_logit_rows: on that many rows, named by an argument."""
        last_only = last_only and not decode
        key = (lens, capacity, decode, last_only, n_logit_rows)
        if key in self._programs:
            return self._programs[key]
        cfg, dt, B, rows = self.config, self.dtype, len(lens), sum(lens)
        fb = FunctionBuilder("main", dt)
        tok = fb.param("Si32", [rows])
        pos = fb.param("Si32", [rows])
        # [0, row, 0] of every sequence: where its new cache rows go, one argument per size of chunk
        starts = {n: fb.param("Si32", [3 * B]) for n in self.chunks}
        layout = {"args": ["tokens", "positions"] + [f"starts_{n}" for n in self.chunks]}
        pick = None
        if n_logit_rows is not None:
            pick = fb.param("Si32", [n_logit_rows])
            layout["args"].append("logit_rows")
        held = [[(fb.param(dt, [L.mixer.kv_heads, L.mixer.rows(capacity), L.mixer.dim]), fb.param(dt, [L.mixer.kv_heads, L.mixer.rows(capacity), L.mixer.vdim]))
                 for L in cfg.layers] for _ in range(B)]
        layout["n_args"] = len(fb.params)
        P = self._declare_params(fb)
        tables: Dict[bytes, Tensor] = {}

        def table_of(m: ChunkedMixerConfig) -> Tensor:
            f = F.pair_frequencies(m.rot_dims, m.rope_base)
            k = f.tobytes()
            if k not in tables:
                tables[k] = F.rope_table(pos, fb.constant(TensorSpec("F32", f.shape), f.astype("<f4").tobytes()))
            return tables[k]

        def part(t: Tensor, b: int) -> Tensor:   # the rows of sequence b
            return t if B == 1 else t.slice([sum(lens[:b]), 0], [lens[b], t.dims[1]])

        for L in cfg.layers:
            if L.mixer.rot_dims:
                table_of(L.mixer)
        hidden = F.embedding_lookup(P["tok_embeddings.weight"], tok)
        if dt != "F32":
            hidden = hidden.cast("F32")
        if cfg.embedding_scale != 1.0:
            hidden = hidden * float(cfg.embedding_scale)
        new = [[()] * cfg.num_layers for _ in range(B)]
        for i, L in enumerate(cfg.layers):
            p, m = f"blocks.{cfg.owner(i)}.", L.mixer
            q = p + "mixer."
            proj = F.linear(self._operand(hidden), P[q + "w_qkvg"], out_dtype="F32")
            cols = [0, m.heads * m.dim, m.keys, m.values, m.heads]
            qs, ks, vs, gate = (proj.slice([0, sum(cols[:j + 1])], [rows, cols[j + 1]]) for j in range(4))
            qs, ks = (F.rope_pairs(t, table_of(m), n, 0) if m.rot_dims else t for t, n in ((qs, m.heads), (ks, m.kv_heads)))
            qs, ks = (F.head_rms_norm(t, n, cfg.eps, dt) for t, n in ((qs, m.heads), (ks, m.kv_heads)))
            vs = self._operand(vs)
            ctxs = []
            for b in range(B):
                kb, vb, sink = part(ks, b), part(vs, b), P[q + "sink"]
                first = 0 if decode else (lens[b] - 1) // m.chunk * m.chunk   # the rows of the chunk that the next token may go on with
                at = starts[m.chunk] if B == 1 else starts[m.chunk].slice([3 * b], [3])
                slot = []
                for t, width, base in ((kb, m.dim, held[b][i][0]), (vb, m.vdim, held[b][i][1])):
                    n = lens[b] - first
                    t = t if first == 0 else t.slice([first, 0], [n, t.dims[1]])
                    slot.append(F.dynamic_update_slice_into(base, t.reshape([n, m.kv_heads, width]).transpose([1, 0, 2]), at))
                new[b][i] = tuple(slot)
                if decode:
                    ctxs.append(F.chunk_attention_cache(part(qs, b), slot[0], slot[1], sink, pos if B == 1 else pos.slice([b], [1]), m.heads, m.chunk, m.scale))
                else:   # a prompt starts at its first token: its keys and values are the rows at hand
                    ctxs.append(F.chunk_attention(part(qs, b), kb, vb, sink, m.heads, m.kv_heads, m.chunk, m.scale))
            ctx = F.head_gate(self._stack(ctxs), gate, m.heads)
            y = F.linear(ctx, P[q + "w_out"], out_dtype="F32")
            hidden = F.post_norm_add(hidden, y, P[p + "norm_1.gamma"], cfg.residual_mult, cfg.eps)
            if L.ffn_dim is not None:
                f, h = p + "feed_forward.", self._operand(hidden)
                act = F.swiglu(F.linear(h, P[f + "w_gate"]), F.linear(h, P[f + "w_up"]))
                y = F.linear(act, P[f + "w_down"], out_dtype="F32")
                hidden = F.post_norm_add(hidden, y, P[p + "norm_2.gamma"], cfg.residual_mult, cfg.eps)
        if pick is not None:
            hidden = hidden.take(pick)
        elif last_only:
            hidden = self._stack([hidden.slice([sum(lens[:b + 1]) - 1, 0], [1, cfg.embed_dim]) for b in range(B)])
        normed, *_ = F.rms_norm(hidden, P["final_norm.gamma"], cfg.eps)
        logits = F.linear(self._operand(normed), P["lm_head"], out_dtype="F32")
        if cfg.logit_softcap is not None:
            logits = F.softcap(logits, cfg.logit_softcap)
        fb.set_results([t for b in range(B) for slot in new[b] for t in slot] + [logits])
        prog = Program(fb)
        self._programs[key] = (prog, layout)
        return prog, layout

    # -- what a layer keeps per sequence -------------------------------------------------
    def _position_args(self, offs):
        return [self._upload_i32([v for o in offs for v in (0, o % n, 0)]) for n in self.chunks]

    def _slot_dims(self, i, rows):
        m = self.config.layers[i].mixer
        return (m.kv_heads, rows, m.dim), (m.kv_heads, rows, m.vdim)

    def _fresh_slot(self, i, capacity):
        return [self._zeros(d) for d in self._slot_dims(i, self.config.layers[i].mixer.rows(capacity))]

    def _slot_handles(self, slot):
        return [slot.keys, slot.values]

    def _grown_slot(self, i, slot, capacity):
        rows = self.config.layers[i].mixer.rows(capacity)
        if slot.capacity >= rows:
            return slot
        return DecodeKvCache(*(self._grow_rows(h, d, rows) for h, d in zip((slot.keys, slot.values), self._slot_dims(i, slot.capacity))), slot.len, rows)

    def _new_slot(self, i, handles, length, capacity):
        return DecodeKvCache(next(handles), next(handles), length, self.config.layers[i].mixer.rows(capacity))


# kind of a checkpoint -> (class, default storage dtype); `architecture` of a model folder's config.json -> kind
MODEL_KINDS = {"gpt": (Gpt, "F32"), "ministral": (Ministral, "Bf16"), "dadupel": (Dadupel, "Bf16"), "fuzazen": (Fuzazen, "Bf16")}
KIND_OF_ARCHITECTURE = {"Dadupel": "dadupel", "Fuzazen": "fuzazen"}


# ================================================================================ BatchGenerator
class BatchGenerator:
    """Greedy generation for several independent sequences at once, of equal prompt length unless the model takes batches of
    unequal rows (`ragged_batches`) (the reference decodes one
    sequence per model call; its batch is a host-side loop): rows stacked through `forward_batch`, one attention launch
    per layer for all of them.  On a backend with sample_decode_rows_begin / _wait the loop is pipelined like
    `Generator`: the tokens of step t stay on the device as the input of step t + 1, which is queued before the host
    has seen them; elsewhere the rows are arg-maxed on the host (sampler.rs:96-103, last maximum... first index wins
    here as on the device).  The context window does not slide: generation stops at the context length."""

    def __init__(self, model, prompts: Sequence[Sequence[int]], kv_cache_capacity: Optional[int] = None):
        if len(prompts) == 0 or len(prompts[0]) == 0:
            raise ValueError("prompts must be non-empty")
        if any(len(p) == 0 for p in prompts):
            raise ValueError("prompts must be non-empty")
        if any(len(p) != len(prompts[0]) for p in prompts) and not getattr(model, "ragged_batches", False):
            raise ValueError("all prompts of a batch must have equal length")
        self.model = model
        self.batch = len(prompts)
        self.tokens = [list(p) for p in prompts]
        self.capacity = kv_cache_capacity
        self.caches = [[None] * model.num_layers for _ in prompts]
        self.pipelined = hasattr(model.backend, "sample_decode_rows_begin")
        self.logits = model.forward_batch(self.tokens, 0, self.caches, self.capacity, last_logits_only=True)
        self.lens = [len(p) for p in prompts]

    @property
    def processed_len(self) -> int:
        """Tokens of the longest sequence that have gone through the model."""
        return max(self.lens)

    def _offset(self):
        """Positions of the next tokens: one number while all sequences have one length."""
        return self.lens[0] if min(self.lens) == max(self.lens) else list(self.lens)

    def step(self) -> List[int]:
        """Samples one token per sequence and runs the forward that consumes them."""
        be, B = self.model.backend, self.batch
        if self.processed_len >= self.model.context_length:
            raise ValueError("context length reached")
        if self.pipelined:
            ticket = be.sample_decode_rows_begin(self.logits)
            self.logits = self.model.forward_batch([[None]] * B, self._offset(), self.caches, self.capacity,
                                                   token_handle=be.decode_rows_tensor(B))
            nxt = be.sample_decode_rows_wait(ticket, B)
        else:
            rows = be.to_numpy(self.logits)
            nxt = [int(np.argmax(rows[b])) for b in range(B)]
            self.logits = self.model.forward_batch([[t] for t in nxt], self._offset(), self.caches, self.capacity)
        self.lens = [n + 1 for n in self.lens]
        for b in range(B):
            self.tokens[b].append(nxt[b])
        return nxt

    def generate(self, max_new_tokens: int) -> List[List[int]]:
        out = [[] for _ in range(self.batch)]
        for _ in range(max_new_tokens):
            for b, t in enumerate(self.step()):
                out[b].append(t)
        return out


# ================================================================================ host sampler
class Sampler:
    """The reference's host sampler (crates/gpt-rs/src/inference/sampler.rs:7-104): what a generation loop falls back to
    when the backend answers `Ok(None)` to sample_decode_token, and the only path for top-k (sampler.rs:74-76: a request
    with top_k is never offered to the backend).

    `sample(row, rng)`: temperature <= 0 -> arg-max (the LAST of equal maxima, as `Iterator::max_by` returns it).  Otherwise
    logits / temperature in f32; with top_k = k < len every value below the k-th largest becomes -inf (values equal to it
    stay); softmax with the maximum taken out; a sum that is not finite or not positive falls back to arg-max; the token is
    drawn from the cumulative f32 weights as `WeightedIndex` does (a uniform draw in [0, total), first cumulative weight
    above it).  The reference draws from `thread_rng()`, which no one can replay: `rng` is a numpy Generator here, so the
    distribution is the reference's and the stream is this implementation's own."""

    def __init__(self, temperature: float, top_k: Optional[int] = None):
        self.temperature = float(temperature)
        self.top_k = None if top_k is None else max(int(top_k), 1)   # with_top_k: k.max(1)

    @staticmethod
    def argmax(values: np.ndarray) -> int:
        v = np.asarray(values, np.float32).reshape(-1)
        if v.size == 0:
            return 0
        return int(v.size - 1 - np.argmax(v[::-1]))

    def adjusted(self, row: np.ndarray) -> np.ndarray:
        """logits / temperature with everything below the k-th largest value at -inf (sampler.rs:34-50)."""
        adj = (np.asarray(row, np.float32).reshape(-1) / np.float32(self.temperature)).astype(np.float32)
        k = self.top_k
        if k is not None and 0 < k < adj.size:
            kth = np.partition(adj, adj.size - k)[adj.size - k]
            adj = np.where(adj < kth, np.float32(-np.inf), adj).astype(np.float32)
        return adj

    def probabilities(self, row: np.ndarray) -> Optional[np.ndarray]:
        """The f32 weights the draw is made from; None where the reference falls back to arg-max."""
        adj = self.adjusted(row)
        with np.errstate(over="ignore", invalid="ignore"):
            probs = np.exp(adj - np.max(adj), dtype=np.float32)
            total = np.cumsum(probs, dtype=np.float32)[-1]   # the f32 running sum, in order, of `iter().sum()`
        if not np.isfinite(total) or total <= 0.0:
            return None
        return (probs * (np.float32(1.0) / total)).astype(np.float32)

    def sample(self, row: np.ndarray, rng: np.random.Generator) -> int:
        row = np.asarray(row, np.float32).reshape(-1)
        if row.size == 0:
            raise ValueError("cannot sample from empty logits")
        if self.temperature <= 0.0:
            return self.argmax(row)
        probs = self.probabilities(row)
        if probs is None or not np.all(np.isfinite(probs)):
            return self.argmax(row)
        cum = np.cumsum(probs, dtype=np.float32)
        total = cum[-1]
        if not total > 0.0:
            return self.argmax(row)
        # WeightedIndex draws in [0, total): the f32 rounding of the draw must not reach `total`, or the last index would
        # be picked even where its weight is zero (a token that top-k masked)
        x = min(np.float32(rng.uniform(0.0, float(total))), np.nextafter(total, np.float32(0.0)))
        return int(min(np.searchsorted(cum, x, side="right"), row.size - 1))

    def supports_backend_decode_sampling(self) -> bool:
        return self.top_k is None

    def decode_sample_request(self, rng: np.random.Generator) -> Optional[dict]:
        """sampler.rs:78-93: None with top-k; greedy; or the temperature with a uniform draw in [eps, 1 - eps)."""
        if not self.supports_backend_decode_sampling():
            return None
        if self.temperature <= 0.0:
            return {"temperature": 0.0, "top_k": None, "random_u": None}
        eps = float(np.finfo(np.float32).eps)
        return {"temperature": self.temperature, "top_k": None, "random_u": float(np.float32(rng.uniform(eps, 1.0 - eps)))}


# ================================================================================ Generator
class Generator:
    """Generation loop, greedy by default (crates/gpt-rs/src/inference/generate.rs:37-203).

    With `device_sampling` the token comes from backend.sample_decode_token (spec.rs:1333-1348)
    and only 8 bytes cross PCIe per step; otherwise, where the backend declines (`Ok(None)`), and always with `top_k`
    (sampler.rs:74-76), the last logits row is read back and the host `Sampler` draws the token.

    `pipelined` (default: on when the backend offers sample_decode_token_begin / _wait and sampling is on the
    device): a step queues the sampling of token t, then the forward of step t + 1 fed by the device copy of that
    token, and only then waits for token t, so the device never idles for the host round trip.  Same tokens as
    the unpipelined loop; an error of step t + 1's launch surfaces one step later.
    """

    def __init__(self, model, prompt: Sequence[int], kv_cache_capacity: Optional[int] = None,
                 device_sampling: bool = True, temperature: float = 0.0, seed: int = 0,
                 pipelined: Optional[bool] = None, last_logits_only: bool = True, top_k: Optional[int] = None):
        if len(prompt) == 0:
            raise ValueError("prompt must be non-empty")
        self.sampler = Sampler(temperature, top_k)
        if not self.sampler.supports_backend_decode_sampling():
            if pipelined:
                raise ValueError("pipelined generation needs device sampling: top-k is sampled on the host")
            device_sampling = False
        self.model = model
        self.tokens = list(prompt)
        self.capacity = kv_cache_capacity
        self.device_sampling = device_sampling
        # temperature > 0: the backend samples from softmax(logits / temperature) given a uniform draw per
        # step (DecodeSampleRequest.random_u, spec.rs:1270-1284; sampler.rs:83-93 draws it in (eps, 1 - eps))
        self.temperature = float(temperature)
        # the loop only ever samples from the last row: prefill runs the head on that row alone (`self.logits` is then
        # [1, V] after a prefill as after a decode step); False keeps every row as the reference's forward does
        self.last_logits_only = bool(last_logits_only)
        self._rng = np.random.default_rng(seed)
        can_pipeline = device_sampling and hasattr(model.backend, "sample_decode_token_begin") and \
            hasattr(model, "forward_decode_device_token")
        if pipelined and not can_pipeline:
            raise ValueError("pipelined generation needs device sampling and a backend with sample_decode_token_begin")
        self.pipelined = can_pipeline if pipelined is None else bool(pipelined)
        self.caches: List[Optional[DecodeKvCache]] = [None] * model.num_layers
        self.window_start = max(0, len(self.tokens) - model.context_length)
        context = self.tokens[self.window_start:]
        self.logits = self._prefill(context)
        self.processed_len = len(context)

    def _sample(self) -> int:
        be = self.model.backend
        if self.device_sampling:
            req = self.sampler.decode_sample_request(self._rng)
            if req is not None:
                state = self._rng.bit_generator.state
                tok = be.sample_decode_token(self.logits, temperature=req["temperature"], random_u=req["random_u"])
                if tok is not None:
                    return tok
                self._rng.bit_generator.state = state   # Ok(None): the host sampler draws instead
        row = be.to_numpy(self.logits)
        return self.sampler.sample(row[-1] if row.ndim == 2 else row, self._rng)

    def _prefill(self, context):
        if self.last_logits_only:
            return self.model.forward_with_decode_cache(context, 0, self.caches, self.capacity, last_logits_only=True)
        return self.model.forward_with_decode_cache(context, 0, self.caches, self.capacity)

    def _draw_u(self) -> float:
        eps = float(np.finfo(np.float32).eps)
        return float(np.float32(self._rng.uniform(eps, 1.0 - eps)))

    def _step_pipelined(self) -> Optional[int]:
        """Queue sampling + next forward, then wait for the token.  None: the backend declined (nothing queued)."""
        be = self.model.backend
        if self.temperature > 0.0:
            state = self._rng.bit_generator.state
            ticket = be.sample_decode_token_begin(self.logits, temperature=self.temperature, random_u=self._draw_u())
            if ticket is None:
                self._rng.bit_generator.state = state   # the unpipelined path draws again
                return None
        else:
            ticket = be.sample_decode_token_begin(self.logits, temperature=0.0)
            if ticket is None:
                return None
        self.logits = self.model.forward_decode_device_token(be.decode_token_tensor(), self.processed_len, self.caches,
                                                             self.capacity)
        self.processed_len += 1
        nxt = be.sample_decode_token_wait(ticket)
        self.tokens.append(nxt)
        return nxt

    def step(self) -> int:
        if self.pipelined and self.processed_len < self.model.context_length:
            nxt = self._step_pipelined()
            if nxt is not None:
                return nxt
        nxt = self._sample()
        self.tokens.append(nxt)
        if self.processed_len >= self.model.context_length:
            # generate.rs:127-134: slide the window and rebuild the caches
            self.caches = [None] * self.model.num_layers
            self.window_start = len(self.tokens) - self.model.context_length
            context = self.tokens[self.window_start:]
            self.logits = self._prefill(context)
            self.processed_len = len(context)
        else:
            self.logits = self.model.forward_with_decode_cache([nxt], self.processed_len, self.caches, self.capacity)
            self.processed_len += 1
        return nxt

    def step_final(self) -> int:
        nxt = self._sample()
        self.tokens.append(nxt)
        return nxt

    def generate(self, max_new_tokens: int) -> List[int]:
        out = []
        for i in range(max_new_tokens):
            out.append(self.step() if i + 1 < max_new_tokens else self.step_final())
        return out
