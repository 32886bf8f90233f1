"""Small Dadupel models for tests: configurations, random weights in the layout of a model folder, and a writer of such folders.
Nothing here uses the product's code."""
import json
import os
import struct

import numpy as np


def ssm(heads=4, vdim=16, state=16, groups=2, conv=4, norm_groups=2, ff=64, limit=1.2):
    return {"type": "mamba2", "mixer": dict(heads=heads, vdim=vdim, state=state, groups=groups, conv=conv, norm_groups=norm_groups),
            "mlp": None if ff is None else {"kind": "dense", "ff": ff, "limit": limit}}


def latent(heads=3, dim=16, rot_dim=8, vdim=24, q_rank=40, kv_rank=24, scale=None, base=500.0, scaling=(4.0, 64, 8.0, 1.0), kv_from=None, ff=64, limit=1.2):
    rot = {"dims": rot_dim, "base": base}
    if scaling is not None:
        rot["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    m = dict(heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, q_rank=q_rank, kv_rank=kv_rank, rot=rot,
             scale=(dim + rot_dim) ** -0.5 if scale is None else scale)
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m, "mlp": None if ff is None else {"kind": "dense", "ff": ff, "limit": limit}}


def config(layers, width=64, vocab=96, eps=1e-5):
    return {"architecture": "Dadupel", "layers": layers, "norm": {"eps": eps}, "vocab": vocab, "width": width}


def bf16(x):
    """Nearest bf16 values, as f32."""
    u = np.ascontiguousarray(x, np.float32).view(np.uint32)
    return (((u + 0x7FFF + ((u >> 16) & 1)) >> 16) << 16).astype(np.uint32).view(np.float32)


def weights(cfg, seed=0, sharp=2.5):
    """bf16-representable tensors of a model folder.  `sharp` widens the attention scores, so that single keys matter."""
    rng = np.random.default_rng(seed)
    d, W = cfg["width"], {}

    def mat(name, rows, cols, gain=1.0):
        W[name] = rng.standard_normal((rows, cols)) * gain * cols ** -0.5

    def vec(name, n, mean=0.0, std=0.1):
        W[name] = mean + std * rng.standard_normal(n)

    W["embed"] = rng.standard_normal((cfg["vocab"], d))
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        vec(p + "norm1", d, 1.0)
        vec(p + "norm1.b", d)
        q = p + "mix."
        if L["type"] == "mamba2":
            inner, bc = m["heads"] * m["vdim"], m["groups"] * m["state"]
            mat(q + "in", 2 * inner + 2 * bc + m["heads"], d)
            W[q + "conv"] = rng.standard_normal((inner + 2 * bc, m["conv"])) * 0.5
            vec(q + "conv.b", inner + 2 * bc)
            vec(q + "dt_bias", m["heads"], -3.0, 0.5)       # small steps: states reach far back
            vec(q + "A_log", m["heads"], -1.0, 0.5)
            vec(q + "D", m["heads"], 1.0)
            vec(q + "norm", inner, 1.0)
            mat(q + "o", d, inner)
        else:
            H, hd = m["heads"], m["dim"] + m["rot_dim"]
            mat(q + "dq", m["q_rank"], d)
            vec(q + "dq.norm", m["q_rank"], 1.0)
            mat(q + "uq", H * hd, m["q_rank"], sharp)
            if m.get("kv_from") is None:
                mat(q + "dkv", m["kv_rank"] + m["rot_dim"], d)
                vec(q + "dkv.norm", m["kv_rank"], 1.0)
            mat(q + "uk", H * m["dim"], m["kv_rank"])
            mat(q + "uv", H * m["vdim"], m["kv_rank"])
            mat(q + "o", d, H * m["vdim"])
        vec(p + "ls1", d, 0.8, 0.2)
        if L["mlp"] is not None:
            ff = L["mlp"]["ff"]
            mat(p + "mlp.gate", ff, d)
            mat(p + "mlp.up", ff, d)
            mat(p + "mlp.down", d, ff)
            vec(p + "ls2", d, 0.6, 0.2)
    vec("final.norm", d, 1.0)
    vec("final.norm.b", d)
    return {k: bf16(v) for k, v in W.items()}


def write_folder(path, cfg, W, extra=None):
    """config.json and model.safetensors (BF16) under `path`."""
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    head, blobs, off = {"__metadata__": {"format": "pt"}}, [], 0
    tensors = dict(W, **(extra or {}))
    for name, a in tensors.items():
        data = (np.ascontiguousarray(a, np.float32).view(np.uint32) >> 16).astype("<u2").tobytes()
        head[name] = {"dtype": "BF16", "shape": list(a.shape), "data_offsets": [off, off + len(data)]}
        blobs.append(data)
        off += len(data)
    js = json.dumps(head).encode()
    js += b" " * (-len(js) % 8)
    with open(os.path.join(path, "model.safetensors"), "wb") as f:
        f.write(struct.pack("<Q", len(js)) + js + b"".join(blobs))
    return path


# Layer stacks whose sizes differ from each other in every respect: one head, one group, no feed-forward, no scaling, short and
# long filters, widths and ranks on and off the tilings of the kernels
STACKS = {
    "mixed": config([ssm(), latent(), ssm(heads=6, vdim=8, state=8, groups=3, conv=3, norm_groups=1), latent(heads=5, dim=8, vdim=16, q_rank=24, kv_from=1)]),
    "tiled": config([latent(heads=4, dim=32, rot_dim=32, vdim=32, q_rank=64, kv_rank=64, ff=128), ssm(heads=8, vdim=32, state=64, groups=4, norm_groups=4, ff=128),
                     latent(heads=24, dim=16, rot_dim=32, vdim=8, q_rank=64, kv_rank=64, kv_from=0, ff=128)], width=128, vocab=160),
    "odd": config([ssm(heads=3, vdim=20, state=12, groups=1, conv=2, norm_groups=3, ff=None), latent(heads=1, dim=10, rot_dim=6, vdim=7, q_rank=9, kv_rank=11, scaling=None, ff=36),
                   ssm(heads=5, vdim=4, state=5, groups=5, conv=5, norm_groups=1, ff=52)], width=36, vocab=50),
    "deep_share": config([latent(scaling=(2.0, 32, 16.0, 2.0)), latent(kv_from=0, ff=None), latent(heads=2, base=50.0, scaling=None, ff=None), latent(heads=7, dim=24, kv_from=0, scaling=(2.0, 32, 16.0, 2.0))]),
}
