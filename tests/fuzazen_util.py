"""Small Fuzazen models for tests: configurations and random weights in the layout of a model folder.  Nothing here uses the
product's code."""
import numpy as np

from dadupel_util import bf16, write_folder  # noqa: F401


def layer(heads=4, kv_heads=2, dim=16, vdim=24, rot=8, base=500.0, chunk=7, scale=0.3, ff=48, weights_of=None):
    e = {"type": "attention", "mlp": None if ff is None else {"kind": "dense", "ff": ff},
         "mixer": dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale, rot={"dims": rot, "base": base}, mask={"size": chunk})}
    if weights_of is not None:
        e["weights_of"] = weights_of
    return e


def same(layers, i):
    """A layer that uses the weights of layers[i]."""
    return dict(layers[i], weights_of=i)


def config(layers, width=64, vocab=96, eps=1e-5, scale=0.7, mult=0.4, cap=20.0):
    return {"architecture": "Fuzazen", "layers": layers, "norm": {"eps": eps}, "vocab": vocab, "width": width, "embedding": {"scale": scale},
            "residual_mult": mult, "logit_softcap": cap}


def weights(cfg, seed=0):
    """bf16-representable tensors of a model folder."""
    rng = np.random.default_rng(seed)
    d, W = cfg["width"], {}

    def mat(name, rows, cols, gain=1.0):
        W[name] = rng.standard_normal((rows, cols)) * gain * cols ** -0.5

    def vec(name, n, mean=0.0, std=0.1):
        W[name] = mean + std * rng.standard_normal(n)

    W["embed"] = rng.standard_normal((cfg["vocab"], d))
    for i, L in enumerate(cfg["layers"]):
        if L.get("weights_of") is not None:
            continue
        p, m = f"l{i}.", L["mixer"]
        H, G, q = m["heads"], m["kv_heads"], f"l{i}.mix."
        mat(q + "q", H * m["dim"], d)
        mat(q + "k", G * m["dim"], d)
        mat(q + "v", G * m["vdim"], d)
        vec(q + "sink", H, 1.0, 1.0)
        mat(q + "g", H, d, 1.5)
        mat(q + "o", d, H * m["vdim"])
        vec(p + "norm1", d, 1.0, 0.2)
        if L["mlp"] is not None:
            ff = L["mlp"]["ff"]
            mat(p + "mlp.gate", ff, d)
            mat(p + "mlp.up", ff, d)
            mat(p + "mlp.down", d, ff)
            vec(p + "norm2", d, 1.0, 0.2)
    vec("final.norm", d, 1.0, 0.2)
    mat("head", cfg["vocab"], d, 6.0)
    return {k: bf16(v) for k, v in W.items()}


# Layer stacks whose sizes differ from each other in every respect: one key / value head, as many as queries, more queries per key
# head than a workgroup takes, partial and whole rotations, chunks of one position and longer than the sequence, no feed-forward,
# weights used by earlier and by later layers, sizes on and off the tilings of the kernels
_mixed = [layer(), layer(heads=6, kv_heads=1, dim=32, vdim=16, rot=32, chunk=20, scale=0.15, ff=None), layer(heads=3, kv_heads=3, dim=24, vdim=8, rot=4, chunk=64, ff=80)]
_tiled = [layer(heads=8, kv_heads=2, dim=128, vdim=64, rot=64, base=1e4, chunk=96, scale=0.1, ff=192),
          layer(heads=8, kv_heads=4, dim=64, vdim=128, rot=64, base=1e4, chunk=33, scale=0.12, ff=128)]
_wide = [layer(heads=40, kv_heads=2, dim=40, vdim=72, rot=24, chunk=50, scale=0.2, ff=64), layer(heads=17, kv_heads=1, dim=72, vdim=136, rot=72, chunk=300, scale=0.1, ff=32)]
_shared = [layer(chunk=16, weights_of=2), layer(heads=2, chunk=9, base=50.0, ff=None), layer(chunk=16)]
STACKS = {
    "mixed": config(_mixed + [same(_mixed, 1), same(_mixed, 0)]),
    "tiled": config(_tiled + [same(_tiled, 0)], width=128, vocab=160, scale=1.0, mult=0.25, cap=25.0),
    "odd": config([layer(heads=3, kv_heads=1, dim=10, vdim=7, rot=4, chunk=5, ff=36), layer(heads=2, kv_heads=2, dim=7, vdim=5, rot=6, chunk=1, ff=None),
                   layer(heads=5, kv_heads=5, dim=9, vdim=11, rot=8, chunk=1000, ff=52)], width=36, vocab=50, eps=1e-3, mult=1.0, cap=5.0),
    "wide": config(_wide, width=96, vocab=101),
    "shared": config(_shared + [same(_shared, 1), dict(_shared[2], weights_of=0)], mult=0.5),
}
