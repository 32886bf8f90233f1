"""Plain, slow CPU implementation of the Fuzazen design (test infrastructure: nothing in the product imports it).

One function per mechanism, written from the design's equations with numpy and plain loops over tokens; it shares no
code with the product path.  `dt` chooses the arithmetic (float64 by default, float32 for rounding studies).

Notation: x[T, width] rows of one sequence; a weight W is stored [out, in] and applied as x @ W.T.
"""
from __future__ import annotations

import numpy as np


# ------------------------------------------------------------------------------------------ row functions
def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def over_rms(x, eps):
    """Every last-axis row divided by its root mean square."""
    return x / np.sqrt((x * x).mean(axis=-1, keepdims=True) + eps)


def post_norm_add(x, y, w, mult, eps):
    """The residual update of a sublayer whose OUTPUT is normed: x + mult * y / rms(y) * w."""
    return x + mult * (over_rms(y, eps) * w)


def softcap(z, cap):
    return cap * np.tanh(z / cap)


# ------------------------------------------------------------------------------------------ attention
def rotate_leading_pairs(x, positions, dims, base):
    """x[T, heads, D]: the pairs (2i, 2i + 1), i < dims / 2, turn by position * base^(-2i / dims); the rest stays."""
    out = x.copy()
    for i in range(dims // 2):
        a = np.asarray(positions, np.float64) * float(base) ** (-2.0 * i / dims)
        c, s = np.cos(a).astype(x.dtype)[:, None], np.sin(a).astype(x.dtype)[:, None]
        u, v = x[:, :, 2 * i], x[:, :, 2 * i + 1]
        out[:, :, 2 * i] = u * c - v * s
        out[:, :, 2 * i + 1] = v * c + u * s
    return out


def sink_softmax(s, sink):
    """Weights of the scores s when the denominator also holds exp(sink)."""
    top = max(s.max(), sink)
    e = np.exp(s - top)
    return e / (e.sum() + np.exp(sink - top))


def chunk_attend(q, k, v, sink, scale, chunk, start):
    """Queries q[T, H, D] at positions start, start + 1, ... over keys k[L, G, D] and values v[L, G, V] of positions 0 .. L - 1:
    a query sees the keys of its own chunk of `chunk` positions up to itself."""
    T, H = q.shape[:2]
    G = k.shape[1]
    out = np.empty((T, H, v.shape[2]), q.dtype)
    for t in range(T):
        p = start + t
        lo = p // chunk * chunk
        for h in range(H):
            g = h // (H // G)
            w = sink_softmax((k[lo:p + 1, g] @ q[t, h]) * scale, sink[h])
            out[t, h] = w @ v[lo:p + 1, g]
    return out


def attention_mixer(x, W, p, m, eps, held, start):
    """held: (k[L, G, D], v[L, G, V]) of the positions before `start`, or None; returns (rows, (k, v) with the new ones)."""
    T = x.shape[0]
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    pos = np.arange(start, start + T)
    q = (x @ W[p + "q"].T).reshape(T, H, D)
    k = (x @ W[p + "k"].T).reshape(T, G, D)
    v = (x @ W[p + "v"].T).reshape(T, G, V)
    q, k = (over_rms(rotate_leading_pairs(t, pos, m["rot"]["dims"], m["rot"]["base"]), eps) for t in (q, k))
    if held is not None:
        k, v = np.concatenate([held[0], k]), np.concatenate([held[1], v])
    ctx = chunk_attend(q, k, v, W[p + "sink"], m["scale"], m["mask"]["size"], start)
    ctx = ctx * sigmoid(x @ W[p + "g"].T)[:, :, None]
    return ctx.reshape(T, H * V) @ W[p + "o"].T, (k, v)


# ------------------------------------------------------------------------------------------ feed-forward, model
def gated_feed_forward(x, W, p):
    return (silu(x @ W[p + "gate"].T) * (x @ W[p + "up"].T)) @ W[p + "down"].T


def owner(config, i):
    """The layer whose tensors layer i uses."""
    while config["layers"][i].get("weights_of") is not None:
        i = config["layers"][i]["weights_of"]
    return i


class Reference:
    """The whole model over the mechanisms above.  `state` (per sequence) holds every layer's keys and values."""

    def __init__(self, config, weights, dt_type=np.float64):
        self.c, self.dt = config, dt_type
        self.W = {k: np.asarray(v, dt_type) for k, v in weights.items()}

    def forward(self, tokens, state=None, layers_out=None):
        """Runs `tokens` after what `state` already holds; returns (logits [T, vocab], state)."""
        c, W, eps, mult = self.c, self.W, self.c["norm"]["eps"], self.c["residual_mult"]
        st = {"n": 0, "layer": [None] * len(c["layers"])} if state is None else state
        start = st["n"]
        x = W["embed"][np.asarray(tokens)] * self.dt(c["embedding"]["scale"])
        new = [None] * len(c["layers"])
        for i, L in enumerate(c["layers"]):
            p = f"l{owner(c, i)}."
            y, new[i] = attention_mixer(x, W, p + "mix.", L["mixer"], eps, st["layer"][i], start)
            x = post_norm_add(x, y, W[p + "norm1"], mult, eps)
            if L["mlp"] is not None:
                x = post_norm_add(x, gated_feed_forward(x, W, p + "mlp."), W[p + "norm2"], mult, eps)
            if layers_out is not None:
                layers_out.append(x.copy())
        logits = softcap((over_rms(x, eps) * W["final.norm"]) @ W["head"].T, c["logit_softcap"])
        return logits, {"n": start + len(tokens), "layer": new}
