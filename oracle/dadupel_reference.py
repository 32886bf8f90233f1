"""Plain, slow CPU implementation of the Dadupel design (test infrastructure: nothing in the product imports it).

One function per mechanism, written from the design's equations with numpy and plain loops over tokens; it shares no
code with the product path.  `dt` chooses the arithmetic (float64 by default, float32 for rounding studies).

Notation: h[T, width] rows of one sequence; a weight W is stored [out, in] and applied as h @ W.T.
"""
from __future__ import annotations

import math

import numpy as np


# ------------------------------------------------------------------------------------------ row functions
def sigmoid(x):
    return 1.0 / (1.0 + np.exp(-x))


def silu(x):
    return x * sigmoid(x)


def softplus(x):
    return np.logaddexp(np.zeros_like(x), x)


def layer_norm(x, w, b, eps):
    mean = x.mean(axis=-1, keepdims=True)
    var = ((x - mean) ** 2).mean(axis=-1, keepdims=True)
    return (x - mean) / np.sqrt(var + eps) * w + b


def rms_norm(x, w, eps):
    return x / np.sqrt((x * x).mean(axis=-1, keepdims=True) + eps) * w


def grouped_rms_norm(x, w, groups, eps):
    """Each of `groups` equal parts of a row is divided by its own root mean square; then one gain per element."""
    T, n = x.shape
    parts = x.reshape(T, groups, n // groups)
    parts = parts / np.sqrt((parts * parts).mean(axis=-1, keepdims=True) + eps)
    return parts.reshape(T, n) * w


# ------------------------------------------------------------------------------------------ Mamba-2
def causal_conv_silu(x, taps, bias, history):
    """Depthwise convolution over time; taps[:, -1] meets the current row.  history: the K - 1 rows before x[0]."""
    T, C = x.shape
    K = taps.shape[1]
    rows = np.concatenate([history, x], axis=0)
    out = np.empty_like(x)
    for t in range(T):
        acc = bias.copy()
        for k in range(K):
            acc = acc + taps[:, k] * rows[t + k]
        out[t] = silu(acc)
    return out, rows[rows.shape[0] - (K - 1):].copy()


def selective_state_scan(x, B, C, dt, A_log, D, state):
    """x[T, heads, vdim], B / C[T, groups, N], dt[T, heads] (step sizes, after softplus), state[heads, N, vdim].
    S <- exp(-exp(A_log) dt) S + dt B x^T ;  y = S^T C + D x."""
    T, H, V = x.shape
    G = B.shape[1]
    S = state.copy()
    y = np.empty_like(x)
    for t in range(T):
        for h in range(H):
            g = h // (H // G)
            S[h] = np.exp(-np.exp(A_log[h]) * dt[t, h]) * S[h] + dt[t, h] * np.outer(B[t, g], x[t, h])
            y[t, h] = S[h].T @ C[t, g] + D[h] * x[t, h]
    return y, S


def mamba2_mixer(h, W, p, m, eps, st, dt_type=np.float64):
    """st: {"conv": [taps - 1, channels], "ssm": [heads, N, vdim]} or None; returns (rows, new state)."""
    H, V, N, G = m["heads"], m["vdim"], m["state"], m["groups"]
    inner, bc = H * V, G * N
    T = h.shape[0]
    pr = h @ W[p + "in"].T
    z, xbc, dt = pr[:, :inner], pr[:, inner:2 * inner + 2 * bc], pr[:, 2 * inner + 2 * bc:]
    if st is None:
        st = {"conv": np.zeros((m["conv"] - 1, xbc.shape[1]), dt_type), "ssm": np.zeros((H, N, V), dt_type)}
    xbc, conv = causal_conv_silu(xbc, W[p + "conv"], W[p + "conv.b"], st["conv"])
    dt = softplus(dt + W[p + "dt_bias"])
    x = xbc[:, :inner].reshape(T, H, V)
    B = xbc[:, inner:inner + bc].reshape(T, G, N)
    C = xbc[:, inner + bc:].reshape(T, G, N)
    y, ssm = selective_state_scan(x, B, C, dt, W[p + "A_log"], W[p + "D"], st["ssm"])
    y = grouped_rms_norm(y.reshape(T, inner) * silu(z), W[p + "norm"], m["norm_groups"], eps)
    return y @ W[p + "o"].T, {"conv": conv, "ssm": ssm}


# ------------------------------------------------------------------------------------------ latent attention
def rotary_tables(rot, positions):
    """cos / sin [T, dims / 2] of the interleaved rotation, with the YaRN blend of frequencies when rot["scaling"]."""
    n, base = rot["dims"], float(rot["base"])
    sc = rot.get("scaling")
    freqs, mag = [], 1.0
    for i in range(n // 2):
        f = base ** (-2.0 * i / n)
        if sc:
            def dim_of(turns):
                return n * math.log(sc["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
            lo = max(math.floor(dim_of(sc["fast"])), 0)
            hi = min(math.ceil(dim_of(sc["slow"])), n - 1)
            ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
            f = f / sc["factor"] * ramp + f * (1.0 - ramp)
        freqs.append(f)
    if sc:
        mag = 0.1 * math.log(sc["factor"]) + 1.0
    ang = np.asarray(positions, np.float64)[:, None] * np.asarray(freqs)[None, :]
    return np.cos(ang) * mag, np.sin(ang) * mag


def rotate_pairs(x, cos, sin):
    """Dimensions (2i, 2i + 1) of the last axis turn together; x[T, ..., 2 * half], cos / sin [T, half]."""
    shape = (x.shape[0],) + (1,) * (x.ndim - 2) + (cos.shape[1],)
    c, s = cos.reshape(shape), sin.reshape(shape)
    u, v = x[..., 0::2], x[..., 1::2]
    out = np.empty_like(x)
    out[..., 0::2] = u * c - v * s
    out[..., 1::2] = v * c + u * s
    return out


def latent_rows(h, W, p, m, eps, cos, sin):
    """(normed latent [T, kv_rank], rotated shared key part [T, rot_dim])."""
    r = h @ W[p + "dkv"].T
    R = m["kv_rank"]
    return rms_norm(r[:, :R], W[p + "dkv.norm"], eps), rotate_pairs(r[:, R:], cos, sin)


def latent_queries(h, W, p, m, eps, cos, sin):
    q = rms_norm(h @ W[p + "dq"].T, W[p + "dq.norm"], eps) @ W[p + "uq"].T
    q = q.reshape(h.shape[0], m["heads"], m["dim"] + m["rot_dim"])
    return q[..., :m["dim"]], rotate_pairs(q[..., m["dim"]:], cos, sin)


def latent_attend(qn, qr, c, kr, Wuk, Wuv, m, start):
    """Queries at positions start, start + 1, ... over latents c[L, R] and shared key parts kr[L, rot_dim]."""
    T, H = qn.shape[:2]
    L = c.shape[0]
    k = (c @ Wuk.T).reshape(L, H, m["dim"])
    v = (c @ Wuv.T).reshape(L, H, m["vdim"])
    out = np.empty((T, H, m["vdim"]), qn.dtype)
    for t in range(T):
        n = start + t + 1
        for h in range(H):
            s = (k[:n, h] @ qn[t, h] + kr[:n] @ qr[t, h]) * m["scale"]
            w = np.exp(s - s.max())
            out[t, h] = (w / w.sum()) @ v[:n, h]
    return out.reshape(T, H * m["vdim"])


# ------------------------------------------------------------------------------------------ feed-forward, model
def clamped_glu(gate, up, limit):
    g = np.minimum(gate, limit)
    u = np.clip(up, -limit, limit)
    return g * sigmoid(1.702 * g) * (u + 1.0)


class Reference:
    """The whole model over the mechanisms above.  `state` (per sequence) is a dict of what each layer keeps."""

    def __init__(self, config, weights, dt_type=np.float64):
        self.c, self.dt = config, dt_type
        self.W = {k: (v if v.dtype.kind == "i" else np.asarray(v, dt_type)) for k, v in weights.items()}

    def forward(self, tokens, state=None, layers_out=None):
        """Runs `tokens` after what `state` already holds; returns (logits [T, vocab], state)."""
        c, W, eps = self.c, self.W, self.c["norm"]["eps"]
        st = {"n": 0, "layer": [None] * len(c["layers"])} if state is None else state
        start, T = st["n"], len(tokens)
        pos = np.arange(start, start + T)
        x = W["embed"][np.asarray(tokens)].astype(self.dt)
        new = [None] * len(c["layers"])
        for i, L in enumerate(c["layers"]):
            p, m = f"l{i}.mix.", L["mixer"]
            h = layer_norm(x, W[f"l{i}.norm1"], W[f"l{i}.norm1.b"], eps)
            if L["type"] == "mamba2":
                mix, new[i] = mamba2_mixer(h, W, p, m, eps, st["layer"][i], self.dt)
            else:
                cos, sin = (t.astype(self.dt) for t in rotary_tables(m["rot"], pos))
                if m.get("kv_from") is None:
                    cl, kr = latent_rows(h, W, p, m, eps, cos, sin)
                    old = st["layer"][i]
                    new[i] = (cl, kr) if old is None else (np.concatenate([old[0], cl]), np.concatenate([old[1], kr]))
                cl, kr = new[i if m.get("kv_from") is None else m["kv_from"]]
                qn, qr = latent_queries(h, W, p, m, eps, cos, sin)
                mix = latent_attend(qn, qr, cl, kr, W[p + "uk"], W[p + "uv"], m, start) @ W[p + "o"].T
            delta = mix * W[f"l{i}.ls1"]
            if L["mlp"] is not None:
                q = f"l{i}.mlp."
                a = clamped_glu(h @ W[q + "gate"].T, h @ W[q + "up"].T, L["mlp"]["limit"])
                delta = delta + (a @ W[q + "down"].T) * W[f"l{i}.ls2"]
            x = x + delta
            if layers_out is not None:
                layers_out.append(x.copy())
        logits = layer_norm(x, W["final.norm"], W["final.norm.b"], eps) @ W["embed"].T
        return logits, {"n": start + T, "layer": new}
