"""A plain, slow implementation of the Ruzolorn decoder: whole sequences, no cache, no state carried
between calls, one function per mechanism, numpy float64.  It shares no code with the engine: the
tests compare the two.

The design in short.  x = scale E[token].  A norm LN (layer norm, a gain and no bias) stands in front
of every sublayer and another behind it: x += m LN_1b(mixer(LN_1(x))), x += m LN_2b(ff(LN_2(x))) with
one number m; the second is missing where a layer has no feed-forward.  Mixers: `parallel`, a softmax
attention (grouped queries, an RMS norm on every q and k head, no positions, a sliding window) beside
a Mamba-2 layer (a short convolution on its inputs, per head a matrix state under a decay that the
token sets, a gate before a norm in parts), added with fixed factors; `retention`, linear attention
with a fixed decay per head, rotated queries and keys, each head's output divided by its root mean
square and gated.  Feed-forward: routed experts (softmax scores, a correction for the choice only,
the last few router rows standing for the input itself) and a shared expert.  Logits: W_head LN(x).

`config` is the model's config.json as a dict, `w` maps tensor names to arrays.
"""
from __future__ import annotations

from typing import Dict, List, Optional, Sequence

import numpy as np

Weights = Dict[str, np.ndarray]


def layer_norm(x: np.ndarray, g: np.ndarray, eps: float) -> np.ndarray:
    """(x - mean) / sqrt(var + eps) * g along the last axis, var the mean squared deviation."""
    d = x - np.mean(x, axis=-1, keepdims=True)
    return d / np.sqrt(np.mean(d * d, axis=-1, keepdims=True) + eps) * g


def over_rms(x: np.ndarray, eps: float) -> np.ndarray:
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def sigmoid(z: np.ndarray) -> np.ndarray:
    return 1.0 / (1.0 + np.exp(-z))


def silu(z: np.ndarray) -> np.ndarray:
    return z * sigmoid(z)


def softplus(z: np.ndarray) -> np.ndarray:
    return np.logaddexp(0.0, z)


def window_softmax(scores: np.ndarray, window: int) -> np.ndarray:
    """scores [T, T] -> weights; row i sees the columns j with 0 <= i - j < window."""
    T = scores.shape[0]
    back = np.arange(T)[:, None] - np.arange(T)[None, :]
    s = np.where((back >= 0) & (back < window), scores, -np.inf)
    e = np.exp(s - s.max(axis=-1, keepdims=True))
    return e / e.sum(axis=-1, keepdims=True)


def window_attention(h: np.ndarray, m: dict, w: Weights, name: str, eps: float) -> np.ndarray:
    T = h.shape[0]
    H, d = m["heads"], m["dim"]
    G, dv = m.get("kv_heads", H), m.get("vdim", d)
    q = over_rms((h @ w[name + ".q"].T).reshape(T, H, d), eps) * w[name + ".q.norm"]
    k = over_rms((h @ w[name + ".k"].T).reshape(T, G, d), eps) * w[name + ".k.norm"]
    v = (h @ w[name + ".v"].T).reshape(T, G, dv)
    window = m["mask"]["size"] if m.get("mask") else T
    o = np.zeros((T, H, dv))
    for j in range(H):
        g = j // (H // G)
        o[:, j] = window_softmax(q[:, j] @ k[:, g].T * m["scale"], window) @ v[:, g]
    return o.reshape(T, H * dv) @ w[name + ".o"].T


def causal_convolution(u: np.ndarray, taps: np.ndarray, bias: np.ndarray) -> np.ndarray:
    """u [T, C], taps [C, K], the last column the current token's, zeros in front of the sequence."""
    T, C = u.shape
    K = taps.shape[1]
    padded = np.concatenate([np.zeros((K - 1, C)), u])
    return sum(padded[j:j + T] * taps[:, j] for j in range(K)) + bias


def mamba2(h: np.ndarray, m: dict, w: Weights, name: str, eps: float) -> np.ndarray:
    T = h.shape[0]
    H, N, G, P = m["heads"], m["state"], m["groups"], m["vdim"]
    inner = H * P
    z, xbc, dt = np.split(h @ w[name + ".in"].T, [inner, 2 * inner + 2 * G * N], axis=-1)
    xbc = silu(causal_convolution(xbc, w[name + ".conv"], w[name + ".conv.b"]))
    x = xbc[:, :inner].reshape(T, H, P)
    B = xbc[:, inner:inner + G * N].reshape(T, G, N)
    C = xbc[:, inner + G * N:].reshape(T, G, N)
    dt = softplus(dt + w[name + ".dt_bias"])
    y = np.zeros((T, H, P))
    for j in range(H):
        g = j // (H // G)
        S = np.zeros((N, P))
        for t in range(T):
            S = np.exp(-np.exp(w[name + ".A_log"][j]) * dt[t, j]) * S + dt[t, j] * np.outer(B[t, g], x[t, j])
            y[t, j] = S.T @ C[t, g] + w[name + ".D"][j] * x[t, j]
    y = y.reshape(T, inner) * silu(z)
    parts = m.get("norm_groups", 1)
    y = over_rms(y.reshape(T, parts, inner // parts), eps).reshape(T, inner) * w[name + ".norm"]
    return y @ w[name + ".o"].T


def parallel_mixer(h: np.ndarray, m: dict, w: Weights, name: str, eps: float) -> np.ndarray:
    left = window_attention(h, m["left"], w, name + ".left", eps)
    right = mamba2(h, m["right"], w, name + ".right", eps)
    return m["left_scale"] * left + m["right_scale"] * right


def rotate_half(x: np.ndarray, rot: Optional[dict]) -> np.ndarray:
    """x [T, heads, d]: entry i of the first rot.dims turns with entry i + dims/2 by p * base^(-2i/dims)."""
    if not rot or not rot.get("dims"):
        return x
    dims, base = rot["dims"], rot["base"]
    half = dims // 2
    a = np.arange(x.shape[0])[:, None] * np.array([base ** (-2.0 * i / dims) for i in range(half)])
    c, s = np.cos(a)[:, None, :], np.sin(a)[:, None, :]
    u, v = x[..., :half], x[..., half:dims]
    return np.concatenate([u * c - v * s, v * c + u * s, x[..., dims:]], axis=-1)


def retention(h: np.ndarray, m: dict, w: Weights, name: str, eps: float) -> np.ndarray:
    T = h.shape[0]
    H, d = m["heads"], m["dim"]
    dv = m.get("vdim", d)
    q = rotate_half((h @ w[name + ".q"].T).reshape(T, H, d), m.get("rot"))
    k = rotate_half((h @ w[name + ".k"].T).reshape(T, H, d), m.get("rot")) * d ** -0.5
    v = (h @ w[name + ".v"].T).reshape(T, H, dv)
    o = np.zeros((T, H, dv))
    for j in range(H):
        S = np.zeros((d, dv))
        for t in range(T):
            S = m["decay"][j] * S + np.outer(k[t, j], v[t, j])
            o[t, j] = S.T @ q[t, j]
    o = over_rms(o, eps).reshape(T, H * dv) * silu(h @ w[name + ".g"].T)
    return o @ w[name + ".o"].T


def gated_ff(h: np.ndarray, w: Weights, name: str) -> np.ndarray:
    return (silu(h @ w[name + ".gate"].T) * (h @ w[name + ".up"].T)) @ w[name + ".down"].T


def route(h: np.ndarray, r: dict, w: Weights, name: str):
    """(chosen [T, top], weights [T, top]); numbers from `experts` on stand for the input itself."""
    z = h @ w[name + ".router"].T
    s = np.exp(z - z.max(axis=-1, keepdims=True))
    s = s / s.sum(axis=-1, keepdims=True)
    ids = np.argsort(-(s + w[name + ".correction"]), axis=-1, kind="stable")[:, :r["top"]]
    return ids, np.take_along_axis(s, ids, axis=-1)


def experts(h: np.ndarray, mlp: dict, w: Weights, name: str) -> np.ndarray:
    ids, wts = route(h, mlp["router"], w, name)
    out = np.zeros_like(h)
    for t in range(h.shape[0]):
        for e, a in zip(ids[t], wts[t]):
            out[t] += a * (h[t] if e >= mlp["router"]["experts"] else gated_ff(h[t:t + 1], w, f"{name}.e{e}")[0])
    if mlp.get("shared"):
        out = out + gated_ff(h, w, name + ".shared")
    return out


def forward(config: dict, w: Weights, tokens: Sequence[int], trace: Optional[List[np.ndarray]] = None) -> np.ndarray:
    """Logits [T, vocab] of one sequence from position 0.  `trace` collects the residual after every layer."""
    w = {k: np.asarray(v, dtype=np.float64) for k, v in w.items()}
    eps, m = config["norm"]["eps"], config.get("residual_mult", 1.0)
    x = w["embed"][np.asarray(tokens)] * (config.get("embedding") or {}).get("scale", 1.0)
    mixers = {"parallel": parallel_mixer, "retention": retention}
    for i, layer in enumerate(config["layers"]):
        name = f"l{i}"
        y = mixers[layer["type"]](layer_norm(x, w[name + ".norm1"], eps), layer["mixer"], w, name + ".mix", eps)
        x = x + m * layer_norm(y, w[name + ".norm1b"], eps)
        if layer.get("mlp"):
            y = experts(layer_norm(x, w[name + ".norm2"], eps), layer["mlp"], w, name + ".mlp")
            x = x + m * layer_norm(y, w[name + ".norm2b"], eps)
        if trace is not None:
            trace.append(x.copy())
    return layer_norm(x, w["final.norm"], eps) @ w["head"].T
