"""A plain, slow implementation of the Lupolorn decoder: whole sequences, no cache, no state
carried between calls, one function per mechanism, numpy float64.  It shares no code with the
engine: the tests compare the two.

The design in short.  x = s E[token].  Each sublayer has an RMS norm in front and another behind:
x <- x + N1b(mixer(N1 x)), x <- x + N2b(ff(N2 x)).  Mixers: `mingru` (an element-wise recurrence
S <- (1 - z) S + z c whose gate and candidate read the current token only), `latent_attention`
(queries through a normed latent, keys and values per head from another, no positions, a sliding
window) and `attention` (grouped queries, neighbouring entries rotated in pairs by frequencies that
may be stretched, queries and keys divided by their root mean square behind the rotation, one more
in the softmax's denominator, a sigmoid gate a head).  Feed-forward: down(relu(up h)^2), or routed
experts of that form (softmax scores, not renormalised) beside a shared one behind a sigmoid gate.
Logits: E N(x).

`config` is the model's config.json as a dict, `w` maps tensor names to arrays.
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional, Sequence

import numpy as np


def unit_rms(x: np.ndarray, eps: float) -> np.ndarray:
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def rms_norm(x: np.ndarray, g: np.ndarray, eps: float) -> np.ndarray:
    return unit_rms(x, eps) * g


def sigmoid(z: np.ndarray) -> np.ndarray:
    e = np.exp(-np.abs(z))
    return np.where(z >= 0, 1.0, e) / (1.0 + e)


def silu(z: np.ndarray) -> np.ndarray:
    return z * sigmoid(z)


def relu_squared(z: np.ndarray) -> np.ndarray:
    return np.maximum(z, 0.0) ** 2


def frequencies(rot: dict) -> np.ndarray:
    """base^(-2i/dims), i < dims/2; with `scaling` the long wavelengths divided by factor, the short ones kept, and a
    straight mix of the two in between."""
    out = []
    for i in range(rot["dims"] // 2):
        f = rot["base"] ** (-2.0 * i / rot["dims"])
        sc = rot.get("scaling")
        if sc:
            turns = sc["original"] / (2.0 * math.pi / f)       # whole turns inside the original length
            if turns < sc["low"]:
                f = f / sc["factor"]
            elif turns <= sc["high"]:
                s = (turns - sc["low"]) / (sc["high"] - sc["low"])
                f = (1.0 - s) * f / sc["factor"] + s * f
        out.append(f)
    return np.array(out)


def rotate_pairs(x: np.ndarray, positions: Sequence[int], rot: Optional[dict]) -> np.ndarray:
    """x [T, heads, d]: entries 2i and 2i + 1 turn together by p f_i; the entries from rot.dims on pass."""
    if not rot or not rot.get("dims"):
        return x
    f = frequencies(rot)
    out = x.copy()
    for t, p in enumerate(positions):
        for i in range(len(f)):
            c, s = math.cos(p * f[i]), math.sin(p * f[i])
            u, v = x[t, :, 2 * i], x[t, :, 2 * i + 1]
            out[t, :, 2 * i] = u * c - v * s
            out[t, :, 2 * i + 1] = v * c + u * s
    return out


def visible(T: int, window: Optional[int]) -> np.ndarray:
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    vis = j <= i
    if window:
        vis &= i - j < window
    return vis


def softmax_over(scores: np.ndarray, vis: np.ndarray, one_more: bool) -> np.ndarray:
    """Row-wise weights over the visible columns; `one_more`: the denominator holds 1 + the sum."""
    s = np.where(vis, scores, -np.inf)
    m = s.max(axis=-1, keepdims=True)
    if one_more:
        m = np.maximum(m, 0.0)
    e = np.exp(s - m)
    den = e.sum(axis=-1, keepdims=True)
    if one_more:
        den = den + np.exp(-m)
    return e / den


def mingru(h: np.ndarray, w: Dict[str, np.ndarray], name: str) -> np.ndarray:
    z = sigmoid(h @ w[name + ".z"].T + w[name + ".z.b"])
    u = h @ w[name + ".x"].T + w[name + ".x.b"]
    cand = np.where(u >= 0, u + 0.5, sigmoid(u))
    S = np.zeros(z.shape[1])
    states = np.zeros_like(z)
    for t in range(h.shape[0]):
        S = (1.0 - z[t]) * S + z[t] * cand[t]
        states[t] = S
    return (states * silu(h @ w[name + ".g"].T)) @ w[name + ".o"].T


def latent_attention(h: np.ndarray, m: dict, w: Dict[str, np.ndarray], name: str, eps: float) -> np.ndarray:
    T = h.shape[0]
    H, d, dv = m["heads"], m["dim"], m["vdim"]
    cq = rms_norm(h @ w[name + ".dq"].T, w[name + ".dq.norm"], eps)
    q = (cq @ w[name + ".uq"].T).reshape(T, H, d)
    c = rms_norm(h @ w[name + ".dkv"].T, w[name + ".dkv.norm"], eps)
    k = (c @ w[name + ".uk"].T).reshape(T, H, d)
    v = (c @ w[name + ".uv"].T).reshape(T, H, dv)
    vis = visible(T, (m.get("mask") or {}).get("size"))
    o = np.zeros((T, H, dv))
    for j in range(H):
        o[:, j] = softmax_over(q[:, j] @ k[:, j].T * m["scale"], vis, False) @ v[:, j]
    return o.reshape(T, H * dv) @ w[name + ".o"].T


def attention(h: np.ndarray, positions, m: dict, w: Dict[str, np.ndarray], name: str, eps: float) -> np.ndarray:
    T = h.shape[0]
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = (h @ w[name + ".q"].T).reshape(T, H, d)
    k = (h @ w[name + ".k"].T).reshape(T, G, d)
    v = (h @ w[name + ".v"].T).reshape(T, G, dv)
    q = unit_rms(rotate_pairs(q, positions, m.get("rot")), eps)
    k = unit_rms(rotate_pairs(k, positions, m.get("rot")), eps)
    gate = sigmoid(h @ w[name + ".g"].T)
    vis = visible(T, None)
    o = np.zeros((T, H, dv))
    for j in range(H):
        g = j // (H // G)
        o[:, j] = softmax_over(q[:, j] @ k[:, g].T * m["scale"], vis, True) @ v[:, g] * gate[:, j:j + 1]
    return o.reshape(T, H * dv) @ w[name + ".o"].T


def two_layer(h: np.ndarray, w: Dict[str, np.ndarray], name: str) -> np.ndarray:
    return relu_squared(h @ w[name + ".up"].T) @ w[name + ".down"].T


def route(h: np.ndarray, r: dict, w: Dict[str, np.ndarray], name: str):
    """(chosen experts [T, top], their softmax scores as they are [T, top])."""
    z = h @ w[name + ".router"].T
    s = np.exp(z - z.max(axis=-1, keepdims=True))
    s = s / s.sum(axis=-1, keepdims=True)
    ids = np.argsort(-s, axis=-1, kind="stable")[:, :r["top"]]
    return ids, np.take_along_axis(s, ids, axis=-1)


def experts(h: np.ndarray, mlp: dict, w: Dict[str, np.ndarray], name: str) -> np.ndarray:
    ids, wts = route(h, mlp["router"], w, name)
    out = np.zeros((h.shape[0], w[name + ".e0.down"].shape[0]))
    for t in range(h.shape[0]):
        for e, a in zip(ids[t], wts[t]):
            out[t] += a * two_layer(h[t], w, f"{name}.e{e}")
    if mlp.get("shared"):
        out += sigmoid(h @ w[name + ".shared.sg"].T) * two_layer(h, w, name + ".shared")
    return out


def forward(config: dict, w: Dict[str, np.ndarray], tokens: Sequence[int], trace: Optional[List[np.ndarray]] = None) -> np.ndarray:
    """Logits [T, vocab] of one sequence from position 0.  `trace` collects the residual after every layer."""
    w = {k: np.asarray(v, dtype=np.float64) for k, v in w.items()}
    eps = config["norm"]["eps"]
    positions = list(range(len(tokens)))
    x = w["embed"][np.asarray(tokens)] * config["embedding"]["scale"]
    for i, layer in enumerate(config["layers"]):
        name, m = f"l{i}", layer["mixer"]
        h = rms_norm(x, w[name + ".norm1"], eps)
        if layer["type"] == "mingru":
            y = mingru(h, w, name + ".mix")
        elif layer["type"] == "latent_attention":
            y = latent_attention(h, m, w, name + ".mix", eps)
        elif layer["type"] == "attention":
            y = attention(h, positions, m, w, name + ".mix", eps)
        else:
            raise ValueError(layer["type"])
        x = x + rms_norm(y, w[name + ".norm1b"], eps)
        mlp = layer.get("mlp")
        if mlp:
            h = rms_norm(x, w[name + ".norm2"], eps)
            y = two_layer(h, w, name + ".mlp") if mlp["kind"] == "dense" else experts(h, mlp, w, name + ".mlp")
            x = x + rms_norm(y, w[name + ".norm2b"], eps)
        if trace is not None:
            trace.append(x.copy())
    return rms_norm(x, w["final.norm"], eps) @ w["embed"].T
