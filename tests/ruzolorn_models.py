"""Small Ruzolorn configurations and random weights for the tests.  The weights are drawn here with numpy (not by the
framework's own generator), rounded to bfloat16 and written with the safetensors package, so that the engine and the
plain implementation read the same numbers.  Scales are chosen so that activations stay of order one, attention is far
from uniform, the states remember for a while, and every gate, correction and identity expert matters."""
import json
import os

import numpy as np


def parallel(left, right, scales=(0.9, 1.2), mlp=None):
    return dict(type="parallel", mixer=dict(left=left, right=right, left_scale=scales[0], right_scale=scales[1]), mlp=mlp)


def left(heads, kv_heads, dim, vdim, scale, window=None):
    m = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale)
    if window:
        m["mask"] = dict(size=window)
    return m


def right(heads, vdim, state, groups=1, conv=4, norm_groups=1):
    return dict(heads=heads, vdim=vdim, state=state, groups=groups, conv=conv, norm_groups=norm_groups)


def retention(heads, dim, vdim, decay, rot_dims=None, base=10000.0, mlp=None):
    m = dict(heads=heads, dim=dim, vdim=vdim, decay=decay)
    if rot_dims is not None:
        m["rot"] = dict(base=base, dims=rot_dims)
    return dict(type="retention", mixer=m, mlp=mlp)


def moe(experts, top, ff, identity=0, shared=None):
    d = dict(kind="moe", expert=dict(ff=ff), router=dict(experts=experts, top=top, identity=identity))
    if shared:
        d["shared"] = dict(ff=shared)
    return d


CONFIGS = {
    # both mixers with and without a feed-forward; two kv heads under four heads, values larger and smaller than keys; a window
    # that is no multiple of a page and none at all; rotation on part of a head, on all of it, none; groups of B and C, a norm in
    # parts; experts with and without identities and a shared one
    "mixed": dict(architecture="Ruzolorn", width=48, vocab=97, norm=dict(eps=1e-5), embedding=dict(scale=2.5), residual_mult=0.8,
                  layers=[retention(3, 16, 24, [0.999, 0.9, 0.6], 8, 100.0, moe(5, 2, 24, 2, 40)),
                          parallel(left(4, 2, 16, 24, 0.5, 11), right(6, 12, 20, 3, 3, 2), (0.9, 1.2), moe(4, 1, 16, 1)),
                          retention(2, 12, 8, [1.0, 0.97], 12, 50.0, None),
                          parallel(left(2, 1, 12, 8, 0.6), right(4, 16, 8, 2, 4, 4), (1.5, 0.4), moe(6, 3, 20, 0, 24)),
                          parallel(left(3, 3, 20, 20, 0.4, 40), right(2, 10, 16, 1, 2, 1), (1.0, 1.0), None)]),
    # sizes that are no multiples of four; a window of one position and one longer than any request; every head its own kv head;
    # more identities than experts, more choices than experts; a convolution of one tap and one of five; no factors
    "plain": dict(architecture="Ruzolorn", width=50, vocab=61, norm=dict(eps=3e-6), embedding=dict(scale=1.0), residual_mult=1.0,
                  layers=[parallel(left(5, 5, 7, 9, 0.7, 1), right(3, 5, 7, 3, 5, 5), (0.7, 0.7), moe(1, 3, 9, 3, 15)),
                          retention(1, 10, 6, [0.95], None, mlp=moe(6, 4, 21, 5, None)),
                          parallel(left(1, 1, 6, 5, 0.8, 500), right(5, 6, 9, 1, 1, 3), (1.0, -0.5), None),
                          retention(3, 6, 7, [0.5, 0.99, 0.9], 2, 20.0, moe(3, 2, 10, 1, 10))]),
    # sizes the matrix cores serve: keys of 64, 32 and 128, values of their size and smaller (padded in the pages), windows of two
    # pages and one more, of a page less one, none; states of several blocks of 64 and of a part of one
    "wide": dict(architecture="Ruzolorn", width=128, vocab=320, norm=dict(eps=1e-6), embedding=dict(scale=6.0), residual_mult=0.6,
                 layers=[parallel(left(4, 2, 64, 64, 0.2, 33), right(4, 64, 128, 2, 4, 2), (0.8, 1.1), moe(8, 3, 64, 2, 96)),
                         retention(2, 64, 128, [0.998, 0.97], 64, 30000.0, moe(6, 2, 32, 1, 64)),
                         parallel(left(6, 2, 32, 16, 0.3, 15), right(8, 32, 48, 1, 4, 1), (1.1, 0.6), None),
                         retention(3, 128, 40, [0.999, 0.95, 0.9], 32, 10000.0, moe(4, 1, 32, 4, 32)),
                         parallel(left(2, 1, 128, 128, 0.12), right(2, 72, 64, 2, 3, 1), (0.7, 1.0), moe(4, 2, 32, 0, None))]),
    # a state without any pages
    "states": dict(architecture="Ruzolorn", width=32, vocab=40, norm=dict(eps=1e-5), embedding=dict(scale=4.0), residual_mult=0.5,
                   layers=[retention(2, 16, 16, [0.99, 0.8], 16, 100.0, moe(2, 1, 8, 1, 8)), retention(4, 8, 4, [0.9, 0.99, 0.95, 1.0], 4, mlp=None)]),
    # scores so far apart that a head mostly reads one key: a key lost or won at a window's edge stands out
    "edges": dict(architecture="Ruzolorn", width=32, vocab=40, norm=dict(eps=1e-5), embedding=dict(scale=3.0), residual_mult=1.0,
                  layers=[parallel(left(4, 2, 16, 16, 2.0, 17), right(2, 8, 8), (2.0, 0.2), None)]),
}


def to_bf16(a):
    import torch
    return torch.from_numpy(np.ascontiguousarray(np.asarray(a, dtype=np.float32))).to(torch.bfloat16)


def draw_weights(config, seed):
    """{name: torch bfloat16 tensor} for every tensor the configuration's model holds."""
    rng = np.random.default_rng(seed)
    W, V = config["width"], config["vocab"]
    t = {}

    def mat(rows, cols, gain=1.0):
        return rng.normal(0.0, gain / np.sqrt(cols), size=(rows, cols))

    def norm(name, n=W, around=1.0):
        t[name] = around + rng.normal(0.0, 0.2, size=n)

    def gated(pre, F):
        t[pre + ".gate"], t[pre + ".up"] = mat(F, W, 1.5), mat(F, W, 1.5)
        t[pre + ".down"] = mat(W, F)

    t["embed"] = rng.normal(0.0, 1.0 / config["embedding"]["scale"], size=(V, W))
    t["head"] = mat(V, W)
    norm("final.norm")
    for i, lay in enumerate(config["layers"]):
        p, m = f"l{i}", lay["mixer"]
        norm(p + ".norm1")
        norm(p + ".norm1b", around=0.7)
        x = p + ".mix"
        if lay["type"] == "retention":
            H, d, dv = m["heads"], m["dim"], m["vdim"]
            t[x + ".q"], t[x + ".k"] = mat(H * d, W, 1.3), mat(H * d, W, 1.3)
            t[x + ".v"], t[x + ".g"] = mat(H * dv, W), mat(H * dv, W, 1.5)
            t[x + ".o"] = mat(W, H * dv)
        else:
            a, y = m["left"], x + ".left"
            H, G, d, dv = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
            t[y + ".q"], t[y + ".k"], t[y + ".v"] = mat(H * d, W), mat(G * d, W), mat(G * dv, W)
            norm(y + ".q.norm", d)
            norm(y + ".k.norm", d)
            t[y + ".o"] = mat(W, H * dv)
            b, y = m["right"], x + ".right"
            H, P, N, G = b["heads"], b["vdim"], b["state"], b["groups"]
            inner, ch = H * P, H * P + 2 * G * N
            t[y + ".in"] = mat(inner + ch + H, W, 1.2)
            t[y + ".conv"] = rng.normal(0.0, 0.7, size=(ch, b["conv"]))
            t[y + ".conv.b"] = rng.normal(0.0, 0.3, size=ch)
            t[y + ".dt_bias"] = rng.normal(-1.5, 1.0, size=H)
            t[y + ".A_log"] = rng.uniform(-3.0, 1.0, size=H)      # from forgetting within a few tokens to remembering a hundred
            t[y + ".D"] = rng.normal(0.0, 0.7, size=H)
            norm(y + ".norm", inner)
            t[y + ".o"] = mat(W, inner)
        mlp = lay.get("mlp")
        if mlp:
            norm(p + ".norm2")
            norm(p + ".norm2b", around=0.7)
            rows = mlp["router"]["experts"] + mlp["router"]["identity"]
            t[p + ".mlp.router"] = mat(rows, W, 2.0)
            t[p + ".mlp.correction"] = rng.normal(0.0, 0.1, size=rows)
            for e in range(mlp["router"]["experts"]):
                gated(f"{p}.mlp.e{e}", mlp["expert"]["ff"])
            if mlp.get("shared"):
                gated(p + ".mlp.shared", mlp["shared"]["ff"])
    return {k: to_bf16(v) for k, v in t.items()}


def write_folder(path, config, seed, weights=None):
    from safetensors.torch import save_file
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(config, f)
    w = weights if weights is not None else draw_weights(config, seed)
    save_file({k: v.contiguous() for k, v in w.items()}, os.path.join(path, "model.safetensors"))
    return path


def as_float64(weights):
    import torch
    return {k: v.to(torch.float64).numpy() for k, v in weights.items()}
