"""Small Lupolorn configurations and random weights for the tests.  The weights are drawn here with numpy (not by the
framework's own generator), rounded to bfloat16 and written with the safetensors package, so that the engine and the
plain implementation read the same numbers.  Scales are chosen so that activations stay of order one, attention is far
from uniform, the one more in the denominators and the gates matter, and the recurrences remember for a while."""
import json
import os

import numpy as np


def wavelengths(factor, low, high, original):
    return dict(factor=factor, low=low, high=high, original=original)


def attention(heads, kv_heads, dim, vdim, scale, rot_dims, base=10000.0, scaling=None, mlp=None):
    m = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale)
    if rot_dims is not None:
        m["rot"] = dict(base=base, dims=rot_dims)
        if scaling:
            m["rot"]["scaling"] = scaling
    return dict(type="attention", mixer=m, mlp=mlp)


def latent(heads, dim, vdim, q_rank, kv_rank, scale, window=None, mlp=None):
    m = dict(heads=heads, dim=dim, vdim=vdim, q_rank=q_rank, kv_rank=kv_rank, scale=scale)
    if window:
        m["mask"] = dict(size=window)
    return dict(type="latent_attention", mixer=m, mlp=mlp)


def mingru(width, mlp=None):
    return dict(type="mingru", mixer=dict(width=width), mlp=mlp)


def dense(ff):
    return dict(kind="dense", ff=ff)


def moe(experts, top, ff, shared=None):
    d = dict(kind="moe", expert=dict(ff=ff), router=dict(experts=experts, top=top))
    if shared:
        d["shared"] = dict(ff=shared)
    return d


CONFIGS = {
    # every mixer behind every kind of feed-forward; the first layer a recurrence; two kv heads under four heads, values larger and
    # smaller than keys; rotation on part of a head with stretched frequencies, on all of it, none; a window that is no multiple
    # of a page; a latent layer without a window
    "mixed": dict(architecture="Lupolorn", width=48, vocab=97, norm=dict(eps=1e-5), embedding=dict(scale=2.5),
                  layers=[mingru(72, dense(40)),
                          latent(3, 16, 24, 20, 32, 0.4, 11, moe(5, 2, 24, 56)),
                          attention(4, 2, 16, 24, 0.5, 8, 100.0, wavelengths(3.0, 1.0, 4.0, 64), dense(64)),
                          latent(2, 12, 8, 16, 24, 0.5, None, None),
                          attention(2, 1, 12, 8, 0.6, 12, 50.0, None, moe(4, 1, 16, None)),
                          mingru(20, moe(3, 3, 12, 20))]),
    # sizes that are no multiples of four; a window of one position and one longer than any request; one head; every head its
    # own kv head; a layer without a feed-forward; one expert of one; no factor on the embedding; the second sort of
    # frequencies all stretched
    "plain": dict(architecture="Lupolorn", width=50, vocab=61, norm=dict(eps=3e-6), embedding=dict(scale=1.0),
                  layers=[latent(5, 7, 9, 11, 13, 0.7, 1, dense(33)),
                          attention(3, 3, 6, 7, 0.9, 2, 20.0, wavelengths(8.0, 1.5, 2.5, 6), None),
                          mingru(37, moe(1, 1, 9, 15)),
                          latent(1, 10, 6, 5, 18, 0.6, 500, moe(6, 3, 21, 10)),
                          attention(1, 1, 10, 13, 0.8, None, mlp=dense(22))]),
    # sizes the matrix cores serve: keys and values of 64, 32 and 128, values smaller than keys (padded in the pages), latents of 64
    # and 128 under 20 heads (two groups of them), windows of two pages and one more and of a page less one
    "wide": dict(architecture="Lupolorn", width=128, vocab=320, norm=dict(eps=1e-6), embedding=dict(scale=11.3),
                 layers=[attention(4, 2, 64, 64, 0.2, 64, 30000.0, wavelengths(4.0, 1.0, 4.0, 256), moe(8, 3, 64, 96)),
                         latent(20, 16, 16, 48, 64, 0.35, 33, dense(160)),
                         mingru(192, dense(96)),
                         attention(6, 2, 32, 16, 0.3, 16, 10000.0, None, moe(6, 2, 32, 64)),
                         latent(4, 32, 48, 64, 128, 0.25, 15, moe(4, 1, 32, None)),
                         attention(2, 1, 128, 128, 0.12, 32, 10000.0, None, None),
                         mingru(64, None)]),
    # one layer of each sort with a feed-forward of one sort only: a state without any pages, pages without any state
    "states": dict(architecture="Lupolorn", width=32, vocab=40, norm=dict(eps=1e-5), embedding=dict(scale=4.0),
                   layers=[mingru(32, dense(24)), mingru(16, moe(2, 1, 8, 8))]),
    "windows": dict(architecture="Lupolorn", width=32, vocab=40, norm=dict(eps=1e-5), embedding=dict(scale=3.0),
                    layers=[latent(2, 8, 16, 8, 16, 0.6, 5, dense(24))]),
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

    def two_layer(pre, F):
        t[pre + ".up"] = mat(F, W, 1.5)
        t[pre + ".down"] = mat(W, F)

    t["embed"] = rng.normal(0.0, 1.0 / config["embedding"]["scale"], size=(V, W))
    norm("final.norm")
    for i, lay in enumerate(config["layers"]):
        p, m = f"l{i}", lay["mixer"]
        norm(p + ".norm1")
        norm(p + ".norm1b", around=0.7)
        x = p + ".mix"
        if lay["type"] == "mingru":
            n = m["width"]
            for g in ("z", "x", "g"):
                t[f"{x}.{g}"] = mat(n, W, 2.0)
            t[x + ".z.b"] = rng.normal(-2.0, 1.0, size=n)      # most channels forget slowly
            t[x + ".x.b"] = rng.normal(0.0, 0.5, size=n)
            t[x + ".o"] = mat(W, n)
        elif lay["type"] == "latent_attention":
            H, d, dv, qr, r = m["heads"], m["dim"], m["vdim"], m["q_rank"], m["kv_rank"]
            t[x + ".dq"], t[x + ".dkv"] = mat(qr, W), mat(r, W)
            norm(x + ".dq.norm", qr)
            norm(x + ".dkv.norm", r)
            t[x + ".uq"], t[x + ".uk"] = mat(H * d, qr, 1.6), mat(H * d, r, 1.6)
            t[x + ".uv"] = mat(H * dv, r)
            t[x + ".o"] = mat(W, H * dv)
        else:
            H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            t[x + ".q"], t[x + ".k"] = mat(H * d, W, 1.5), mat(G * d, W, 1.5)
            t[x + ".v"] = mat(G * dv, W)
            t[x + ".g"] = mat(H, W, 1.5)
            t[x + ".o"] = mat(W, H * dv)
        mlp = lay.get("mlp")
        if mlp:
            norm(p + ".norm2")
            norm(p + ".norm2b", around=0.7)
        if mlp and mlp["kind"] == "dense":
            two_layer(p + ".mlp", mlp["ff"])
        elif mlp:
            E = mlp["router"]["experts"]
            t[p + ".mlp.router"] = mat(E, W, 2.0)
            for e in range(E):
                two_layer(f"{p}.mlp.e{e}", mlp["expert"]["ff"])
            if mlp.get("shared"):
                two_layer(p + ".mlp.shared", mlp["shared"]["ff"])
                t[p + ".mlp.shared.sg"] = mat(1, W, 1.5)
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
