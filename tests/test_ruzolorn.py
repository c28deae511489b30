"""Ruzolorn without a GPU: the configuration reader, the model as data (tensors, run order, cache needs), and the plain
implementation's mechanisms against other ways of writing the same formulas."""
import copy
import math

import numpy as np
import pytest

import ruzolorn_models as rm
from plain import ruzolorn_plain as plain


def spec_of(config):
    import tinyinfer_amd  # noqa: F401
    from tinyinfer_amd.registry import config_and_spec
    return config_and_spec(config)


def test_architecture_is_registered():
    import tinyinfer_amd  # noqa: F401
    from tinyinfer_amd.registry import registered_architectures
    assert "Ruzolorn" in registered_architectures()


@pytest.mark.parametrize("name", sorted(rm.CONFIGS))
def test_spec_asks_for_the_tensors_of_the_configuration(name):
    from tinyinfer_amd.models.model import Model
    config = rm.CONFIGS[name]
    typed, spec = spec_of(config)
    model = Model(spec)
    want = {k: tuple(v.shape) for k, v in rm.draw_weights(config, 1).items()}
    got = {k: tuple(v.shape) for k, v in model.tensors().items() if not v.optional}
    assert got == want
    assert typed["width"] == config["width"] and typed["residual_mult"] == config["residual_mult"]
    assert typed["embedding"]["scale"] == config["embedding"]["scale"]


def test_cache_needs_of_every_mixer():
    from tinyinfer_amd.models.model import Model
    model = Model(spec_of(rm.CONFIGS["wide"])[1])
    kinds = {}
    for need, count in model.cache_groups:
        kinds.setdefault(type(need).__name__, []).append((need, count))
    # matrix states (heads x key size x value size) and the last taps - 1 rows of the convolutions
    assert sorted(tuple(n.shape) for n, _ in kinds["StateNeed"]) == sorted(
        [(4, 128 * 64), (3, 4 * 64 + 2 * 2 * 128), (2, 64 * 128), (8, 48 * 32), (3, 8 * 32 + 2 * 48), (3, 128 * 40), (2, 64 * 72),
         (2, 2 * 72 + 2 * 2 * 64)])
    # values of 16 under keys of 32 are padded: no value size of their own; windows where a layer has one
    assert sorted((n.kv_heads, n.head_dim, n.v_dim or 0, n.window or 0) for n, _ in kinds["PagedKVNeed"]) == [(1, 128, 0, 0), (2, 32, 0, 15), (2, 64, 0, 33)]
    model = Model(spec_of(rm.CONFIGS["plain"])[1])
    kv = sorted((n.kv_heads, n.head_dim, n.v_dim, n.window) for n, _ in model.cache_groups if type(n).__name__ == "PagedKVNeed")
    assert kv == [(1, 6, 5, 500), (5, 7, 9, 1)]
    # a convolution of one tap keeps nothing
    assert sorted(tuple(n.shape) for n, _ in model.cache_groups if type(n).__name__ == "StateNeed") == sorted(
        [(3, 35), (4, 15 + 2 * 3 * 7), (1, 60), (5, 54), (3, 42)])


def test_defaults_are_filled_in():
    config = copy.deepcopy(rm.CONFIGS["plain"])
    del config["embedding"], config["residual_mult"]
    par = config["layers"][0]["mixer"]
    del par["left"]["kv_heads"], par["left"]["vdim"], par["left"]["scale"], par["left"]["mask"], par["left_scale"], par["right_scale"]
    del par["right"]["groups"], par["right"]["norm_groups"]
    ret = config["layers"][3]["mixer"]
    del ret["vdim"], ret["rot"]
    ret["decay"] = 0.75
    del config["layers"][3]["mlp"]["shared"], config["layers"][3]["mlp"]["router"]["identity"], config["layers"][3]["mlp"]["kind"]
    typed, _ = spec_of(config)
    got = typed["layers"][0]["mixer"]
    assert got["left"]["kv_heads"] == 5 and got["left"]["vdim"] == 7 and abs(got["left"]["scale"] - 7 ** -0.5) < 1e-12
    assert got["left"]["mask"] is None and got["left_scale"] == got["right_scale"] == 1.0
    assert got["right"]["groups"] == got["right"]["norm_groups"] == 1
    assert typed["embedding"]["scale"] == 1.0 and typed["residual_mult"] == 1.0
    got = typed["layers"][3]["mixer"]
    assert got["vdim"] == 6 and got["rot"] is None and got["decay"] == [0.75] * 3
    assert typed["layers"][3]["mlp"]["shared"] is None and typed["layers"][3]["mlp"]["router"]["identity"] == 0
    assert typed["layers"][2]["mlp"] is None


@pytest.mark.parametrize("change,word", [
    (lambda c: c["layers"][1]["mixer"]["left"].update(heads=5), "kv_heads"),
    (lambda c: c["layers"][1]["mixer"]["left"].update(dim=300), "dim"),
    (lambda c: c["layers"][1]["mixer"]["left"]["mask"].update(size=0), "size"),
    (lambda c: c["layers"][1]["mixer"].pop("right"), "right"),
    (lambda c: c["layers"][1]["mixer"]["right"].update(groups=4), "groups"),
    (lambda c: c["layers"][1]["mixer"]["right"].update(norm_groups=5), "norm_groups"),
    (lambda c: c["layers"][1]["mixer"]["right"].pop("conv"), "conv"),
    (lambda c: c["layers"][1]["mixer"]["right"].update(state=400), "state"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=7), "dims"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=18), "dims"),
    (lambda c: c["layers"][0]["mixer"].update(decay=[0.9]), "decay"),
    (lambda c: c["layers"][0]["mixer"].update(decay=["a", 1, 2]), "decay"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(top=8), "top"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(identity=-1), "identity"),
    (lambda c: c["layers"][0]["mlp"]["shared"].update(ff=0), "ff"),
    (lambda c: c["layers"][0]["mlp"].update(kind="dense"), "dense"),
    (lambda c: c["layers"][0].update(type="mamba"), "mamba"),
    (lambda c: c["norm"].pop("eps"), "eps"),
    (lambda c: c.update(residual_mult="half"), "residual_mult"),
])
def test_what_is_not_served_is_refused_by_name(change, word):
    from tinyinfer_amd import ConfigError
    config = copy.deepcopy(rm.CONFIGS["mixed"])
    change(config)
    with pytest.raises(ConfigError) as e:
        spec_of(config)
    assert word in str(e.value)


def test_libraries_of_the_architecture_are_built_for_it_and_for_no_other():
    import tinyinfer_amd  # noqa: F401
    from tinyinfer_amd.csrc import build
    mine = build.libraries_for("bfloat16", "Ruzolorn")
    assert {"linear_attention", "short_conv", "residual", "hyper", "gated_attention", "attention_bf16", "moe_bf16"} <= set(mine)
    assert not {"mingru", "latent_attention", "recurrent", "diff_attention", "pointwise"} & set(mine)
    assert "short_conv" not in build.libraries_for("bfloat16", "Qwen3ForCausalLM")
    assert not any(n.endswith("_bf16") for n in build.libraries_for("float32", "Ruzolorn"))


# ------------------------------------------------------------------------ the plain implementation against itself
def test_layer_norm_takes_the_mean_off_and_divides_by_the_deviation():
    rng = np.random.default_rng(0)
    x = rng.normal(3.0, 2.0, size=(5, 40))
    y = plain.layer_norm(x, np.full(40, 2.0), 1e-12)
    assert np.abs(y.mean(axis=1)).max() < 1e-12 and np.abs(y.std(axis=1) - 2.0).max() < 1e-9
    assert np.abs(plain.layer_norm(x + 7.0, np.ones(40), 1e-5) - plain.layer_norm(x, np.ones(40), 1e-5)).max() < 1e-12


def test_the_window_keeps_its_own_position_and_those_before_it():
    p = plain.window_softmax(np.zeros((8, 8)), 3)
    for i in range(8):
        assert [j for j in range(8) if p[i, j] > 0] == [j for j in (i - 2, i - 1, i) if j >= 0]
    assert np.array_equal(plain.window_softmax(np.ones((5, 5)), 1), np.eye(5))


def test_mamba2_is_a_masked_product_of_c_and_b():
    """y_t = sum_(s <= t) exp(sum of the log decays behind s) d_s (C_t . B_s) x_s + D x_t: the other form of the recurrence."""
    rng = np.random.default_rng(1)
    W, T = 9, 12
    m = rm.right(4, 3, 5, 2, 3, 2)
    config = dict(width=W, vocab=4, embedding=dict(scale=1.0), layers=[rm.parallel(rm.left(1, 1, 2, 2, 1.0), m)])
    w = {k[len("l0.mix.right"):]: v for k, v in rm.as_float64(rm.draw_weights(config, 3)).items() if k.startswith("l0.mix.right")}
    w = {"m" + k: v for k, v in w.items()}
    w["m.o"] = np.eye(12)
    h = rng.normal(size=(T, W))
    got = plain.mamba2(h, m, w, "m", 1e-6)
    p = h @ w["m.in"].T
    z, xbc, dt = p[:, :12], p[:, 12:12 + 32], p[:, 44:]
    conv = np.zeros_like(xbc)
    for t in range(T):
        for j in range(3):
            if t - 2 + j >= 0:
                conv[t] += xbc[t - 2 + j] * w["m.conv"][:, j]
    xbc = conv + w["m.conv.b"]
    xbc = xbc / (1 + np.exp(-xbc))
    d = np.log1p(np.exp(dt + w["m.dt_bias"]))
    y = np.zeros((T, 4, 3))
    for j in range(4):
        x, B, C = xbc[:, 3 * j:3 * j + 3], xbc[:, 12 + 5 * (j // 2):17 + 5 * (j // 2)], xbc[:, 22 + 5 * (j // 2):27 + 5 * (j // 2)]
        log_a = -np.exp(w["m.A_log"][j]) * d[:, j]
        for t in range(T):
            y[t, j] = w["m.D"][j] * x[t] + sum(math.exp(log_a[s + 1:t + 1].sum()) * d[s, j] * (C[t] @ B[s]) * x[s] for s in range(t + 1))
    y = y.reshape(T, 12) * z / (1 + np.exp(-z))
    for part in range(2):
        run = slice(6 * part, 6 * part + 6)
        y[:, run] /= np.sqrt((y[:, run] ** 2).mean(axis=1, keepdims=True) + 1e-6)
    assert np.abs(got - y * w["m.norm"]).max() < 1e-10


def test_retention_is_a_decayed_product_of_rotated_queries_and_keys():
    rng = np.random.default_rng(2)
    W, T, d, dv = 7, 11, 6, 4
    m = rm.retention(2, d, dv, [0.9, 1.0], 4, 30.0)["mixer"]
    w = {"m.q": rng.normal(size=(2 * d, W)), "m.k": rng.normal(size=(2 * d, W)), "m.v": rng.normal(size=(2 * dv, W)),
         "m.g": rng.normal(size=(2 * dv, W)), "m.o": np.eye(2 * dv)}
    h = rng.normal(size=(T, W))
    got = plain.retention(h, m, w, "m", 1e-5)
    freq = np.array([1.0, 30.0 ** -0.5])

    def turned(x):      # as multiplication by a complex number of angle p f
        z = (x[..., 0:2] + 1j * x[..., 2:4]) * np.exp(1j * np.outer(np.arange(T), freq))[:, None, :]
        return np.concatenate([z.real, z.imag, x[..., 4:]], axis=-1)
    q, k = turned((h @ w["m.q"].T).reshape(T, 2, d)), turned((h @ w["m.k"].T).reshape(T, 2, d))
    v = (h @ w["m.v"].T).reshape(T, 2, dv)
    o = np.zeros((T, 2, dv))
    for j in range(2):
        for t in range(T):
            o[t, j] = sum(m["decay"][j] ** (t - s) * (q[t, j] @ k[s, j]) / math.sqrt(d) * v[s, j] for s in range(t + 1))
            o[t, j] /= math.sqrt((o[t, j] ** 2).mean() + 1e-5)
    g = h @ w["m.g"].T
    assert np.abs(got - o.reshape(T, -1) * g / (1 + np.exp(-g))).max() < 1e-10


def test_the_correction_counts_for_the_choice_only_and_identities_return_their_input():
    rng = np.random.default_rng(4)
    W, E, N = 8, 3, 2
    w = {"m.router": rng.normal(size=(E + N, W)), "m.correction": np.array([0.0, 0.0, -5.0, 5.0, 0.0])}
    for e in range(E):
        for t in ("gate", "up", "down"):
            w[f"m.e{e}.{t}"] = rng.normal(size=(W, W))
    h = rng.normal(size=(20, W))
    mlp = rm.moe(E, 2, W, N)
    ids, wts = plain.route(h, mlp["router"], w, "m")
    out = plain.experts(h, mlp, w, "m")
    for t in range(20):
        s = np.exp(h[t] @ w["m.router"].T)
        s = s / s.sum()
        assert ids[t, 0] == 3 and 2 not in ids[t] and np.abs(wts[t] - s[ids[t]]).max() < 1e-12
        want = s[3] * h[t]                                     # the first choice is an identity everywhere
        e = ids[t, 1]
        want = want + s[e] * (h[t] if e == 4 else plain.gated_ff(h[t:t + 1], w, f"m.e{e}")[0])
        assert np.abs(out[t] - want).max() < 1e-12
    assert {0, 1, 4} <= set(ids[:, 1])


def test_every_learned_tensor_moves_the_logits():
    config = rm.CONFIGS["mixed"]
    w = rm.as_float64(rm.draw_weights(config, 5))
    toks = [int(t) for t in np.random.default_rng(6).integers(0, config["vocab"], size=24)]
    base = plain.forward(config, w, toks)
    for name in w:
        if ".mlp.e" in name:
            continue                # an expert that no token of this prompt chose moves nothing
        rng = np.random.default_rng(len(name))
        changed = dict(w)
        changed[name] = w[name] * 1.3 + rng.normal(0.0, 0.3, size=w[name].shape)
        assert np.abs(plain.forward(config, changed, toks) - base).max() > 1e-9, name


def test_factors_of_the_embedding_and_of_every_sublayer():
    config = copy.deepcopy(rm.CONFIGS["states"])
    w = rm.as_float64(rm.draw_weights(config, 7))
    toks = [3, 1, 4, 1, 5]
    trace = []
    plain.forward(config, w, toks, trace)
    x0 = w["embed"][toks] * 4.0
    config["residual_mult"] = 1.0
    other = []
    plain.forward(config, w, toks, other)
    # the first sublayer reads the same row: its share is half as large
    config["layers"] = config["layers"][:1]
    config["layers"][0]["mlp"] = None
    one, half = [], []
    plain.forward(config, w, toks, one)
    config["residual_mult"] = 0.5
    plain.forward(config, w, toks, half)
    assert np.abs((one[0] - x0) - 2.0 * (half[0] - x0)).max() < 1e-12 and np.abs(trace[0] - other[0]).max() > 1e-3
    config["layers"] = []
    assert np.abs(plain.forward(config, w, toks) - plain.layer_norm(x0, w["final.norm"], 1e-5) @ w["head"].T).max() < 1e-12
