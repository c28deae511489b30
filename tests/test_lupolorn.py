"""Lupolorn without a GPU: the configuration reader, the model as data (tensors, run order, cache needs), and the plain
implementation's mechanisms against other ways of writing the same formulas."""
import copy
import math

import numpy as np
import pytest

import lupolorn_models as lm
from plain import lupolorn_plain as plain


def spec_of(config):
    import tinyinfer_amd  # noqa: F401
    from tinyinfer_amd.registry import config_and_spec
    return config_and_spec(config)


def test_architecture_is_registered():
    import tinyinfer_amd  # noqa: F401
    from tinyinfer_amd.registry import registered_architectures
    assert "Lupolorn" in registered_architectures()


@pytest.mark.parametrize("name", sorted(lm.CONFIGS))
def test_spec_asks_for_the_tensors_of_the_configuration(name):
    from tinyinfer_amd.models.model import Model
    config = lm.CONFIGS[name]
    typed, spec = spec_of(config)
    model = Model(spec)
    want = {k: tuple(v.shape) for k, v in lm.draw_weights(config, 1).items()}
    got = {k: tuple(v.shape) for k, v in model.tensors().items() if not v.optional}
    assert got == want
    assert typed["width"] == config["width"] and typed["vocab"] == config["vocab"]
    assert typed["embedding"]["scale"] == config["embedding"]["scale"]


def test_cache_needs_of_every_mixer():
    from tinyinfer_amd.models.model import Model
    model = Model(spec_of(lm.CONFIGS["wide"])[1])
    kinds = {}
    for need, count in model.cache_groups:
        kinds.setdefault(type(need).__name__, []).append((need, count))
    # the recurrences: one 32-bit number a channel and request
    assert sorted((tuple(n.shape), c) for n, c in kinds["StateNeed"]) == [((64,), 1), ((192,), 1)]
    # latents twice (as rows and transposed) where the matrix cores serve the sizes, under their windows
    assert sorted((tuple(n.row_shape), n.window, c) for n, c in kinds["PagedRowsNeed"]) == [((128,), 33, 1), ((256,), 15, 1)]
    # values of 16 under keys of 32 are padded: no value size of their own
    assert sorted((n.kv_heads, n.head_dim, n.v_dim) for n, _ in kinds["PagedKVNeed"]) == [(1, 128, None), (2, 32, None), (2, 64, None)]
    model = Model(spec_of(lm.CONFIGS["plain"])[1])
    rows = sorted((tuple(n.row_shape), n.window) for n, _ in model.cache_groups if type(n).__name__ == "PagedRowsNeed")
    assert rows == [((13,), 1), ((18,), 500)]      # once: no matrix-core kernel takes these sizes
    kv = sorted((n.kv_heads, n.head_dim, n.v_dim) for n, _ in model.cache_groups if type(n).__name__ == "PagedKVNeed")
    assert kv == [(1, 10, 13), (3, 6, 7)]


def test_defaults_are_filled_in():
    config = copy.deepcopy(lm.CONFIGS["plain"])
    del config["embedding"]
    m = config["layers"][1]["mixer"]
    del m["kv_heads"], m["vdim"], m["scale"]
    del config["layers"][0]["mixer"]["mask"]
    del config["layers"][0]["mixer"]["scale"]
    del config["layers"][2]["mlp"]["shared"]
    typed, _ = spec_of(config)
    got = typed["layers"][1]["mixer"]
    assert got["kv_heads"] == 3 and got["vdim"] == 6 and abs(got["scale"] - 6 ** -0.5) < 1e-12
    assert typed["embedding"]["scale"] == 1.0
    assert typed["layers"][0]["mixer"]["mask"] is None and abs(typed["layers"][0]["mixer"]["scale"] - 7 ** -0.5) < 1e-12
    assert typed["layers"][2]["mlp"]["shared"] is None and typed["layers"][1]["mlp"] is None


@pytest.mark.parametrize("change,word", [
    (lambda c: c["layers"][2]["mixer"].update(heads=5), "kv_heads"),
    (lambda c: c["layers"][2]["mixer"]["rot"].update(dims=7), "dims"),
    (lambda c: c["layers"][2]["mixer"]["rot"].update(dims=18), "dims"),
    (lambda c: c["layers"][2]["mixer"]["rot"]["scaling"].pop("original"), "original"),
    (lambda c: c["layers"][2]["mixer"]["rot"]["scaling"].update(low=5.0), "low"),
    (lambda c: c["layers"][2]["mixer"].update(dim=300), "dim"),
    (lambda c: c["layers"][1]["mixer"].pop("q_rank"), "q_rank"),
    (lambda c: c["layers"][1]["mixer"]["mask"].update(size=0), "size"),
    (lambda c: c["layers"][1]["mlp"]["router"].update(top=6), "top"),
    (lambda c: c["layers"][1]["mlp"]["shared"].update(ff=0), "ff"),
    (lambda c: c["layers"][0]["mixer"].pop("width"), "width"),
    (lambda c: c["layers"][0].update(type="mamba"), "mamba"),
    (lambda c: c["layers"][0]["mlp"].update(kind="sparse"), "sparse"),
    (lambda c: c["norm"].pop("eps"), "eps"),
    (lambda c: c["embedding"].update(scale="big"), "scale"),
])
def test_what_is_not_served_is_refused_by_name(change, word):
    from tinyinfer_amd import ConfigError
    config = copy.deepcopy(lm.CONFIGS["mixed"])
    change(config)
    with pytest.raises(ConfigError) as e:
        spec_of(config)
    assert word in str(e.value)


def test_libraries_of_the_architecture_are_built_for_it_and_for_no_other():
    import tinyinfer_amd  # noqa: F401
    from tinyinfer_amd.csrc import build
    mine = build.libraries_for("bfloat16", "Lupolorn")
    assert {"mingru", "residual", "latent_attention_bf16", "gated_attention", "moe_bf16"} <= set(mine)
    assert not {"hyper", "linear_attention", "recurrent", "diff_attention"} & set(mine)
    assert "mingru" not in build.libraries_for("bfloat16", "Qwen3ForCausalLM")
    assert not any(n.endswith("_bf16") for n in build.libraries_for("float32", "Lupolorn"))


# ------------------------------------------------------------------------ the plain implementation against itself
def test_the_recurrence_is_a_weighted_sum_of_candidates():
    """S_t = sum_j (prod over later steps of (1 - z)) z_j c_j, the weights summing to one less what is left of the start."""
    rng = np.random.default_rng(0)
    W, N, T = 7, 5, 12
    w = {"m.z": rng.normal(size=(N, W)), "m.x": rng.normal(size=(N, W)), "m.g": np.zeros((N, W)), "m.o": np.eye(N),
         "m.z.b": rng.normal(size=N), "m.x.b": rng.normal(size=N)}
    w["m.g"][:, 0] = 1.0
    h = rng.normal(size=(T, W))
    h[:, 0] = 1.0                                              # g = 1 everywhere: the output is S silu(1)
    got = plain.mingru(h, w, "m") / plain.silu(np.array(1.0))
    z = plain.sigmoid(h @ w["m.z"].T + w["m.z.b"])
    u = h @ w["m.x"].T + w["m.x.b"]
    assert (u > 0).any() and (u < 0).any()
    c = np.array([[v + 0.5 if v >= 0 else 1.0 / (1.0 + math.exp(-v)) for v in row] for row in u])
    for t in range(T):
        want = sum(np.prod(1.0 - z[j + 1:t + 1], axis=0) * z[j] * c[j] for j in range(t + 1))
        assert np.abs(got[t] - want).max() < 1e-12
    # the candidate is continuous at zero and grows without bound above it
    assert abs(plain.sigmoid(np.array(-1e-9)) - 0.5) < 1e-8


def test_wavelengths_are_kept_stretched_or_mixed():
    rot = dict(base=500.0, dims=16, scaling=lm.wavelengths(4.0, 1.0, 8.0, 100))
    f = plain.frequencies(rot)
    g = plain.frequencies(dict(base=500.0, dims=16))
    lengths = 2 * math.pi / g
    seen = set()
    for i in range(8):
        if lengths[i] < 100 / 8.0:
            assert f[i] == g[i]
            seen.add("kept")
        elif lengths[i] > 100 / 1.0:
            assert abs(f[i] - g[i] / 4.0) < 1e-15
            seen.add("stretched")
        else:
            assert g[i] / 4.0 < f[i] < g[i]
            seen.add("mixed")
    assert seen == {"kept", "stretched", "mixed"}
    # the mix meets both ends: at a wavelength of original / high it keeps, at original / low it stretches
    for turns, want in ((8.0, 1.0), (1.0, 0.25)):
        base_f = turns * 2 * math.pi / 100
        got = plain.frequencies(dict(base=1.0 / base_f ** 2, dims=4, scaling=lm.wavelengths(4.0, 1.0, 8.0, 100)))[1]
        assert abs(got / base_f - want) < 1e-9


def test_rotation_turns_neighbours_and_keeps_lengths():
    rng = np.random.default_rng(1)
    x = rng.normal(size=(6, 2, 10))
    rot = dict(base=30.0, dims=6)
    y = plain.rotate_pairs(x, [0, 1, 2, 3, 4, 50], rot)
    assert np.array_equal(y[0], x[0]) and np.array_equal(y[:, :, 6:], x[:, :, 6:])
    for i in range(3):
        assert np.abs((y[:, :, 2 * i:2 * i + 2] ** 2).sum(-1) - (x[:, :, 2 * i:2 * i + 2] ** 2).sum(-1)).max() < 1e-12
    # as multiplication by a complex number of angle p f
    z = (x[:, :, 0:6:2] + 1j * x[:, :, 1:6:2]) * np.exp(1j * np.outer([0, 1, 2, 3, 4, 50], plain.frequencies(rot)))[:, None, :]
    assert np.abs(z.real - y[:, :, 0:6:2]).max() < 1e-12 and np.abs(z.imag - y[:, :, 1:6:2]).max() < 1e-12


def test_one_more_in_the_denominator_is_a_key_of_score_zero_without_a_value():
    rng = np.random.default_rng(2)
    T = 9
    s = rng.normal(size=(T, T)) * 3 - 1
    p = plain.softmax_over(s, plain.visible(T, None), True)
    wide = np.concatenate([s, np.zeros((T, 1))], axis=1)
    vis = np.concatenate([plain.visible(T, None), np.ones((T, 1), dtype=bool)], axis=1)
    ref = plain.softmax_over(wide, vis, False)
    assert np.abs(p - ref[:, :T]).max() < 1e-12 and (p.sum(axis=1) < 1.0).all()
    # far below zero nearly nothing is left of the keys, far above the one more does not count; neither overflows
    assert plain.softmax_over(s - 60, plain.visible(T, None), True).sum(axis=1).max() < 1e-20
    assert np.abs(plain.softmax_over(s + 900, plain.visible(T, None), True).sum(axis=1) - 1).max() < 1e-12


def test_the_window_keeps_its_own_position_and_those_before_it():
    v = plain.visible(8, 3)
    for i in range(8):
        assert [j for j in range(8) if v[i, j]] == [j for j in (i - 2, i - 1, i) if j >= 0]
    assert np.array_equal(plain.visible(5, 1), np.eye(5, dtype=bool)) and np.array_equal(plain.visible(5, 9), plain.visible(5, None))


def test_latent_attention_equals_attention_over_the_latents_themselves():
    """q . (W_uk c) = (W_uk^T q) . c and sum p (W_uv c) = W_uv sum p c: what the kernels compute."""
    rng = np.random.default_rng(3)
    W, T, H, d, dv, qr, R = 10, 14, 3, 4, 6, 5, 8
    m = dict(heads=H, dim=d, vdim=dv, q_rank=qr, kv_rank=R, scale=0.7, mask=dict(size=4))
    w = {"m.dq": rng.normal(size=(qr, W)), "m.dq.norm": rng.normal(1, 0.2, size=qr), "m.uq": rng.normal(size=(H * d, qr)),
         "m.dkv": rng.normal(size=(R, W)), "m.dkv.norm": rng.normal(1, 0.2, size=R), "m.uk": rng.normal(size=(H * d, R)),
         "m.uv": rng.normal(size=(H * dv, R)), "m.o": rng.normal(size=(W, H * dv))}
    h = rng.normal(size=(T, W))
    got = plain.latent_attention(h, m, w, "m", 1e-6)
    c = plain.rms_norm(h @ w["m.dkv"].T, w["m.dkv.norm"], 1e-6)
    q = (plain.rms_norm(h @ w["m.dq"].T, w["m.dq.norm"], 1e-6) @ w["m.uq"].T).reshape(T, H, d)
    o = np.zeros((T, H, dv))
    for j in range(H):
        qa = q[:, j] @ w["m.uk"][j * d:(j + 1) * d]
        for t in range(T):
            keys = range(max(0, t - 3), t + 1)
            s = np.array([qa[t] @ c[k] for k in keys]) * 0.7
            p = np.exp(s - s.max())
            o[t, j] = w["m.uv"][j * dv:(j + 1) * dv] @ sum(a * c[k] for a, k in zip(p / p.sum(), keys))
    assert np.abs(got - o.reshape(T, -1) @ w["m.o"].T).max() < 1e-10


def test_router_weights_are_the_scores_as_they_are():
    rng = np.random.default_rng(4)
    w = {"m.router": rng.normal(size=(6, 8))}
    h = rng.normal(size=(20, 8))
    ids, wts = plain.route(h, dict(experts=6, top=2), w, "m")
    for t in range(20):
        e = np.exp(h[t] @ w["m.router"].T)
        s = e / e.sum()
        assert set(ids[t]) == set(np.argsort(-s)[:2]) and np.abs(wts[t] - s[ids[t]]).max() < 1e-12
        assert wts[t].sum() < 1.0
    _, wts = plain.route(h, dict(experts=6, top=6), w, "m")
    assert np.abs(wts.sum(axis=1) - 1.0).max() < 1e-12


def test_every_learned_tensor_moves_the_logits():
    config = lm.CONFIGS["mixed"]
    w = lm.as_float64(lm.draw_weights(config, 5))
    toks = [int(t) for t in np.random.default_rng(6).integers(0, config["vocab"], size=24)]
    base = plain.forward(config, w, toks)
    for name in w:
        if ".mlp.e" in name:
            continue                # an expert that no token of this prompt chose moves nothing
        rng = np.random.default_rng(len(name))
        changed = dict(w)
        changed[name] = w[name] * 1.3 + rng.normal(0.0, 0.05, size=w[name].shape)
        assert np.abs(plain.forward(config, changed, toks) - base).max() > 1e-9, name


def test_the_embedding_is_scaled_and_the_head_is_not():
    config = copy.deepcopy(lm.CONFIGS["states"])
    w = lm.as_float64(lm.draw_weights(config, 7))
    toks = [3, 1, 4, 1, 5]
    trace = []
    base = plain.forward(config, w, toks, trace)
    config["layers"] = []
    x = w["embed"][toks] * 4.0
    assert np.abs(plain.forward(config, w, toks) - plain.rms_norm(x, w["final.norm"], 1e-5) @ w["embed"].T).max() < 1e-12
    assert np.abs(base - plain.rms_norm(trace[-1], w["final.norm"], 1e-5) @ w["embed"].T).max() < 1e-12
