"""Ruzolorn on the GPU against the plain implementation: every mechanism alone through the kernels' own object, and the
engine under every way of cutting the work (each request whole; most of it in one step and its last tokens one by
one; portions of changing size down to two tokens; up to four live requests mixed, with so few pages and slots that they
are used again), in 32-bit and in bfloat16, and greedy generation through the entry point and the scheduler."""
import math

import numpy as np
import pytest
import torch

import ruzolorn_models as rm
import traces
from helpers import random_tokens
from plain import ruzolorn_plain as plain

pytestmark = pytest.mark.gpu

DT = {"float32": torch.float32, "bfloat16": torch.bfloat16}
# rms of (engine - plain) over rms of the plain logits, per position.  float32: rounding of 32-bit sums against float64.
# bfloat16: operands of every product, cached keys, values and latents and the queries are rounded to 8 bits, which moves the
# logits by a per cent or two, while a lost key, a lost state or a wrong expert moves them by tens of per cent.
# Where two experts' scores lie within that rounding of each other, bfloat16 may pick the other one with nothing
# wrong: in bfloat16 the bound holds for all but 8 % of the positions and the median error stays under 2 %.
TOL = {"float32": 2e-4, "bfloat16": 8e-2}


@pytest.fixture(scope="module")
def ops():
    import tinyinfer_amd  # noqa: F401
    from tinyinfer_amd.ops.kernels import get_ops
    return get_ops()


def dev(a, dtype=torch.float32):
    return torch.as_tensor(np.asarray(a)).to(dtype).to("cuda")


def f64(t):
    return t.detach().to("cpu", torch.float64).numpy()


def bf16_round(a):
    return torch.as_tensor(np.asarray(a, dtype=np.float32)).to(torch.bfloat16).to(torch.float64).numpy()


def f32_round(a):
    return np.asarray(a, dtype=np.float32).astype(np.float64)


# ---------------------------------------------------------------------------------- each mechanism alone
@pytest.mark.parametrize("W", [50, 192, 1030, 2048, 4100, 8192, 9000])
def test_layer_norms_on_either_side_of_a_sublayer(ops, W):
    """x += m LN(f1 y + f2 plus), then LN of the new x, in one kernel, whatever form y comes in; and each norm of either sort.
    The rows lie far from zero, so that a mean left in would show."""
    rng = np.random.default_rng(W)
    M, m, f1, f2 = 9, 0.7, 0.8, 1.3
    g, ng = rng.normal(1.0, 0.3, size=W), rng.normal(1.0, 0.3, size=W)
    x0 = rng.normal(-1.0, 2.0, size=(M, W))
    plus, gate = rng.normal(2.0, 3.0, size=(M, W)), rng.uniform(0.1, 0.9, size=M)
    lists = {"row": (rng.normal(3.0, 1.0, size=(M, W)), None, 0), "side by side": (rng.normal(3.0, 1.0, size=(3 * M, W)), None, 3),
             "listed": (rng.normal(3.0, 1.0, size=(2 * M + 5, W)), rng.permutation(2 * M + 5)[:2 * M].reshape(M, 2).astype(np.int32), 0)}
    norms = {True: plain.layer_norm, False: lambda x, w, eps: plain.over_rms(x, eps) * w}
    for kind, (y, gather, n_sum) in lists.items():
        y32 = f32_round(y)
        rows = y32 if kind == "row" else y32.reshape(M, 3, W).sum(1) if gather is None else y32[gather].sum(1)
        for centered, next_centered in ((True, True), (True, False), (False, True)):
            for branch in (False, True, "ungated"):
                tot = f1 * rows + (0 if not branch else f2 * f32_round(plus) * (f32_round(gate)[:, None] if branch is True else 1.0))
                want = f32_round(x0) + m * norms[centered](tot, f32_round(g), 1e-3)
                for dtype in ("float32", "bfloat16", None):
                    x = dev(x0)
                    out = torch.full((M, W), float("nan"), device="cuda", dtype=DT[dtype]) if dtype else None
                    ops.norm_residual_next(x, dev(y), dev(g), 1e-3, None if gather is None else dev(gather, torch.int32), n_sum,
                                           dev(plus) if branch else None, dev(gate) if branch is True else None, dev(ng) if dtype else None, 1e-2,
                                           out, centered, next_centered, m, f1, f2)
                    assert np.abs(f64(x) - want).max() < 2e-5 * np.abs(want).max(), (kind, branch, dtype)
                    if dtype:
                        nxt = norms[next_centered](want, f32_round(ng), 1e-2)
                        assert np.abs(f64(out) - nxt).max() < (5e-5 if dtype == "float32" else 2.0 ** -7) * np.abs(nxt).max(), (kind, branch, dtype)


@pytest.mark.parametrize("K", [1, 2, 3, 4, 5, 7])
@pytest.mark.parametrize("C", [5, 96, 1030, 2304])
def test_short_convolution_with_bias_and_silu(ops, K, C):
    """Columns of wider rows, three requests in slots of their own under every cut: whole, portions beside single tokens, single
    tokens alone.  Every cut gives the same bits; the state is left with the last rows; a zeroed slot starts anew."""
    rng = np.random.default_rng(10 * K + C)
    T, pad = (37, 21, 12), 12
    u = [f32_round(rng.normal(size=(n, C))) for n in T]
    taps, bias = f32_round(rng.normal(size=(C, K))), f32_round(rng.normal(size=C))
    want = [plain.silu(plain.causal_convolution(x, taps, bias)) for x in u]
    bare = [plain.causal_convolution(x, taps, np.zeros(C)) for x in u]

    def run(steps, state, activate=True):
        at, got = [0, 0, 0], [[], [], []]
        for step in steps:
            rows, meta, entry_of, pos = [], [], [], []
            for r, n in step:
                meta.append([len(entry_of), n, at[r], 2 - r])
                rows.append(u[r][at[r]:at[r] + n])
                entry_of += [len(meta) - 1] * n
                pos += range(at[r], at[r] + n)
                at[r] += n
            wide = torch.full((len(pos), C + 2 * pad), float("nan"), device="cuda")
            wide[:, pad:pad + C] = dev(np.concatenate(rows))
            out = torch.full((len(pos), C), float("nan"), device="cuda")
            ops.short_conv(wide[:, pad:pad + C], dev(taps), state, dev(meta, torch.int32), dev(entry_of, torch.int32), dev(pos, torch.int32), out,
                           dev(bias) if activate else None, activate)
            o, i = f64(out), 0
            for r, n in step:
                got[r].append(o[i:i + n])
                i += n
        assert tuple(at) == T
        return [np.concatenate(g) for g in got]

    def fresh():
        return torch.zeros(3, K - 1, C, device="cuda") if K > 1 else None
    whole_steps = [[(0, 37)], [(1, 21)], [(2, 12)]]
    state = fresh()
    whole = run(whole_steps, state)
    for g, w in zip(whole, want):
        assert np.abs(g - w).max() < 1e-5 * max(1.0, np.abs(w).max())
    for g, w in zip(run(whole_steps, fresh(), False), bare):
        assert np.abs(g - w).max() < 1e-5 * max(1.0, np.abs(w).max())
    mixed = [[(0, 2), (1, 9), (2, 1)], [(0, 1), (2, 1)], [(1, 1), (0, 20), (2, 2)], [(0, 1), (1, 1), (2, 1)], [(2, 7)], [(1, 10), (0, 13)]]
    single = [[(0, 1), (1, 1), (2, 1)]] * 12 + [[(1, 1), (0, 1)]] * 9 + [[(0, 1)]] * 16
    for steps in (mixed, single, [[(2, 12), (0, 37), (1, 21)]]):
        other = fresh()
        for g, w in zip(run(steps, other), whole):
            assert np.array_equal(g, w)
        if K > 1:
            assert np.array_equal(f64(other), f64(state))
    if K > 1:
        for r in range(3):
            tail = np.concatenate([np.zeros((K - 1, C)), u[r]])[-(K - 1):]
            assert np.array_equal(f64(state[2 - r]), tail)
        state.zero_()
        assert all(np.array_equal(g, w) for g, w in zip(run(single, state), whole))


def scan_by_hand(q, k, v, a, d, skip):
    """q, k [T, H, dk], v [T, H, dv], a, d [T, H] -> (o [T, H, dv], S [H, dk, dv])."""
    T, H, dk = q.shape
    S = np.zeros((H, dk, v.shape[2]))
    o = np.zeros((T, H, v.shape[2]))
    for t in range(T):
        for j in range(H):
            S[j] = a[t, j] * S[j] + d[t, j] * np.outer(k[t, j], v[t, j])
            o[t, j] = S[j].T @ q[t, j] + skip[j] * v[t, j]
    return o, S


def chunk_lists(entries):
    """entries [(row0, tokens)] -> chunks and spans of at most 64 tokens."""
    chunks, spans = [], []
    for e, (row0, n) in enumerate(entries):
        cuts = [(i, min(64, n - i)) for i in range(0, n, 64)]
        spans.append([len(chunks), len(cuts)])
        chunks += [[e, row0 + i, c, (1 if i == 0 else 0) | (2 if i + c == n else 0)] for i, c in cuts]
    return dev(chunks, torch.int32), dev(spans, torch.int32)


def check_scan(ops, rows, cols, kw, heads, dk, dv, want, S, cuts):
    """The scan of one request under every cut against (want, S): token by token forms agree bit for bit, chunks up to rounding;
    two requests in one step, in either form; a slot beside it is never touched."""
    T, scale = want.shape[0], np.abs(want).max()
    state = torch.zeros(4, heads, dk * dv, device="cuda")
    state[1].fill_(float("nan"))
    per_row = ("dt", "positions")

    def step(at, n, slot, o, chunked):
        part = {x: (y[at:at + n] if x in per_row else y) for x, y in kw.items()}
        chunks, spans = chunk_lists([(0, n)]) if chunked else (None, None)
        ops.linear_scan(rows[at:at + n].clone(), state, dev([[0, n, at, slot]], torch.int32), o[at:at + n], heads, dk, dv, cols,
                        chunks=chunks, spans=spans, **part)

    def run(sizes, slot, chunked):
        o = torch.full((T, heads * dv), float("nan"), device="cuda")
        at = 0
        for n in sizes:
            step(at, n, slot, o, chunked(n))
            at += n
        assert at == T
        return f64(o).reshape(T, heads, dv)

    whole = run([T], 0, lambda n: False)
    assert np.abs(whole - want).max() < 3e-5 * scale
    assert np.abs(f64(state[0]).reshape(heads, dk, dv) - S).max() < 3e-5 * np.abs(S).max()
    assert np.array_equal(run(cuts, 2, lambda n: False), whole)
    assert np.array_equal(f64(state[2]), f64(state[0]))
    for sizes, chunked in (([T], lambda n: True), (cuts, lambda n: True), (cuts, lambda n: n >= 10), ([1, 65, T - 66], lambda n: n > 1)):
        state[3].zero_()
        got = run(sizes, 3, chunked)
        assert np.abs(got - want).max() < 3e-5 * scale
        assert np.abs(f64(state[3]).reshape(heads, dk, dv) - S).max() < 3e-5 * np.abs(S).max()
    # two requests in one step
    n1 = T - 7
    both = {x: (torch.cat([y[:n1], y]) if x in per_row else y) for x, y in kw.items()}
    for chunked in (False, True):
        state[0].zero_()
        state[2].zero_()
        o = torch.full((n1 + T, heads * dv), float("nan"), device="cuda")
        chunks, spans = chunk_lists([(0, n1), (n1, T)]) if chunked else (None, None)
        ops.linear_scan(torch.cat([rows[:n1], rows]), state, dev([[0, n1, 0, 2], [n1, T, 0, 0]], torch.int32), o, heads, dk, dv, cols, chunks=chunks,
                        spans=spans, **both)
        got = f64(o).reshape(n1 + T, heads, dv)
        assert np.abs(got[:n1] - want[:n1]).max() < 3e-5 * scale and np.abs(got[n1:] - want).max() < 3e-5 * scale
    assert torch.isnan(state[1]).all()


@pytest.mark.parametrize("heads,dk,dv,rot_dims", [(3, 16, 24, 8), (1, 10, 7, 10), (2, 64, 64, 64), (4, 128, 40, 32), (2, 30, 130, 0),
                                                  (1, 256, 256, 256), (5, 1, 3, 0), (2, 72, 68, 2)])
def test_retention_scan(ops, heads, dk, dv, rot_dims):
    """Rotated queries and keys under a fixed decay; decays of 1, of next to nothing and between; a key that stands far out at the
    start reaches the last token."""
    rng = np.random.default_rng(dk + dv)
    T = 150
    nq, nv = heads * dk, heads * dv
    rows = f32_round(rng.normal(size=(T, 2 * nq + nv + 4)))
    rows[2, 2 + nq:2 + 2 * nq] *= 30.0
    decay = f32_round(np.array([1.0, 0.03, 0.9, 0.997, 0.6])[:heads])
    rot = dict(base=50.0, dims=rot_dims)
    q = plain.rotate_half(rows[:, 2:2 + nq].reshape(T, heads, dk), rot)
    k = plain.rotate_half(rows[:, 2 + nq:2 + 2 * nq].reshape(T, heads, dk), rot) * 0.37
    v = rows[:, 4 + 2 * nq:].reshape(T, heads, dv)
    want, S = scan_by_hand(q, k, v, np.tile(decay, (T, 1)), np.ones((T, heads)), np.zeros(heads))
    kw = dict(decay=dev(decay), k_scale=0.37)
    for tabled in ((False, True) if rot_dims else (False,)):
        if rot_dims:
            freq = np.array([50.0 ** (-2.0 * i / rot_dims) for i in range(rot_dims // 2)])
            angles = np.outer(np.arange(T), freq)
            kw.update(inv_freq=dev(freq), positions=dev(np.arange(T), torch.int32), rot_dims=rot_dims,
                      rope_table=dev(np.stack([np.cos(angles), np.sin(angles)], axis=-1)) if tabled else None)
        check_scan(ops, dev(rows), (2, 2 + nq, 4 + 2 * nq), kw, heads, dk, dv, want, S, [17, 1, 1, 2, 33, 64, 31, 1])


@pytest.mark.parametrize("heads,groups,dk,dv", [(4, 2, 16, 24), (3, 1, 9, 7), (6, 3, 64, 64), (2, 2, 128, 48), (4, 1, 130, 72), (1, 1, 256, 16), (8, 4, 4, 4)])
def test_selective_scan(ops, heads, groups, dk, dv):
    """Step sizes from next to nothing to hundreds (everything before is forgotten, and the differences of the chunk's large sums must
    keep their digits), groups of heads that share B and C, and the input itself passed through."""
    rng = np.random.default_rng(dk + dv)
    T = 150
    nq, nv = groups * dk, heads * dv
    rows = f32_round(rng.normal(size=(T, nv + 2 * nq + 4)))
    dt = f32_round(rng.normal(-1.0, 1.5, size=(T, heads + 3)))
    dt[60, 3:] = 300.0                                        # (the state's share of this token's own value is large too)
    bias, a_log, skip = f32_round(rng.normal(size=heads)), f32_round(rng.uniform(-4.0, 2.0, size=heads)), f32_round(rng.normal(size=heads))
    v = rows[:, :nv].reshape(T, heads, dv)
    k = np.repeat(rows[:, nv:nv + nq].reshape(T, groups, dk), heads // groups, axis=1)
    q = np.repeat(rows[:, nv + nq + 4:].reshape(T, groups, dk), heads // groups, axis=1)
    d = plain.softplus(dt[:, 3:] + bias)
    want, S = scan_by_hand(q, k, v, np.exp(-np.exp(a_log) * d), d, skip)
    kw = dict(dt=dev(dt), dt_col=3, dt_bias=dev(bias), a_log=dev(a_log), skip=dev(skip), qk_heads=groups)
    # (the tokens in front of the large step are compared on their own scale below)
    check_scan(ops, dev(rows), (nv + nq + 4, nv, 0), kw, heads, dk, dv, want, S, [17, 1, 1, 2, 33, 64, 31, 1])
    early = want[:60]
    state = torch.zeros(1, heads, dk * dv, device="cuda")
    chunks, spans = chunk_lists([(0, T)])
    for form in ((None, None), (chunks, spans)):
        state.zero_()
        o = torch.empty(T, nv, device="cuda")
        ops.linear_scan(dev(rows), state, dev([[0, T, 0, 0]], torch.int32), o, heads, dk, dv, (nv + nq + 4, nv, 0), chunks=form[0], spans=form[1], **kw)
        assert np.abs(f64(o).reshape(T, heads, dv)[:60] - early).max() < 3e-5 * np.abs(early).max()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("W,groups", [(96, 4), (84, 1), (60, 12), (2048, 1), (1024, 8), (1036, 2), (5000, 1), (4096, 2), (6600, 3), (9000, 1), (20001, 1), (70, 70)])
def test_norms_in_parts_with_a_gate_behind_or_in_front(ops, dtype, W, groups):
    rng = np.random.default_rng(W + groups)
    M = 11
    o = f32_round(rng.normal(size=(M, W)) * np.linspace(0.1, 5.0, W))      # parts of very different size
    for off, extra in ((9, 3), (8, 0)):
        proj = f32_round(rng.normal(size=(M, W + off + extra)))
        w = f32_round(rng.normal(1.0, 0.3, size=W))
        z = proj[:, off:off + W]
        for weight in (w, None):
            for silu in (False, True):
                for first in (False, True):
                    act = plain.silu(z) if silu else plain.sigmoid(z)
                    y = o * act if first else o
                    want = plain.over_rms(y.reshape(M, groups, W // groups), 1e-3).reshape(M, W) * (w if weight is not None else 1.0) * (1.0 if first else act)
                    out = torch.full((M, W), float("nan"), device="cuda", dtype=DT[dtype])
                    ops.gated_group_norm(dev(o), dev(proj), off, None if weight is None else dev(w), 1e-3, out, groups, silu, first)
                    assert np.abs(f64(out) - want).max() < (3e-5 if dtype == "float32" else 2.0 ** -7) * np.abs(want).max(), (off, silu, first)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("heads,kv,dk,dv,P,window", [(4, 2, 16, 24, 16, 20), (3, 3, 7, 9, 4, 1), (5, 1, 64, 40, 16, 33), (2, 1, 128, 128, 16, 64), (2, 2, 32, 16, 8, 15),
                                                     (1, 1, 10, 130, 16, 100)])
def test_windowed_attention_with_normed_heads(ops, dtype, heads, kv, dk, dv, P, window):
    """Preparation and attention without positions over pages in any order.  Three queries each stand far out against one key: the
    first their window still holds, the next one back, and their own."""
    rng = np.random.default_rng(dk * 10 + window)
    T, eps, scale = 130, 1e-5, 0.9 * dk ** -0.5
    nq, nk, nv = heads * dk, kv * dk, kv * dv
    proj = rng.normal(size=(T, nq + nk + nv))
    qw, kw = rng.normal(1.0, 0.3, size=dk), rng.normal(1.0, 0.3, size=dk)
    k = proj[:, nq:nq + nk].reshape(T, kv, dk)
    per = heads // kv
    for t, back in ((T - 1, window - 1), (T - 2, window), (T - 3, 0)):
        if 0 <= t - back:
            for h in range(heads):      # a query along its key: the norm of both makes the score the largest there is
                proj[t, h * dk:(h + 1) * dk] = k[t - back, h // per] * kw / np.maximum(np.abs(qw), 0.1) * np.sign(qw)
    p32 = f32_round(proj)
    q = plain.over_rms(p32[:, :nq].reshape(T, heads, dk), eps) * f32_round(qw)
    k = plain.over_rms(p32[:, nq:nq + nk].reshape(T, kv, dk), eps) * f32_round(kw)
    v = p32[:, nq + nk:].reshape(T, kv, dv)
    if dtype == "bfloat16":
        q, k, v = bf16_round(q), bf16_round(k), bf16_round(v)
    sharp = 8.0 * scale
    want = np.zeros((T, heads, dv))
    for h in range(heads):
        want[:, h] = plain.window_softmax(q[:, h] @ k[:, h // per].T * sharp, window) @ v[:, h // per]
    n_pages = -(-T // P)
    ids = rng.permutation(n_pages + 3)[:n_pages]
    padded = dk if (dv < dk and dk in (32, 64, 128)) else dv
    pool = torch.full((n_pages + 3, kv, P, dk + padded), float("nan"), device="cuda", dtype=DT[dtype])
    table = dev(np.asarray(ids, dtype=np.int32)[None, :], torch.int32)
    pos, slot = dev(np.arange(T), torch.int32), torch.zeros(T, device="cuda", dtype=torch.int32)
    q_out = torch.empty(T, nq, device="cuda", dtype=DT[dtype])
    for at, n in ((0, 70), (70, T - 70)):
        ops.gated_qkv_prep(dev(proj)[at:at + n].contiguous(), dev(qw), dev(kw), None, None, pos[at:at + n].contiguous(), slot[:n].contiguous(), table, pool,
                           q_out[at:at + n], heads, kv, dk, dv, (0, nq, nq + nk), eps=eps)
    out = torch.empty(T, heads * dv, device="cuda", dtype=DT[dtype])
    ops.gated_attention(q_out, pool, table, pos, slot, None, None, out, heads, kv, dk, dv, sharp, window)
    got = f64(out).reshape(T, heads, dv)
    assert np.abs(got - want).max() < (5e-5 if dtype == "float32" else 2e-2) * np.abs(want).max()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("E,N,top,W,F", [(5, 2, 2, 64, 96), (1, 3, 3, 33, 17), (8, 2, 3, 128, 64), (4, 4, 1, 96, 32), (6, 1, 4, 1024, 320), (3, 0, 2, 40, 24),
                                         (7, 7, 5, 2080, 64)])
def test_router_with_a_correction_and_experts_beside_identities(ops, dtype, E, N, top, W, F):
    """Few tokens (row by row) and many (grouped on the matrix cores where the sizes allow); at many there are tokens whose choices
    are identities alone."""
    rng = np.random.default_rng(E * 100 + W)
    r = bf16_round if dtype == "bfloat16" else f32_round
    w = {"m.router": f32_round(rng.normal(0.0, 2.0 / math.sqrt(W), size=(E + N, W))), "m.correction": f32_round(rng.normal(0.0, 0.1, size=E + N))}
    for e in range(E):
        w[f"m.e{e}.gate"], w[f"m.e{e}.up"] = r(rng.normal(0.0, 1.5 / math.sqrt(W), size=(F, W))), r(rng.normal(0.0, 1.5 / math.sqrt(W), size=(F, W)))
        w[f"m.e{e}.down"] = r(rng.normal(0.0, 1.0 / math.sqrt(F), size=(W, F)))
    gate_up = dev(np.concatenate([np.concatenate([w[f"m.e{e}.gate"], w[f"m.e{e}.up"]]) for e in range(E)]), DT[dtype])
    down = dev(np.concatenate([w[f"m.e{e}.down"] for e in range(E)]), DT[dtype])
    alone = 0
    for M in (1, 3, 40, 400):
        h = r(rng.normal(size=(M, W)))
        ids = torch.empty(M, top, device="cuda", dtype=torch.int32)
        wts = torch.empty(M, top, device="cuda")
        ops.moe_route_grouped(dev(h, DT[dtype]), dev(w["m.router"]), ids, wts, dev(w["m.correction"]), top, renormalize=False, score="softmax")
        ids_want, wts_want = plain.route(h, dict(top=top), w, "m")
        z = h @ w["m.router"].T
        p = np.exp(z - z.max(axis=1, keepdims=True))
        choice = np.sort(p / p.sum(axis=1, keepdims=True) + w["m.correction"], axis=1)
        sure = np.diff(choice, axis=1).min(axis=1) > 1e-5 if E + N > 1 else np.ones(M, dtype=bool)
        assert np.array_equal(ids.cpu().numpy()[sure], ids_want[sure]) and np.abs(f64(wts)[sure] - wts_want[sure]).max() < 1e-5
        y = torch.full((M, W), float("nan"), device="cuda")
        ops.moe_experts_gated(dev(h, DT[dtype]), ids, wts, gate_up, down, y, E, "silu", identity=N)
        want = np.zeros((M, W))
        ids_got, wts_got = ids.cpu().numpy(), f64(wts)
        alone += int((ids_got >= E).all(axis=1).sum())
        for e in range(E):
            t, k = np.nonzero(ids_got == e)
            if len(t):
                np.add.at(want, t, wts_got[t, k][:, None] * plain.gated_ff(h[t], w, f"m.e{e}"))
        t, k = np.nonzero(ids_got >= E)
        np.add.at(want, t, wts_got[t, k][:, None] * h[t])
        assert np.abs(f64(y) - want).max() < (5e-5 if dtype == "float32" else 1.5e-2) * np.abs(want).max(), M
    assert alone > 0 or N < top or top > 3


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_identities_beside_ungated_experts(ops, dtype):
    """The same places beside experts of two matrices, the weight on their inputs or their outputs; few tokens and many."""
    rng = np.random.default_rng(3)
    r = bf16_round if dtype == "bfloat16" else f32_round
    E, N, top, W, F = 4, 2, 2, 64, 96
    up, down = r(rng.normal(0.0, 0.2, size=(E, F, W))), r(rng.normal(0.0, 0.1, size=(E, W, F)))
    for M in (5, 300):
        h = r(rng.normal(size=(M, W)))
        ids = np.stack([rng.permutation(E + N)[:top] for _ in range(M)]).astype(np.int32)
        wts = f32_round(rng.uniform(0.2, 0.8, size=(M, top)))
        for scale_input in (True, False):
            y = torch.full((M, W), float("nan"), device="cuda")
            ops.moe_experts(dev(h, DT[dtype]), dev(ids, torch.int32), dev(wts), dev(up.reshape(E * F, W), DT[dtype]), dev(down.reshape(E * W, F), DT[dtype]), y, E,
                            scale_input, identity=N)
            want = np.zeros((M, W))
            for t in range(M):
                for e, a in zip(ids[t], wts[t]):
                    if e >= E:
                        want[t] += a * h[t]
                    elif scale_input:
                        want[t] += down[e] @ np.maximum(up[e] @ (a * h[t]), 0.0) ** 2
                    else:
                        want[t] += a * (down[e] @ np.maximum(up[e] @ h[t], 0.0) ** 2)
            assert np.abs(f64(y) - want).max() < (5e-5 if dtype == "float32" else 1.5e-2) * np.abs(want).max(), (M, scale_input)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("M", [1, 5, 40, 300])
def test_a_gated_feed_forward_takes_silu_inside_its_product(ops, dtype, M):
    rng = np.random.default_rng(M)
    r = bf16_round if dtype == "bfloat16" else f32_round
    W, F = 96, 160
    h, gate, up = r(rng.normal(size=(M, W))), r(rng.normal(0.0, 0.2, size=(F, W))), r(rng.normal(0.0, 0.2, size=(F, W)))
    out = torch.full((M, F), float("nan"), device="cuda", dtype=DT[dtype])
    ops.linear(dev(h, DT[dtype]), dev(np.concatenate([gate, up]), DT[dtype]), out, "swiglu")
    want = plain.silu(h @ gate.T) * (h @ up.T)
    assert np.abs(f64(out) - want).max() < (3e-5 if dtype == "float32" else 2.0 ** -7) * np.abs(want).max()


# ---------------------------------------------------------------------------------- the engine
REQUEST_LENGTHS = {"a": 97, "b": 45, "c": 130, "d": 33, "e": 71, "f": 58}
PROMPT_LENGTHS = {"a": 60, "b": 12, "c": 101, "d": 30, "e": 2, "f": 41}
_made = {}


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    def get(name):
        if name not in _made:
            config = rm.CONFIGS[name]
            weights = rm.draw_weights(config, seed=len(name) * 13 + 2)
            path = rm.write_folder(str(tmp_path_factory.mktemp("ruzolorn_" + name)), config, 0, weights)
            requests = {r: random_tokens(n, config["vocab"], 17 + i) for i, (r, n) in enumerate(REQUEST_LENGTHS.items())}
            w = rm.as_float64(weights)
            want = {r: plain.forward(config, w, t) for r, t in requests.items()}
            _made[name] = (path, requests, want, w)
        return _made[name]
    return get


def build_engine(folder, dtype, max_tokens, page_size=16, max_requests=4):
    import tinyinfer_amd  # noqa: F401
    from tinyinfer_amd.engine import Engine
    return Engine.from_folder(folder, dtype, page_size=page_size, max_tokens=max_tokens, max_requests=max_requests, max_seq=max_tokens)


def replay(engine, trace):
    from tinyinfer_amd.engine import StepEntry
    got = {}
    for step in trace:
        logits = engine.step([StepEntry(r, t, w) for r, t, w in step["entries"]])
        rows = None if logits is None else logits.cpu().numpy().astype(np.float64)
        i = 0
        for r, _, w in step["entries"]:
            for _ in w:
                got.setdefault(r, []).append(rows[i])
                i += 1
        for r in step["end"]:
            engine.release(r)
        engine.cache.check()
    return {r: np.stack(v) for r, v in got.items()}


def errors(got, want):
    assert got.shape == want.shape, (got.shape, want.shape)
    d = got - want
    d = d - d.mean(axis=1, keepdims=True)
    ref = want - want.mean(axis=1, keepdims=True)
    return np.sqrt((d ** 2).mean(axis=1)) / np.sqrt((ref ** 2).mean(axis=1))


def worst(got, want):
    w, where = 0.0, None
    for r in want:
        e = errors(got[r], want[r])
        if e.max() > w:
            w, where = float(e.max()), (r, int(e.argmax()))
    return w, where


def within(got, want, dtype):
    """32-bit: every position within the bound.  bfloat16: all but 8 % of them, and the median far below it."""
    if dtype == "float32":
        w, where = worst(got, want)
        return w < TOL[dtype], (w, where)
    e = np.concatenate([errors(got[r], want[r]) for r in want])
    over = float((e > TOL[dtype]).mean())
    return over <= 0.08 and float(np.median(e)) < 2e-2, (over, float(np.median(e)), float(e.max()))


def make_trace(mode, requests):
    if mode == "whole":
        return traces.whole(requests)
    if mode == "tail":
        return traces.tail_one_by_one(requests, 32)
    if mode == "portions":
        return traces.portions(requests)
    return traces.mixed(requests, PROMPT_LENGTHS, live=4)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name,page_size", [("mixed", 8), ("plain", 4), ("wide", 16), ("states", 16), ("edges", 4)])
@pytest.mark.parametrize("mode", ["whole", "tail", "portions", "mixed"])
def test_engine_matches_plain(folders, name, page_size, dtype, mode):
    folder, requests, want, _ = folders(name)
    trace = make_trace(mode, requests)
    n_tok = traces.max_pages(trace, page_size) * page_size      # the tightest pool: pages are handed out again
    engine = build_engine(folder, dtype, n_tok, page_size)       # four state slots for six requests: slots are used again
    got = replay(engine, trace)
    assert not engine.cache.live_requests()
    ok, seen = within(got, want, dtype)
    assert ok, (name, mode, dtype, seen)


@pytest.mark.parametrize("name", ["mixed", "plain"])
def test_cuts_agree_bit_for_bit_in_float32(folders, name):
    """Token by token from the first token on, in portions, and whole: in 32-bit every sum is taken in an order that does
    not depend on the step, so the logits are the same bits."""
    folder, requests, _, _ = folders(name)
    some = {r: requests[r][:40] for r in ("b", "d")}
    results = []
    for trace in (traces.whole(some), traces.tail_one_by_one(some, 39), traces.portions(some), traces.mixed(some, {"b": 20, "d": 3}, live=2)):
        engine = build_engine(folder, "float32", 256)
        results.append(replay(engine, trace))
    for other in results[1:]:
        for r in some:
            assert np.array_equal(results[0][r], other[r]), r


def test_pages_and_slots_used_again_hold_nothing_of_their_last_owner(folders):
    """One request at a time in the smallest pool that holds it and one state slot: the second gets the pages and the slot
    the first gave back, and must find an empty memory there."""
    folder, requests, want, _ = folders("mixed")
    engine = build_engine(folder, "float32", 144, page_size=8, max_requests=1)
    for r in ("c", "b", "c"):
        got = replay(engine, traces.portions({r: requests[r]}))
        w, where = worst(got, {r: want[r]})
        assert w < TOL["float32"], (r, w, where)


def test_long_decoding(folders):
    """A prompt of 50 tokens in portions of 32, then 250 tokens one by one: the states of both recurrences and the convolutions'
    rows are carried through every step, every window passes over decoded tokens, and where there is none the first keys stay visible."""
    from tinyinfer_amd.engine import StepEntry
    folder, _, _, w = folders("mixed")
    config = rm.CONFIGS["mixed"]
    toks = random_tokens(300, config["vocab"], 99)
    want = plain.forward(config, w, toks)
    for dtype in ("float32", "bfloat16"):
        engine = build_engine(folder, dtype, 320, page_size=8)
        rows, at = [], 0
        while at < 50:
            n = min(32, 50 - at)
            rows.append(engine.step([StepEntry("x", toks[at:at + n], list(range(n)))]).cpu().numpy())
            at += n
        for t in toks[50:]:
            rows.append(engine.step([StepEntry("x", [t], [0])]).cpu().numpy())
            engine.cache.check()
        got = np.concatenate(rows).astype(np.float64)
        ok, seen = within({"x": got}, {"x": want}, dtype)
        assert ok, (dtype, seen)


def test_a_token_far_back_reaches_the_last_position(folders):
    """Changing token 3 of 120 moves the last position's logits, through the cached keys and through the carried state alike
    (the plain model says by how much; the engine, fed in a portion and then token by token, agrees with it)."""
    from tinyinfer_amd.engine import StepEntry
    folder, requests, _, w = folders("mixed")
    config = rm.CONFIGS["mixed"]
    toks = list(requests["c"][:120])
    other = list(toks)
    other[3] = (other[3] + 1) % config["vocab"]
    engine = build_engine(folder, "float32", 256, page_size=8)
    outs = []
    for i, t in enumerate((toks, other)):
        engine.step([StepEntry(str(i), t[:100], [])])
        for tok in t[100:119]:
            engine.step([StepEntry(str(i), [tok], [])])
        outs.append(engine.step([StepEntry(str(i), [t[119]], [0])]).cpu().numpy()[0].astype(np.float64))
        engine.release(str(i))
    want = [plain.forward(config, w, t)[-1] for t in (toks, other)]
    assert np.abs(want[0] - want[1]).max() > 1e-3
    for g, wnt in zip(outs, want):
        assert errors(g[None], wnt[None])[0] < TOL["float32"]


@pytest.mark.parametrize("use_graph", [False, True])
def test_greedy_generation_through_the_entry_point(folders, use_graph):
    """Several prompts of unequal length at once through LLM.generate: the scheduler cuts the prompts into portions of 16
    and batches decoding requests; every generated token is the plain model's argmax."""
    import tinyinfer_amd as ti
    folder, requests, _, w = folders("mixed")
    config = rm.CONFIGS["mixed"]
    prompts = [requests["b"][:37], requests["d"][:5], requests["e"][:50], requests["f"][:1]]
    n_new = 12
    llm = ti.LLM(folder, dtype="float32", max_seq=128, max_requests=3, chunk_size=16, max_batched_tokens=40, use_graph=use_graph)
    got = llm.generate(prompts, max_new_tokens=n_new, temperature=0.0)
    for p, g in zip(prompts, got):
        toks = list(p)
        for _ in range(n_new):
            logits = plain.forward(config, w, toks)[-1]
            best = int(np.argmax(logits))
            margin = logits[best] - np.partition(logits, -2)[-2]
            toks.append(best)
            if margin < 1e-3:          # a tie within rounding: what follows may differ legitimately
                break
        n = len(toks) - len(p)
        assert g[:n] == toks[len(p):], (p[:3], g, toks[len(p):])


def test_graphs_replay_the_bfloat16_kernels(folders):
    """bfloat16 at sizes the matrix cores serve: decoding from captured graphs gives the tokens that decoding step by step gives."""
    import tinyinfer_amd as ti
    folder, requests, _, _ = folders("wide")
    prompts = [requests["b"][:37], requests["d"][:5], requests["e"][:50]]
    outs = []
    for use_graph in (False, True):
        llm = ti.LLM(folder, dtype="bfloat16", max_seq=128, max_requests=3, chunk_size=32, max_batched_tokens=64, use_graph=use_graph)
        outs.append(llm.generate(prompts, max_new_tokens=20, temperature=0.0))
    assert outs[0] == outs[1]


def test_matrix_core_kernels_agree_with_the_row_wise_ones(folders):
    """bfloat16 at sizes the matrix cores serve: a long prompt whole (tiles, in pairs and one by one), then single tokens with every
    context split over workgroups and not split.  Every way agrees with the row-wise kernels and with the plain model."""
    from tinyinfer_amd.engine import StepEntry
    folder, _, _, w = folders("wide")
    config = rm.CONFIGS["wide"]
    toks = random_tokens(420, config["vocab"], 5)
    want = plain.forward(config, w, toks)

    def run(fast, splits=0, paired=None):
        engine = build_engine(folder, "bfloat16", 448)
        engine.ops.use_fast_attention = fast
        engine.ops.force_decode_splits = splits
        engine.ops.force_paired_tiles = paired
        engine.ops.count_calls(True)
        rows = [engine.step([StepEntry("x", toks[:400], list(range(400)))]).cpu().numpy()]
        for t in toks[400:]:
            rows.append(engine.step([StepEntry("x", [t], [0])]).cpu().numpy())
        names = [r["name"] for r in engine.ops.timing_report()]
        engine.ops.count_calls(False)
        return np.concatenate(rows).astype(np.float64), names

    slow, names = run(False)
    mine = [n for n in names if n.startswith("gated_attention")]
    assert mine and all(n.endswith("[generic]") for n in mine)
    ok, seen = within({"x": slow}, {"x": want}, "bfloat16")
    assert ok, seen
    for splits, paired in ((0, None), (4, True), (1, False)):
        fast, names = run(True, splits, paired)
        mine = [n for n in names if n.startswith("gated_attention")]
        assert mine and all(n.endswith("[mfma]") for n in mine), mine
        scans = [n for n in names if n.startswith("linear_scan")]
        assert {("selective" in n, n.endswith("[chunked]")) for n in scans} == {(a, b) for a in (True, False) for b in (True, False)}
        assert any(n.startswith("moe_experts") and "+identity" in n and "grouped, sums left" in n for n in names)
        assert any(n.startswith("norm_residual_next") and "centered plus +norm" in n for n in names)
        ok, seen = within({"x": fast}, {"x": want}, "bfloat16")
        assert ok, (splits, paired, seen)
        # a router's choice within rounding of a tie may fall the other way at a position or two
        e = errors(fast, slow)
        assert np.median(e) < 2e-2 and (e > 0.08).mean() <= 0.05, (splits, paired, float(np.median(e)), float(e.max()))


def test_long_portions_beside_single_tokens(folders):
    """Steps in which a portion goes through the chunks of both recurrences while other requests decode one token each: their states sit in
    the same step's chunks."""
    folder, _, _, w = folders("mixed")
    config = rm.CONFIGS["mixed"]
    reqs = {r: random_tokens(n, config["vocab"], 40 + i) for i, (r, n) in enumerate((("p", 330), ("q", 40), ("s", 300)))}
    want = {r: plain.forward(config, w, t) for r, t in reqs.items()}
    cuts = {"p": [130, 70, 128, 1, 1], "q": [20] + [1] * 20, "s": [1, 2, 150, 147]}
    at = {r: 0 for r in reqs}
    trace = []
    for k in range(max(len(c) for c in cuts.values())):
        step = {"entries": [], "end": []}
        for r in reqs:
            if k < len(cuts[r]):
                n = cuts[r][k]
                step["entries"].append((r, reqs[r][at[r]:at[r] + n], list(range(n))))
                at[r] += n
                if at[r] == len(reqs[r]):
                    step["end"].append(r)
        trace.append(step)
    for dtype in ("float32", "bfloat16"):
        got = replay(build_engine(folder, dtype, 704, page_size=8), trace)
        ok, seen = within(got, want, dtype)
        assert ok, (dtype, seen)


def plain_greedy(config, w, prompt, n_new):
    """(generated ids, how many of them stand clear of a tie within rounding)."""
    toks, sure = list(prompt), 0
    for k in range(n_new):
        logits = plain.forward(config, w, toks)[-1]
        best = int(np.argmax(logits))
        if sure == k and logits[best] - np.partition(logits, -2)[-2] > 1e-3:
            sure = k + 1
        toks.append(best)
    return toks[len(prompt):], sure


def test_command_line_generates_from_a_ruzolorn_folder(folders):
    """bin/tinyinfer picks the model by config.json: token ids in, the plain model's greedy tokens out; with --cuda-graph too."""
    import os
    import subprocess
    import sys
    folder, requests, _, w = folders("plain")
    config = rm.CONFIGS["plain"]
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    p1, p2 = requests["b"][:11], requests["d"][:4]
    for extra in ([], ["--cuda-graph"]):
        run = subprocess.run([sys.executable, os.path.join(root, "bin", "tinyinfer"), "-m", folder, "-n", "6", "-p", ",".join(map(str, p1)),
                              "-p", " ".join(map(str, p2)), "--dtype", "float32", "--max-seq", "64"] + extra,
                             capture_output=True, text=True, timeout=300)
        assert run.returncode == 0, run.stderr[-2000:]
        outputs = [l[len("[output] "):].split() for l in run.stdout.split("\n") if l.startswith("[output] ")]
        assert len(outputs) == 2
        for p, got in zip((p1, p2), outputs):
            want, sure = plain_greedy(config, w, p, 6)
            assert [int(t) for t in got][:sure] == want[:sure], (got, want)


def test_random_weights_drawn_on_the_device_run():
    """A config.json alone: the parts' declared distributions give a model that steps (what the bench tool measures)."""
    from tinyinfer_amd.engine import Engine, StepEntry
    for name in ("mixed", "wide"):
        engine = Engine.from_config(rm.CONFIGS[name], seed=3, dtype="bfloat16", page_size=16, max_tokens=256, max_requests=2, max_seq=256)
        toks = random_tokens(70, rm.CONFIGS[name]["vocab"], 1)
        a = engine.step([StepEntry("x", toks, [69])]).cpu().numpy()
        engine.release("x")
        assert engine.step([StepEntry("y", toks[:69], [])]) is None
        b = engine.step([StepEntry("y", toks[69:], [0])]).cpu().numpy()
        assert np.isfinite(a).all() and a.std() > 0
        assert np.abs(a - b).max() < 0.08 * max(1e-6, np.abs(a).max())


def test_trace_replay_program(folders, tmp_path):
    """The replay program on a Ruzolorn folder: it picks the model by config.json and writes the logits the engine gives."""
    import os
    import subprocess
    import sys
    folder, requests, want, _ = folders("plain")
    some = {r: requests[r] for r in ("b", "d", "f")}
    trace = traces.mixed(some, PROMPT_LENGTHS, live=2)
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    out = tmp_path / "out"
    proc = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", folder, "--dtype", "float32", "--out", str(out),
                           "--max-tokens", str(traces.max_tokens(trace))], input=traces.to_jsonl(trace), text=True,
                          capture_output=True, timeout=600)
    assert proc.returncode == 0, proc.stderr[-2000:]
    V = rm.CONFIGS["plain"]["vocab"]
    got = {}
    for i, step in enumerate(trace):
        assert f"done {i}" in proc.stdout
        rows = np.fromfile(out / f"{i}.f32", dtype="<f4").reshape(-1, V).astype(np.float64)
        k = 0
        for r, _, wnt in step["entries"]:
            for _ in wnt:
                got.setdefault(r, []).append(rows[k])
                k += 1
    w, where = worst({r: np.stack(v) for r, v in got.items()}, {r: want[r] for r in some})
    assert w < TOL["float32"], (w, where)
