"""Lupolorn on the GPU against the plain implementation: every mechanism alone through the kernels' own object, and the
engine under every way of cutting the work (each request whole; most of it in one step and its last tokens one by
one; portions of changing size down to two tokens; up to four live requests mixed, with so few pages and slots that they
are used again), in 32-bit and in bfloat16, and greedy generation through the entry point and the scheduler."""
import math

import numpy as np
import pytest
import torch

import lupolorn_models as lm
import traces
from helpers import random_tokens
from plain import lupolorn_plain as plain

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


def paged(rng, n_tokens, P, extra_pages=3):
    n_pages = -(-n_tokens // P)
    ids = rng.permutation(n_pages + extra_pages)[:n_pages]
    return np.asarray(ids, dtype=np.int32)[None, :], n_pages + extra_pages


# ---------------------------------------------------------------------------------- each mechanism alone
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_embedding_times_a_factor(ops, dtype):
    rng = np.random.default_rng(0)
    table = rng.normal(size=(31, 50))
    toks = np.array([30, 0, 7, 7, 15], dtype=np.int32)
    x = torch.full((5, 50), float("nan"), device="cuda")
    ops.embed(dev(table, DT[dtype]), dev(toks, torch.int32), x, 13.37)
    t = bf16_round(table) if dtype == "bfloat16" else f32_round(table)
    assert np.abs(f64(x) - t[toks] * 13.37).max() < 1e-5 * np.abs(t).max() * 13.37


@pytest.mark.parametrize("W", [50, 192, 1030, 2048, 4100, 8192, 9000])
def test_norms_on_either_side_of_a_sublayer(ops, W):
    """x += rms norm of what a sublayer left (one row, a sum of listed rows, of rows side by side, a gated branch beside it), then
    the next sublayer's rms norm of the new x, in the same kernel; and the first half alone."""
    rng = np.random.default_rng(W)
    M = 9
    g, ng = rng.normal(1.0, 0.3, size=W), rng.normal(1.0, 0.3, size=W)
    x0 = rng.normal(size=(M, W)) * 2
    plus, gate = rng.normal(size=(M, W)) * 3, rng.uniform(0.1, 0.9, size=M)
    lists = {"row": (rng.normal(size=(M, W)), None, 0), "side by side": (rng.normal(size=(3 * M, W)), None, 3),
             "listed": (rng.normal(size=(2 * M + 5, W)), rng.permutation(2 * M + 5)[:2 * M].reshape(M, 2).astype(np.int32), 0)}
    for kind, (y, gather, n_sum) in lists.items():
        y32 = f32_round(y)
        rows = y32 if kind == "row" else y32.reshape(M, 3, W).sum(1) if gather is None else y32[gather].sum(1)
        for branch in (False, True, "ungated"):
            tot = rows + (0 if not branch else f32_round(plus) * (f32_round(gate)[:, None] if branch is True else 1.0))
            want = f32_round(x0) + plain.rms_norm(tot, f32_round(g), 1e-3)
            for dtype in ("float32", "bfloat16", None):
                x = dev(x0)
                out = torch.full((M, W), float("nan"), device="cuda", dtype=DT[dtype]) if dtype else None
                ops.norm_residual_next(x, dev(y), dev(g), 1e-3, None if gather is None else dev(gather, torch.int32), n_sum,
                                       dev(plus) if branch else None, dev(gate) if branch is True else None, dev(ng) if dtype else None, 1e-2, out)
                assert np.abs(f64(x) - want).max() < 2e-5 * np.abs(want).max(), (kind, branch, dtype)
                if dtype:
                    nxt = plain.rms_norm(want, f32_round(ng), 1e-2)
                    assert np.abs(f64(out) - nxt).max() < (3e-5 if dtype == "float32" else 2.0 ** -7) * np.abs(nxt).max(), (kind, branch, dtype)
    y = dev(x0)
    ops.add_gated_rows(y, dev(plus), dev(gate))
    want = f32_round(x0) + f32_round(gate)[:, None] * f32_round(plus)
    assert np.abs(f64(y) - want).max() < 1e-5


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("N,K", [(33, 50), (96, 128), (3072, 1024), (4160, 2048), (520, 2304)])
def test_square_of_relu_in_the_products_epilogue(ops, dtype, N, K):
    """Every kernel that the row counts pick: a row per wavefront, workgroups of 16 rows, tiles, pieces of a long K."""
    rng = np.random.default_rng(N)
    w = rng.normal(size=(N, K)) / math.sqrt(K)
    for M in (1, 3, 8, 16, 40, 64, 130, 700):
        if dtype == "float32" and M * N * K > 2e8:
            continue
        a = rng.normal(size=(M, K)) * 2
        r = bf16_round if dtype == "bfloat16" else f32_round
        want = plain.relu_squared(r(a) @ r(w).T)
        out = torch.full((M, N), float("nan"), device="cuda", dtype=DT[dtype])
        ops.linear(dev(a, DT[dtype]), dev(w, DT[dtype]), out, "relu2")
        err = np.abs(f64(out) - want)
        assert (err <= (2e-5 if dtype == "float32" else 2.0 ** -8) * want + 1e-4 * (0.02 if dtype == "float32" else 1.0) * want.max()).all(), (M, err.max())
        assert (f64(out) == 0).mean() > 0.3


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("W", [5, 64, 100, 320])
def test_minimal_gru(ops, dtype, W):
    """The recurrence over a request's tokens whole, in portions down to single tokens, in chunks of one and of several blocks,
    and beside another request; the state in its slot carries from step to step; a slot that is zeroed serves the next
    request; gates at both ends (a channel that forgets everything, one that keeps everything)."""
    rng = np.random.default_rng(W)
    T = 290
    proj = rng.normal(size=(T, 3 * W + 7)) * 2
    oz, ox, og = 3, 3 + W, 7 + 2 * W
    bz, bx = rng.normal(-2.0, 1.0, size=W), rng.normal(0.0, 0.5, size=W)
    bz[0], bz[1] = 90.0, -90.0
    p32, bz32, bx32 = f32_round(proj), f32_round(bz), f32_round(bx)
    z = plain.sigmoid(p32[:, oz:oz + W] + bz32)
    u = p32[:, ox:ox + W] + bx32
    c = np.where(u >= 0, u + 0.5, plain.sigmoid(u))
    S, states = np.zeros(W), np.zeros((T, W))
    for t in range(T):
        S = (1.0 - z[t]) * S + z[t] * c[t]
        states[t] = S
    want = states * plain.silu(p32[:, og:og + W])
    state = torch.zeros(3, W, device="cuda")
    state[1].fill_(float("nan"))                              # another request's slot: never touched
    pj, zb, xb = dev(proj), dev(bz), dev(bx)
    cols = (oz, ox, og)
    tol = (3e-5 if dtype == "float32" else 2.0 ** -7) * np.abs(want).max()

    def run(cuts, slot, chunk=0):
        o = torch.full((T, W), float("nan"), device="cuda", dtype=DT[dtype])
        at = 0
        for n in cuts:
            lists = (None, None)
            if chunk:
                sizes = [min(chunk, n - k) for k in range(0, n, chunk)]
                lists = (dev([[0, at + sum(sizes[:k]), s, (1 if k == 0 else 0) | (2 if k == len(sizes) - 1 else 0)] for k, s in enumerate(sizes)],
                             torch.int32), dev([[0, len(sizes)]], torch.int32))
            ops.mingru_scan(pj, zb, xb, state, dev([[at, n, at, slot]], torch.int32), o, W, cols, *lists)
            at += n
        assert at == T
        return f64(o)

    whole = run([T], 0)
    assert np.abs(whole - want).max() < tol
    assert np.abs(f64(state[0]) - S).max() < 3e-5 * max(1.0, np.abs(S).max())
    cut = run([17, 1, 1, 2, 33, 16, 1, 64, T - 135], 2)
    assert np.array_equal(cut, whole) and np.array_equal(f64(state[2]), f64(state[0]))
    for chunk in (64, 128, 5):
        for cuts in ([T], [65, 1, 2, 100, T - 168]):
            state[0].zero_()                                  # the slot goes to the next request
            got = run(cuts, 0, chunk)
            assert np.abs(got - want).max() < tol, (chunk, cuts)
            assert np.abs(f64(state[0]) - S).max() < 3e-5 * max(1.0, np.abs(S).max()), (chunk, cuts)
    # three requests in one step in chunks: one of several chunks, one of a single token, one of a single chunk, each from its state
    start = rng.normal(size=(3, W))
    state = dev(start)
    meta = [[0, 150, 0, 2], [150, 1, 9, 0], [151, 40, 3, 1]]
    chunks = [[0, 0, 64, 1], [0, 64, 64, 0], [0, 128, 22, 2], [1, 150, 1, 3], [2, 151, 40, 3]]
    o = torch.full((T, W), float("nan"), device="cuda", dtype=DT[dtype])
    ops.mingru_scan(pj, zb, xb, state, dev(meta, torch.int32), o, W, cols, dev(chunks, torch.int32), dev([[0, 3], [3, 1], [4, 1]], torch.int32))
    got = f64(o)
    assert np.isnan(got[191:]).all()
    for row0, n, _, slot in meta:
        S = f32_round(start[slot])
        for t in range(row0, row0 + n):
            S = (1.0 - z[t]) * S + z[t] * c[t]
            ref = S * plain.silu(p32[t, og:og + W])
            assert np.abs(got[t] - ref).max() < 3 * tol, (slot, t)
        assert np.abs(f64(state[slot]) - S).max() < 3e-5 * max(1.0, np.abs(S).max()), slot


def rotation_inputs(rot, n_table):
    if not rot or not rot["dims"]:
        return None, None
    f = plain.frequencies(rot)
    ang = np.arange(n_table)[:, None] * f[None, :]
    return dev(f), dev(np.stack([np.cos(ang), np.sin(ang)], axis=-1))


@pytest.mark.parametrize("dims,base,scaling", [(16, 500.0, lm.wavelengths(4.0, 1.0, 8.0, 100)), (8, 30.0, None), (64, 500000.0, lm.wavelengths(2.0, 2.0, 2.0, 3000)),
                                               (2, 7.0, lm.wavelengths(9.0, 0.5, 3.0, 10))])
def test_the_parts_table_holds_the_stretched_frequencies(dims, base, scaling):
    from tinyinfer_amd.parts import build_part
    from tinyinfer_amd.spec import PartSpec
    rot = dict(base=base, dims=dims)
    params = dict(dims=dims, base=base, layout="pairs")
    if scaling:
        rot["scaling"] = scaling
        params["scaling"] = dict(scaling, kind="wavelength")
    part = build_part("pos", PartSpec("rope_partial", params), "")
    part.prepare(None, 700)
    f = plain.frequencies(rot)
    assert np.abs(f64(part.held("inv_freq")) / f - 1).max() < 1e-6
    ang = np.arange(700)[:, None] * f[None, :]
    assert np.abs(f64(part.held("table")) - np.stack([np.cos(ang), np.sin(ang)], -1)).max() < 1e-6


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("heads,kv,dk,dv,P,rot_dims,scaled", [
    (4, 2, 16, 24, 16, 8, True), (3, 3, 7, 5, 4, 6, True), (5, 1, 40, 33, 64, 40, False), (2, 2, 64, 64, 16, 64, True), (2, 1, 64, 32, 16, 0, False),
    (8, 2, 128, 128, 32, 64, True), (1, 1, 256, 256, 16, 2, False), (7, 7, 32, 32, 8, 32, True), (3, 1, 130, 100, 16, 130, False),
    (20, 10, 24, 16, 16, 16, True), (18, 9, 72, 40, 32, 70, False)])
def test_attention_with_paired_rotation_unit_norms_and_one_more_in_the_denominator(ops, dtype, heads, kv, dk, dv, P, rot_dims, scaled):
    """The projections of a whole request are rotated, divided by their root mean square and written into the pages in three
    portions (the last a single token); then the attention of every row with a gate a head.  The last row's query points at
    key 1, far back among hundreds, once the rotation has turned both; the first rows see one, two, three keys, where the one
    more weighs most."""
    rng = np.random.default_rng(dk * 1000 + dv + heads)
    T, eps = 333, 1e-2                                        # an eps that shows beside small heads
    scale = 2.0 / dk                                          # a head against itself scores 2: the one more weighs a tenth
    per = heads // kv
    nq, nk, nv = heads * dk, kv * dk, kv * dv
    proj = rng.normal(size=(T, nq + nk + nv + heads)) * 0.3
    rot = dict(base=300.0, dims=rot_dims)
    if scaled:
        rot["scaling"] = lm.wavelengths(3.0, 1.0, 6.0, 90)
    pos = np.arange(T, dtype=np.int32)
    # key 1 as the last row's query sees it: turned to position 1 and back from position T - 1
    k1 = plain.rotate_pairs(proj[None, 1, nq:nq + nk].reshape(1, kv, dk), [1], rot)
    back = plain.rotate_pairs(k1, [-(T - 1)], rot)
    for h in range(heads):
        proj[T - 1, h * dk:(h + 1) * dk] = back[0, h // per]
    p32 = f32_round(proj)
    q = plain.unit_rms(plain.rotate_pairs(p32[:, :nq].reshape(T, heads, dk), pos, rot), eps)
    k = plain.unit_rms(plain.rotate_pairs(p32[:, nq:nq + nk].reshape(T, kv, dk), pos, rot), eps)
    v = p32[:, nq + nk:nq + nk + nv].reshape(T, kv, dv)
    inv, tab = rotation_inputs(rot, 100)                      # beyond the table the angle is taken in 32-bit on the device
    table, n_pages = paged(rng, T, P)
    pool = torch.full((n_pages, kv, P, dk + dv), float("nan"), device="cuda", dtype=DT[dtype])
    q_out = torch.empty(T, nq, device="cuda", dtype=DT[dtype])
    slots = np.zeros(T, dtype=np.int32)
    for lo, hi in ((0, 37), (37, T - 1), (T - 1, T)):
        ops.gated_qkv_prep(dev(proj[lo:hi]), None, None, inv, tab, dev(pos[lo:hi], torch.int32), dev(slots[lo:hi], torch.int32),
                           dev(table, torch.int32), pool, q_out[lo:hi], heads, kv, dk, dv, (0, nq, nq + nk), eps=eps, rot_dims=rot_dims,
                           pairs=True, unit_norm=True)
    tol = 2e-4 if dtype == "float32" else 2.0 ** -7
    assert np.abs(f64(q_out).reshape(T, heads, dk) - q).max() < tol * np.abs(q).max()
    flat = f64(pool).reshape(n_pages, -1)
    for t in (0, 1, P - 1, P, 36, 37, T - 2, T - 1):
        pg = flat[table[0, t // P]]
        assert np.abs(pg[:kv * P * dk].reshape(kv, P, dk)[:, t % P] - k[t]).max() < tol * np.abs(k).max(), t
        assert np.abs(pg[kv * P * dk:].reshape(kv, dv, P)[:, :, t % P] - v[t]).max() < tol * np.abs(v).max(), t
    if dtype == "bfloat16":
        q, k, v = bf16_round(q), bf16_round(k), bf16_round(v)
    gates = plain.sigmoid(p32[:, nq + nk + nv:])
    want = np.zeros((T, heads, dv))
    for h in range(heads):
        p = plain.softmax_over(q[:, h] @ k[:, h // per].T * scale, plain.visible(T, None), True)
        assert dk < 16 or p[T - 1, 1] > 4.0 / T               # the far key stands out
        want[:, h] = p @ v[:, h // per] * gates[:, h:h + 1]
    zeros = torch.zeros(heads, device="cuda")
    out = torch.empty(T, heads * dv, device="cuda", dtype=DT[dtype])
    args = (q_out, pool, dev(table, torch.int32), dev(pos, torch.int32), dev(slots, torch.int32))
    ops.gated_attention(*args, zeros, dev(proj), out, heads, kv, dk, dv, scale, gate_col=nq + nk + nv, gate_mode=2)
    bound = 5e-5 if dtype == "float32" else 2e-2
    err = np.abs(f64(out).reshape(T, heads, dv) - want)
    assert err.max() < bound * np.abs(want).max(), (np.unravel_index(err.argmax(), err.shape), err.max())
    ops.gated_attention(*args, None, dev(proj), out, heads, kv, dk, dv, scale, gate_col=nq + nk + nv, gate_mode=2)
    assert np.abs(f64(out).reshape(T, heads, dv)[:3] - want[:3]).max() > 4 * bound * np.abs(want[:3]).max()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("H,d,dv,qr,R,P,window", [(3, 5, 7, 11, 13, 4, 9), (2, 16, 16, 24, 32, 16, 0), (20, 16, 32, 48, 64, 16, 33), (4, 32, 48, 300, 128, 16, 31),
                                                  (17, 8, 16, 16, 256, 32, 1), (2, 64, 64, 96, 512, 16, 40)])
def test_latent_attention_with_a_query_latent(ops, dtype, H, d, dv, qr, R, P, window):
    """Both latents normed by one kernel, in portions over page borders; the queries from theirs; then the attention under the
    window: row by row, and where the matrix cores serve the sizes as tiles of a portion, as single tokens, mixed, and with a
    context split over workgroups.  For the last row the oldest key the window keeps is made to stand out (no window: the
    third token) and the key just behind the window has the same latent."""
    rng = np.random.default_rng(H * 100 + R)
    T, eps = 150, 1e-4
    scale = 1.2 / math.sqrt(d)
    proj = rng.normal(size=(T, qr + R + 3)) * 0.5
    off = qr + 3
    target = T - window if window else 2
    if window:
        proj[target - 1, off:] = proj[target, off:]
    qn, kn = rng.normal(1.0, 0.2, size=qr), rng.normal(1.0, 0.2, size=R)
    uk, uv = bf16_round(rng.normal(size=(H * d, R)) / math.sqrt(R) * 1.5), bf16_round(rng.normal(size=(H * dv, R)) / math.sqrt(R))
    p32 = f32_round(proj)
    cq = plain.rms_norm(p32[:, :qr], f32_round(qn), eps)
    c = plain.rms_norm(p32[:, off:], f32_round(kn), eps)
    twice = dtype == "bfloat16" and d % 8 == 0 and R % 16 == 0 and dv % 16 == 0
    table, n_pages = paged(rng, T, P)
    pool = torch.full((n_pages, P, 2 * R if twice else R), float("nan"), device="cuda", dtype=DT[dtype])      # rows never written hold anything
    pos, slots = np.arange(T, dtype=np.int32), np.zeros(T, dtype=np.int32)
    out_q = torch.empty(T, qr, device="cuda", dtype=DT[dtype])
    for lo, hi in ((0, 37), (37, T - 1), (T - 1, T)):
        ops.latent_prep_queries(dev(proj[lo:hi]), dev(kn), dev(qn), dev(pos[lo:hi], torch.int32), dev(slots[lo:hi], torch.int32),
                                dev(table, torch.int32), pool, out_q[lo:hi], off, eps, 0, qr, R)
    tol = 3e-5 if dtype == "float32" else 2.0 ** -7
    assert np.abs(f64(out_q) - cq).max() < tol * np.abs(cq).max()
    flat = f64(pool).reshape(n_pages, -1)
    for t in (0, 1, P - 1, P, 36, 37, T - 1):
        pg = flat[table[0, t // P]]
        assert np.abs(pg[:P * R].reshape(P, R)[t % P] - c[t]).max() < tol * np.abs(c).max(), t
        if twice:
            assert np.array_equal(pg[:P * R].reshape(P, R)[t % P], pg[P * R:].reshape(R, P)[:, t % P]), t
    if dtype == "bfloat16":
        c = bf16_round(c)
    q = rng.normal(size=(T, H, d)) * 0.6                      # the queries as the product behind cq leaves them, 32-bit
    for h in range(H):
        keys = c @ uk[h * d:(h + 1) * d].T
        dq = keys[target] - keys[max(0, target - 30):].mean(axis=0)
        if window != 1:
            q[T - 1, h] = dq * (14.0 / (dq @ keys[target] * scale))
    q32 = f32_round(q)
    vis = plain.visible(T, window or None)
    want = np.zeros((T, H, dv))
    for h in range(H):
        p = plain.softmax_over(q32[:, h] @ (c @ uk[h * d:(h + 1) * d].T).T * scale, vis, False)
        assert (d < 16 or p[T - 1, target] > 0.2) and (not window or p[T - 1, target - 1] == 0.0)
        want[:, h] = p @ (c @ uv[h * dv:(h + 1) * dv].T)
    qd, ukd, uvd = dev(q.reshape(T, H * d)), dev(uk, DT[dtype]), dev(uv, DT[dtype])
    args = (qd, ukd, uvd, None, pool, dev(table, torch.int32), dev(pos, torch.int32), dev(slots, torch.int32))
    sizes = (H, d, 0, R, dv, scale, window)
    bound = (1e-4 if dtype == "float32" else 4e-2) * max(1.0, np.abs(want).max())
    out = torch.zeros(T, H * dv, device="cuda", dtype=DT[dtype])
    ops.latent_attention(*args, out, *sizes)
    err = np.abs(f64(out).reshape(T, H, dv) - want)
    assert err.max() < bound, ("rows", np.unravel_index(err.argmax(), err.shape), err.max())
    if not twice:
        return
    uk_t = torch.empty(H * R, d, device="cuda", dtype=torch.bfloat16)
    ops.latent_transpose(ukd, uk_t, H)
    entries = dev([[0, T, 0, 0]], torch.int32)
    tiles = dev([[0, r0, min(64, T - r0)] for r0 in range(0, T, 64)], torch.int32)
    ops.count_calls(True)
    for splits, lists in ((0, dict(tiles=tiles, entries=entries)), (0, dict(all_rows=True)), (0, dict(all_rows=True, context=T)),
                          (3, dict(all_rows=True, context=T)), (0, dict(tiles=tiles[:1], entries=entries, rows=dev(list(range(64, T)), torch.int32)))):
        ops.force_decode_splits = splits
        fast = torch.zeros(T, H * dv, device="cuda", dtype=torch.bfloat16)
        ops.latent_attention(*args, fast, *sizes, w_uk_t=uk_t, **lists)
        err = np.abs(f64(fast).reshape(T, H, dv) - want)
        assert err.max() < bound, (splits, list(lists), np.unravel_index(err.argmax(), err.shape), err.max())
    ops.force_decode_splits = 0
    took = [c["name"] for c in ops.timing_report() if c["name"].startswith("latent_attention")]
    ops.count_calls(False)
    assert took and all("[mfma]" in n for n in took), took


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("E,top,W,F", [(6, 2, 64, 32), (5, 5, 40, 24), (12, 4, 96, 64), (1, 1, 50, 9), (70, 3, 128, 32)])
def test_router_and_experts_weighted_on_their_outputs(ops, dtype, E, top, W, F):
    """Softmax scores as they are, the gate's row beside the router's, squared-relu experts times their weights, few tokens (row by
    row) and many (grouped on the matrix cores where they serve the sizes)."""
    rng = np.random.default_rng(E * 10 + top)
    router, sg = rng.normal(size=(E, W)) * 2.0 / math.sqrt(W), rng.normal(size=W) / math.sqrt(W)
    r = bf16_round if dtype == "bfloat16" else f32_round
    w = {"m.router": f32_round(router)}
    for e in range(E):
        w[f"m.e{e}.up"], w[f"m.e{e}.down"] = r(rng.normal(size=(F, W)) * 1.5 / math.sqrt(W)), r(rng.normal(size=(W, F)) / math.sqrt(F))
    up = dev(np.concatenate([w[f"m.e{e}.up"] for e in range(E)]), DT[dtype])
    down = dev(np.concatenate([w[f"m.e{e}.down"] for e in range(E)]), DT[dtype])
    for M in (3, 200):
        h = r(rng.normal(size=(M, W)))
        ids_want, wts_want = plain.route(h, dict(experts=E, top=top), w, "m")
        s = h @ w["m.router"].T
        best = -np.sort(-s, axis=1)[:, :top + 1]
        sure = (best[:, :-1] - best[:, 1:]).min(axis=1) > 1e-5 if E > top else np.diff(best, axis=1).max(axis=1, initial=-1.0) < -1e-5
        ids = torch.empty(M, top, device="cuda", dtype=torch.int32)
        wts, gate = torch.empty(M, top, device="cuda"), torch.full((M,), float("nan"), device="cuda")
        hd = dev(h, DT[dtype])
        ops.moe_route_grouped(hd, dev(router), ids, wts, None, top, renormalize=False, score="softmax", gate_row=dev(sg), gate_out=gate)
        assert sure.mean() > 0.8 and np.array_equal(ids.cpu().numpy()[sure], ids_want[sure])
        assert np.abs(f64(wts)[sure] - wts_want[sure]).max() < 1e-5
        assert np.abs(f64(gate) - plain.sigmoid(h @ f32_round(sg))).max() < 1e-5
        y = torch.full((M, W), float("nan"), device="cuda")
        ops.moe_experts(hd, ids, wts, up, down, y, E, scale_input=False)
        want = np.zeros((M, W))
        for t in range(M):
            for e, a in zip(ids.cpu().numpy()[t], f64(wts)[t]):
                want[t] += a * plain.two_layer(h[t], w, f"m.e{e}")
        assert np.abs(f64(y) - want).max() < (5e-5 if dtype == "float32" else 1e-2) * np.abs(want).max(), M


def test_equal_scores_go_to_the_lower_index(ops):
    h = torch.zeros(3, 16, device="cuda")
    ids, wts = torch.empty(3, 3, device="cuda", dtype=torch.int32), torch.empty(3, 3, device="cuda")
    ops.moe_route_grouped(h, torch.ones(8, 16, device="cuda"), ids, wts, None, 3, renormalize=False, score="softmax")
    assert ids.cpu().tolist() == [[0, 1, 2]] * 3 and np.abs(f64(wts) - 0.125).max() < 1e-6


def test_a_row_that_is_not_a_number_still_names_experts_that_exist(ops):
    h = torch.full((2, 16), float("nan"), device="cuda")
    ids, wts = torch.empty(2, 3, device="cuda", dtype=torch.int32), torch.empty(2, 3, device="cuda")
    ops.moe_route_grouped(h, torch.ones(8, 16, device="cuda"), ids, wts, None, 3, renormalize=False, score="softmax")
    assert all(0 <= i < 8 for row in ids.cpu().tolist() for i in row)


# ---------------------------------------------------------------------------------- the engine
REQUEST_LENGTHS = {"a": 97, "b": 45, "c": 130, "d": 33, "e": 71, "f": 58}
PROMPT_LENGTHS = {"a": 60, "b": 12, "c": 101, "d": 30, "e": 2, "f": 41}
_made = {}


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    def get(name):
        if name not in _made:
            config = lm.CONFIGS[name]
            weights = lm.draw_weights(config, seed=len(name) * 13 + 2)
            path = lm.write_folder(str(tmp_path_factory.mktemp("lupolorn_" + name)), config, 0, weights)
            requests = {r: random_tokens(n, config["vocab"], 17 + i) for i, (r, n) in enumerate(REQUEST_LENGTHS.items())}
            w = lm.as_float64(weights)
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
@pytest.mark.parametrize("name,page_size", [("mixed", 8), ("plain", 4), ("wide", 16), ("states", 16), ("windows", 16)])
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
    """A prompt of 50 tokens in portions of 32, then 250 tokens one by one: the states of the recurrences are carried through
    every step, every window passes over decoded tokens, and the keys of the first tokens stay visible to the last."""
    from tinyinfer_amd.engine import StepEntry
    folder, _, _, w = folders("mixed")
    config = lm.CONFIGS["mixed"]
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
    config = lm.CONFIGS["mixed"]
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
    config = lm.CONFIGS["mixed"]
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
    config = lm.CONFIGS["wide"]
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
    mine = [n for n in names if n.startswith(("gated_attention", "latent_attention"))]
    assert mine and all(n.endswith("[generic]") for n in mine)
    ok, seen = within({"x": slow}, {"x": want}, "bfloat16")
    assert ok, seen
    for splits, paired in ((0, None), (4, True), (1, False)):
        fast, names = run(True, splits, paired)
        mine = [n for n in names if n.startswith(("gated_attention", "latent_attention"))]
        assert mine and all(n.endswith("[mfma]") for n in mine), mine
        assert any(n.startswith("mingru_scan") and n.endswith("[chunked]") for n in names)
        assert any(n.startswith("moe_experts") and "grouped" in n for n in names)
        assert any(n.startswith("norm_residual_next") and "plus +norm" in n for n in names)
        ok, seen = within({"x": fast}, {"x": want}, "bfloat16")
        assert ok, (splits, paired, seen)
        # a router's choice within rounding of a tie may fall the other way at a position or two
        e = errors(fast, slow)
        assert np.median(e) < 2e-2 and (e > 0.08).mean() <= 0.05, (splits, paired, float(np.median(e)), float(e.max()))


def test_long_portions_beside_single_tokens(folders):
    """Steps in which a portion goes through the chunked recurrence while other requests decode one token each: their states sit in
    the same step's chunks."""
    folder, _, _, w = folders("mixed")
    config = lm.CONFIGS["mixed"]
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


def test_command_line_generates_from_a_lupolorn_folder(folders):
    """bin/tinyinfer picks the model by config.json: token ids in, the plain model's greedy tokens out; with --cuda-graph too."""
    import os
    import subprocess
    import sys
    folder, requests, _, w = folders("plain")
    config = lm.CONFIGS["plain"]
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
        engine = Engine.from_config(lm.CONFIGS[name], seed=3, dtype="bfloat16", page_size=16, max_tokens=256, max_requests=2, max_seq=256)
        toks = random_tokens(70, lm.CONFIGS[name]["vocab"], 1)
        a = engine.step([StepEntry("x", toks, [69])]).cpu().numpy()
        engine.release("x")
        assert engine.step([StepEntry("y", toks[:69], [])]) is None
        b = engine.step([StepEntry("y", toks[69:], [0])]).cpu().numpy()
        assert np.isfinite(a).all() and a.std() > 0
        assert np.abs(a - b).max() < 0.08 * max(1e-6, np.abs(a).max())


def test_trace_replay_program(folders, tmp_path):
    """The replay program on a Lupolorn folder: it picks the model by config.json and writes the logits the engine gives."""
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
    V = lm.CONFIGS["plain"]["vocab"]
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
