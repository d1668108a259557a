"""The Famidra design on the GPU against the plain implementation (plain_famidra.py): every mechanism alone, then whole models through the
stage, the compute kernel and the trace runner -- whole prompts, portions, token by token, batches, slots that are used again."""
import json
import os
import subprocess

import numpy as np
import pytest

import famidra_models as M
import plain_famidra as P

pytestmark = pytest.mark.gpu

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
DTYPES = ("f32", "bf16")
# root mean square of the difference over that of the expected values, worst row
MODEL_TOL = {"f32": 5e-5, "bf16": 8e-2}


def torch_dtype(dtype):
    import torch
    return torch.float32 if dtype == "f32" else torch.bfloat16


def dev(a, dtype):
    import torch
    return torch.from_numpy(np.ascontiguousarray(a, dtype=np.float32)).cuda().to(torch_dtype(dtype)).contiguous()


def back(t):
    return t.float().cpu().numpy().astype(np.float64)


def row_error(got, want):
    got, want = np.asarray(got, np.float64), np.asarray(want, np.float64)
    return np.sqrt(((got - want) ** 2).mean(-1)) / np.sqrt((want ** 2).mean())


def assert_rows(got, want, tol, what="", stretch=1.0):
    """`stretch`: one row in fifty may be off by that many times more (a head whose output almost cancels is blown up by its norm,
    rounding included)."""
    e = row_error(got, want)
    ok = bool(np.isfinite(got).all()) and e.max() <= tol * stretch and (e > tol).sum() <= max(1, e.size // 50)
    assert ok if stretch > 1 else bool(np.isfinite(got).all()) and e.max() <= tol, f"{what}: worst row {int(e.argmax())} of {e.size} off by {e.max():.2e} (tol {tol})"


def logit_error(got, want):
    d = np.asarray(got, np.float64) - want
    d -= d.mean(-1, keepdims=True)
    w = want - want.mean(-1, keepdims=True)
    return np.sqrt((d ** 2).mean(-1)) / np.sqrt((w ** 2).mean())


def assert_logits(got, want, dtype, what=""):
    """fp32 storage holds every position; in bf16 a few may stray further, where a norm blows up the rounding of a small vector."""
    e, tol = logit_error(got, want), MODEL_TOL[dtype]
    ok = e.max() <= tol if dtype == "f32" else e.max() <= 5 * tol and (e > tol).sum() <= max(1, e.size // 25)
    assert ok, f"{what}: row {int(e.argmax())} of {e.size} off by {e.max():.2e} (tol {tol})"


# ---- mechanisms alone ----------------------------------------------------------------------------
@pytest.mark.parametrize("b,s,r", [(1, 64, 40), (3, 52, 17), (7, 256, 512), (70, 136, 200), (200, 256, 384), (300, 512, 2048), (200, 512, 8), (333, 1024, 24), (1030, 2048, 32), (2048, 1024, 8192)])
def test_bf16_products(b, s, r):
    import torch
    from glinthawk_amd import ops
    g = torch.Generator().manual_seed(b * s + r)
    x = torch.randn((b, s), generator=g).cuda().bfloat16()
    w = (torch.randn((r, s), generator=g) / s ** 0.5).cuda().bfloat16()
    want = x.float() @ w.float().T
    got = ops.matmul(x, w).float()
    assert (got - want).abs().max() <= 2 ** -8 * want.abs().max() + 1e-6
    assert (ops.matmul_scaled(x, w, 0.5) - 0.5 * want).abs().max() <= 1e-5 * want.abs().max()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,s,width", [(1, 24, 52), (5, 128, 128), (33, 40, 1000), (200, 64, 256), (260, 64, 50)])
def test_stream_step(dtype, rows, s, width):
    """Every part of the residual update: bias, norm behind the projection, sum or replacement, added vector, norm in front of the next product."""
    import torch
    from glinthawk_amd import ops
    rng = np.random.default_rng(rows * width)
    rnd = lambda *shape: M.to_bf16(rng.standard_normal(shape))
    inp, w, bias, post, add, nxt = rnd(rows, s), rnd(width, s), rnd(width), 1 + 0.3 * rnd(width), rnd(width), 1 + 0.3 * rnd(width)
    post, nxt = M.to_bf16(post), M.to_bf16(nxt)
    x0 = rng.standard_normal((rows, width)).astype(np.float32)
    y = inp.astype(np.float64) @ w.T
    eps = 2e-3
    for parts in (dict(bias=bias, post_norm=post, accumulate=True, next_norm=nxt), dict(accumulate=False, add=add, next_norm=nxt), dict(post_norm=post, accumulate=True),
                  dict(bias=bias, accumulate=True, next_norm=None)):
        v = y + (parts["bias"] if "bias" in parts else 0)
        if "post_norm" in parts:
            v = P.rms_norm(v, eps, post.astype(np.float64))
        want = (x0 if parts["accumulate"] else 0) + v + (parts["add"] if "add" in parts else 0)
        out = torch.zeros((rows, 2 * width), dtype=torch_dtype(dtype), device="cuda")      # a row stride of its own
        x = torch.from_numpy(x0).cuda()
        dparts = {k: (dev(a, dtype) if isinstance(a, np.ndarray) else a) for k, a in parts.items()}
        ops.matmul_stream(x, dev(inp, dtype), dev(w, dtype), eps, out=out[:, width:], **dparts)
        want_out = P.rms_norm(want, eps, nxt.astype(np.float64)) if parts.get("next_norm") is not None else want
        tol = 1e-5 if dtype == "f32" else 1e-2
        assert_rows(back(x), want, tol, f"stream {sorted(parts)}")
        assert_rows(back(out[:, width:]), want_out, tol, f"out {sorted(parts)}")
        assert float(out[:, :width].abs().max()) == 0.0
    one = torch.zeros((rows, width), dtype=torch_dtype(dtype), device="cuda")
    ops.stream_out(torch.from_numpy(x0).cuda(), one, dev(nxt, dtype), eps)
    assert_rows(back(one), P.rms_norm(x0.astype(np.float64), eps, nxt.astype(np.float64)), 1e-5 if dtype == "f32" else 5e-3, "norm alone")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,s,hidden", [(1, 32, 20), (9, 64, 30), (64, 256, 128), (210, 64, 72)])
def test_gate(dtype, rows, s, hidden):
    from glinthawk_amd import ops
    rng = np.random.default_rng(hidden)
    x, w, b = (M.to_bf16(rng.standard_normal(n)) for n in ((rows, s), (2 * hidden, s), (2 * hidden,)))
    w = M.to_bf16(w / np.sqrt(s))
    y = x.astype(np.float64) @ w.T + b
    want = P.gelu_tanh(y[:, :hidden]) * y[:, hidden:]
    assert_rows(back(ops.matmul_gate(dev(x, dtype), dev(w, dtype), dev(b, dtype))), want, 1e-5 if dtype == "f32" else 1e-2)


def test_embedding():
    import torch
    from glinthawk_amd import ops
    rng = np.random.default_rng(1)
    e, p = rng.standard_normal((31, 20)).astype(np.float32), rng.standard_normal((40, 20)).astype(np.float32)
    tok = rng.integers(0, 31, (2, 5)).astype(np.int32)
    copy = torch.zeros((10, 40), device="cuda")
    x = ops.embed_positions(torch.from_numpy(tok.reshape(-1)).cuda(), torch.tensor([0, 33], dtype=torch.int32, device="cuda"), 5, dev(e, "f32"), dev(p, "f32"), copy[:, 20:])
    want = e[tok] + np.stack([p[0:5], p[33:38]])
    assert np.array_equal(x.cpu().numpy().reshape(2, 5, 20), want) and np.array_equal(copy[:, 20:].cpu().numpy(), x.cpu().numpy())


ATTENTIONS = {
    # heads, kv heads, dim, vdim, window, kept, table rows, bias_max
    "grouped": (6, 2, 24, 16, 11, 3, 10, 40),
    "matrix": (8, 2, 64, 64, 40, 5, 16, 64),
    "ten": (10, 1, 72, 40, 30, 20, 8, 33),
    "own": (3, 3, 128, 96, 70, 0, 32, 100),
    "deep": (2, 1, 200, 136, 17, 1, 6, 25),
    "deeper": (1, 1, 300, 280, 20, 2, 4, 9),
    "open": (4, 2, 32, 32, 0, 0, 12, 50),        # no window
}


class Cache:
    """One attention layer's cache rows of a few contexts, filled by hand (heads padded to 8 elements with zeros)."""

    def __init__(self, shape, k, v, dtype, offset=256):
        import torch
        from glinthawk_amd import ops
        heads, kv, d, dv, window, keep, rows, bias_max = shape
        self.attn = ops.window_attn(heads, kv, d, dv, d ** -0.5, window, keep, int(bias_max) + 1)
        dp, vp = -(-d // 8) * 8, -(-dv // 8) * 8
        self.offset = offset
        self.regions = []
        for kk, vv in zip(k, v):
            T = kk.shape[0]
            full = np.zeros((T, kv * (dp + vp)), np.float32)
            full[:, : kv * dp].reshape(T, kv, dp)[:, :, :d] = kk
            full[:, kv * dp:].reshape(T, kv, vp)[:, :, :dv] = vv
            t = dev(full, dtype)
            assert t.shape[1] * t.element_size() == ops.window_row_bytes(self.attn, t.dtype)
            pad = torch.full((offset // t.element_size(),), float("nan"), dtype=t.dtype, device="cuda")
            self.regions.append(torch.cat([pad, t.reshape(-1)]).contiguous())
        self.rows = ops.row_table([r.data_ptr() for r in self.regions])
        self.dp = dp


def attend(shape, q, k, v, rel, start, n, dtype):
    """Rows [start_i, start_i + n) of every sequence as one call."""
    import torch
    from glinthawk_amd import ops
    heads, kv, d, dv, window, keep, rows, bias_max = shape
    cache = Cache(shape, k, v, dtype)
    qp = np.zeros((len(q), n, heads, cache.dp), np.float32)
    for i, (qq, s) in enumerate(zip(q, start)):
        qp[i, :, :, :d] = qq[s:s + n]
    bias = np.array([[rel[P.distance_bucket(t, rows, bias_max), h] for t in range(int(bias_max) + 1)] for h in range(heads)], np.float32)
    out = ops.attn_window(dev(qp.reshape(len(q) * n, -1), dtype), cache.attn, cache.rows, torch.tensor(start, dtype=torch.int32, device="cuda"), n, max(start),
                          torch.from_numpy(bias).cuda(), cache.offset)
    return back(out).reshape(len(q), n, heads, dv)


def attention_case(name, T, seed, n_seq=1, sharp=False):
    shape = ATTENTIONS[name]
    heads, kv, d, dv, window, keep, rows, bias_max = shape
    rng = np.random.default_rng(seed)
    q = [M.to_bf16(rng.standard_normal((T, heads, d))) for _ in range(n_seq)]
    k = [M.to_bf16(rng.standard_normal((T, kv, d))) for _ in range(n_seq)]
    v = [M.to_bf16(rng.standard_normal((T, kv, dv))) for _ in range(n_seq)]
    rel = rng.standard_normal((rows, heads)).astype(np.float32)
    want = [P.windowed_attention(*(a.astype(np.float64) for a in (qq, kk, vv)), d ** -0.5, rel.astype(np.float64), bias_max, window or T + 1, keep)
            for qq, kk, vv in zip(q, k, v)]
    return shape, q, k, v, rel, want


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(ATTENTIONS))
def test_windowed_attention(name, dtype):
    """A whole prompt, portions from anywhere, single tokens at and around the window's edges, two sequences in a call."""
    T = 150
    shape, q, k, v, rel, want = attention_case(name, T, 3, n_seq=2)
    tol = 1e-5 if dtype == "f32" else 8e-3
    assert_rows(np.stack(attend(shape, q, k, v, rel, [0, 0], T, dtype)).reshape(2 * T, -1), np.stack(want).reshape(2 * T, -1), tol, "whole")
    window, keep = shape[4], shape[5]
    for start, n in (([0, 70], 2), ([13, 90], 33), ([64, 1], 64), ([100, 37], 17), ([16, 48], 80)):
        w = np.stack([a[s:s + n] for a, s in zip(want, start)])
        assert_rows(attend(shape, q, k, v, rel, start, n, dtype).reshape(2 * n, -1), w.reshape(2 * n, -1), tol, f"portion {start}+{n}")
    for p in sorted({0, 1, max(0, keep - 1), keep, window - 1, window, window + 1, window + keep, T - 1} & set(range(T))):
        w = np.stack([a[p] for a in want])
        assert_rows(attend(shape, q, k, v, rel, [p, p], 1, dtype)[:, 0].reshape(2, -1), w.reshape(2, -1), tol, f"token {p}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["grouped", "matrix", "ten", "own"])
def test_one_key_stands_out(name, dtype):
    """Every key in turn made the one that its query's score picks: seen exactly where the window or the kept tokens show it, and just
    not seen one position further."""
    shape = ATTENTIONS[name]
    heads, kv, d, dv, window, keep, rows, bias_max = shape
    T = window + keep + 70
    rng = np.random.default_rng(4)
    q0 = rng.standard_normal((heads, d))
    q0 *= np.sqrt(d) * 4 / np.linalg.norm(q0, axis=-1, keepdims=True)
    q = M.to_bf16(np.broadcast_to(q0, (T, heads, d)))
    v = M.to_bf16(rng.standard_normal((T, kv, dv)))
    rel = np.zeros((rows, heads), np.float32)
    for j in (0, keep - 1, keep, keep + 1, 31, T - 2 * window // 3):
        if j < 0:
            continue
        k = M.to_bf16(0.02 * rng.standard_normal((T, kv, d)))
        k[j] = M.to_bf16(np.stack([q[0, g * (heads // kv)] for g in range(kv)]))
        want = P.windowed_attention(*(a.astype(np.float64) for a in (q, k, v)), d ** -0.5, rel.astype(np.float64), bias_max, window, keep)
        got = attend(shape, [q], [k], [v], rel, [0], T, dtype)[0]
        tol = 1e-5 if dtype == "f32" else 1e-2
        assert_rows(got.reshape(T, -1), want.reshape(T, -1), tol, f"key {j} in a prompt")
        seen = np.abs(got[:, 0] - v[j, 0]).max(-1) < 0.2
        expect = [P.visible(i, j, window, keep) for i in range(T)]
        assert seen.tolist() == expect, f"key {j}"
        for p in (j, j + window - 1, j + window, T - 1):
            if p < T:
                one = attend(shape, [q], [k], [v], rel, [p], 1, dtype)[0]
                assert_rows(one.reshape(1, -1), want[p].reshape(1, -1), tol, f"key {j} decoded at {p}")


@pytest.mark.parametrize("dtype", DTYPES)
def test_bias_by_distance_in_every_row_of_the_table(dtype):
    """Scores from the bias alone: each query's output is the bias-weighted mean of the values."""
    shape = (4, 2, 16, 24, 90, 8, 14, 77)
    T = 130
    rng = np.random.default_rng(5)
    q, k = np.zeros((T, 4, 16), np.float32), np.zeros((T, 2, 16), np.float32)
    v = M.to_bf16(rng.standard_normal((T, 2, 24)))
    rel = (3 * rng.standard_normal((14, 4))).astype(np.float32)
    want = P.windowed_attention(*(a.astype(np.float64) for a in (q, k, v)), 0.25, rel.astype(np.float64), 77, 90, 8)
    got = attend(shape, [q], [k], [v], rel, [0], T, dtype)[0]
    assert_rows(got.reshape(T, -1), want.reshape(T, -1), 1e-5 if dtype == "f32" else 5e-3)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n_tokens", [1, 4, 250, 600])
def test_query_key_norm_and_append(dtype, n_tokens):
    import torch
    from glinthawk_amd import ops
    heads, kv, d, dv, width, eps = 6, 3, 20, 12, 88, 2e-3
    rng = np.random.default_rng(6)
    nq, nk, nv = heads * d, kv * d, kv * dv
    a = ops.window_attn(heads, kv, d, dv, 1.0, 9, 2, 5)
    x = M.to_bf16(rng.standard_normal((2 * n_tokens, width)))
    w, b = M.to_bf16(rng.standard_normal((nq + nk + nv, width)) / 9), M.to_bf16(rng.standard_normal(nq + nk + nv))
    qn, kn = M.to_bf16(1 + 0.3 * rng.standard_normal(nq)), M.to_bf16(1 + 0.3 * rng.standard_normal(nk))
    y = x.astype(np.float64) @ w.T + b
    T = n_tokens + 40
    row = ops.window_row_bytes(a, torch_dtype(dtype)) // (4 if dtype == "f32" else 2)
    regions = [torch.full((T, row), 7.0, dtype=torch_dtype(dtype), device="cuda") for _ in range(3)]
    start = [3, 39]
    q = ops.matmul_window_append(dev(x, dtype), dev(w, dtype), a, ops.row_table([regions[0].data_ptr(), regions[1].data_ptr()]),
                                 torch.tensor(start, dtype=torch.int32, device="cuda"), n_tokens, dev(b, dtype), dev(qn, dtype), dev(kn, dtype), eps)
    tol = 1e-5 if dtype == "f32" else 1e-2
    dp, vp = 24, 16
    got_q = back(q).reshape(-1, heads, dp)
    assert_rows(got_q[:, :, :d].reshape(len(x), -1), P.rms_norm(y[:, :nq], eps, qn.astype(np.float64)), tol, "q")
    assert np.abs(got_q[:, :, d:]).max() == 0
    for i in range(2):
        c = back(regions[i])
        part = y[i * n_tokens:(i + 1) * n_tokens]
        mine = c[start[i]:start[i] + n_tokens]
        gk, gv = mine[:, : kv * dp].reshape(-1, kv, dp), mine[:, kv * dp:].reshape(-1, kv, vp)
        assert_rows(gk[:, :, :d].reshape(n_tokens, -1), P.rms_norm(part[:, nq:nq + nk], eps, kn.astype(np.float64)), tol, "k")
        assert_rows(gv[:, :, :dv].reshape(n_tokens, -1), part[:, nq + nk:], tol, "v")
        assert np.abs(gk[:, :, d:]).max() == 0 and np.abs(gv[:, :, dv:]).max() == 0
        c[start[i]:start[i] + n_tokens] = 7.0
        assert (c == 7.0).all(), "rows outside the call were written"


MLSTMS = {"small": (3, 12, 20, 9.0), "round": (2, 64, 64, 15.0), "tall": (1, 130, 40, 5.0), "broad": (2, 32, 200, 15.0), "big": (1, 256, 136, 15.0), "huge": (1, 300, 70, 15.0)}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(MLSTMS))
def test_mlstm(name, dtype):
    """Mixer up to its output projection, for gates from never forgetting to forgetting at once: a whole prompt, portions, token by token;
    the state behind the last token as well."""
    import torch
    from glinthawk_amd import ops
    H, d, dv, cap = MLSTMS[name]
    width, eps, T = 72, 1e-4, 214
    from glinthawk_amd._lib import GhMlstm
    m = GhMlstm(H, d, dv, cap, eps)
    rng = np.random.default_rng(8)
    rows, gate_row = ops.mlstm_weight_rows(m)
    hd, hv = H * d, H * dv
    w = np.zeros((rows, width), np.float32)
    w[:2 * hd + 2 * hv] = rng.standard_normal((2 * hd + 2 * hv, width)) / np.sqrt(width)
    w[gate_row:gate_row + 2 * H] = rng.standard_normal((2 * H, width)) / 3
    w = M.to_bf16(w)
    bi, bf = M.to_bf16(2 * rng.standard_normal(H)), M.to_bf16(np.linspace(-6, 7, H) if H > 1 else np.array([3.0]))
    norm = M.to_bf16(1 + 0.2 * rng.standard_normal(hv))
    x = M.to_bf16(rng.standard_normal((T, width)))
    X, W = x.astype(np.float64), w.astype(np.float64)
    split = np.split(W[:2 * hd + 2 * hv], [hd, 2 * hd, 2 * hd + hv])
    q = (X @ split[0].T).reshape(T, H, d) * d ** -0.5
    k, v, g = (X @ split[1].T).reshape(T, H, d), (X @ split[2].T).reshape(T, H, dv), X @ split[3].T
    li = P.soft_cap(X @ W[gate_row:gate_row + H].T + bi, cap)
    lf = P.log_sigmoid(P.soft_cap(X @ W[gate_row + H:gate_row + 2 * H].T + bf, cap))
    o, (S, n, mm) = P.mlstm_recurrence(q, k, v, li, lf)
    want = P.rms_norm(o, eps).reshape(T, hv) * norm / (1 + np.exp(-g))
    tol = 5e-5 if dtype == "f32" else 4e-2
    weights = [dev(a, dtype) for a in (w, bi, bf, norm)]
    offset = 512

    def run(cuts, label):
        state = torch.full((offset // 4 + ops.mlstm_state_bytes(m) // 4,), float("nan"), device="cuda")     # position 0 needs no cleared slot
        table = ops.row_table([state.data_ptr()])
        outs, at = [], 0
        for c in cuts:
            outs.append(back(ops.mlstm_forward(dev(x[at:at + c], dtype), weights[0], m, *weights[1:], table, torch.tensor([at], dtype=torch.int32, device="cuda"), c, offset)))
            at += c
        got = np.concatenate(outs)
        assert_rows(got, want[:at], tol, label, 1.0 if dtype == "f32" else 5.0)
        if at == T:
            vp = -(-dv // 4) * 4
            st = state[offset // 4:].cpu().numpy().astype(np.float64)
            gS = st[:H * d * vp].reshape(H, d, vp)
            assert_rows(gS[:, :, :dv].reshape(H, -1), S.reshape(H, -1), tol, label + ": S")
            assert_rows(st[H * d * vp:H * d * vp + H * d].reshape(1, -1), n.reshape(1, -1), tol, label + ": n")
            assert np.abs(st[-H:] - mm).max() <= (1e-4 if dtype == "f32" else 5e-2), label + ": m"

    run([T], "whole")
    run([2, 3, 5, 64, 1, 63, 65, 11], "portions")
    run([130, 1, 1, 1, 81], "tokens between portions")
    run([1] * 40, "token by token")


@pytest.mark.parametrize("dtype", DTYPES)
def test_mlstm_extreme_gates(dtype):
    """A far token written once with a strong input gate and kept by open forget gates must still be read, and a closed forget gate
    must wipe it."""
    import torch
    from glinthawk_amd import ops
    from glinthawk_amd._lib import GhMlstm
    H, d, dv, cap, T = 2, 16, 24, 15.0, 300
    m = GhMlstm(H, d, dv, cap, 1e-5)
    rows, gate_row = ops.mlstm_weight_rows(m)
    width = d + dv + 4
    # input columns: [key | value | query switch, unused, input gate, forget gate]
    w = np.zeros((rows, width), np.float32)
    for h in range(H):
        w[h * d:(h + 1) * d, :d] = np.eye(d) * np.sqrt(d)
        w[H * d + h * d:H * d + (h + 1) * d, :d] = np.eye(d)
        w[2 * H * d + h * dv:2 * H * d + (h + 1) * dv, d:d + dv] = np.eye(dv)
        w[gate_row + h, d + dv + 2] = 1
        w[gate_row + H + h, d + dv + 3] = 1 if h == 0 else -1        # the second head forgets where the first keeps
    rng = np.random.default_rng(2)
    x = np.zeros((T, width), np.float32)
    x[:, d:d + dv] = rng.standard_normal((T, dv))
    x[:, :d] = 0.05 * rng.standard_normal((T, d))
    x[:, d + dv + 2] = -8.0
    x[:, d + dv + 3] = 12.0
    x[5, 3], x[5, d + dv + 2] = 4.0, 6.0
    x[T - 1, 3] = 4.0
    x, w = M.to_bf16(x), M.to_bf16(w)
    X, W = x.astype(np.float64), w.astype(np.float64)
    q = (X @ W[:H * d].T).reshape(T, H, d) * d ** -0.5
    k, v = (X @ W[H * d:2 * H * d].T).reshape(T, H, d), (X @ W[2 * H * d:2 * H * d + H * dv].T).reshape(T, H, dv)
    li, lf = P.soft_cap(X @ W[gate_row:gate_row + H].T, cap), P.log_sigmoid(P.soft_cap(X @ W[gate_row + H:gate_row + 2 * H].T, cap))
    o, _ = P.mlstm_recurrence(q, k, v, li, lf)
    want = P.rms_norm(o, 1e-5).reshape(T, -1) / 2           # the output gate sees zero
    far = P.rms_norm(v[5], 1e-5)
    assert np.abs(want[-1, :dv] * 2 - far[0]).max() < 0.05 and np.abs(want[-1, dv:] * 2 - far[1]).max() > 0.5
    zeros, ones = dev(np.zeros(H), dtype), dev(np.ones(H * dv), dtype)
    for cuts in ([T], [100, 7, 193], [299, 1]):
        state = torch.empty((ops.mlstm_state_bytes(m) // 4,), device="cuda").fill_(float("nan"))
        table, at = ops.row_table([state.data_ptr()]), 0
        for c in cuts:
            got = back(ops.mlstm_forward(dev(x[at:at + c], dtype), dev(w, dtype), m, zeros, zeros, ones, table, torch.tensor([at], dtype=torch.int32, device="cuda"), c))
            assert_rows(got, want[at:at + c], 1e-4 if dtype == "f32" else 3e-2, f"{cuts} at {at}")
            at += c


# ---- whole models ---------------------------------------------------------------------------------
@pytest.fixture(scope="module")
def models(tmp_path_factory):
    made = {}

    def get(name, T=120):
        if name not in made:
            cfg = M.CONFIGS[name]
            weights = M.random_weights(cfg, seed=sum(map(ord, name)))
            path = M.write_model(tmp_path_factory.mktemp(name), cfg, weights)
            rng = np.random.default_rng(11)
            # At a first token a head's normed output is v times the sign of k . q: where that product almost vanishes, rounding decides.
            # Sequences that rounding errors of weights in bf16 throw off like that say nothing about the code and are drawn again.
            noisy = {k: a * (1 + 2.0 ** -9 * rng.standard_normal(a.shape)) for k, a in weights.items()}
            seqs, want, residuals = [], [], []
            while len(seqs) < 4:
                s, res = rng.integers(0, cfg["vocab"], T), []
                w = P.forward(cfg, weights, s, residuals=res)
                if np.sort(logit_error(P.forward(cfg, noisy, s), w))[-2:].mean() < 0.06:
                    seqs.append(s)
                    want.append(w)
                    residuals = residuals or res
            made[name] = (path, cfg, weights, seqs, want, residuals)
        return made[name]

    return get


def open_stage(path, dtype, n=4, **kw):
    from glinthawk_amd.stage import DesignStage
    return DesignStage(path, dtype, n, n, **kw)


NAMES = list(M.CONFIGS)


def decode_step(st, ids, tokens, positions):
    st.new_state(len(ids))
    st.set_prompts(ids, tokens, positions, prompt_length=1, max_completion_length=st.max_positions)
    assert st.forward()
    return st.logits(len(ids))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
def test_prompt_and_residual_stream(models, name, dtype):
    path, cfg, _, seqs, want, residuals = models(name)
    st = open_stage(path, dtype)
    T = len(seqs[0])
    logits, nxt, res = st.prefill_logits([5], [0], seqs[0][None], range(T), True, cfg["width"])
    for i, (a, b) in enumerate(zip(res, residuals)):
        assert_rows(a, b, MODEL_TOL[dtype], f"stream behind run {i}", 1.0 if dtype == "f32" else 5.0)
    assert_logits(logits, want[0], dtype)
    assert int(nxt[0]) == int(np.argmax(logits[-1]))
    if dtype == "f32":
        assert (np.argmax(logits, -1) == np.argmax(want[0], -1)).all()
    st.close()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
def test_decoding_token_by_token(models, name, dtype):
    path, cfg, _, seqs, want, _ = models(name)
    st = open_stage(path, dtype)
    got = []
    for i, tok in enumerate(seqs[1]):
        got.append(decode_step(st, [3], [tok], [i])[0])
    assert_logits(np.stack(got), want[1], dtype)
    st.close()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
@pytest.mark.parametrize("cuts", [[2] * 30 + [60], [3, 7, 2, 64, 5, 39], [65, 2, 53], [119, 1], [31, 33, 1, 1, 54]])
def test_portions(models, name, dtype, cuts):
    path, cfg, _, seqs, want, _ = models(name)
    st = open_stage(path, dtype)
    at, got = 0, []
    for c in cuts:
        part = seqs[0][at:at + c]
        logits = decode_step(st, [9], part, [at]) if c == 1 else st.prefill_logits([9], [at], part[None], range(c))[0]
        got.append(logits)
        at += c
    assert_logits(np.concatenate(got), want[0], dtype)
    st.close()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
@pytest.mark.parametrize("paged", [False, True])
def test_unequal_requests_in_a_batch_and_slots_used_again(models, name, dtype, paged):
    """Four requests of different lengths, prefilled in pairs at different positions and decoded together, then all over again in the
    slots they gave back: each answers as if it were alone."""
    path, cfg, _, seqs, want, _ = models(name)
    st = open_stage(path, dtype, 4, paged=paged)
    for turn in range(2):
        ids = [10 * turn + k for k in range(4)]
        order = [0, 1, 2, 3] if turn == 0 else [2, 0, 3, 1]            # other sequences in other slots the second time
        at = [0, 0, 0, 0]

        def go(which, n):
            toks = np.stack([seqs[order[k]][at[k]:at[k] + n] for k in which])
            logits, _, _ = st.prefill_logits([ids[k] for k in which], [at[k] for k in which], toks, range(len(which) * n))
            w = np.concatenate([want[order[k]][at[k]:at[k] + n] for k in which])
            assert_logits(logits, w, dtype, f"turn {turn}, contexts {which}")
            for k in which:
                at[k] += n

        go([0], 40)
        go([1], 7)
        go([2, 3], 21)
        go([1, 2], 30)          # at positions 7 and 21
        for _ in range(12):
            logits = decode_step(st, ids, [seqs[order[k]][at[k]] for k in range(4)], at)
            w = np.stack([want[order[k]][at[k]] for k in range(4)])
            assert_logits(logits, w, dtype, f"turn {turn}, decoding at {at}")
            at = [a + 1 for a in at]
        go([3, 0, 2], 20)
        assert st.slot_counts() == dict(free=0, allocated=4, total=4)
        assert st.prefill_logits([99], [0], seqs[0][None, :3]) is None       # no slot left: nothing runs
        for i in ids:
            assert st.release_context(i)
    if paged:
        assert st.paging_info(0, 0)["clears"] >= 1
    # a context that starts again without being given back
    st.prefill_logits([77], [0], seqs[3][None, :50])
    logits, _, _ = st.prefill_logits([77], [0], seqs[1][None, :60], range(60))
    assert_logits(logits, want[1][:60], dtype)
    st.close()


@pytest.mark.parametrize("name", ["odd", "round"])
def test_tokens_out_of_order_are_refused(models, name):
    from glinthawk_amd._lib import GlintError
    path, cfg, _, seqs, want, _ = models(name)
    st = open_stage(path, "f32")
    st.prefill_logits([1], [0], seqs[0][None, :10])
    with pytest.raises(GlintError):
        st.prefill_logits([1], [12], seqs[0][None, 12:20])
    with pytest.raises(GlintError):
        decode_step(st, [1], [3], [9])
    with pytest.raises(GlintError):
        st.prefill_logits([2], [0], np.zeros((1, cfg["max_positions"] + 1), int))
    with pytest.raises(GlintError):
        decode_step(st, [1, 1], [3, 4], [10, 10])
    logits, _, _ = st.prefill_logits([1], [10], seqs[0][None, 10:20], range(10))       # and nothing of that has touched the context
    assert_logits(logits, want[0][10:20], "f32")
    st.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding(models, dtype):
    """Decoding far beyond the window, the table of distances and the prompt, up to the last position the model has."""
    path, cfg, weights, _, _, _ = models("odd")
    T = cfg["max_positions"]
    seq = np.random.default_rng(5).integers(0, cfg["vocab"], T)
    want = P.forward(cfg, weights, seq)
    st = open_stage(path, dtype, 2)
    st.prefill_logits([4], [0], seq[None, :10])
    got = [decode_step(st, [4], [seq[i]], [i])[0] for i in range(10, T)]
    assert_logits(np.stack(got), want[10:], dtype)
    assert st.row(0)["finished"]
    st.close()


@pytest.mark.parametrize("name", ["odd", "round"])
def test_greedy_generation_through_the_compute_kernel(models, name):
    """The serving entry point: states pushed and popped as wire records, prompts fed token by token, then the sampled tokens; each row
    must get the tokens the plain implementation generates."""
    from glinthawk_amd import stage as S, wire
    from glinthawk_amd.kernel import ComputeKernel
    path, cfg, weights, seqs, _, _ = models(name)
    prompts = [list(map(int, seqs[0][:5])), list(map(int, seqs[1][:9])), list(map(int, seqs[2][:1]))]
    new = 12
    want = []
    for p in prompts:
        toks = list(p)
        for _ in range(new):
            toks.append(int(np.argmax(P.forward(cfg, weights, toks)[-1])))
        want.append(toks[len(p):])
    kernel = ComputeKernel(model_dir=path, dtype="f32", concurrency=3, max_contexts=3)
    rows = wire.new_prompts(3)
    rows["active"], rows["kv_tier"], rows["context_id"] = 1, 0, [21, 22, 23]
    rows["prompt_length"], rows["max_completion_length"] = [len(p) for p in prompts], new
    rows["token"] = [p[0] for p in prompts]
    got = [[] for _ in prompts]
    meta = dict(dtype=wire.DTYPE_CODE["f32"], next_layer=0, next_stage=S.STAGE_PRE)
    for _ in range(max(map(len, prompts)) + new + 2):
        if not rows["active"].any():
            break
        kernel.push(wire.pack_state(meta, rows))
        assert kernel.wait(30.0)
        kernel.read_event()
        _, rows, *_ = wire.unpack_state(kernel.pop(), 0, 0)
        for i, p in enumerate(prompts):
            if not rows["active"][i]:
                continue
            pos = int(rows["token_pos"][i])
            if pos < len(p):
                rows["token"][i] = p[pos]                    # still inside the prompt: the sampled token is not used
            else:
                got[i].append(int(rows["token"][i]))
                if len(got[i]) == new:
                    rows["active"][i] = 0
    assert got == want
    kernel.close()


def test_float32_weights_load_as_well(models, tmp_path):
    path, cfg, weights, seqs, want, _ = models("odd")
    st = open_stage(M.write_model(tmp_path / "f32", cfg, weights, dtype="F32"), "f32")
    assert_logits(st.prefill_logits([1], [0], seqs[0][None, :30], range(30))[0], want[0][:30], "f32")
    st.close()


@pytest.mark.parametrize("dtype", ["bfloat16", "float32"])
def test_trace_runner(models, tmp_path, dtype):
    path, cfg, _, seqs, want, _ = models("odd")
    steps = [
        {"step": 0, "entries": [{"id": "a", "tokens": seqs[0][:30].tolist(), "want": [0, 7, 29]}], "end": []},
        {"step": 1, "entries": [{"id": "b", "tokens": seqs[1][:2].tolist(), "want": []}], "end": []},
        {"step": 2, "entries": [{"id": "a", "tokens": [int(seqs[0][30])], "want": [0]}, {"id": "b", "tokens": [int(seqs[1][2])], "want": [0]}], "end": ["a"]},
        {"step": 5, "entries": [{"id": "b", "tokens": seqs[1][3:50].tolist(), "want": [46]}, {"id": "c", "tokens": [int(seqs[2][0])], "want": [0]}], "end": ["b", "c"]},
        {"step": 6, "entries": [{"id": "a", "tokens": seqs[3][:9].tolist(), "want": [8]}], "end": ["a"]},
    ]
    expect = {0: want[0][[0, 7, 29]], 2: np.stack([want[0][30], want[1][2]]), 5: np.stack([want[1][49], want[2][0]]), 6: want[3][8:9]}
    run = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", path, "--dtype", dtype, "--out", str(tmp_path), "--max-tokens", "100"],
                         input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=110)
    assert run.returncode == 0, run.stderr
    assert [l for l in run.stdout.splitlines() if l.startswith("done")] == [f"done {s['step']}" for s in steps]
    for n, w in expect.items():
        got = np.fromfile(tmp_path / f"{n}.f32", np.float32).reshape(-1, cfg["vocab"])
        assert got.shape == w.shape
        assert_logits(got, w, "f32" if dtype == "float32" else "bf16", f"step {n}")
    assert not (tmp_path / "1.f32").exists()
