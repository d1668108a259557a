"""The Dirozen design on the GPU against the plain implementation (plain_dirozen.py): every mechanism alone, then whole models through the
stage, the compute kernel and the trace runner -- whole prompts, portions, token by token, batches, slots and pages that are used again."""
import json
import os
import subprocess

import numpy as np
import pytest

import dirozen_models as M
import plain_dirozen as P
import plain_famidra as PF

pytestmark = pytest.mark.gpu

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
DTYPES = ("f32", "bf16")
# root mean square of the difference of the logits over that of the expected ones, worst row
MODEL_TOL = {"f32": 2e-5, "bf16": 3e-2}


def torch_dtype(dtype):
    import torch
    return torch.float32 if dtype == "f32" else torch.bfloat16


def dev(a, dtype):
    import torch
    return torch.from_numpy(np.ascontiguousarray(a, dtype=np.float32)).cuda().to(torch_dtype(dtype)).contiguous()


def positions(p):
    import torch
    return torch.tensor(p, dtype=torch.int32, device="cuda")


def back(t):
    return t.float().cpu().numpy().astype(np.float64)


def assert_rows(got, want, tol, what=""):
    """Each row's error over its own size, or the rows' common one where that is larger."""
    got, want = np.asarray(got, np.float64), np.asarray(want, np.float64)
    rms = lambda a: np.sqrt((a ** 2).mean(-1))
    e = rms(got - want) / np.maximum(rms(want), np.sqrt((want ** 2).mean()))
    assert bool(np.isfinite(got).all()) and e.max() <= tol, f"{what}: worst row {int(e.argmax())} of {e.size} off by {e.max():.2e} (tol {tol})"


def assert_logits(got, want, dtype, what=""):
    d = np.asarray(got, np.float64) - want
    d -= d.mean(-1, keepdims=True)
    w = want - want.mean(-1, keepdims=True)
    e, tol = np.sqrt((d ** 2).mean(-1)) / np.sqrt((w ** 2).mean()), MODEL_TOL[dtype]
    assert np.isfinite(got).all() and e.max() <= tol, f"{what}: row {int(e.argmax())} of {e.size} off by {e.max():.2e} (tol {tol})"


# ---- mechanisms alone ----------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,s,width", [(1, 24, 52), (5, 128, 128), (200, 64, 256), (1100, 40, 1000), (260, 64, 50)])
def test_norms_around_zero(dtype, rows, s, width):
    import torch
    from glinthawk_amd import ops
    rng = np.random.default_rng(rows)
    inp, w, nxt, post = (M.to_bf16(rng.standard_normal(n)) for n in ((rows, s), (width, s), (width,), (width,)))
    nxt, post, eps = M.to_bf16(0.01 * nxt), M.to_bf16(0.01 * post), 2e-3
    x0 = rng.standard_normal((rows, width)).astype(np.float32)
    y = inp.astype(np.float64) @ w.T
    tol = 1e-5 if dtype == "f32" else 5e-3
    for parts, v in ((dict(), y), (dict(post_norm=dev(post, dtype)), P.rms_norm_around_zero(y, post.astype(np.float64), eps))):
        x, out = torch.from_numpy(x0).cuda(), torch.zeros((rows, width), dtype=torch_dtype(dtype), device="cuda")
        ops.matmul_stream(x, dev(inp, dtype), dev(w, dtype), eps, out=out, next_norm=dev(nxt, dtype), norm_base=1.0, **parts)
        assert_rows(back(x), x0 + v, tol, "stream")
        assert_rows(back(out), P.rms_norm_around_zero(x0 + v, nxt.astype(np.float64), eps), tol, "norm behind the update")
    ops.stream_out(torch.from_numpy(x0).cuda(), out, dev(nxt, dtype), eps, 1.0)
    assert_rows(back(out), P.rms_norm_around_zero(x0.astype(np.float64), nxt.astype(np.float64), eps), tol, "norm alone")


@pytest.mark.parametrize("n_tokens", [1, 20, 70])
def test_projections_with_a_large_feed_forward(n_tokens):
    """Sizes at which few rows take the feed-forward's gate in the launch of its own product, into rows that lie apart."""
    import torch
    from glinthawk_amd import ops
    heads, kv, d, ff, width = 4, 2, 64, 28672, 256
    a = ops.window_attn(heads, kv, d, d, 1.0, values_are_keys=True)
    rows, ff_row = ops.parallel_weight_rows(a, True, ff)
    g = torch.Generator().manual_seed(n_tokens)
    w = (torch.randn((rows, width), generator=g) / 16).cuda().bfloat16()
    x = torch.randn((n_tokens, width), generator=g).cuda().bfloat16()
    keys = torch.zeros((-(-(n_tokens + 4) // 32) * 32, kv * d), dtype=torch.bfloat16, device="cuda")
    at = keys.numel() * 2
    region = torch.cat([keys.reshape(-1).view(torch.uint8), torch.zeros(keys.shape[0] * kv * 4, dtype=torch.uint8, device="cuda")])
    wide = torch.full((n_tokens, ff + 48), 5.0, dtype=torch.bfloat16, device="cuda")
    q, gates = ops.matmul_parallel(x, w, a, ops.row_table([region.data_ptr()]), positions([4]), n_tokens, 1e-3, 0.5, 8, True, wide[:, 40:40 + ff], factor_offset=at)
    y = x.float() @ w.float().T
    h = torch.nn.functional.silu(y[:, ff_row:ff_row + ff]) * y[:, ff_row + ff:ff_row + 2 * ff]
    assert_rows(back(wide[:, 40:40 + ff]), back(h), 1e-2, "hidden")
    assert bool((wide[:, :40] == 5).all()) and bool((wide[:, 40 + ff:] == 5).all())
    y = back(y)
    temp = np.array([P.query_temperature(p, 0.5, 8) for p in range(4, 4 + n_tokens)])[:, None, None]
    assert_rows(back(q), (P.unit_rms(y[:, :256].reshape(-1, heads, d), 1e-3) * temp).reshape(n_tokens, -1), 1e-2, "q")
    assert_rows(back(gates), P.sigmoid(y[:, 384:388]), 1e-2, "head gates")
    assert_rows(back(region[:at].view(torch.bfloat16)).reshape(-1, kv * d)[4:4 + n_tokens], y[:, 256:384], 1e-2, "keys")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n_tokens", [1, 4, 250, 600])
@pytest.mark.parametrize("heads,kv,d,ff,gated,every", [(6, 3, 20, 44, True, 7), (4, 1, 64, 0, True, 1), (5, 5, 96, 72, False, 33), (3, 1, 136, 21, True, 64), (2, 2, 300, 40, True, 0),
                                                       (16, 2, 128, 256, True, 10)])
def test_projections_of_a_parallel_layer(heads, kv, d, ff, gated, every, n_tokens, dtype):
    """Everything one product feeds: queries with norm and temperature, cache rows and key factors, head gates, the feed-forward's hidden
    values; at positions on both sides of a step of the temperature, and nothing written outside."""
    import torch
    from glinthawk_amd import ops
    width, eps, coef = 88, 2e-3, 0.6
    rng = np.random.default_rng(d + n_tokens)
    a = ops.window_attn(heads, kv, d, d, 1.0, values_are_keys=True)
    rows, ff_row = ops.parallel_weight_rows(a, gated, ff)
    nq, nk, ng = heads * d, kv * d, heads if gated else 0
    assert ff_row >= nq + nk + ng and rows >= ff_row + 2 * ff
    w = np.zeros((rows, width), np.float32)
    w[:nq + nk + ng] = rng.standard_normal((nq + nk + ng, width)) / 9
    w[ff_row:ff_row + 2 * ff] = rng.standard_normal((2 * ff, width)) / 9
    w = M.to_bf16(w)
    x = M.to_bf16(rng.standard_normal((3 * n_tokens, width)))
    y = x.astype(np.float64) @ w.T
    T = n_tokens + 72
    dp = -(-d // 8) * 8
    row, group = kv * dp, 32
    size = 4 if dtype == "f32" else 2
    assert ops.window_row_bytes(a, torch_dtype(dtype)) == row * size and ops.window_factor_bytes(a) == 4 * kv
    keys = [torch.full((T, row), 7.0, dtype=torch_dtype(dtype), device="cuda") for _ in range(2)]
    factors = [torch.full((-(-T // group), kv, group), 7.0, device="cuda") for _ in range(2)]
    # one region per context: the factors behind the keys
    at = -(-T * row * size // 256) * 256
    regions = [torch.cat([k.reshape(-1).view(torch.uint8), torch.zeros(at - k.numel() * size, dtype=torch.uint8, device="cuda"), f.reshape(-1).view(torch.uint8)]) for k, f in zip(keys, factors)]
    start = [31, 3, max(0, every - 1)]
    wide = torch.full((len(x), ff + 24), 5.0, dtype=torch_dtype(dtype), device="cuda")
    hidden = wide[:, 16:16 + ff] if ff else None
    q, gates = ops.matmul_parallel(dev(x, dtype), dev(w, dtype), a, ops.row_table([regions[0].data_ptr(), 0, regions[1].data_ptr()]), positions(start), n_tokens, eps,
                                   coef, every, gated, hidden, factor_offset=at)
    tol = 1e-5 if dtype == "f32" else 1e-2
    got_q, got_h = back(q).reshape(-1, heads, dp), back(wide)
    assert (got_h[:, :16] == 5).all() and (got_h[:, 16 + ff:] == 5).all(), "columns beside the hidden values were written"
    for i, region in ((0, regions[0]), (2, regions[1])):
        part = slice(i * n_tokens, (i + 1) * n_tokens)
        pos = start[i] + np.arange(n_tokens)
        temp = np.array([P.query_temperature(p, coef, every) if every else 1.0 for p in pos])[:, None, None]
        raw_q, raw_k = y[part, :nq].reshape(-1, heads, d), y[part, nq:nq + nk].reshape(-1, kv, d)
        assert_rows(got_q[part, :, :d].reshape(n_tokens, -1), (P.unit_rms(raw_q, eps) * temp).reshape(n_tokens, -1), tol, "q")
        assert np.abs(got_q[part, :, d:]).max(initial=0) == 0
        if gated:
            assert_rows(back(gates)[part], P.sigmoid(y[part, nq + nk:nq + nk + ng]), tol, "head gates")
        if ff:
            g, u = y[part, ff_row:ff_row + ff], y[part, ff_row + ff:ff_row + 2 * ff]
            assert_rows(got_h[part, 16:16 + ff], P.silu(g) * u, tol, "hidden")
        cache = back(region[:T * row * size].view(torch_dtype(dtype))).reshape(T, kv, dp)
        fac = region[at:].view(torch.float32).cpu().numpy().reshape(-1, kv, group).transpose(0, 2, 1).reshape(-1, kv)
        assert_rows(cache[pos, :, :d].reshape(n_tokens, -1), raw_k.reshape(n_tokens, -1), tol, "keys")
        assert np.abs(cache[pos, :, d:]).max(initial=0) == 0
        assert_rows(fac[pos], 1 / np.sqrt((raw_k ** 2).mean(-1) + eps), tol, "key factors")
        cache[pos], fac[pos] = 7.0, 7.0
        assert (cache == 7).all() and (fac == 7).all(), "rows outside the call were written"
    # the context without a region: nothing of it is written
    assert np.abs(got_q[n_tokens:2 * n_tokens]).max() == 0 and (got_h[n_tokens:2 * n_tokens] == 5).all()


ATTENTIONS = {  # heads, kv heads, dim
    "small": (6, 2, 24), "matrix": (8, 2, 64), "ten": (10, 1, 72), "own": (3, 3, 128), "between": (4, 4, 88), "many": (48, 1, 96), "one": (1, 1, 40), "deep": (2, 1, 200),
    "deeper": (2, 2, 300), "deepest": (1, 1, 512),
}


class Cache:
    """One layer's keys of a few contexts, filled by hand: rows padded to 8 elements a head, the factors of 32 tokens of a head together;
    what lies behind the last token is NaN."""

    def __init__(self, shape, k, dtype, eps, scale, room=40, **window):
        import torch
        from glinthawk_amd import ops
        heads, kv, d = shape
        self.attn = ops.window_attn(heads, kv, d, d, scale, values_are_keys=True, **window)
        dp = self.dp = -(-d // 8) * 8
        self.offset, self.regions = 256, []
        size = 4 if dtype == "f32" else 2
        longest = max(len(kk) for kk in k) + room
        self.factor_offset = self.offset + -(-longest * kv * dp * size // 256) * 256
        for kk in k:
            T = kk.shape[0]
            full = np.full((longest, kv, dp), np.nan, np.float32)
            full[:T] = 0
            full[:T, :, :d] = kk
            f = np.full((-(-longest // 32) * 32, kv), np.nan, np.float32)
            f[:T] = 1 / np.sqrt((kk.astype(np.float64) ** 2).mean(-1) + eps)
            region = torch.full(((self.factor_offset + f.size * 4) // 4,), float("nan"), device="cuda").view(torch.uint8)
            region[self.offset:self.offset + full.size * size] = dev(full, dtype).reshape(-1).view(torch.uint8)
            region[self.factor_offset:] = torch.from_numpy(np.ascontiguousarray(f.reshape(-1, 32, kv).transpose(0, 2, 1))).cuda().reshape(-1).view(torch.uint8)
            self.regions.append(region)
        self.rows = ops.row_table([r.data_ptr() for r in self.regions])


def attend(shape, q, k, start, n, dtype, eps=1e-3, scale=None, gates=None, bias=None, **window):
    """Queries of positions [start_i, start_i + n) of every sequence as one call; q as it meets the keys."""
    import torch
    from glinthawk_amd import ops
    heads, kv, d = shape
    cache = Cache(shape, k, dtype, eps, scale, **window)
    qp = np.zeros((len(q), n, heads, cache.dp), np.float32)
    for i, (qq, s) in enumerate(zip(q, start)):
        qp[i, :, :, :d] = qq[s:s + n]
    wide = torch.full((len(q) * n, heads * d + 20), 3.0, dtype=torch_dtype(dtype), device="cuda")
    if gates is not None:
        gates = torch.from_numpy(np.concatenate([g[s:s + n] for g, s in zip(gates, start)]).astype(np.float32)).cuda()
    if bias is not None:
        bias = torch.from_numpy(np.ascontiguousarray(bias, np.float32)).cuda()
    out = ops.attn_window(dev(qp.reshape(len(q) * n, -1), dtype), cache.attn, cache.rows, positions(start), n, max(start), bias, cache.offset, cache.factor_offset,
                          gates, wide[:, 8:8 + heads * d])
    full = back(wide)
    assert (full[:, :8] == 3).all() and (full[:, 8 + heads * d:] == 3).all(), "columns beside the output were written"
    return back(out).reshape(len(q), n, heads, d)


def attention_case(name, T, seed, n_seq, eps, scale):
    """Keys of very different lengths, so that one that is not divided by its root mean square shows."""
    heads, kv, d = ATTENTIONS[name]
    rng = np.random.default_rng(seed)
    q = [M.to_bf16(rng.standard_normal((T, heads, d))) for _ in range(n_seq)]
    k = [M.to_bf16(rng.standard_normal((T, kv, d)) * np.exp(rng.standard_normal((T, kv, 1)))) for _ in range(n_seq)]
    want = [np.stack([[P.read_keys(qq[t, h].astype(np.float64), kk[: t + 1, h // (heads // kv)].astype(np.float64), eps, scale) for h in range(heads)] for t in range(T)])
            for qq, kk in zip(q, k)]
    return (heads, kv, d), q, k, want


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(ATTENTIONS))
def test_attention_over_keys_that_are_values(name, dtype):
    """A whole prompt, portions from anywhere, single tokens around the borders of the kernels' tiles, two sequences in a call."""
    T, eps, scale = 200, 1e-3, 2.0 / ATTENTIONS[name][2] ** 0.5
    shape, q, k, want = attention_case(name, T, 3, 2, eps, scale)
    tol = 1e-5 if dtype == "f32" else 8e-3
    run = lambda start, n, **kw: attend(shape, q, k, start, n, dtype, eps, scale, **kw)
    assert_rows(run([0, 0], T).reshape(2 * T, -1), np.stack(want).reshape(2 * T, -1), tol, "whole")
    for start, n in (([0, 70], 2), ([13, 90], 33), ([64, 1], 64), ([100, 37], 17), ([16, 48], 128), ([127, 128], 15), ([31, 32], 16)):
        w = np.stack([a[s:s + n] for a, s in zip(want, start)])
        assert_rows(run(start, n).reshape(2 * n, -1), w.reshape(2 * n, -1), tol, f"portion {start}+{n}")
    gates = [np.random.default_rng(i).random((T, shape[0])) for i in range(2)]
    for p in (0, 1, 31, 32, 63, 64, 127, 128, T - 1):
        w = np.stack([a[p] for a in want])
        assert_rows(run([p, p], 1).reshape(2, -1), w.reshape(2, -1), tol, f"token {p}")
    for start, n in (([5, 60], 1), ([150, 2], 1), ([0, 0], T), ([40, 9], 50)):
        w = np.stack([a[s:s + n] * g[s:s + n, :, None] for a, g, s in zip(want, gates, start)])
        assert_rows(run(start, n, gates=gates).reshape(2 * n, -1), w.reshape(2 * n, -1), tol, f"gated {start}+{n}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["small", "matrix", "ten", "own", "between", "deep"])
def test_one_key_stands_out(name, dtype):
    """Every key in turn made the one its queries' scores pick, among hundreds: read from its own position on by every later query, near or
    far, and by none before it.  One head long and one short, which their norms make alike."""
    heads, kv, d = shape = ATTENTIONS[name]
    T, scale, eps = 700, 14.0 / d, 1e-4
    rng = np.random.default_rng(4)
    q0 = rng.standard_normal((kv, d))
    q0 /= np.sqrt((q0 ** 2).mean(-1, keepdims=True))
    q = M.to_bf16(np.broadcast_to(np.repeat(q0, heads // kv, axis=0), (T, heads, d)))
    tol = 2e-5 if dtype == "f32" else 1e-2
    base = M.to_bf16(rng.standard_normal((T, kv, d)))
    for j in (0, 1, 31, 32, 63, 64, 127, 128, 255, 256, 300, 511, 513, T - 2):
        k = base.copy()
        k[j] = M.to_bf16(q0 * (0.2 if j % 2 else 3.0))
        want = np.stack([[P.read_keys(q[t, h].astype(np.float64), k[: t + 1, h // (heads // kv)].astype(np.float64), eps, scale) for h in range(0, heads, heads // kv)] for t in range(T)])
        got = attend(shape, [q], [k], [0], T, dtype, eps, scale)[0][:, ::heads // kv]
        assert_rows(got.reshape(T, -1), want.reshape(T, -1), tol, f"key {j} in a prompt")
        seen = np.array([np.corrcoef(got[t, 0], q0[0])[0, 1] > 0.95 for t in range(T)])
        assert seen[j:].all() and not seen[:j].any(), f"key {j}"
        for p in sorted({j, j + 1, 64, 300, 511, 512, 640, T - 1}):
            if p < T:
                one = attend(shape, [q], [k], [p], 1, dtype, eps, scale)[0][:, ::heads // kv]
                assert_rows(one.reshape(1, -1), want[p].reshape(1, -1), tol, f"key {j} decoded at {p}")
        s = max(0, j - 20)
        n = min(40, T - s)
        some = attend(shape, [q], [k], [s], n, dtype, eps, scale)[0][:, ::heads // kv]
        assert_rows(some.reshape(n, -1), want[s:s + n].reshape(n, -1), tol, f"key {j} in a portion from {s}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["matrix", "own", "deep"])
def test_values_that_are_keys_under_a_window_and_a_bias(name, dtype):
    """The mechanism beside those other designs use: a sliding window, kept first tokens and a bias by distance."""
    heads, kv, d = shape = ATTENTIONS[name]
    T, window, keep, rows, bias_max, eps, scale = 150, 37, 5, 12, 50, 1e-3, 1.5 * ATTENTIONS[name][2] ** -0.5
    rng = np.random.default_rng(7)
    q = M.to_bf16(rng.standard_normal((T, heads, d)))
    k = M.to_bf16(rng.standard_normal((T, kv, d)) * np.exp(rng.standard_normal((T, kv, 1))))
    rel = rng.standard_normal((rows, heads))
    want = PF.windowed_attention(q.astype(np.float64), P.unit_rms(k.astype(np.float64), eps), k.astype(np.float64), scale, rel, bias_max, window, keep)
    bias = np.array([[rel[PF.distance_bucket(t, rows, bias_max), h] for t in range(bias_max + 1)] for h in range(heads)])
    for start, n in ((0, T), (60, 33), (36, 1), (37, 1), (43, 1), (T - 1, 1)):
        got = attend(shape, [q], [k], [start], n, dtype, eps, scale, bias=bias, window=window, keep_first=keep, n_dist=bias_max + 1)[0]
        assert_rows(got.reshape(n, -1), want[start:start + n].reshape(n, -1), 1e-5 if dtype == "f32" else 8e-3, f"{start}+{n}")


def test_rows_copied_apart():
    import torch
    from glinthawk_amd import _lib
    src = np.arange(60, dtype=np.float32).reshape(12, 5)
    dst = torch.full((12, 9), -1.0, device="cuda")
    torch.cuda.synchronize()
    _lib.check(_lib.lib().gh_memcpy_rows(dst.data_ptr() + 8, 36, src.ctypes.data, 20, 20, 12, _lib.GH_H2D, None), "gh_memcpy_rows")
    got = dst.cpu().numpy()
    assert (got[:, 2:7] == src).all() and (got[:, :2] == -1).all() and (got[:, 7:] == -1).all()


# ---- whole models ---------------------------------------------------------------------------------
@pytest.fixture(scope="module")
def models(tmp_path_factory):
    made = {}

    def get(name, T=150):
        if name not in made:
            cfg = M.CONFIGS[name]
            weights = M.random_weights(cfg, seed=sum(map(ord, name)))
            path = M.write_model(tmp_path_factory.mktemp(name), cfg, weights)
            rng = np.random.default_rng(11)
            seqs = [rng.integers(0, cfg["vocab"], T) for _ in range(4)]
            residuals = []
            want = [P.forward(cfg, weights, s, residuals=residuals if i == 0 else None) for i, s in enumerate(seqs)]
            made[name] = (path, cfg, weights, seqs, want, residuals)
        return made[name]

    return get


def open_stage(path, dtype, n=4, max_positions=400, **kw):
    from glinthawk_amd.stage import DesignStage
    return DesignStage(path, dtype, n, n, max_positions=max_positions, **kw)


NAMES = list(M.CONFIGS)


def decode_step(st, ids, tokens, at):
    st.new_state(len(ids))
    st.set_prompts(ids, tokens, at, prompt_length=1, max_completion_length=st.max_positions)
    assert st.forward()
    return st.logits(len(ids))


def run_portions(st, ctx, seq, cuts):
    at, got = 0, []
    for c in cuts:
        part = seq[at:at + c]
        got.append(decode_step(st, [ctx], part, [at]) if c == 1 else st.prefill_logits([ctx], [at], part[None], range(c))[0])
        at += c
    return np.concatenate(got)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
def test_prompt_and_residual_stream(models, name, dtype):
    path, cfg, _, seqs, want, residuals = models(name)
    st = open_stage(path, dtype)
    T = len(seqs[0])
    logits, nxt, res = st.prefill_logits([5], [0], seqs[0][None], range(T), True, cfg["width"])
    assert st.layer_runs == len(cfg["layers"]) and st.vocab_size == cfg["vocab"]
    for i, (a, b) in enumerate(zip(res, residuals)):
        assert_rows(a, b, MODEL_TOL[dtype], f"stream behind layer {i}")
    assert_logits(logits, want[0], dtype)
    assert int(nxt[0]) == int(np.argmax(logits[-1]))
    if dtype == "f32":
        assert (np.argmax(logits, -1) == np.argmax(want[0], -1)).all()
    st.close()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
@pytest.mark.parametrize("cuts", [[1] * 150, [2] * 40 + [70], [3, 7, 2, 64, 5, 69], [65, 2, 83], [149, 1], [31, 33, 1, 1, 84]], ids=lambda c: f"{len(c)}cuts")
def test_portions_and_decoding(models, name, dtype, cuts):
    path, _, _, seqs, want, _ = models(name)
    st = open_stage(path, dtype)
    assert_logits(run_portions(st, 9, seqs[0], cuts), want[0], dtype)
    st.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_far_token(tmp_path, dtype):
    """A token that reads one other token, hundreds of positions away: in a prompt, decoded, and behind portions that end next to either."""
    cfg = M.CONFIGS["round"]
    reader, needle = 5, 9
    w = M.with_needle(cfg, M.random_weights(cfg, 3), reader, needle)
    st = open_stage(M.write_model(tmp_path, cfg, w), dtype, max_positions=700)
    rng = np.random.default_rng(2)
    seq = rng.integers(10, cfg["vocab"], 600)
    readers = [40, 96, 320, 321, 511, 599]
    seq[readers] = reader
    seq[31] = needle
    want = P.forward(cfg, w, seq)
    without = seq.copy()
    without[31] = 12
    shift = np.abs(P.forward(cfg, w, without) - want).max(-1)
    assert shift[readers].min() > 0.4
    for i, cuts in enumerate(([600], [31, 1, 8, 1, 279, 1, 1, 278], [32, 64, 2, 222, 1, 279], [30, 2, 287, 2, 190, 88, 1])):
        assert_logits(run_portions(st, i % 2, seq, cuts), want, dtype, f"{cuts}")
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
            assert_logits(logits, np.concatenate([want[order[k]][at[k]:at[k] + n] for k in which]), dtype, f"turn {turn}, contexts {which}")
            for k in which:
                at[k] += n

        go([0], 90 if turn == 0 else 40)      # the second time the last sequence's keys lie behind
        go([1], 7)
        go([2, 3], 21)
        go([1, 2], 30)          # at positions 7 and 21
        for _ in range(12):
            logits = decode_step(st, ids, [seqs[order[k]][at[k]] for k in range(4)], at)
            assert_logits(logits, np.stack([want[order[k]][at[k]] for k in range(4)]), dtype, f"turn {turn}, decoding at {at}")
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


@pytest.mark.parametrize("dtype", DTYPES)
def test_across_pages(tmp_path, dtype):
    """Cache rows so long that a sequence crosses 2 MiB pages, in a prompt, in portions and while decoding; then a short one in the same slot."""
    heads = 8 if dtype == "f32" else 16
    cfg = M.config(48, 60, [M.layer(heads, heads, 128, 90, ff=32), M.layer(1, 1, 24, 90)])
    w = M.random_weights(cfg, 8)
    st = open_stage(M.write_model(tmp_path, cfg, w), dtype, 1, max_positions=1100, paged=True)
    seq = np.random.default_rng(3).integers(0, 60, 540)
    want = P.forward(cfg, w, seq)
    pages = lambda: st.paging_info(0, 0)["blocks_committed"]      # a page holds 512 tokens of the first layer
    st.prefill_logits([1], [0], seq[None, :500])
    before = pages()
    got = [decode_step(st, [1], [seq[i]], [i])[0] for i in range(500, 530)]
    assert pages() == before + 1
    assert_logits(np.stack(got), want[500:530], dtype, "decoded")
    assert_logits(run_portions(st, 1, seq, [7, 504, 2, 27]), want, dtype, "portions")
    assert_logits(st.prefill_logits([1], [0], seq[None], range(540))[0], want, dtype, "prompt")
    assert st.release_context(1)
    short = np.random.default_rng(4).integers(0, 60, 30)
    assert_logits(run_portions(st, 2, short, [20, 1, 9]), P.forward(cfg, w, short), dtype, "slot used again")
    assert pages() == before and st.paging_info(0, 0)["clears"] >= 3
    st.close()


def test_tokens_out_of_order_are_refused(models):
    from glinthawk_amd._lib import GlintError
    path, cfg, _, seqs, want, _ = models("odd")
    st = open_stage(path, "f32", max_positions=60)
    st.prefill_logits([1], [0], seqs[0][None, :10])
    with pytest.raises(GlintError):
        st.prefill_logits([1], [12], seqs[0][None, 12:20])
    with pytest.raises(GlintError):
        st.prefill_logits([2], [0], seqs[0][None, :61])
    with pytest.raises(GlintError):
        decode_step(st, [1, 1], [3, 4], [10, 10])
    assert_logits(st.prefill_logits([1], [10], seqs[0][None, 10:60], range(50))[0], want[0][10:60], "f32")       # up to the last position
    with pytest.raises(GlintError):
        decode_step(st, [1], [3], [60])
    st.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding(models, dtype):
    """Hundreds of tokens decoded behind a short prompt, through many steps of the temperature, up to the last position of the context."""
    path, cfg, weights, _, _, _ = models("odd")
    T = 400
    seq = np.random.default_rng(5).integers(0, cfg["vocab"], T)
    want = P.forward(cfg, weights, seq)
    st = open_stage(path, dtype, 2)
    st.prefill_logits([4], [0], seq[None, :10])
    got = [decode_step(st, [4], [seq[i]], [i])[0] for i in range(10, T)]
    assert_logits(np.stack(got), want[10:], dtype)
    assert st.row(0)["finished"]
    st.close()


def test_the_default_number_of_positions(models):
    path, cfg, _, seqs, want, _ = models("odd")
    st = open_stage(path, "f32", 1, max_positions=0)
    assert st.max_positions == 4096
    assert_logits(st.prefill_logits([1], [0], seqs[0][None], range(150))[0], want[0], "f32")
    st.close()


@pytest.mark.parametrize("name", ["odd", "between"])
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
    kernel = ComputeKernel(model_dir=path, dtype="f32", concurrency=3, max_contexts=3, max_positions=64)
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


def test_loading(models, tmp_path):
    """fp32 tensors load as well as bf16 ones; a missing or misshapen tensor is named."""
    from glinthawk_amd._lib import GlintError
    path, cfg, weights, seqs, want, _ = models("odd")
    st = open_stage(M.write_model(tmp_path / "f32", cfg, weights, dtype="F32"), "f32")
    assert_logits(st.prefill_logits([1], [0], seqs[0][None, :30], range(30))[0], want[0][:30], "f32")
    st.close()
    with pytest.raises(GlintError, match="l1.mix.g is missing"):
        open_stage(M.write_model(tmp_path / "less", cfg, weights, drop=("l1.mix.g",)), "f32")
    with pytest.raises(GlintError, match="l0.mlp.down has another shape"):
        open_stage(M.write_model(tmp_path / "other", cfg, dict(weights, **{"l0.mlp.down": weights["l0.mlp.down"].T.copy()})), "f32")


@pytest.mark.parametrize("dtype", ["bfloat16", "float32"])
def test_trace_runner(models, tmp_path, dtype):
    path, cfg, _, seqs, want, _ = models("odd")
    steps = [
        {"step": 0, "entries": [{"id": "a", "tokens": seqs[0][:30].tolist(), "want": [0, 7, 29]}], "end": []},
        {"step": 1, "entries": [{"id": "b", "tokens": seqs[1][:2].tolist(), "want": []}], "end": []},
        {"step": 2, "entries": [{"id": "a", "tokens": [int(seqs[0][30])], "want": [0]}, {"id": "b", "tokens": [int(seqs[1][2])], "want": [0]}], "end": ["a"]},
        {"step": 5, "entries": [{"id": "b", "tokens": seqs[1][3:50].tolist(), "want": [46]}, {"id": "c", "tokens": [int(seqs[2][0])], "want": [0]}], "end": ["b", "c"]},
        {"step": 6, "entries": [{"id": "a", "tokens": seqs[3][:100].tolist(), "want": [8, 99]}], "end": ["a"]},
    ]
    expect = {0: want[0][[0, 7, 29]], 2: np.stack([want[0][30], want[1][2]]), 5: np.stack([want[1][49], want[2][0]]), 6: want[3][[8, 99]]}
    run = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", path, "--dtype", dtype, "--out", str(tmp_path), "--max-tokens", "100"],
                         input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=110)
    assert run.returncode == 0, run.stderr
    assert [l for l in run.stdout.splitlines() if l.startswith("done")] == [f"done {s['step']}" for s in steps]
    for n, w in expect.items():
        got = np.fromfile(tmp_path / f"{n}.f32", np.float32).reshape(-1, cfg["vocab"])
        assert got.shape == w.shape
        assert_logits(got, w, "f32" if dtype == "float32" else "bf16", f"step {n}")
    assert not (tmp_path / "1.f32").exists()
