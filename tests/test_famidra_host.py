"""Host side of the run-time sized designs: the configuration reader and its refusals, the order of layer runs, the distance table, the
paged contexts, the registry, the trace runner's arguments -- and the plain implementation against itself."""
import copy
import json
import os
import subprocess

import numpy as np
import pytest

import famidra_models as M
import plain_famidra as P
from glinthawk_amd import stage as S
from glinthawk_amd._lib import GlintError

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


def text_of(cfg):
    return json.dumps(dict(cfg, layers=[{k: v for k, v in l.items() if not k.startswith("_")} for l in cfg["layers"]]))


@pytest.mark.parametrize("name", list(M.CONFIGS))
def test_order_of_layer_runs(name):
    cfg = M.CONFIGS[name]
    want = [(i, t) for i, t, _ in P.run_order(len(cfg["layers"]), cfg["loop"])]
    assert S.famidra_runs(text_of(cfg)) == want


def test_without_a_loop_every_layer_runs_once():
    cfg = copy.deepcopy(M.CONFIGS["odd"])
    cfg["loop"] = None
    assert S.famidra_runs(text_of(cfg)) == [(i, None) for i in range(4)]


@pytest.mark.parametrize("change", [
    lambda c: c.pop("width"), lambda c: c.update(width=0), lambda c: c.update(width=2.5), lambda c: c.update(width="52"), lambda c: c.update(layers=[]),
    lambda c: c["layers"][0].update(type="convolution"), lambda c: c["layers"][0]["mixer"].pop("kv_heads"), lambda c: c["layers"][0]["mixer"].update(heads=5),
    lambda c: c["layers"][0]["mixer"]["mask"].pop("size"), lambda c: c["layers"][1]["mixer"].update(gate_cap=0), lambda c: c["layers"][0]["mlp"].update(kind="sparse"),
    lambda c: c["loop"].update(stop=9), lambda c: c["loop"].update(start=3), lambda c: c["loop"].update(times=0), lambda c: c["norm"].pop("eps")])
def test_bad_configurations_are_refused(change):
    cfg = copy.deepcopy(M.CONFIGS["odd"])
    change(cfg)
    with pytest.raises(GlintError, match="config.json"):
        S.famidra_runs(text_of(cfg))


@pytest.mark.parametrize("text", ["", "{", "[1,2", '{"width": }', '{"a": 1} x', '{"a": "\\q"}', "nul", '{"a": +1}', "[" * 100 + "]" * 100])
def test_malformed_json_is_refused(text):
    with pytest.raises(GlintError, match="JSON"):
        S.famidra_runs(text)


def test_json_numbers_and_escapes():
    cfg = copy.deepcopy(M.CONFIGS["odd"])
    text = text_of(cfg).replace('"architecture": "Famidra"', '"archi\\u0074ecture":"Fami\\u0064ra\\n\\"\\ud83d\\ude00"').replace('"width": 52', '"width":\t5.2e1')
    assert len(S.famidra_runs(text)) == 8


@pytest.mark.parametrize("rows,bias_max", [(16, 64.0), (10, 23), (7, 40), (32, 200), (2, 5), (24, 96), (9, 30.5), (1, 3)])
def test_distance_table(rows, bias_max):
    half = rows // 2
    got = [S.host_lib().glint_book_distance_bucket(n, rows, bias_max) for n in range(3 * int(bias_max))]
    if half:
        assert got == [P.distance_bucket(n, rows, bias_max) for n in range(3 * int(bias_max))]
    assert got[:half] == list(range(half)) and got == sorted(got) and max(got) <= rows - 1
    assert all(b == rows - 1 for b in got[int(np.ceil(bias_max)):])
    assert S.host_lib().glint_book_distance_bucket(10 ** 12, rows, bias_max) == rows - 1


def test_distance_table_where_the_logarithm_is_a_whole_number():
    # half 8, 8 rows over a factor of 16: a row for every half power of two, exactly
    got = [S.host_lib().glint_book_distance_bucket(n, 16, 128.0) for n in (8, 15, 16, 31, 32, 63, 64, 127, 128)]
    assert got == [8, 9, 10, 11, 12, 13, 14, 15, 15]


def test_paged_contexts_commit_what_a_sequence_needs():
    MiB = 1 << 20
    ctx = S.BookLayeredContext(4096, [("rows", 1024), ("state", 3 * MiB), ("rows", 2048)])      # 4 MiB, 3 MiB, 8 MiB
    blocks = lambda rows: len({b for off, n in ((0, 1024 * rows), (4 * MiB, 3 * MiB), (7 * MiB, 2048 * rows)) for b in range(off // (2 * MiB), (off + n - 1) // (2 * MiB) + 1)})
    assert ctx.append(0, 10) == (blocks(10), 0)
    assert ctx.append(10, 1) == (blocks(11), 0)
    assert ctx.append(12, 1) is None and ctx.append(10, 1) is None          # not the next token
    assert ctx.append(11, 3000) == (blocks(3011), 0)
    assert ctx.append(0, 1) == (blocks(1), 1)                               # started again: dropped and committed anew
    assert ctx.append(11, 1) is None
    assert ctx.append(1, 1) == (blocks(2), 1)


def test_registry_refuses_what_it_does_not_know(tmp_path):
    def refused(dtype="f32", match=""):
        with pytest.raises(GlintError, match=match):
            S.DesignStage(str(tmp_path), dtype)
    refused(match="cannot read")
    (tmp_path / "config.json").write_text('{"architecture": "Somethingelse"}')
    refused(match="unknown architecture")
    (tmp_path / "config.json").write_text('{"architecture": "Famidra"}')
    refused(match="is missing")


def test_trace_runner_arguments():
    def run(*args):
        return subprocess.run([os.path.join(ROOT, "bin", "trace_run"), *args], input="", capture_output=True, text=True, timeout=300)
    for args in ((), ("--model", "x", "--out", "y", "--dtype", "float16"), ("--what", "1"), ("--model", "/nonexistent", "--out", "/tmp", "--dtype", "float32")):
        r = run(*args)
        assert r.returncode == 1 and r.stderr.startswith("trace-run:"), args


# ---- the plain implementation against itself: what the GPU tests compare with has to hold together ----
def test_plain_recurrence_continues_from_its_state():
    rng = np.random.default_rng(1)
    T, H, d, dv = 30, 2, 5, 7
    q, k, v = (rng.standard_normal((T, H, n)) for n in (d, d, dv))
    li, lf = rng.standard_normal((T, H)), P.log_sigmoid(rng.standard_normal((T, H)))
    whole, state = P.mlstm_recurrence(q, k, v, li, lf)
    a, mid = P.mlstm_recurrence(q[:13], k[:13], v[:13], li[:13], lf[:13])
    b, end = P.mlstm_recurrence(q[13:], k[13:], v[13:], li[13:], lf[13:], mid)
    assert np.allclose(np.concatenate([a, b]), whole) and all(np.allclose(x, y) for x, y in zip(end, state))
    # and equals the sum over all earlier tokens that the recurrence unrolls to
    for t in (0, 7, 29):
        b_cum = np.cumsum(lf, 0)
        m = np.maximum(b_cum[t], (b_cum[t] - b_cum[:t + 1] + li[:t + 1]).max(0))
        w = np.exp(b_cum[t] - b_cum[:t + 1] + li[:t + 1] - m) * np.einsum("shd,hd->sh", k[:t + 1], q[t])
        den = np.maximum(np.abs(w.sum(0)), np.exp(-m)) + 1e-6
        assert np.allclose(np.einsum("sh,shv->hv", w, v[:t + 1]) / den[:, None], whole[t])


def test_plain_attention_shows_the_visible_keys_only():
    T, window, keep = 20, 5, 3
    q, k = np.zeros((T, 1, 4)), np.zeros((T, 1, 4))
    v = np.eye(T)[:, None, :]
    out = P.windowed_attention(q, k, v, 1.0, np.zeros((4, 1)), 9, window, keep)[:, 0]
    for i in range(T):
        seen = {j for j in range(T) if out[i, j] > 0}
        assert seen == {j for j in range(i + 1) if j > i - window or j < keep}
        assert np.allclose(out[i].sum(), 1)
