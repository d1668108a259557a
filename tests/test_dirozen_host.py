"""Host side of the Dirozen design: the configuration reader and its refusals, cache rows that are laid out in groups, the registry -- and
the plain implementation against itself."""
import copy
import json

import numpy as np
import pytest

import dirozen_models as M
import plain_dirozen as P
import plain_famidra as PF
from glinthawk_amd import stage as S
from glinthawk_amd._lib import GlintError


@pytest.mark.parametrize("name", list(M.CONFIGS))
def test_every_size_and_constant_is_read(name):
    cfg = M.CONFIGS[name]
    got = S.dirozen_config(json.dumps(cfg))
    f32 = lambda v: float(np.float32(v))
    assert (got["width"], got["vocab"], got["eps"]) == (cfg["width"], cfg["vocab"], f32(cfg["norm"]["eps"]))
    assert len(got["layers"]) == len(cfg["layers"])
    for g, want in zip(got["layers"], cfg["layers"]):
        m = want["mixer"]
        assert [g[k] for k in ("heads", "kv_heads", "dim")] == [m[k] for k in ("heads", "kv_heads", "dim")]
        assert g["ff"] == (want["mlp"]["ff"] if want["mlp"] else 0)
        assert (g["scale"], g["temp_coef"], g["temp_every"]) == (f32(m["scale"]), f32(m["q_temp"]["coef"]), m["q_temp"]["every"])


def test_no_temperature():
    cfg = copy.deepcopy(M.CONFIGS["odd"])
    cfg["layers"][0]["mixer"]["q_temp"] = None
    del cfg["layers"][1]["mixer"]["q_temp"]
    assert [l["temp_every"] for l in S.dirozen_config(json.dumps(cfg))["layers"]] == [0, 0, 1]


@pytest.mark.parametrize("change", [
    lambda c: c.pop("width"), lambda c: c.update(vocab=0), lambda c: c.update(width=2.5), lambda c: c.update(layers=[]), lambda c: c["norm"].pop("eps"),
    lambda c: c["layers"][0].update(type="mlstm"), lambda c: c["layers"][0]["mixer"].pop("scale"), lambda c: c["layers"][0]["mixer"].update(heads=5),
    lambda c: c["layers"][1]["mixer"].update(vdim=10), lambda c: c["layers"][2]["mixer"]["q_temp"].update(every=0),
    lambda c: c["layers"][2]["mixer"]["q_temp"].pop("coef"), lambda c: c["layers"][0]["mlp"].update(kind="sparse"), lambda c: c["layers"][0]["mlp"].pop("ff")])
def test_bad_configurations_are_refused(change):
    cfg = copy.deepcopy(M.CONFIGS["odd"])
    change(cfg)
    with pytest.raises(GlintError, match="config.json"):
        S.dirozen_config(json.dumps(cfg))


def test_rows_in_groups_are_committed_by_whole_groups():
    MiB = 1 << 20
    # a group of 32 tokens is 3 MiB: the first token needs all of it, the 33rd another
    ctx = S.BookLayeredContext(100, [("rows", 3 * MiB // 32, 32)])
    assert ctx.append(0, 1) == (2, 0)
    assert ctx.append(1, 31) == (2, 0)
    assert ctx.append(32, 1) == (3, 0)
    assert ctx.append(33, 67) == (6, 0)          # 100 positions: four groups, 12 MiB
    # and what lies behind starts after the last whole group
    ctx = S.BookLayeredContext(33, [("rows", 65536, 32), ("rows", 16)])       # 4 MiB, then 528 bytes
    assert ctx.append(0, 1) == (2, 0)
    ctx = S.BookLayeredContext(33, [("rows", 65536), ("rows", 16)])           # 33 x 64 KiB: the second part is in the second block
    assert ctx.append(0, 1) == (2, 0)


def test_the_registry_knows_the_design(tmp_path):
    (tmp_path / "config.json").write_text('{"architecture": "Dirozen"}')
    with pytest.raises(GlintError, match="is missing"):
        S.DesignStage(str(tmp_path), "f32")


# ---- the plain implementation against itself and against the mechanisms it shares with another design ----
def test_plain_attention_continues():
    rng = np.random.default_rng(1)
    q, k = rng.standard_normal((30, 4, 6)), rng.standard_normal((30, 2, 6))
    whole = P.attention(q, k, 0.7, 0.4, 5, 1e-3)
    assert np.allclose(P.attention(q[17:], k, 0.7, 0.4, 5, 1e-3, first=17), whole[17:])
    # the same with the temperature and the norms taken out first
    t = np.array([P.query_temperature(p, 0.4, 5) for p in range(30)])[:, None, None]
    assert np.allclose(PF.windowed_attention(P.unit_rms(q, 1e-3) * t, P.unit_rms(k, 1e-3), k, 0.7, np.zeros((2, 4)), 9, 31, 0), whole)
    assert np.allclose(whole[0, :2], k[0, 0]) and np.allclose(whole[0, 2:], k[0, 1])          # one key: its value, unnormed


def test_plain_temperature():
    got = [P.query_temperature(p, 0.5, 4) for p in range(9)]
    want = 1 + 0.5 * np.log([1, 1, 1, 2, 2, 2, 2, 3, 3])
    assert np.allclose(got, want)


def test_plain_norm_and_gate():
    x = np.array([[3.0, -4.0]])
    assert np.allclose(P.rms_norm_around_zero(x, np.array([0.0, 1.0]), 0.0), [[3 / np.sqrt(12.5), -8 / np.sqrt(12.5)]])
    assert np.allclose(P.silu(np.array([0.0, 2.0])), [0, 2 / (1 + np.exp(-2))])


def test_needle_weights_show_the_needle():
    """What the far-key tests rest on: the one needle among hundreds of tokens changes the reader's logits, and only from the reader on."""
    cfg = M.CONFIGS["round"]
    w = M.with_needle(cfg, M.random_weights(cfg, 3), 5, 9)
    rng = np.random.default_rng(2)
    seq = rng.integers(10, cfg["vocab"], 200)
    seq[3], seq[150] = 9, 5
    other = seq.copy()
    other[3] = 11
    d = np.abs(P.forward(cfg, w, seq) - P.forward(cfg, w, other)).max(-1)
    assert d[150] > 0.5 and d[:3].max() == 0 and np.median(d[100:150]) < 0.5 * d[150]
