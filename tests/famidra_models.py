"""Small random Famidra models for the tests: configurations, weights (rounded to bf16, so that every path starts from the same numbers)
and a writer of the model directory."""
from __future__ import annotations

import json
import os
import struct

import numpy as np


def mlstm(heads, dim, vdim, cap=15.0, ff=None):
    return {"type": "mlstm", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}, "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def attention(heads, kv_heads, dim, vdim, window, keep, rows, bias_max, scale=None, ff=None):
    """`rows`: rows of the distance-bias table (a tensor's size, not part of config.json)."""
    return {"type": "attention", "mlp": None if ff is None else {"kind": "dense", "ff": ff}, "_rows": rows,
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "bias_max": bias_max, "scale": dim ** -0.5 if scale is None else scale,
                      "mask": {"size": window, "keep_first": keep}}}


def config(width, vocab, layers, loop, positions=512, eps=1e-5, logit_scale=1.0):
    return {"architecture": "Famidra", "width": width, "vocab": vocab, "max_positions": positions, "norm": {"eps": eps}, "logit_scale": logit_scale,
            "layers": layers, "loop": dict(zip(("start", "stop", "times"), loop))}


# sizes that are equal, 1 or a round number in many a model are none of it in at least one of these
CONFIGS = {
    # odd sizes everywhere, three passes over a middle run of layers, attention first
    "odd": config(52, 91, [attention(6, 2, 20, 12, 9, 3, 10, 23, ff=44), mlstm(3, 12, 20, cap=9.0), attention(2, 2, 9, 15, 5, 0, 7, 40), mlstm(1, 7, 5, ff=20)],
                  (1, 3, 3), positions=300, eps=3e-4, logit_scale=0.6),
    # sizes the matrix-core kernels take, grouped queries, the loop from the first layer on
    "round": config(128, 320, [mlstm(2, 64, 64, cap=6.0), attention(8, 2, 64, 32, 33, 5, 16, 64, ff=192), mlstm(4, 32, 96)], (0, 2, 2), logit_scale=0.4),
    # one head, one pass, one kept token, a window of many keys, the whole stack in the loop
    "plain": config(64, 200, [attention(1, 1, 128, 128, 150, 1, 32, 200, ff=80), mlstm(1, 128, 64)], (0, 2, 1), positions=600),
    # heads wider than the common kernels, a group of ten
    "wide": config(96, 150, [attention(10, 1, 136, 40, 12, 6, 8, 30, ff=52), mlstm(2, 300, 130), attention(4, 4, 24, 200, 70, 20, 12, 50)], (1, 2, 2), positions=400),
}


def to_bf16(a):
    bits = np.ascontiguousarray(a, dtype=np.float32).view(np.uint32)
    rounded = (bits + 0x7FFF + ((bits >> 16) & 1)) >> 16
    return (rounded << 16).astype(np.uint32).view(np.float32)


def random_weights(cfg, seed=0, rel_std=1.0, qk_gain=1.5):
    rng = np.random.default_rng(seed)
    W, V = cfg["width"], cfg["vocab"]

    def lin(out, inp, gain=1.0):
        return rng.standard_normal((out, inp)) * gain / np.sqrt(inp)

    def norm(n, gain=1.0):
        return gain * (1 + 0.2 * rng.standard_normal(n))

    w = {"embed": rng.standard_normal((V, W)), "pos": 0.4 * rng.standard_normal((cfg["max_positions"], W)), "final.norm": norm(W),
         "loop.in": lin(W, 2 * W, 1.4), "loop.step": 0.5 * rng.standard_normal((cfg["loop"]["times"], W))}
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        w[p + "norm1"], w[p + "norm1b"] = norm(W), norm(W)
        H, d, dv = m["heads"], m["dim"], m["vdim"]
        if layer["type"] == "mlstm":
            for n, rows in (("q", H * d), ("k", H * d), ("v", H * dv), ("g", H * dv)):
                w[p + "mix." + n] = lin(rows, W)
            w[p + "mix.i"], w[p + "mix.f"] = lin(H, W, 2.0), lin(H, W, 2.0)
            w[p + "mix.i.b"], w[p + "mix.f.b"] = rng.standard_normal(H), 3 + 2 * rng.standard_normal(H)
            w[p + "mix.norm"], w[p + "mix.o"] = norm(H * dv), lin(W, H * dv)
        else:
            G = m["kv_heads"]
            for n, rows in (("q", H * d), ("k", G * d), ("v", G * dv)):
                w[p + "mix." + n] = lin(rows, W)
                w[p + f"mix.{n}.b"] = 0.3 * rng.standard_normal(rows)
            w[p + "mix.q.norm"], w[p + "mix.k.norm"] = norm(H * d, qk_gain), norm(G * d, qk_gain)
            w[p + "mix.rel"], w[p + "mix.o"] = rel_std * rng.standard_normal((layer["_rows"], H)), lin(W, H * dv)
        if layer["mlp"] is not None:
            ff = layer["mlp"]["ff"]
            w[p + "norm2"], w[p + "norm2b"] = norm(W), norm(W)
            for n, rows, cols in (("gate", ff, W), ("up", ff, W), ("down", W, ff)):
                w[p + "mlp." + n], w[p + f"mlp.{n}.b"] = lin(rows, cols), 0.2 * rng.standard_normal(rows)
    return {k: to_bf16(a) for k, a in w.items()}


def write_model(path, cfg, weights, dtype="BF16", drop=()):
    """config.json and model.safetensors; `dtype` of the stored tensors, `drop`: tensors left out."""
    os.makedirs(path, exist_ok=True)
    clean = dict(cfg, layers=[{k: v for k, v in layer.items() if not k.startswith("_")} for layer in cfg["layers"]])
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(clean, f)
    header, blobs, at = {}, [], 0
    for name, a in weights.items():
        if name in drop:
            continue
        a = np.ascontiguousarray(a, dtype=np.float32)
        blob = (a.view(np.uint32) >> 16).astype(np.uint16).tobytes() if dtype == "BF16" else a.tobytes()
        header[name] = {"dtype": dtype, "shape": list(a.shape), "data_offsets": [at, at + len(blob)]}
        blobs.append(blob)
        at += len(blob)
    raw = json.dumps(header).encode()
    with open(os.path.join(path, "model.safetensors"), "wb") as f:
        f.write(struct.pack("<Q", len(raw)) + raw + b"".join(blobs))
    return str(path)
