"""Small random Dirozen models for the tests: configurations and weights, rounded to bf16 so that every path starts from the same numbers."""
from __future__ import annotations

import numpy as np

from famidra_models import to_bf16, write_model  # noqa: F401  (the model directory's format is the designs' common one)


def layer(heads, kv_heads, dim, every, coef=0.35, ff=None, scale=None):
    return {"type": "attention", "mlp": None if ff is None else {"kind": "dense", "ff": ff},
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": 1.1 * dim ** -0.5 if scale is None else scale,
                      "q_temp": {"coef": coef, "every": every}}}


def config(width, vocab, layers, eps=1e-5):
    return {"architecture": "Dirozen", "width": width, "vocab": vocab, "norm": {"eps": eps}, "layers": layers}


# sizes that are equal, 1 or a round number in many a model are none of it in at least one of these
CONFIGS = {
    # odd sizes everywhere, layers of unlike shapes, one without a feed-forward
    "odd": config(52, 91, [layer(6, 2, 20, 7, 0.25, ff=44), layer(3, 3, 9, 50, 0.9), layer(4, 1, 15, 1, 0.1, ff=21)], eps=3e-3),
    # sizes the matrix-core kernels take, grouped queries
    "round": config(128, 320, [layer(8, 2, 64, 32, ff=192), layer(4, 4, 32, 40, 0.5, ff=128), layer(2, 1, 128, 16)]),
    # one head, one layer with and one without a feed-forward of its width
    "plain": config(64, 200, [layer(1, 1, 128, 24, 0.0, ff=64), layer(1, 1, 64, 100, 1.2)], eps=1e-6),
    # head sizes between the kernels' steps
    "between": config(80, 150, [layer(12, 3, 88, 20, 0.4, ff=72), layer(6, 6, 72, 9, 0.2, ff=40), layer(32, 1, 104, 64, 0.8, ff=88)]),
    # heads wider than the common kernels, a group of ten
    "wide": config(96, 150, [layer(10, 1, 136, 12, ff=52), layer(2, 2, 300, 33, 0.7, ff=48), layer(4, 2, 260, 5)], eps=1e-3),
}


def random_weights(cfg, seed=0):
    rng = np.random.default_rng(seed)
    W, V = cfg["width"], cfg["vocab"]

    def lin(out, inp, gain=1.0):
        return rng.standard_normal((out, inp)) * gain / np.sqrt(inp)

    def norm(n):
        return 0.2 * rng.standard_normal(n)

    w = {"embed": rng.standard_normal((V, W)), "head": lin(V, W), "final.norm": norm(W)}
    for i, spec in enumerate(cfg["layers"]):
        p, m = f"l{i}.", spec["mixer"]
        H, G, d = m["heads"], m["kv_heads"], m["dim"]
        w[p + "norm1"] = norm(W)
        w[p + "mix.q"], w[p + "mix.k"], w[p + "mix.g"], w[p + "mix.o"] = lin(H * d, W), lin(G * d, W), lin(H, W, 2.0), lin(W, H * d, 1.5)
        if spec["mlp"] is not None:
            ff = spec["mlp"]["ff"]
            w[p + "mlp.gate"], w[p + "mlp.up"], w[p + "mlp.down"] = lin(ff, W), lin(ff, W), lin(W, ff)
    return {k: to_bf16(a) for k, a in w.items()}


def with_needle(cfg, weights, reader, needle, gain=6.0):
    """Weights whose first layer makes every head of token `reader` look for token `needle`, wherever that is."""
    w = dict(weights)
    m = cfg["layers"][0]["mixer"]
    H, G, d = m["heads"], m["kv_heads"], m["dim"]
    rng = np.random.default_rng(1)
    u = rng.standard_normal((G, d))
    u /= np.linalg.norm(u, axis=-1, keepdims=True)

    def direction(token):          # what the first layer sees of a token, as a vector that reads 1 there
        e = weights["embed"][token].astype(np.float64)
        h = e / np.sqrt(np.mean(e * e)) * (1 + weights["l0.norm1"])
        return h / (h @ h)

    u_q = np.repeat(u, H // G, axis=0).reshape(-1)
    w["l0.mix.q"] = to_bf16(weights["l0.mix.q"] + gain * np.sqrt(d) * np.outer(u_q, direction(reader)))
    w["l0.mix.k"] = to_bf16(weights["l0.mix.k"] + gain * np.sqrt(d) * np.outer(u.reshape(-1), direction(needle)))
    w["l0.mix.g"] = to_bf16(0.2 * weights["l0.mix.g"])
    return w
