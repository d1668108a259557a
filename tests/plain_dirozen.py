"""Plain, slow implementation of the Dirozen design in numpy: one function per mechanism, a loop over positions and heads where it is an
attention.  It shares no code with the product; the GPU tests compare against it.  `dt` picks the precision everything is computed in
(float64 by default)."""
from __future__ import annotations

import numpy as np


def unit_rms(x, eps):
    """x over its root mean square along the last axis."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def rms_norm_around_zero(x, w, eps):
    return unit_rms(x, eps) * (1 + w)


def sigmoid(z):
    return 1 / (1 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def query_temperature(p, coef, every):
    """Factor of a query at position p: grows with the logarithm of how many whole stretches of `every` tokens end at or before it."""
    return 1 + coef * np.log((p + 1) // every + 1)


def softmax(score):
    w = np.exp(score - score.max())
    return w / w.sum()


def read_keys(query, k, eps, scale):
    """query (d) as it meets the keys, k (n, d) the visible keys as projected: their mean under the softmax of the scores, taken of the
    keys before their norm."""
    return softmax((unit_rms(k, eps) @ query) * scale) @ k


def attention(q, k, scale, coef, every, eps, first=0):
    """q (T, H, d) of positions first .. first + T - 1, k (first + T, G, d) of the whole sequence, both as projected.  Returns (T, H, d)."""
    T, H, _ = q.shape
    per = H // k.shape[1]
    out = np.zeros_like(q)
    for t in range(T):
        p = first + t
        for h in range(H):
            query = unit_rms(q[t, h], eps) * query_temperature(p, coef, every)
            out[t, h] = read_keys(query, k[: p + 1, h // per], eps, scale)
    return out


def attention_mixer(h, w, mix, eps):
    """h (T, width); w: tensor name without the mixer's prefix -> array."""
    T, H, G, d = h.shape[0], mix["heads"], mix["kv_heads"], mix["dim"]
    q, k = (h @ w["q"].T).reshape(T, H, d), (h @ w["k"].T).reshape(T, G, d)
    o = attention(q, k, mix["scale"], mix["q_temp"]["coef"], mix["q_temp"]["every"], eps)
    o = o * sigmoid(h @ w["g"].T)[:, :, None]
    return o.reshape(T, H * d) @ w["o"].T


def feed_forward(h, w):
    return (silu(h @ w["gate"].T) * (h @ w["up"].T)) @ w["down"].T


def sub(weights, prefix):
    return {k[len(prefix):]: a for k, a in weights.items() if k.startswith(prefix)}


def forward(config, weights, tokens, dt=np.float64, residuals=None):
    """Logits (T, vocab) of one sequence from its first token on; `residuals` (a list) gets the stream behind every layer."""
    w = {k: np.asarray(a).astype(dt) for k, a in weights.items()}
    eps = config["norm"]["eps"]
    x = w["embed"][np.asarray(tokens)]
    for i, layer in enumerate(config["layers"]):
        h = rms_norm_around_zero(x, w[f"l{i}.norm1"], eps)
        y = attention_mixer(h, sub(w, f"l{i}.mix."), layer["mixer"], eps)
        if layer["mlp"] is not None:
            y = y + feed_forward(h, sub(w, f"l{i}.mlp."))
        x = x + y
        if residuals is not None:
            residuals.append(x)
    return rms_norm_around_zero(x, w["final.norm"], eps) @ w["head"].T
