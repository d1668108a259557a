"""Plain, slow implementation of the Famidra design in numpy: one function per mechanism, one token at a time where the
mechanism is a recurrence, a loop over visible keys where it is an attention.  It shares no code with the product; the
GPU tests compare against it.  `dt` picks the precision everything is computed in (float64 by default)."""
from __future__ import annotations

import numpy as np


def rms_norm(x, eps, weight=None):
    y = x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)
    return y if weight is None else y * weight


def gelu_tanh(z):
    return 0.5 * z * (1 + np.tanh(np.sqrt(2 / np.pi) * (z + 0.044715 * z ** 3)))


def log_sigmoid(z):
    return -np.logaddexp(0.0, -z)


def soft_cap(z, cap):
    return cap * np.tanh(z / cap)


def distance_bucket(n, rows, bias_max):
    """Which row of a distance-bias table of `rows` rows a distance n falls into: one row a distance up to half of them, then
    rows that widen with the logarithm; everything from bias_max on (and a little before) in the last one."""
    half = rows // 2
    if n < half:
        return n
    return min(rows - 1, half + int(np.floor(np.log(n / half) / np.log(bias_max / half) * (rows - half) + 1e-9)))


def visible(i, j, window, keep_first):
    return j <= i and (i - j < window or j < keep_first)


def windowed_attention(q, k, v, scale, rel, bias_max, window, keep_first):
    """q (T, H, d), k (T, G, d), v (T, G, dv) of one whole sequence -> (T, H, dv)."""
    T, H, _ = q.shape
    group = H // k.shape[1]
    out = np.zeros((T, H, v.shape[2]), dtype=q.dtype)
    for i in range(T):
        js = [j for j in range(i + 1) if visible(i, j, window, keep_first)]
        rows = [distance_bucket(i - j, rel.shape[0], bias_max) for j in js]
        for h in range(H):
            g = h // group
            score = (k[js, g] @ q[i, h]) * scale + rel[rows, h]
            p = np.exp(score - score.max())
            out[i, h] = (p / p.sum()) @ v[js, g]
    return out


def mlstm_recurrence(q, k, v, log_i, log_f, state=None):
    """q, k (T, H, d), v (T, H, dv), log gates (T, H); q already scaled.  Returns (T, H, dv) and the state (S, n, m) behind the last token."""
    T, H, d = q.shape
    dv = v.shape[2]
    if state is None:
        state = (np.zeros((H, d, dv), q.dtype), np.zeros((H, d), q.dtype), np.zeros(H, q.dtype))
    S, n, m = (a.copy() for a in state)
    out = np.zeros((T, H, dv), q.dtype)
    for t in range(T):
        m_new = np.maximum(log_f[t] + m, log_i[t])
        decay = np.exp(log_f[t] + m - m_new)
        inp = np.exp(log_i[t] - m_new)
        S = decay[:, None, None] * S + inp[:, None, None] * k[t][:, :, None] * v[t][:, None, :]
        n = decay[:, None] * n + inp[:, None] * k[t]
        m = m_new
        num = np.einsum("hdv,hd->hv", S, q[t])
        den = np.maximum(np.abs(np.sum(n * q[t], axis=-1)), np.exp(-m)) + 1e-6
        out[t] = num / den[:, None]
    return out, (S, n, m)


def mlstm_mixer(h, w, mix, eps):
    """h (T, width); w: tensor name without the layer's prefix -> array."""
    T = h.shape[0]
    H, d, dv, cap = mix["heads"], mix["dim"], mix["vdim"], mix["gate_cap"]
    q = (h @ w["q"].T).reshape(T, H, d) * h.dtype.type(d) ** -0.5
    k = (h @ w["k"].T).reshape(T, H, d)
    v = (h @ w["v"].T).reshape(T, H, dv)
    log_i = soft_cap(h @ w["i"].T + w["i.b"], cap)
    log_f = log_sigmoid(soft_cap(h @ w["f"].T + w["f.b"], cap))
    o, _ = mlstm_recurrence(q, k, v, log_i, log_f)
    o = rms_norm(o, eps).reshape(T, H * dv) * w["norm"]
    return (o / (1 + np.exp(-(h @ w["g"].T)))) @ w["o"].T


def attention_mixer(h, w, mix, eps):
    T = h.shape[0]
    H, G, d, dv = mix["heads"], mix["kv_heads"], mix["dim"], mix["vdim"]
    q = rms_norm(h @ w["q"].T + w["q.b"], eps, w["q.norm"]).reshape(T, H, d)
    k = rms_norm(h @ w["k"].T + w["k.b"], eps, w["k.norm"]).reshape(T, G, d)
    v = (h @ w["v"].T + w["v.b"]).reshape(T, G, dv)
    o = windowed_attention(q, k, v, mix["scale"], w["rel"], mix["bias_max"], mix["mask"]["size"], mix["mask"]["keep_first"])
    return o.reshape(T, H * dv) @ w["o"].T


def feed_forward(h, w):
    return (gelu_tanh(h @ w["gate"].T + w["gate.b"]) * (h @ w["up"].T + w["up.b"])) @ w["down"].T + w["down.b"]


def run_order(n_layers, loop):
    """(layer, pass or None, first layer of its pass) in the order the layers run."""
    order = [(i, None, False) for i in range(loop["start"])]
    for t in range(loop["times"]):
        order += [(i, t, i == loop["start"]) for i in range(loop["start"], loop["stop"])]
    return order + [(i, None, False) for i in range(loop["stop"], n_layers)]


def sub(weights, prefix):
    return {k[len(prefix):]: a for k, a in weights.items() if k.startswith(prefix)}


def forward(config, weights, tokens, dt=np.float64, residuals=None):
    """Logits (T, vocab) of one sequence from its first token on; `residuals` (a list) gets the stream behind every layer run."""
    w = {k: np.asarray(a).astype(dt) for k, a in weights.items()}
    eps = config["norm"]["eps"]
    x = w["embed"][np.asarray(tokens)] + w["pos"][: len(tokens)]
    x0 = x
    for i, t, first in run_order(len(config["layers"]), config["loop"]):
        layer = config["layers"][i]
        if first:
            x = np.concatenate([x, x0], axis=-1) @ w["loop.in"].T + w["loop.step"][t]
        mixer = {"mlstm": mlstm_mixer, "attention": attention_mixer}[layer["type"]]
        y = mixer(rms_norm(x, eps, w[f"l{i}.norm1"]), sub(w, f"l{i}.mix."), layer["mixer"], eps)
        x = x + rms_norm(y, eps, w[f"l{i}.norm1b"])
        if layer["mlp"] is not None:
            y = feed_forward(rms_norm(x, eps, w[f"l{i}.norm2"]), sub(w, f"l{i}.mlp."))
            x = x + rms_norm(y, eps, w[f"l{i}.norm2b"])
        if residuals is not None:
            residuals.append(x)
    return rms_norm(x, eps, w["final.norm"]) @ w["embed"].T * config["logit_scale"]
