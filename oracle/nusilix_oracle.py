"""Slow NumPy restatement of the Nusilix decoder, for tests only: one function per mechanism, float64 throughout, whole
sequences at a time, no caches and no shared code with the library.

Notation: x is [T, width], one row per position p = 0 .. T - 1.  Weights are a dict name -> array, matrices [out, in].
"""
from __future__ import annotations

import numpy as np


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def softplus(z):
    return np.logaddexp(0.0, z)


def sinusoid(positions, width):
    """Column 2i: sin(p * 10000^(-2i / width)), column 2i + 1: the cosine of the same angle."""
    col = np.arange(width)
    angle = np.asarray(positions, dtype=np.float64)[:, None] * 10000.0 ** (-(col // 2 * 2) / width)
    return np.where(col % 2 == 0, np.sin(angle), np.cos(angle))


def rms_norm(x, w, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * w


def grouped_rms_norm(x, w, eps, groups):
    parts = x.reshape(*x.shape[:-1], groups, x.shape[-1] // groups)
    parts = parts / np.sqrt(np.mean(parts * parts, axis=-1, keepdims=True) + eps)
    return parts.reshape(x.shape) * w


def query_temperature(positions, coef, every):
    p = np.asarray(positions, dtype=np.float64)
    return 1.0 + coef * np.log(np.floor((p + 1.0) / every) + 1.0)


def distance_slopes(heads):
    return 2.0 ** (-8.0 * (np.arange(heads) + 1.0) / heads)


def shared_kv_attention(q, k_rows, v_rows, scale, slopes, first_pos):
    """q [T, H, D] at positions first_pos + t, k_rows / v_rows [N, G, D] at positions 0 .. N - 1; causal softmax with
    slope_h * distance taken off the scaled scores."""
    T, H, _ = q.shape
    N, G, _ = k_rows.shape
    out = np.zeros((T, H, v_rows.shape[2]))
    for h in range(H):
        g = h // (H // G)
        dist = (first_pos + np.arange(T))[:, None] - np.arange(N)[None, :]
        s = (q[:, h] @ k_rows[:, g].T) * scale - slopes[h] * dist
        s = np.where(dist >= 0, s, -np.inf)
        e = np.exp(s - s.max(axis=1, keepdims=True))
        out[:, h] = (e / e.sum(axis=1, keepdims=True)) @ v_rows[:, g]
    return out


def attention_mixer(h, w, pre, m, eps):
    T = h.shape[0]
    H, G, D = m["heads"], m["kv_heads"], m["dim"]
    q = h @ w[pre + "q"].T + w[pre + "q.b"]
    k = h @ w[pre + "k"].T + w[pre + "k.b"]
    v = k
    q = rms_norm(q, w[pre + "q.norm"], eps)
    k = rms_norm(k, w[pre + "k.norm"], eps)
    if m.get("q_temp"):
        q = q * query_temperature(np.arange(T), m["q_temp"]["coef"], m["q_temp"]["every"])[:, None]
    o = shared_kv_attention(q.reshape(T, H, D), k.reshape(T, G, D), v.reshape(T, G, D), m["scale"], distance_slopes(H), 0)
    return o.reshape(T, H * D) @ w[pre + "o"].T + w[pre + "o.b"]


def delta_decay(z, w0):
    return np.exp(-np.exp(-0.5) * sigmoid(z + w0))


def unit_key(k):
    return k / np.sqrt(np.sum(k * k, axis=-1, keepdims=True) + 1e-6)


def generalized_delta_rule(r, k, v, decay, rate, state=None):
    """All [T, H, D]; state [H, D (key), D (value)].  Returns outputs [T, H, D] and the state after the last token."""
    T, H, D = r.shape
    S = np.zeros((H, D, v.shape[2])) if state is None else np.array(state, dtype=np.float64)
    out = np.zeros(v.shape)
    u = unit_key(k)
    for t in range(T):
        for h in range(H):
            old = S[h]
            S[h] = decay[t, h][:, None] * old - np.outer(rate[t, h] * u[t, h], u[t, h] @ old) + np.outer(k[t, h], v[t, h])
            out[t, h] = S[h].T @ r[t, h]
    return out, S


def delta_mixer(h, w, pre, m, eps):
    T = h.shape[0]
    H, D = m["heads"], m["dim"]
    r, k, v = (h @ w[pre + n].T for n in ("r", "k", "v"))
    decay = delta_decay(np.tanh(h @ w[pre + "w1"].T) @ w[pre + "w2"].T, w[pre + "w0"])
    rate = sigmoid(h @ w[pre + "a"].T + w[pre + "a.b"])
    o, _ = generalized_delta_rule(*(z.reshape(T, H, D) for z in (r, k, v, decay, rate)))
    o = o / np.sqrt(np.mean(o * o, axis=-1, keepdims=True) + eps)
    o = o.reshape(T, H * D) * w[pre + "norm"] * sigmoid(h @ w[pre + "g"].T)
    return o @ w[pre + "o"].T


def xielu(z, p, q):
    neg = np.minimum(z, 0.0)
    return np.where(z > 0, softplus(p) * z * z, (0.5 + softplus(q)) * (np.expm1(neg) - neg)) + 0.5 * z


def feed_forward(h, w, pre):
    p, q = w[pre + "act"]
    return xielu(h @ w[pre + "up"].T, p, q) @ w[pre + "down"].T


def forward(cfg, weights, tokens, collect=None):
    """cfg: the dictionary of config.json.  Logits [T, vocab] of one sequence; collect receives x after every layer."""
    w = {k: np.asarray(v, dtype=np.float64) for k, v in weights.items()}
    tokens = np.asarray(tokens)
    eps, groups = cfg["norm"]["eps"], cfg["norm"]["groups"]
    x = w["embed"][tokens] + sinusoid(np.arange(len(tokens)), cfg["width"])
    for i, layer in enumerate(cfg["layers"]):
        h = grouped_rms_norm(x, w[f"l{i}.norm1"], eps, groups)
        mixer = {"attention": attention_mixer, "general_delta": delta_mixer}[layer["type"]]
        y = mixer(h, w, f"l{i}.mix.", layer["mixer"], eps)
        if layer.get("mlp"):
            y = y + feed_forward(h, w, f"l{i}.mlp.")
        x = x + cfg["residual_mult"] * y
        if collect is not None:
            collect.append(x.copy())
    return grouped_rms_norm(x, w["final.norm"], eps, groups) @ w["head"].T
