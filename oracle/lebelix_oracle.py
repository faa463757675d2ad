"""Slow NumPy restatement of the Lebelix decoder, for tests only: one function per mechanism, float64 throughout, whole sequences at
a time, no caches and no shared code with the library.

Notation: x is [T, width], one row per position p = 0 .. T - 1.  Weights are a dict name -> array, matrices [out, in].
"""
from __future__ import annotations

import numpy as np

UNIT_EPS = 1e-6


def sigmoid(z):
    return 0.5 * (1.0 + np.tanh(0.5 * z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.logaddexp(0.0, z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(np.sqrt(2.0 / np.pi) * (z + 0.044715 * z ** 3)))


def rms(x, eps):
    """The divisor of an RMS norm over the last axis."""
    return np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def offset_norm(x, w, eps):
    """The model's norm: its weights are stored around zero."""
    return x / rms(x, eps) * (1.0 + w)


def plain_norm(x, w, eps):
    return x / rms(x, eps) * w


def unit(x):
    return x / np.sqrt(np.sum(x * x, axis=-1, keepdims=True) + UNIT_EPS)


def rotate_half(x, positions, base, dims):
    """x [T, ..., D]: elements i and i + dims / 2 of the first `dims` turn by p * base^(-2i / dims)."""
    half = dims // 2
    freq = float(base) ** (-2.0 * np.arange(half) / dims)
    angle = np.asarray(positions, dtype=np.float64).reshape(-1, *([1] * (x.ndim - 1))) * freq
    u, v = x[..., :half], x[..., half:dims]
    return np.concatenate([u * np.cos(angle) - v * np.sin(angle), v * np.cos(angle) + u * np.sin(angle), x[..., dims:]], axis=-1)


def window_mask(T, size):
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    return (j <= i) & (i - j < size)


def chunk_mask(T, size):
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    return (j <= i) & (i // size == j // size)


def soft_cap(s, cap):
    return cap * np.tanh(s / cap)


def softmax(s, mask):
    e = np.where(mask, np.exp(s - np.where(mask, s, -np.inf).max(axis=-1, keepdims=True)), 0.0)
    return e / e.sum(axis=-1, keepdims=True)


def sink_softmax(s, mask):
    """A sink of score 0 takes its share of the weights and gives no value."""
    m = np.maximum(np.where(mask, s, -np.inf).max(axis=-1, keepdims=True), 0.0)
    e = np.where(mask, np.exp(np.where(mask, s, 0.0) - m), 0.0)
    return e / (np.exp(-m) + e.sum(axis=-1, keepdims=True))


def heads_first(x):
    """[T, H, D] to [H, T, D], and back"""
    return np.swapaxes(x, 0, 1)


def causal_conv(x, taps):
    """x [T, C], taps [C, K]: the last column of taps meets the token itself, zeros lie before the start."""
    K = taps.shape[1]
    padded = np.concatenate([np.zeros((K - 1, x.shape[1])), x])
    return sum(padded[j:j + len(x)] * taps[:, j] for j in range(K))


def channel_decay(z, a_log, dt_bias):
    """z [T, H, D] -> the factors of the key channels; a_log [H], dt_bias [H, D]."""
    return np.exp(-np.exp(a_log)[:, None] * softplus(z + dt_bias))


def gated_delta_rule(q, k, v, decay, rate, state=None):
    """q, k, decay [T, H, D], v [T, H, V], rate [T, H]; state [H, D, V].  -> outputs [T, H, V], the state after the last token."""
    T, H, D = q.shape
    S = np.zeros((H, D, v.shape[2])) if state is None else np.array(state, dtype=np.float64)
    out = np.zeros(v.shape)
    for t in range(T):
        S = decay[t][:, :, None] * S
        u = rate[t][:, None] * (v[t] - np.einsum("hdv,hd->hv", S, k[t]))
        S = S + k[t][:, :, None] * u[:, None, :]
        out[t] = np.einsum("hdv,hd->hv", S, q[t])
    return out, S


def channel_delta_mixer(h, w, pre, m, eps, shared=None):
    T, H, G, D, V = len(h), m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (silu(causal_conv(h @ w[pre + n].T, w[pre + n + ".conv"])) for n in ("q", "k", "v"))
    of_head = np.arange(H) // (H // G)
    q = unit(q.reshape(T, G, D))[:, of_head] * D ** -0.5
    k = unit(k.reshape(T, G, D))[:, of_head]
    rate = sigmoid(h @ w[pre + "b"].T)
    z = ((h @ w[pre + "a1"].T) @ w[pre + "a2"].T).reshape(T, H, D)
    decay = channel_decay(z, w[pre + "A_log"], w[pre + "dt_bias"].reshape(H, D))
    o, _ = gated_delta_rule(q, k, v.reshape(T, H, V), decay, rate)
    o = plain_norm(o, w[pre + "norm"], eps)
    gate = sigmoid((h @ w[pre + "g1"].T) @ w[pre + "g2"].T)
    return (o.reshape(T, H * V) * gate) @ w[pre + "o"].T


def latent_row(h, w, pre, m, eps):
    """What a token leaves behind: its latent and its rotated key part."""
    d = h @ w[pre + "dkv"].T
    c = plain_norm(d[:, :m["kv_rank"]], w[pre + "dkv.norm"], eps)
    return c, rotate_half(d[:, m["kv_rank"]:], np.arange(len(h)), m["rot"]["base"], m["rot_dim"])


def latent_attention_mixer(h, w, pre, m, eps, shared=None):
    T, H, D, R, V = len(h), m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    q = (h @ w[pre + "q"].T).reshape(T, H, D + R)
    q_rot = rotate_half(q[..., D:], np.arange(T), m["rot"]["base"], R)
    c, k_rot = shared if shared is not None else latent_row(h, w, pre, m, eps)
    k = (c @ w[pre + "uk"].T).reshape(T, H, D)
    v = (c @ w[pre + "uv"].T).reshape(T, H, V)
    s = (heads_first(q[..., :D]) @ heads_first(k).swapaxes(1, 2) + heads_first(q_rot) @ k_rot.T) * m["scale"]
    p = softmax(s, window_mask(T, m["mask"]["size"]))
    return heads_first(p @ heads_first(v)).reshape(T, H * V) @ w[pre + "o"].T


def attention_mixer(h, w, pre, m, eps, shared=None):
    T, H, G, D, V = len(h), m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (h @ w[pre + n].T + w[pre + n + ".b"] for n in ("q", "k", "v"))
    q = plain_norm(q.reshape(T, H, D), w[pre + "q.norm"], eps)
    k = plain_norm(k.reshape(T, G, D), w[pre + "k.norm"], eps)
    q, k = (rotate_half(x, np.arange(T), m["rot"]["base"], m["rot"]["dims"]) for x in (q, k))
    of_head = np.arange(H) // (H // G)
    s = soft_cap(heads_first(q) @ heads_first(k[:, of_head]).swapaxes(1, 2) * m["scale"], m["softcap"])
    p = sink_softmax(s, chunk_mask(T, m["mask"]["size"]))
    o = heads_first(p @ heads_first(v.reshape(T, G, V)[:, of_head])).reshape(T, H * V)
    return (o * sigmoid(h @ w[pre + "g"].T)) @ w[pre + "o"].T


MIXERS = {"attention": attention_mixer, "latent_attention": latent_attention_mixer, "channel_delta": channel_delta_mixer}


def feed_forward(h, w, pre):
    return gelu_tanh(h @ w[pre + "up"].T) @ w[pre + "down"].T


def token_side(x, e, w, pre, eps):
    """What a layer adds from the token's own row e [T, dim] of the side table."""
    return plain_norm((gelu_tanh(x @ w[pre + "gate"].T) * e) @ w[pre + "proj"].T, w[pre + "norm"], eps)


def forward(cfg, weights, tokens, collect=None):
    """cfg: the dictionary of config.json.  Logits [T, vocab] of one sequence; collect receives x after every layer."""
    w = {k: np.asarray(v, dtype=np.float64) for k, v in weights.items()}
    tokens = np.asarray(tokens)
    eps, n_side = cfg["norm"]["eps"], cfg["token_side"]["dim"]
    x = w["embed"][tokens] * cfg["embedding"]["scale"]
    rows = {}  # latents by layer
    for i, layer in enumerate(cfg["layers"]):
        m, p = layer["mixer"], f"l{i}."
        h = offset_norm(x, w[p + "norm1"], eps)
        shared = None
        if layer["type"] == "latent_attention":
            if m.get("kv_from") is None:
                rows[i] = latent_row(h, w, p + "mix.", m, eps)
            shared = rows[i if m.get("kv_from") is None else m["kv_from"]]
        x = x + MIXERS[layer["type"]](h, w, p + "mix.", m, eps, shared)
        if layer.get("mlp"):
            x = x + feed_forward(offset_norm(x, w[p + "norm2"], eps), w, p + "mlp.")
        x = x + token_side(x, w["side.embed"][tokens, i * n_side:(i + 1) * n_side], w, p + "side.", eps)
        if collect is not None:
            collect.append(x.copy())
    return offset_norm(x, w["final.norm"], eps) @ w["embed"].T
