"""Prefill and decode throughput of Nusilix models with layers of a real model's sizes (random weights), each beside the
Llama-style Q4_K decoder of equal width, feed-forward, heads and layer count."""
from __future__ import annotations

import time

import numpy as np

from . import llama, nusilix
from .safetensors import f32_to_bf16

HBM_PEAK = 8.0e12
BF16_PEAK = 2.5e15

# name -> (width, feed-forward, attention heads, kv heads, head size, delta heads, their size, rank, layers)
SIZES = {
    "2048": (2048, 8192, 32, 8, 64, 32, 64, 64, 8),
    "4096": (4096, 14336, 32, 8, 128, 64, 64, 128, 4),
}
VOCAB = 32000


def config(size, kinds="both", max_tokens=8192):
    """kinds: "attention", "general_delta", or "both" (alternating)."""
    w, ff, h, kv, d, dh, dd, _, n = SIZES[size]
    attn = nusilix.Layer("attention", heads=h, dim=d, kv_heads=kv, scale=d ** -0.5, temp_coef=0.1, temp_every=1024, ff=ff)
    delta = nusilix.Layer("general_delta", heads=dh, dim=dd, ff=ff)
    pick = {"attention": [attn], "general_delta": [delta], "both": [attn, delta]}[kinds]
    return nusilix.Config(width=w, vocab=VOCAB, norm_groups=4, norm_eps=1e-6, residual_mult=0.5, layers=[pick[i % len(pick)] for i in range(n)],
                          max_tokens=max_tokens)


def random_source(shapes, seed=7):
    """source(name) of a model with these tensors: bfloat16 patterns cut out of one random block, matrices scaled by 1 / sqrt(columns)."""
    rng = np.random.default_rng(seed)
    block = rng.standard_normal(1 << 22).astype(np.float32)
    scaled = {}

    def source(name):
        shape = shapes[name]
        if len(shape) == 1:
            v = 1.0 + 0.1 * rng.standard_normal(shape) if "norm" in name else 0.1 * rng.standard_normal(shape)
            return v.astype(np.float32)
        if shape[1] not in scaled:
            scaled[shape[1]] = f32_to_bf16(block / np.sqrt(shape[1]))
        b = np.roll(scaled[shape[1]], int(rng.integers(1 << 22)))
        return np.resize(b, shape)

    return source


def decode_bytes(cfg, model, ctx_tokens):
    """Bytes one decode step has to move: weights once, cached rows once, recurrent states in and out."""
    total = model.weight_bytes
    for layer in cfg.layers:
        if layer.mixer == "attention":
            total += ctx_tokens * (layer.kv_heads * layer.dim * 2 + 4)
        else:
            total += 2 * layer.heads * layer.dim * layer.dim * 4
    return total


def prompt_flops(cfg, rank, n):
    """Matrix products of the layers plus the two products of causal attention."""
    total = 0
    for name, s in nusilix.tensor_shapes(cfg, rank).items():
        if len(s) == 2 and name not in ("embed", "head"):
            total += 2 * s[0] * s[1] * n
    for layer in cfg.layers:
        if layer.mixer == "attention":
            total += 4 * n * (n + 1) // 2 * layer.columns
    return total


def timed(ctx, fn, reps):
    fn()
    ctx.sync()
    best = 1e9
    for _ in range(reps):
        t0 = time.perf_counter()
        fn()
        ctx.sync()
        best = min(best, time.perf_counter() - t0)
    return best


def measure(ctx, model, prompts, contexts, steps, rng, vocab):
    out = {}
    for n in prompts:
        prompt = rng.integers(0, vocab, n).tolist()

        def prefill():
            model.reset()
            model.prefill(prompt)

        out[f"prefill_{n}"] = timed(ctx, prefill, 3)
    for n in contexts:
        model.reset()
        first = model.prefill(rng.integers(0, vocab, n).tolist())
        model.decode(first, 8)  # (captures the step)
        ctx.sync()
        t0 = time.perf_counter()
        model.decode(first, steps)
        ctx.sync()
        out[f"decode_{n}"] = (time.perf_counter() - t0) / steps
    return out


def run(ctx, size, kinds="both", prompts=(512, 2048), contexts=(512, 4096), steps=64, beside=True):
    """kinds: as in config, or "llama" for the Llama-style decoder alone."""
    if kinds == "llama":
        return run_llama(ctx, size, prompts, contexts, steps)
    _, _, _, _, _, _, _, rank, n_layer = SIZES[size]
    cfg = config(size, kinds)
    model = nusilix.NusilixModel(ctx, cfg, random_source(nusilix.tensor_shapes(cfg, rank)))
    t = measure(ctx, model, prompts, contexts, steps, np.random.default_rng(3), VOCAB)
    out = {"layers": f"{n_layer} x {kinds}", "weight_mb": round(model.weight_bytes / 1e6, 1)}
    report(out, t, {n: prompt_flops(cfg, rank, n) for n in prompts}, {n: decode_bytes(cfg, model, n + steps / 2) for n in contexts})
    model.free()
    if beside:
        out["llama_q4_k_beside"] = run_llama(ctx, size, prompts, contexts, steps)
    return out


def run_llama(ctx, size, prompts, contexts, steps):
    """The Llama-style Q4_K decoder of equal width, feed-forward, heads and layer count."""
    w, ff, h, kv, d, _, _, _, n_layer = SIZES[size]
    cfg = llama.Config(n_layer=n_layer, hidden=w, ffn=ff, n_head=h, head_dim=d, vocab=VOCAB, max_tokens=8192, n_kv_head=kv)
    model = llama.LlamaModel(ctx, cfg, seed=5)
    t = measure(ctx, model, prompts, contexts, steps, np.random.default_rng(3), VOCAB)
    weights = model.weight_bytes_per_token()
    out = {"weight_mb": round(weights / 1e6, 1)}
    params = n_layer * (2 * w * w + 2 * w * kv * d + 3 * w * ff)
    report(out, t, {n: 2 * params * n + n_layer * 4 * n * (n + 1) // 2 * w for n in prompts},
            {n: weights + n_layer * (n + steps / 2) * 2 * 2 * kv * d for n in contexts})
    model.free()
    return out


def report(out, t, flops, nbytes):
    for n, f in flops.items():
        s = t[f"prefill_{n}"]
        out[f"prefill_{n}"] = {"ms": round(s * 1e3, 3), "tok_s": round(n / s, 1), "frac_bf16_peak": round(f / s / BF16_PEAK, 4)}
    for n, b in nbytes.items():
        s = t[f"decode_{n}"]
        out[f"decode_at_{n}"] = {"ms": round(s * 1e3, 4), "tok_s": round(1 / s, 1), "frac_hbm_peak": round(b / HBM_PEAK / s, 4)}
