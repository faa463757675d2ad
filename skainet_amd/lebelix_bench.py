"""Prefill and decode throughput of Lebelix models with layers of a real model's sizes (random weights), each beside a Nusilix decoder
of equal width, feed-forward, attention heads, delta heads and layer count."""
from __future__ import annotations

import numpy as np

from . import lebelix, nusilix, nusilix_bench as base

# name -> width, feed-forward, attention (heads, kv heads, dim), latent (heads, dim, rot, vdim, rank), delta (heads, dim), rank, side, layers
SIZES = {
    "2048": (2048, 8192, (32, 8, 64), (16, 64, 64, 128, 512), (16, 128), 128, 256, 6),
    "4096": (4096, 14336, (32, 8, 128), (32, 128, 64, 128, 512), (32, 128), 128, 256, 3),
}
KINDS = ("attention", "latent_attention", "channel_delta")
VOCAB, MAX_TOKENS = base.VOCAB, 8192
CHUNK, WINDOW = 8192, 4096


def config(size, kinds="all"):
    """kinds: one of KINDS, or "all" (in turn)."""
    w, ff, (h, kv, d), (lh, ld, lr, lv, rank), (dh, dd), _, side, n = SIZES[size]
    layers = {
        "attention": lebelix.Layer("attention", h, d, d, kv_heads=kv, mask_size=CHUNK, scale=d ** -0.5, softcap=30.0, rot_dims=d // 2, ff=ff),
        "latent_attention": lebelix.Layer("latent_attention", lh, ld, lv, mask_size=WINDOW, scale=(ld + lr) ** -0.5, rot_dims=lr, kv_rank=rank, ff=ff),
        "channel_delta": lebelix.Layer("channel_delta", dh, dd, dd, kv_heads=dh, taps=4, ff=ff),
    }
    pick = [layers[k] for k in (KINDS if kinds == "all" else (kinds,))]
    return lebelix.Config(width=w, vocab=VOCAB, norm_eps=1e-6, embed_scale=1.0, side_dim=side, layers=[pick[i % len(pick)] for i in range(n)], max_tokens=MAX_TOKENS)


def beside_config(size, kinds="all"):
    """The Nusilix decoder of the same sizes: its attention stands beside both kinds of attention, its delta rule beside the other."""
    w, ff, (h, kv, d), _, (dh, dd), _, _, n = SIZES[size]
    attn = nusilix.Layer("attention", heads=h, dim=d, kv_heads=kv, scale=d ** -0.5, temp_coef=0.1, temp_every=1024, ff=ff)
    delta = nusilix.Layer("general_delta", heads=dh, dim=dd, ff=ff)
    pick = {"all": [attn, attn, delta], "channel_delta": [delta]}.get(kinds, [attn])
    return nusilix.Config(width=w, vocab=VOCAB, norm_groups=1, norm_eps=1e-6, residual_mult=1.0, layers=[pick[i % len(pick)] for i in range(n)],
                          max_tokens=MAX_TOKENS)


def decode_bytes(cfg, model, ctx_tokens):
    """Bytes one decode step has to move: weights once, the cached rows in its range once, recurrent states in and out."""
    total = model.weight_bytes
    for layer in cfg.layers:
        if layer.mixer == "attention":
            total += min(ctx_tokens, layer.mask_size) * layer.kv_heads * (layer.dim + layer.vdim) * 2
        elif layer.mixer == "latent_attention":
            total += min(ctx_tokens, layer.mask_size) * (layer.kv_rank + layer.rot_dims) * 2
        else:
            total += 2 * layer.heads * layer.dim * layer.vdim * 4
    return total


def prompt_flops(cfg, shapes, n):
    """Matrix products of the layers plus the two products of the attentions."""
    total = sum(2 * s[0] * s[1] * n for name, s in shapes.items() if len(s) == 2 and "embed" not in name and "conv" not in name)
    for layer in cfg.layers:
        if layer.mixer != "channel_delta":
            size = min(layer.mask_size, n)
            keys = size * (size + 1) // 2 + (n - size) * size if layer.mixer == "latent_attention" else n * (n + 1) // 2  # (n within one chunk)
            total += 2 * keys * layer.heads * (layer.dim + layer.vdim + (layer.rot_dims if layer.mixer == "latent_attention" else 0))
    return total


def run(ctx, size, kinds="all", prompts=(512, 2048), contexts=(512, 4096), steps=64, beside=True):
    """kinds: as in config; "nusilix" or "nusilix-KIND": the other decoder alone."""
    if kinds.startswith("nusilix"):
        return run_beside(ctx, size, kinds[8:] or "all", prompts, contexts, steps)
    rank, n_layer = SIZES[size][5], SIZES[size][7]
    cfg = config(size, kinds)
    shapes = lebelix.tensor_shapes(cfg, rank, rank)
    model = lebelix.LebelixModel(ctx, cfg, base.random_source(shapes))
    t = base.measure(ctx, model, prompts, contexts, steps, np.random.default_rng(3), VOCAB)
    out = {"layers": f"{n_layer} x {kinds}", "weight_mb": round(model.weight_bytes / 1e6, 1)}
    base.report(out, t, {n: prompt_flops(cfg, shapes, n) for n in prompts}, {n: decode_bytes(cfg, model, n + steps / 2) for n in contexts})
    model.free()
    if beside:
        out["nusilix_beside"] = run_beside(ctx, size, kinds, prompts, contexts, steps)
    return out


def run_beside(ctx, size, kinds, prompts, contexts, steps):
    rank = SIZES[size][5]
    cfg = beside_config(size, kinds)
    model = nusilix.NusilixModel(ctx, cfg, base.random_source(nusilix.tensor_shapes(cfg, rank)))
    t = base.measure(ctx, model, prompts, contexts, steps, np.random.default_rng(3), VOCAB)
    out = {"weight_mb": round(model.weight_bytes / 1e6, 1)}
    base.report(out, t, {n: base.prompt_flops(cfg, rank, n) for n in prompts}, {n: base.decode_bytes(cfg, model, n + steps / 2) for n in contexts})
    model.free()
    return out
