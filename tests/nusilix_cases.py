"""Small Nusilix models for the tests: configurations as config.json has them, and seeded weights whose logits depend on every
mechanism (matrices of gain about one, decays over their whole range, norms and biases away from 1 and 0)."""
import numpy as np

from skainet_amd import nusilix
from skainet_amd.safetensors import bf16_to_f32, f32_to_bf16


def attention(heads, kv_heads, dim, scale=None, q_temp=(0.4, 7), ff=90):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": dim ** -0.5 * 1.5 if scale is None else scale}
    if q_temp:
        m["q_temp"] = {"coef": q_temp[0], "every": q_temp[1]}
    return {"type": "attention", "mixer": m, "mlp": {"kind": "dense", "ff": ff} if ff else None}


def delta(heads, dim, ff=90):
    return {"type": "general_delta", "mixer": {"heads": heads, "dim": dim}, "mlp": {"kind": "dense", "ff": ff} if ff else None}


def model(layers, width=144, vocab=203, groups=3, eps=1e-5, mult=0.7):
    return {"architecture": "Nusilix", "width": width, "vocab": vocab, "norm": {"groups": groups, "eps": eps}, "residual_mult": mult, "layers": layers}


# name -> (config, rank of the decays).  Between them: head sizes that are padded and that are not, one and many key heads,
# layers without a feed-forward, norms in one group and in many, widths that are no multiple of anything, no temperature.
MODELS = {
    "mixed": (model([attention(6, 2, 48), delta(3, 40), delta(5, 24, ff=70), attention(6, 3, 24, ff=0)]), 12),
    "attention_64": (model([attention(8, 1, 64), attention(3, 3, 64, q_temp=None)], width=128, groups=4), 1),
    "attention_128": (model([attention(4, 4, 128, ff=333), attention(4, 2, 100)], width=200, groups=1, mult=1.0), 1),
    "attention_256": (model([attention(2, 1, 136), attention(2, 2, 256, ff=0)], width=96, groups=2), 1),
    "delta_only": (model([delta(2, 8), delta(1, 64, ff=0), delta(2, 100), delta(1, 136)], width=150, groups=5, vocab=97), 33),
    "odd": (model([delta(3, 7, ff=11), attention(5, 5, 9, ff=13), delta(1, 1, ff=1)], width=45, groups=9, vocab=31), 5),
    "deep": (model([attention(4, 2, 32) if i % 3 == 1 else delta(4, 16) for i in range(9)], width=112, groups=7, mult=0.4), 8),
}


def weights(cfg_dict, rank, seed=0, gains=None):
    """name -> float32 array, every value a bfloat16."""
    cfg = nusilix.config_from_json(cfg_dict)
    rng = np.random.default_rng(seed)
    gains = gains or {}
    out = {}
    for name, shape in nusilix.tensor_shapes(cfg, rank).items():
        last = name.rsplit(".", 1)[-1]
        if last in ("norm", "norm1"):
            a = 1.0 + 0.2 * rng.standard_normal(shape)
        elif last == "w0":
            a = 2.0 * rng.standard_normal(shape)
        elif last == "act":
            a = rng.standard_normal(shape)
        elif len(shape) == 1:
            a = 0.3 * rng.standard_normal(shape)
        else:
            a = rng.standard_normal(shape) * (2.0 if name == "embed" else shape[1] ** -0.5) * gains.get(last, 1.0)
        out[name] = bf16_to_f32(f32_to_bf16(a.astype(np.float32)))
    return out


def device_model(ctx, cfg_dict, w, dtype="float32", max_tokens=512, page_tokens=16):
    cfg = nusilix.config_from_json(cfg_dict, max_tokens=max_tokens, page_tokens=page_tokens, dtype=dtype)
    return nusilix.NusilixModel(ctx, cfg, lambda name: w[name])


def tokens(cfg_dict, n, seed=1):
    return np.random.default_rng(seed).integers(0, cfg_dict["vocab"], n).tolist()


def logit_error(got, want):
    """Per position: root mean square of the difference (means taken off) over that of the wanted logits."""
    d = np.asarray(got, dtype=np.float64) - want
    d -= d.mean(axis=-1, keepdims=True)
    w = want - want.mean(axis=-1, keepdims=True)
    return np.sqrt((d ** 2).mean(axis=-1) / (w ** 2).mean())


# per position, as logit_error; the 16-bit path's own rounding measures 2e-3 to 5e-3 on these models, more at single positions
# of the models with heads of a few channels (a head is divided by its own root mean square: near zero that magnifies)
TOLERANCE = {"float32": 2e-5, "bfloat16": 2e-2}


def check(got, want, dtype, what=None):
    """Every position within the tolerance (16-bit: one in fifty within three times it)."""
    err, tol = logit_error(got, want), TOLERANCE[dtype]
    over = int((err > tol).sum())
    assert over <= (len(err) // 50 if dtype == "bfloat16" else 0) and err.max() < 3 * tol, (what, over, int(err.argmax()), err.max())


def finder(heads, kv_heads, dim, seed=0, match=14.0):
    """One attention layer in which the last token's query (ASK) finds the key of one other token (RARE), whose value is unlike
    any other: keys read the first half of the normalised stream, queries the second half through the same matrices, and
    ASK's second half is RARE's first.  The scale lets a match outweigh hundreds of other keys and, in the heads with flat
    slopes, its distance."""
    cfg = model([attention(heads, kv_heads, dim, scale=match / dim, q_temp=(0.05, 64), ff=0)], width=96, vocab=61, groups=2, mult=1.0)
    w = weights(cfg, 1, seed)
    k = w["l0.mix.k"].reshape(kv_heads, dim, 96) * 2 ** 0.5
    k[:, :, 48:] = 0
    q = np.repeat(np.roll(k, 48, axis=2), heads // kv_heads, axis=0)
    w["l0.mix.k"], w["l0.mix.q"] = k.reshape(-1, 96), q.reshape(-1, 96)
    for n in ("q.b", "k.b"):
        w[f"l0.mix.{n}"][:] = 0
    for n in ("l0.norm1", "l0.mix.q.norm", "l0.mix.k.norm"):
        w[n][:] = 1
    w["embed"] *= 3
    w["l0.mix.o"] *= 4
    w["embed"][ASK, 48:] = w["embed"][RARE, :48]
    return cfg, {n: bf16_to_f32(f32_to_bf16(a)) for n, a in w.items()}


ASK, RARE, COMMON = 60, 59, 58
