"""Small Lebelix models for the tests: configurations as config.json has them, and seeded weights whose logits depend on every
mechanism (matrices of gain about one, decays from nearly nothing to nearly one, norms and biases away from 1 and 0)."""
import numpy as np

from nusilix_cases import TOLERANCE, check, logit_error, tokens  # noqa: F401  (one metric and one tolerance for both designs)
from skainet_amd import lebelix
from skainet_amd.safetensors import bf16_to_f32, f32_to_bf16


def _layer(kind, mixer, ff):
    return {"type": kind, "mixer": mixer, "mlp": {"kind": "dense", "ff": ff} if ff else None}


def attention(heads, kv_heads, dim, vdim, rot, chunk, ff=90, scale=None, softcap=9.0, base=1000.0):
    return _layer("attention", {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "rot": {"dims": rot, "base": base}, "mask": {"size": chunk},
                                "scale": dim ** -0.5 * 2.5 if scale is None else scale, "softcap": softcap}, ff)


def latent(heads, dim, rot, vdim, rank, window, ff=90, scale=None, base=3000.0, kv_from=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": rank, "rot": {"dims": rot, "base": base}, "mask": {"size": window},
         "scale": (dim + rot) ** -0.5 * 2.5 if scale is None else scale}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return _layer("latent_attention", m, ff)


def delta(heads, kv_heads, dim, vdim, taps=4, ff=90):
    return _layer("channel_delta", {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": taps}, ff)


def model(layers, width=144, vocab=203, eps=1e-5, scale=1.7, side=20):
    return {"architecture": "Lebelix", "width": width, "vocab": vocab, "norm": {"eps": eps}, "embedding": {"scale": scale}, "token_side": {"dim": side},
            "layers": layers}


# name -> (config, rank of the decays, rank of the gates).  Between them: sizes that are padded and that are not, keys wider and
# narrower than values, one and many key heads, layers without a feed-forward, rotation of everything and of a part, windows and
# chunks of one token and longer than the sequence, latents read by other layers, convolutions of one tap and of many.
MODELS = {
    "mixed": (model([latent(3, 24, 16, 40, 56, 19), attention(6, 2, 48, 40, 20, 23), delta(6, 3, 40, 24, taps=3, ff=70),
                     latent(5, 40, 16, 24, 56, 33, ff=0, kv_from=0), attention(4, 1, 24, 56, 24, 300, ff=0, softcap=3.0)]), 12, 9),
    "attention_64": (model([attention(8, 1, 64, 64, 32, 37), attention(3, 3, 40, 64, 2, 16)], width=128, side=64), 1, 1),
    "attention_128": (model([attention(4, 4, 128, 100, 64, 41, ff=333), attention(4, 2, 72, 128, 72, 1)], width=200, scale=1.0), 1, 1),
    "attention_256": (model([attention(2, 1, 136, 200, 100, 50), attention(2, 2, 256, 256, 256, 33, ff=0)], width=96, side=1), 1, 1),
    "latent_64": (model([latent(4, 32, 32, 64, 64, 25), latent(2, 8, 32, 20, 64, 1, kv_from=0), latent(3, 17, 8, 33, 30, 500)], width=128), 1, 1),
    "latent_128": (model([latent(4, 64, 64, 128, 192, 30), latent(5, 100, 28, 72, 228, 16)], width=160, side=33), 1, 1),
    "latent_192": (model([latent(3, 128, 64, 128, 320, 40), latent(2, 128, 64, 96, 320, 7, kv_from=0)], width=96), 1, 1),
    "latent_wide": (model([latent(2, 200, 32, 160, 600, 21), latent(2, 24, 8, 136, 900, 35), latent(1, 200, 32, 40, 600, 100, kv_from=0)], width=96), 1, 1),
    "delta_only": (model([delta(2, 2, 8, 8, taps=1), delta(4, 1, 64, 100, ff=0), delta(2, 1, 100, 40, taps=8), delta(1, 1, 136, 256, taps=2)], width=150,
                         vocab=97), 33, 70),
    "odd": (model([delta(3, 1, 7, 5, taps=2, ff=11), attention(5, 5, 9, 3, 4, 5, ff=13), latent(1, 1, 2, 1, 3, 4, ff=1), delta(1, 1, 1, 1, ff=1)], width=45,
                  vocab=31, side=3), 5, 2),
    "deep": (model([attention(4, 2, 32, 32, 16, 29) if i % 3 == 1 else delta(4, 2, 16, 32) if i % 3 else latent(4, 24, 8, 24, 40, 27, kv_from=0 if i else None)
                    for i in range(9)], width=112), 8, 8),
}


def weights(cfg_dict, rank, rank_gate, seed=0):
    """name -> float32 array, every value a bfloat16."""
    cfg = lebelix.config_from_json(cfg_dict)
    rng = np.random.default_rng(seed)
    out = {}
    for name, shape in lebelix.tensor_shapes(cfg, rank, rank_gate).items():
        last = name.rsplit(".", 1)[-1]
        if last in ("norm1", "norm2") or name == "final.norm":
            a = 0.2 * rng.standard_normal(shape)
        elif last == "norm":
            a = 1.0 + 0.2 * rng.standard_normal(shape)
        elif last == "A_log":
            a = rng.uniform(-4.0, 2.0, shape)
        elif last == "dt_bias":
            a = 2.0 * rng.standard_normal(shape) - 1.0
        elif last == "b" and len(shape) == 1:
            a = 0.3 * rng.standard_normal(shape)
        else:
            a = rng.standard_normal(shape) * (1.0 if name in ("embed", "side.embed") else shape[1] ** -0.5)
        out[name] = bf16_to_f32(f32_to_bf16(a.astype(np.float32)))
    return out


def device_model(ctx, cfg_dict, w, dtype="float32", max_tokens=512, page_tokens=16):
    cfg = lebelix.config_from_json(cfg_dict, max_tokens=max_tokens, page_tokens=page_tokens, dtype=dtype)
    return lebelix.LebelixModel(ctx, cfg, lambda name: w[name])


ASK, RARE, COMMON = 60, 59, 58


def finder(kind, size, heads=4, dim=40, vdim=40, seed=0, match=11.0):
    """One attention layer in which a query of ASK finds the key of RARE, whose value is unlike any other: keys read the first half of the
    normalised stream, queries the second half through the same matrices, and ASK's second half is RARE's first.  Only elements that are
    not rotated take part, so the distance does not matter; the scale lets a match outweigh hundreds of other keys."""
    if kind == "attention":
        layer = attention(heads, heads // 2, dim, vdim, 8, size, ff=0, scale=match / (dim - 8), softcap=30.0)
    else:
        layer = latent(heads, dim, 8, vdim, 48, size, ff=0, scale=match / dim)
    cfg = model([layer], width=96, vocab=61, side=4, scale=1.0)
    w = weights(cfg, 1, 1, seed)
    if kind == "attention":
        k = w["l0.mix.k"].reshape(heads // 2, dim, 96) * 2 ** 0.5
        k[:, :8], k[:, :, 48:] = 0, 0
        w["l0.mix.k"], w["l0.mix.q"] = k.reshape(-1, 96), np.repeat(np.roll(k, 48, axis=2), 2, axis=0).reshape(-1, 96)
        for n in ("q", "k"):
            w[f"l0.mix.{n}.b"][:] = 0
            w[f"l0.mix.{n}.norm"][:] = 1
    else:
        d = w["l0.mix.dkv"] * 2 ** 0.5
        d[:, 48:] = 0
        w["l0.mix.dkv"], w["l0.mix.dkv.norm"][:] = d, 1
        q = np.zeros((heads, dim + 8, 96), dtype=np.float32)
        q[:, :dim, 48:] = (w["l0.mix.uk"] @ d[:48, :48]).reshape(heads, dim, 48)
        w["l0.mix.q"] = q.reshape(-1, 96)
    w["l0.norm1"][:] = 0
    w["l0.side.gate"][:] = 0
    w["embed"] *= 3
    w["l0.mix.o"] *= 6
    w["embed"][ASK, 48:] = w["embed"][RARE, :48]
    return cfg, {n: bf16_to_f32(f32_to_bf16(a)) for n, a in w.items()}
