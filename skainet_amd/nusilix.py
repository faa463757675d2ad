"""Nusilix: a decoder over a list of layers (csrc/hybrid.hip) read from a folder with config.json and model.safetensors.

Every layer normalises the residual stream once, in groups, and feeds the result to its mixer and its feed-forward side by side:
x += residual_mult * (mixer(h) + ff(h)).  Mixers: "attention" (values are the keys before their norm; query temperature and
a linear distance bias instead of a rotation; csrc/attention_shared.hip) and "general_delta" (generalized delta rule;
csrc/delta.hip).  Feed-forward: xIELU between two matrices, or none.
"""
from __future__ import annotations

from dataclasses import dataclass, field

import numpy as np

from . import runtime
from .hybrid import DTYPES, HybridModel, Packer, load_folder
from .runtime import BF16

MIXERS = {"attention": 0, "general_delta": 1}  # SKN_MIX_*


@dataclass
class Layer:
    mixer: str
    heads: int
    dim: int
    kv_heads: int = 0
    scale: float = 0.0
    temp_coef: float = 0.0
    temp_every: float = 0.0
    ff: int = 0  # 0: no feed-forward

    @property
    def columns(self):
        return self.heads * self.dim


@dataclass
class Config:
    width: int
    vocab: int
    norm_groups: int
    norm_eps: float
    residual_mult: float
    layers: list = field(default_factory=list)
    max_tokens: int = 2048
    page_tokens: int = 256
    weight_type: int = BF16

    @property
    def n_layer(self):
        return len(self.layers)


def config_from_json(d, max_tokens=2048, page_tokens=256, dtype="bfloat16") -> Config:
    """The decoder's shape from the dictionary of config.json (ValueError for what it does not compute)."""
    layers = []
    for i, e in enumerate(d["layers"]):
        kind, m, mlp = e["type"], e["mixer"], e.get("mlp")
        if kind not in MIXERS:
            raise ValueError(f"layer {i}: unknown type {kind!r}")
        layer = Layer(kind, heads=int(m["heads"]), dim=int(m["dim"]))
        if kind == "attention":
            layer.kv_heads = int(m["kv_heads"])
            layer.scale = float(m["scale"])
            if int(m.get("vdim", layer.dim)) != layer.dim:
                raise ValueError(f"layer {i}: values are keys, so vdim ({m['vdim']}) must be dim ({layer.dim})")
            if m.get("q_temp"):
                layer.temp_coef, layer.temp_every = float(m["q_temp"]["coef"]), float(m["q_temp"]["every"])
        if mlp is not None:
            if mlp.get("kind") != "dense":
                raise ValueError(f"layer {i}: unknown feed-forward kind {mlp.get('kind')!r}")
            layer.ff = int(mlp["ff"])
        layers.append(layer)
    return Config(width=int(d["width"]), vocab=int(d["vocab"]), norm_groups=int(d["norm"]["groups"]), norm_eps=float(d["norm"]["eps"]),
                  residual_mult=float(d["residual_mult"]), layers=layers, max_tokens=int(max_tokens), page_tokens=int(page_tokens),
                  weight_type=DTYPES[dtype])


def tensor_shapes(cfg: Config, rank: int) -> dict:
    """name -> shape of every tensor of a model; rank: of the decay's factors in the general_delta layers."""
    w, s = cfg.width, {"embed": (cfg.vocab, cfg.width)}
    for i, layer in enumerate(cfg.layers):
        p, c, g = f"l{i}.mix.", layer.columns, layer.kv_heads * layer.dim
        s[f"l{i}.norm1"] = (w,)
        if layer.mixer == "attention":
            s.update({p + "q": (c, w), p + "q.b": (c,), p + "k": (g, w), p + "k.b": (g,), p + "q.norm": (c,), p + "k.norm": (g,), p + "o": (w, c),
                      p + "o.b": (w,)})
        else:
            s.update({p + n: (c, w) for n in ("r", "k", "v", "g", "a")})
            s.update({p + "a.b": (c,), p + "w1": (rank, w), p + "w2": (c, rank), p + "w0": (c,), p + "norm": (c,), p + "o": (w, c)})
        if layer.ff:
            s.update({f"l{i}.mlp.up": (layer.ff, w), f"l{i}.mlp.down": (w, layer.ff), f"l{i}.mlp.act": (2,)})
    s["final.norm"], s["head"] = (w,), (cfg.vocab, w)
    return s


def _pack_layer(pk: Packer, cfg: Config, i: int):
    """-> (scalars of the layer's struct, its arrays by field name)"""
    layer, p, w = cfg.layers[i], f"l{i}.mix.", cfg.width
    c, g = layer.columns, layer.kv_heads * layer.dim
    rank, ff = 0, [(f"l{i}.mlp.up", layer.ff)] if layer.ff else []
    no_ff_bias = [(None, layer.ff)] if layer.ff else []
    arrays = {"norm": pk.padded([(f"l{i}.norm1", w)], 64)}
    if layer.mixer == "attention":
        arrays["w_in"] = pk.stack([(p + "q", c), (p + "k", g)] + ff, w)
        arrays["b_in"] = pk.padded([(p + "q.b", c), (p + "k.b", g)] + no_ff_bias, 32)
        arrays["b_out"] = pk.padded([(p + "o.b", w)], 32)
        arrays["q_norm"], arrays["k_norm"] = pk.vector(p + "q.norm", c), pk.vector(p + "k.norm", g)
    else:
        rank = int(pk.get(p + "w1").shape[0])
        arrays["w_in"] = pk.stack([(p + n, c) for n in ("r", "k", "v", "g", "a")] + [(p + "w1", rank)] + ff, w)
        arrays["b_in"] = pk.padded([(None, c)] * 4 + [(p + "a.b", c), (None, rank)] + no_ff_bias, 32)
        arrays["b_out"] = pk.padded([(None, w)], 32)
        arrays["w_decay"] = pk.stack([(p + "w2", c)], rank)
        arrays["b_decay"] = pk.padded([(p + "w0", c)], 32)
        arrays["o_norm"] = pk.vector(p + "norm", c)
    arrays["w_out"] = pk.beside([(p + "o", c)] + ([(f"l{i}.mlp.down", layer.ff)] if layer.ff else []), w)
    scalars = {"mixer": MIXERS[layer.mixer], "heads": layer.heads, "kv_heads": layer.kv_heads, "dim": layer.dim, "rank": rank, "ff": layer.ff,
               "scale": layer.scale, "temp_coef": layer.temp_coef, "temp_every": layer.temp_every}
    if layer.ff:
        act = pk.vector(f"l{i}.mlp.act", 2).astype(np.float64)
        scalars["act_pos"], scalars["act_neg"] = float(np.logaddexp(0.0, act[0])), 0.5 + float(np.logaddexp(0.0, act[1]))
    return scalars, arrays


class NusilixModel(HybridModel):
    def pack_layer(self, pk, i):
        return _pack_layer(pk, self.cfg, i)

    def pack_model(self, pk):
        cfg = self.cfg
        return {"norm_groups": cfg.norm_groups, "residual_mult": cfg.residual_mult, "sinusoid": 1}, {
            "embed": pk.stack([("embed", cfg.vocab)], cfg.width), "final_norm": pk.padded([("final.norm", cfg.width)], 64),
            "head": pk.stack([("head", cfg.vocab)], cfg.width)}


def load(ctx: runtime.Context, path: str, dtype="bfloat16", max_tokens=None, page_tokens=256) -> NusilixModel:
    return load_folder(ctx, path, config_from_json, NusilixModel, dtype, max_tokens, page_tokens)
