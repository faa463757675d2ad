"""Lebelix: a decoder over a list of layers (csrc/hybrid.hip) read from a folder with config.json and model.safetensors.

Every layer runs its mixer and its feed-forward (tanh-form GELU between two matrices, or none) one after the other, each on a norm of its
own (weights around zero), and then adds something of the token's own: a gated part of the token's row in a side table.  Mixers:
"attention" (chunks, partial rotation, per-head norms, capped scores, a sink, an output gate; csrc/attention_ranged.hip),
"latent_attention" (a window over latents that layers may share; csrc/attention_latent.hip) and "channel_delta" (gated delta rule
with a decay per key channel behind short convolutions; csrc/gated_delta.hip).  The head is the embedding.
"""
from __future__ import annotations

from dataclasses import dataclass, field

import numpy as np

from . import runtime
from .hybrid import DTYPES, HybridModel, Packer, load_folder, pad
from .runtime import BF16, MASKS

MIXERS = {"attention": 2, "latent_attention": 3, "channel_delta": 4}  # SKN_MIX_*
MASK_OF = {"attention": "chunk", "latent_attention": "window"}


@dataclass
class Layer:
    mixer: str
    heads: int
    dim: int  # of a query and a key (latent attention: without the rotated part)
    vdim: int
    kv_heads: int = 0  # attention, channel_delta
    mask_size: int = 0
    scale: float = 0.0
    softcap: float = 0.0
    rot_dims: int = 0  # rotated elements: attention the first of dim, latent attention beside dim
    rot_base: float = 10000.0
    kv_rank: int = 0
    kv_from: int = -1
    taps: int = 0
    ff: int = 0  # 0: no feed-forward

    @property
    def columns(self):
        return self.heads * self.vdim


@dataclass
class Config:
    width: int
    vocab: int
    norm_eps: float
    embed_scale: float
    side_dim: int
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
        layer = Layer(kind, heads=int(m["heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]))
        if kind != "latent_attention":
            layer.kv_heads = int(m["kv_heads"])
            if layer.kv_heads < 1 or layer.heads % layer.kv_heads:
                raise ValueError(f"layer {i}: {layer.kv_heads} key heads do not divide {layer.heads} heads")
        if kind == "channel_delta":
            layer.taps = int(m["conv"])
        else:
            layer.scale, layer.mask_size = float(m["scale"]), int(m["mask"]["size"])
            layer.rot_dims, layer.rot_base = int(m["rot"]["dims"]), float(m["rot"]["base"])
        if kind == "attention":
            layer.softcap = float(m.get("softcap") or 0.0)
            if layer.rot_dims > layer.dim:
                raise ValueError(f"layer {i}: {layer.rot_dims} rotated elements of {layer.dim}")
        if kind == "latent_attention":
            layer.kv_rank = int(m["kv_rank"])
            if int(m["rot_dim"]) != layer.rot_dims:
                raise ValueError(f"layer {i}: the rotated part ({m['rot_dim']}) is rotated as a whole, not in {layer.rot_dims} elements")
            if m.get("kv_from") is not None:
                layer.kv_from = j = int(m["kv_from"])
                if not 0 <= j < i or layers[j].mixer != kind or layers[j].kv_from >= 0 or any(
                        getattr(layers[j], n) != getattr(layer, n) for n in ("kv_rank", "rot_dims", "rot_base")):
                    raise ValueError(f"layer {i} cannot read the latents of layer {j}")
        if mlp is not None:
            if mlp.get("kind") != "dense":
                raise ValueError(f"layer {i}: unknown feed-forward kind {mlp.get('kind')!r}")
            layer.ff = int(mlp["ff"])
        layers.append(layer)
    return Config(width=int(d["width"]), vocab=int(d["vocab"]), norm_eps=float(d["norm"]["eps"]), embed_scale=float(d["embedding"]["scale"]),
                  side_dim=int(d["token_side"]["dim"]), layers=layers, max_tokens=int(max_tokens), page_tokens=int(page_tokens), weight_type=DTYPES[dtype])


def tensor_shapes(cfg: Config, rank: int, rank_gate: int) -> dict:
    """name -> shape of every tensor of a model; rank, rank_gate: of the low-rank factors in the channel_delta layers."""
    w, s = cfg.width, {"embed": (cfg.vocab, cfg.width), "side.embed": (cfg.vocab, cfg.n_layer * cfg.side_dim)}
    for i, layer in enumerate(cfg.layers):
        p, h, g, d, v, c = f"l{i}.mix.", layer.heads, layer.kv_heads, layer.dim, layer.vdim, layer.columns
        s[f"l{i}.norm1"] = (w,)
        if layer.mixer == "attention":
            for n, rows in (("q", h * d), ("k", g * d), ("v", g * v)):
                s.update({p + n: (rows, w), p + n + ".b": (rows,)})
            s.update({p + "q.norm": (d,), p + "k.norm": (d,), p + "g": (c, w)})
        elif layer.mixer == "latent_attention":
            s[p + "q"] = (h * (d + layer.rot_dims), w)
            if layer.kv_from < 0:
                s.update({p + "dkv": (layer.kv_rank + layer.rot_dims, w), p + "dkv.norm": (layer.kv_rank,)})
            s.update({p + "uk": (h * d, layer.kv_rank), p + "uv": (c, layer.kv_rank)})
        else:
            for n, rows in (("q", g * d), ("k", g * d), ("v", c)):
                s.update({p + n: (rows, w), p + n + ".conv": (rows, layer.taps)})
            s.update({p + "b": (h, w), p + "A_log": (h,), p + "norm": (v,), p + "a1": (rank, w), p + "a2": (h * d, rank), p + "dt_bias": (h * d,),
                      p + "g1": (rank_gate, w), p + "g2": (c, rank_gate)})
        s[p + "o"] = (w, c)
        if layer.ff:
            s.update({f"l{i}.norm2": (w,), f"l{i}.mlp.up": (layer.ff, w), f"l{i}.mlp.down": (w, layer.ff)})
        if cfg.side_dim:
            s.update({f"l{i}.side.gate": (cfg.side_dim, w), f"l{i}.side.proj": (w, cfg.side_dim), f"l{i}.side.norm": (w,)})
    s["final.norm"] = (w,)
    return s


def _offset_norm(pk: Packer, name, n):
    """A norm whose weights are stored around zero."""
    out = np.zeros(pad(n, 64), dtype=np.float32)
    out[:n] = 1.0 + pk.vector(name, n)
    return out


def _pack_layer(pk: Packer, cfg: Config, i: int):
    """-> (scalars of the layer's struct, its arrays by field name)"""
    layer, p, w = cfg.layers[i], f"l{i}.mix.", cfg.width
    h, g, d, v, c = layer.heads, layer.kv_heads, layer.dim, layer.vdim, layer.columns
    scalars = {"mixer": MIXERS[layer.mixer], "heads": h, "kv_heads": g, "dim": d, "vdim": v, "ff": layer.ff, "scale": layer.scale, "softcap": layer.softcap,
               "mask": MASKS[MASK_OF.get(layer.mixer)], "mask_size": layer.mask_size, "rot_dims": layer.rot_dims, "rot_base": layer.rot_base,
               "kv_rank": layer.kv_rank, "kv_from": layer.kv_from, "taps": layer.taps, "act": 1}
    arrays = {"norm": _offset_norm(pk, f"l{i}.norm1", w), "b_out": np.zeros(pad(w, 32), dtype=np.float32), "w_out": pk.beside([(p + "o", c)], w)}
    if layer.mixer == "attention":
        rows, biases = [(p + "q", h * d), (p + "k", g * d), (p + "v", g * v), (p + "g", c)], {p + "q", p + "k", p + "v"}
        arrays["q_norm"], arrays["k_norm"] = pk.vector(p + "q.norm", d), pk.vector(p + "k.norm", d)
        scalars["sink"] = 1
    elif layer.mixer == "latent_attention":
        rows, biases = [(p + "q", h * (d + layer.rot_dims))], set()
        if layer.kv_from < 0:
            rows.append((p + "dkv", layer.kv_rank + layer.rot_dims))
            arrays["latent_norm"] = pk.vector(p + "dkv.norm", layer.kv_rank)
        arrays["w_latent"] = pk.stack([(p + "uk", h * d), (p + "uv", c)], layer.kv_rank)
    else:
        rank, rank_gate = int(pk.get(p + "a1").shape[0]), int(pk.get(p + "g1").shape[0])
        scalars.update(rank=rank, rank_gate=rank_gate)
        rows, biases = [(p + "q", g * d), (p + "k", g * d), (p + "v", c), (p + "b", h), (p + "a1", rank), (p + "g1", rank_gate)], set()
        arrays["w_decay"], arrays["b_decay"] = pk.stack([(p + "a2", h * d)], rank), pk.padded([(p + "dt_bias", h * d)], 32)
        arrays["w_gate"] = pk.stack([(p + "g2", c)], rank_gate)
        arrays["decay_rate"] = np.exp(pk.vector(p + "A_log", h))
        arrays["o_norm"] = np.tile(pk.vector(p + "norm", v), h)
        arrays["conv"] = np.concatenate([pk.table(p + n + ".conv", (r, layer.taps)) for n, r in (("q", g * d), ("k", g * d), ("v", c))])
    arrays["w_in"] = pk.stack(rows, w)
    arrays["b_in"] = pk.padded([(n + ".b" if n in biases else None, r) for n, r in rows], 32)
    if layer.ff:
        arrays["w_up"], arrays["w_down"] = pk.stack([(f"l{i}.mlp.up", layer.ff)], w), pk.stack([(f"l{i}.mlp.down", w)], layer.ff)
        arrays["norm2"] = _offset_norm(pk, f"l{i}.norm2", w)
    if cfg.side_dim:
        arrays["side_gate"], arrays["side_proj"] = pk.stack([(f"l{i}.side.gate", cfg.side_dim)], w), pk.stack([(f"l{i}.side.proj", w)], cfg.side_dim)
        arrays["side_norm"] = pk.padded([(f"l{i}.side.norm", w)], 64)
    return scalars, arrays


class LebelixModel(HybridModel):
    def pack_layer(self, pk, i):
        return _pack_layer(pk, self.cfg, i)

    def pack_model(self, pk):
        cfg = self.cfg
        arrays = {"embed": pk.stack([("embed", cfg.vocab)], cfg.width), "final_norm": _offset_norm(pk, "final.norm", cfg.width)}
        if cfg.side_dim:
            arrays["side"] = pk.stack([("side.embed", cfg.vocab)], cfg.n_layer * cfg.side_dim)
        return {"embed_scale": cfg.embed_scale, "side_dim": cfg.side_dim}, arrays


def load(ctx: runtime.Context, path: str, dtype="bfloat16", max_tokens=None, page_tokens=256) -> LebelixModel:
    return load_folder(ctx, path, config_from_json, LebelixModel, dtype, max_tokens, page_tokens)
