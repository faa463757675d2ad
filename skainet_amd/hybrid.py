"""What the decoders over a list of layers (csrc/hybrid.hip) have in common on the host side: the layout of their weights, and the
model object that owns them."""
from __future__ import annotations

import ctypes as C
import json
import os

import numpy as np

from . import runtime
from .decoder import DecoderModel
from .runtime import BF16, F32, HybridConfig, HybridLayer, HybridWeights
from .safetensors import SafetensorsReader, bf16_to_f32, f32_to_bf16

DTYPES = {"bfloat16": BF16, "float32": F32}


def pad(n, to):
    return -(-n // to) * to


class Packer:
    """Tensors of a source (name -> float32 array or bfloat16 bit patterns) in the layout of skn_hybrid_layer."""

    def __init__(self, source, weight_type):
        self.get, self.type = source, weight_type

    def matrix(self, name, shape):
        a = self.get(name)
        if tuple(a.shape) != tuple(shape):
            raise ValueError(f"{name} is {tuple(a.shape)}, expected {tuple(shape)}")
        if self.type == F32:
            return bf16_to_f32(a) if a.dtype == np.uint16 else np.asarray(a, dtype=np.float32)
        return a if a.dtype == np.uint16 else f32_to_bf16(a)

    def table(self, name, shape):
        """fp32, without padding"""
        a = self.get(name)
        if tuple(a.shape) != tuple(shape):
            raise ValueError(f"{name} is {tuple(a.shape)}, expected {tuple(shape)}")
        return bf16_to_f32(a) if a.dtype == np.uint16 else np.asarray(a, dtype=np.float32)

    def vector(self, name, n):
        return self.table(name, (n,))

    def zeros(self, rows, cols):
        return np.zeros((rows, cols), dtype=np.float32 if self.type == F32 else np.uint16)

    def stack(self, parts, k):
        """[(name, rows)] one below the other, each from a multiple of 32 rows, columns padded to a multiple of 64."""
        out, at = self.zeros(sum(pad(r, 32) for _, r in parts), pad(k, 64)), 0
        for name, rows in parts:
            out[at:at + rows, :k] = self.matrix(name, (rows, k))
            at += pad(rows, 32)
        return out

    def beside(self, parts, rows):
        """[(name, columns)] side by side, each from a multiple of 64 columns, rows padded to a multiple of 32."""
        out, at = self.zeros(pad(rows, 32), sum(pad(k, 64) for _, k in parts)), 0
        for name, k in parts:
            out[:rows, at:at + k] = self.matrix(name, (rows, k))
            at += pad(k, 64)
        return out

    def padded(self, parts, to):
        """[(name or None, n)] vectors one after the other, each padded to a multiple of `to` (None: zeros)."""
        out, at = np.zeros(sum(pad(n, to) for _, n in parts), dtype=np.float32), 0
        for name, n in parts:
            if name is not None:
                out[at:at + n] = self.vector(name, n)
            at += pad(n, to)
        return out


class HybridModel(DecoderModel):
    """Device-resident model: owns the uploaded weights and the skn_hybrid handle.  Subclasses give their layers' scalars and arrays
    (names as in skn_hybrid_layer) and the model-wide ones."""

    PREFIX = "skn_hybrid"
    STREAMED = ("w_in", "w_out", "w_decay", "w_up", "w_down", "w_latent", "w_gate", "side_gate", "side_proj")  # matrices a decode step reads

    def pack_layer(self, pk, i):
        """-> (scalars of the layer's struct, its arrays by field name)"""
        raise NotImplementedError

    def pack_model(self, pk):
        """-> (further scalars of the configuration, arrays by field name of skn_hybrid_weights; no "head": the embedding)"""
        raise NotImplementedError

    def __init__(self, ctx: runtime.Context, cfg, source):
        """source(name) -> float32 array or bfloat16 bit patterns (uint16)."""
        self.ctx, self.cfg, self.bufs = ctx, cfg, {}
        pk = Packer(source, cfg.weight_type)
        self.weight_bytes = 0  # of the matrices a decode step streams
        layers = (HybridLayer * cfg.n_layer)()
        for i in range(cfg.n_layer):
            scalars, arrays = self.pack_layer(pk, i)
            for k, v in scalars.items():
                setattr(layers[i], k, v)
            for k, a in arrays.items():
                self.bufs[f"l{i}.{k}"] = ctx.to_device(a)
                setattr(layers[i], k, self.bufs[f"l{i}.{k}"].ptr)
                if k in self.STREAMED:
                    self.weight_bytes += a.nbytes
        scalars, arrays = self.pack_model(pk)
        for name, a in arrays.items():
            self.bufs[name] = ctx.to_device(a)
        self.weight_bytes += arrays.get("head", arrays["embed"]).nbytes
        ptr = {name: self.bufs[name].ptr for name in arrays}
        w = HybridWeights(embed=ptr["embed"], final_norm=ptr["final_norm"], head=ptr.get("head", ptr["embed"]), layers=layers, side=ptr.get("side"))
        c = HybridConfig(n_layer=cfg.n_layer, width=cfg.width, vocab=cfg.vocab, max_tokens=cfg.max_tokens, page_tokens=cfg.page_tokens, norm_groups=1,
                         weight_type=cfg.weight_type, norm_eps=cfg.norm_eps, residual_mult=1.0, embed_scale=1.0)
        for k, v in scalars.items():
            setattr(c, k, v)
        h = C.c_void_p()
        ctx._check(ctx.lib.skn_hybrid_create(ctx.handle, C.byref(c), C.byref(w), C.byref(h)))
        self.handle = h.value

    def extend(self, tokens, want=()):
        """The next tokens of the sequence as given; -> logits after the tokens at the places `want` (any order), [len(want), vocab]."""
        toks = np.ascontiguousarray(tokens, dtype=np.int32)
        want = np.asarray(list(want), dtype=np.int32)
        order = np.argsort(want, kind="stable")
        rows = np.ascontiguousarray(want[order])
        out = np.empty((len(rows), self.cfg.vocab), dtype=np.float32)
        i32 = C.POINTER(C.c_int32)
        self._call("extend", toks.ctypes.data_as(i32), len(toks), rows.ctypes.data_as(i32), len(rows), out.ctypes.data)
        res = np.empty_like(out)
        res[order] = out
        return res


def load_folder(ctx: runtime.Context, path: str, config_from_json, model_class, dtype="bfloat16", max_tokens=None, page_tokens=256):
    """A folder with config.json and model.safetensors."""
    with open(os.path.join(path, "config.json")) as f:
        cfg = config_from_json(json.load(f), max_tokens or 2048, page_tokens, dtype)
    reader = SafetensorsReader(os.path.join(path, "model.safetensors"))
    try:
        return model_class(ctx, cfg, lambda name: reader.raw(name) if reader.dtype(name) == "BF16" else reader.f32(name))
    finally:
        reader.close()
