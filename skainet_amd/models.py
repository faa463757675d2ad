"""Model registry: the architecture a path names -> its loader.

A .gguf file names its architecture in the metadata field general.architecture, a folder in the key "architecture" of its
config.json.  Loaders return a decoder.DecoderModel.
"""
from __future__ import annotations

import importlib
import json
import os

# architecture -> (module, loader(ctx, path, dtype, max_tokens, page_tokens))
ARCHITECTURES = {
    "llama": ("skainet_amd.llama", "load"),
    "Nusilix": ("skainet_amd.nusilix", "load"),
    "Lebelix": ("skainet_amd.lebelix", "load"),
}


def architecture_of(path) -> str:
    if os.path.isdir(path):
        with open(os.path.join(path, "config.json")) as f:
            return json.load(f)["architecture"]
    from . import gguf

    reader = gguf.GGUFReader(path)
    try:
        return reader.fields["general.architecture"]
    finally:
        reader.close()


def load_model(ctx, path, dtype="bfloat16", max_tokens=None, page_tokens=256):
    """Opens a model, uploads its weights and returns its decoder.  dtype: of the compute path where a model has a choice
    ("bfloat16" or "float32"; block-quantized files have none and ignore it)."""
    arch = architecture_of(path)
    if arch not in ARCHITECTURES:
        raise ValueError(f"{path}: architecture {arch!r} is not one of {', '.join(sorted(ARCHITECTURES))}")
    module, fn = ARCHITECTURES[arch]
    return getattr(importlib.import_module(module), fn)(ctx, path, dtype=dtype, max_tokens=max_tokens, page_tokens=page_tokens)
