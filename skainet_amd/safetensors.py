"""Safetensors reader (memory-mapped): u64 little-endian header length, JSON header name -> dtype, shape, data_offsets
(into what follows the header), raw little-endian data."""
from __future__ import annotations

import json
import mmap
import struct

import numpy as np

# bfloat16 has no NumPy type: its bit patterns are handed out as uint16
_DTYPES = {"F64": np.float64, "F32": np.float32, "F16": np.float16, "BF16": np.uint16, "I64": np.int64, "I32": np.int32, "I16": np.int16,
           "I8": np.int8, "U8": np.uint8, "BOOL": np.bool_}


class SafetensorsReader:
    """names(); dtype(name); shape(name); raw(name): the array as stored (BF16 as uint16); f32(name): widened to float32."""

    def __init__(self, path):
        self._f = open(path, "rb")
        self._map = mmap.mmap(self._f.fileno(), 0, access=mmap.ACCESS_READ)
        if len(self._map) < 8:
            raise ValueError(f"{path}: not a safetensors file")
        (n,) = struct.unpack_from("<Q", self._map, 0)
        if n > len(self._map) - 8:
            raise ValueError(f"{path}: header of {n} bytes in a file of {len(self._map)}")
        self._entries = {k: v for k, v in json.loads(self._map[8:8 + n]).items() if k != "__metadata__"}
        self._base = 8 + n

    def names(self):
        return list(self._entries)

    def __contains__(self, name):
        return name in self._entries

    def _entry(self, name):
        if name not in self._entries:
            raise ValueError(f"the file has no tensor {name}")
        return self._entries[name]

    def dtype(self, name):
        return self._entry(name)["dtype"]

    def shape(self, name):
        return tuple(self._entry(name)["shape"])

    def raw(self, name):
        e = self._entry(name)
        if e["dtype"] not in _DTYPES:
            raise ValueError(f"{name}: unsupported dtype {e['dtype']}")
        dt = np.dtype(_DTYPES[e["dtype"]])
        lo, hi = e["data_offsets"]
        count = int(np.prod(e["shape"], dtype=np.int64))
        if hi - lo != count * dt.itemsize or self._base + hi > len(self._map):
            raise ValueError(f"{name}: {hi - lo} bytes for shape {e['shape']} of {e['dtype']}")
        return np.frombuffer(self._map, dtype=dt, count=count, offset=self._base + lo).reshape(e["shape"])

    def f32(self, name):
        a = self.raw(name)
        return bf16_to_f32(a) if self.dtype(name) == "BF16" else a.astype(np.float32)

    def close(self):
        try:
            self._map.close()
        except BufferError:  # arrays over the mapping are still alive; it goes with them
            pass
        self._f.close()


def bf16_to_f32(bits):
    return (np.ascontiguousarray(bits).astype(np.uint32) << 16).view(np.float32)


def f32_to_bf16(x):
    """Round to nearest even; bit patterns as uint16."""
    u = np.ascontiguousarray(x, dtype=np.float32).view(np.uint32)
    return ((u + 0x7FFF + ((u >> 16) & 1)) >> 16).astype(np.uint16)


def write_safetensors(path, tensors):
    """tensors: name -> float32 array (stored as BF16), uint16 array (BF16 bit patterns) or int32 array."""
    header, blobs, at = {}, [], 0
    for name, a in tensors.items():
        a = np.ascontiguousarray(a)
        if a.dtype == np.int32:
            dt = "I32"
        else:
            dt = "BF16"
            a = a if a.dtype == np.uint16 else f32_to_bf16(a)
        header[name] = {"dtype": dt, "shape": list(a.shape), "data_offsets": [at, at + a.nbytes]}
        at += a.nbytes
        blobs.append(a.tobytes())
    text = json.dumps(header).encode()
    text += b" " * (-len(text) % 8)
    with open(path, "wb") as f:
        f.write(struct.pack("<Q", len(text)) + text)
        for b in blobs:
            f.write(b)
