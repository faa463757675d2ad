"""What the decoders of the library have in common on the host side: one sequence that is reset, fed a prompt and decoded
greedily, behind entry points that differ by their prefix only (skn_llama_*, skn_hybrid_*)."""
from __future__ import annotations

import ctypes as C

import numpy as np


class DecoderModel:
    PREFIX = ""  # "skn_llama" / "skn_hybrid"

    # subclasses set these: the context, a configuration with `vocab`, the handle, the uploaded buffers by name
    ctx = None
    cfg = None
    handle = None
    bufs: dict = {}

    def _call(self, name, *args):
        self.ctx._check(getattr(self.ctx.lib, f"{self.PREFIX}_{name}")(self.ctx.handle, self.handle, *args))

    def reset(self):
        self._call("reset")

    def prefill(self, tokens):
        """Feeds prompt tokens; returns the greedy next token."""
        arr = (C.c_int32 * len(tokens))(*[int(t) for t in tokens])
        nxt = C.c_int32()
        self._call("prefill", arr, len(tokens), C.byref(nxt))
        return nxt.value

    def decode(self, first_token, n_steps):
        """Greedy decode: feeds first_token, then its own choices; returns the n_steps produced tokens."""
        out = (C.c_int32 * max(n_steps, 1))()
        self._call("decode", int(first_token), n_steps, out)
        return list(out[:n_steps])

    def logits(self):
        p = C.c_void_p()
        self._call("logits", C.byref(p))
        out = np.empty(self.cfg.vocab, dtype=np.float32)
        self.ctx._check(self.ctx.lib.skn_download(self.ctx.handle, out.ctypes.data, p.value, out.nbytes))
        return out

    def generate(self, prompt, n_tokens):
        """The greedy continuation of a prompt, from an empty sequence."""
        self.reset()
        first = self.prefill(prompt)
        return ([first] + self.decode(first, n_tokens - 1))[:n_tokens]

    def free(self):
        if self.handle:
            getattr(self.ctx.lib, f"{self.PREFIX}_free")(self.ctx.handle, self.handle)
            self.handle = None
        for b in {id(b): b for b in self.bufs.values()}.values():
            b.free()
        self.bufs = {}
