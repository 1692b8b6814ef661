"""The Python side of a model handle (mi355x_model_*): what every decoder takes,
whatever its layers are. A subclass makes the handle (self._h) from its own
configuration, which has `batch` and `vocab`."""
from __future__ import annotations

import ctypes as C

import numpy as np

from . import capi


class Decoder:
    lib = None
    config = None
    _h = None

    def close(self):
        if self._h:
            self.lib.mi355x_model_destroy(self._h)
            self._h = C.c_void_p()

    def __del__(self):
        try:
            self.close()
        except Exception:
            pass

    def set_tensor(self, name: str, dtype: int, data: np.ndarray, n_elems: int):
        data = np.ascontiguousarray(data)
        capi.check(self.lib.mi355x_model_set_tensor(self._h, name.encode(), dtype, data.ctypes.data, n_elems))

    def finalize(self, max_tokens: int):
        capi.check(self.lib.mi355x_model_finalize(self._h, max_tokens))

    def reset(self):
        capi.check(self.lib.mi355x_model_reset(self._h))

    @property
    def cache_len(self) -> int:
        return self.lib.mi355x_model_cache_len(self._h)

    def logits(self, tokens, all: bool = False) -> np.ndarray:
        """tokens [batch, n] (or [n] for batch 1) -> [batch, vocab] or [batch, n, vocab]."""
        c = self.config
        t = np.ascontiguousarray(tokens, np.int32).reshape(c.batch, -1)
        n = t.shape[1]
        out = np.empty((c.batch, n, c.vocab) if all else (c.batch, c.vocab), np.float32)
        capi.check(self.lib.mi355x_model_logits(self._h, t.ctypes.data, n, int(all), out.ctypes.data))
        return out

    def logits_at(self, tokens, want) -> np.ndarray:
        """The logits [len(want), vocab] of the rows b * n + t that `want` lists (it may be empty), after tokens [batch, n]."""
        c = self.config
        t = np.ascontiguousarray(tokens, np.int32).reshape(c.batch, -1)
        w = np.ascontiguousarray(want, np.int64).reshape(-1)
        out = np.empty((w.size, c.vocab), np.float32)
        capi.check(self.lib.mi355x_model_logits_at(self._h, t.ctypes.data, t.shape[1], w.ctypes.data, w.size, out.ctypes.data))
        return out

    def generate(self, prompt, n_new: int):
        """Greedy tokens [batch, n_new] and (prompt seconds, decode seconds)."""
        c = self.config
        t = np.ascontiguousarray(prompt, np.int32).reshape(c.batch, -1)
        out = np.empty((c.batch, n_new), np.int32)
        secs = (C.c_double * 2)()
        capi.check(self.lib.mi355x_model_generate(self._h, t.ctypes.data, t.shape[1], n_new, out.ctypes.data, secs))
        return out, (secs[0], secs[1])
