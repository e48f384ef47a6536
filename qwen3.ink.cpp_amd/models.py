"""Models behind one interface (``include/a81w41_model.h``): load a folder by its config.json, feed tokens in
portions, read logits, generate.

``ARCHITECTURES`` says which library holds a model class; a library registers its classes with
``csrc/liba81w41_core.so`` when it is loaded.  ``ensure_built`` compiles what one architecture needs and no more.
"""
from __future__ import annotations

import ctypes as C
import fcntl
import json
import os
import subprocess

import numpy as np

from . import capi

# architecture name in config.json -> (loader of its library, the library's path, make target that builds it)
ARCHITECTURES = {
    "Qwen3": (capi.lib, capi.LIB_PATH, "liba81w41.so"),
    "Takosun": (capi.dense, capi.DENSE_PATH, "dense"),
    "Dimesun": (capi.dense, capi.DENSE_PATH, "dense"),
}


def architecture_of(config: dict) -> str:
    name = config.get("architecture")
    if name not in ARCHITECTURES:
        raise ValueError(f"no model class for architecture {name!r}; known: {', '.join(sorted(ARCHITECTURES))}")
    return name


def read_config(model_dir: str) -> dict:
    with open(os.path.join(model_dir, "config.json"), encoding="utf-8") as f:
        return json.load(f)


def ensure_built(architecture: str) -> None:
    """Compile the architecture's library if it is not there (progress goes to stderr)."""
    _, path, target = ARCHITECTURES[architecture]
    if os.path.exists(path):
        return
    with open(os.path.join(capi.CSRC, ".build.lock"), "w") as lock:
        fcntl.flock(lock, fcntl.LOCK_EX)  # another process may be building the same tree
        if not os.path.exists(path):
            jobs = min(16, os.cpu_count() or 1)
            subprocess.run(["make", "-C", capi.CSRC, f"-j{jobs}", target], check=True, stdout=2)


class Model:
    """One sequence at a time.  ``forward`` runs only the tokens it is given, on top of what the cache holds."""

    def __init__(self, handle, architecture: str):
        self.handle, self.architecture = handle, architecture
        L = capi.core()
        self.vocab, self.max_seq = L.a81w41_model_vocab(handle), L.a81w41_model_max_seq(handle)

    @classmethod
    def load(cls, model_dir: str, max_seq: int, dtype: str = "bfloat16") -> "Model":
        name = architecture_of(read_config(model_dir))
        ARCHITECTURES[name][0]()
        h = C.c_void_p()
        capi.check(capi.core().a81w41_model_load(os.fsencode(model_dir), dtype.encode(), max_seq, C.byref(h)))
        return cls(h, name)

    @classmethod
    def random(cls, config: dict, max_seq: int, dtype: str = "bfloat16", seed: int = 0) -> "Model":
        """Seeded random weights of the configuration's shapes (for benchmarks)."""
        name = architecture_of(config)
        ARCHITECTURES[name][0]()
        h = C.c_void_p()
        capi.check(capi.core().a81w41_model_create_random(json.dumps(config).encode(), dtype.encode(), max_seq, seed, C.byref(h)))
        return cls(h, name)

    def reset(self) -> None:
        capi.check(capi.core().a81w41_model_reset(self.handle))

    @property
    def position(self) -> int:
        return capi.core().a81w41_model_position(self.handle)

    def forward(self, token_ids, want=None) -> np.ndarray:
        """Logits [len(want)][vocab] at the rising places ``want`` among the new tokens (default: the last one)."""
        ids = np.ascontiguousarray(token_ids, np.int32)
        w = np.ascontiguousarray([len(ids) - 1] if want is None else want, np.int32)
        out = np.empty((len(w), self.vocab), np.float32)
        capi.check(capi.core().a81w41_model_forward(self.handle, ids.ctypes.data, len(ids), w.ctypes.data, len(w),
                                                    out.ctypes.data))
        return out

    def generate_greedy(self, prompt, n_new: int):
        """-> (n_new token ids, prefill ms, decode ms)"""
        ids = np.ascontiguousarray(prompt, np.int32)
        out = np.empty(n_new, np.int32)
        t_pre, t_dec = C.c_double(), C.c_double()
        capi.check(capi.core().a81w41_model_generate_greedy(self.handle, ids.ctypes.data, len(ids), n_new, out.ctypes.data,
                                                            C.byref(t_pre), C.byref(t_dec)))
        return out, t_pre.value, t_dec.value

    def set_option(self, name: str, value: int) -> None:
        capi.check(capi.core().a81w41_model_set_option(self.handle, name.encode(), int(value)))

    def read_buffer(self, name: str, *shape: int) -> np.ndarray:
        out = np.empty(shape, np.float32)
        capi.check(capi.core().a81w41_model_read_buffer(self.handle, name.encode(), out.ctypes.data, out.size))
        return out

    def resident_bytes(self) -> dict:
        a, b = C.c_size_t(), C.c_size_t()
        total = capi.core().a81w41_model_resident_bytes(self.handle, C.byref(a), C.byref(b))
        return {"total": int(total), "weights": a.value, "cache": b.value}

    def close(self) -> None:
        h, self.handle = getattr(self, "handle", None), None
        if h and capi is not None:  # module globals are gone at interpreter shutdown
            capi.core().a81w41_model_destroy(h)

    __del__ = close
