"""Front end of the library's resident models of any registered design: load_model() picks the class
from what the path holds (a folder with config.json and model.safetensors, a GGUF file, a LiteNN
archive), create_model() builds one from a configuration and tensors in host memory.

    model = load_model("folder")
    tokens, prefill_ms, decode_ms = model.generate(prompt_ids, 64)
"""
from __future__ import annotations

import ctypes as C
import json

import numpy as np

from . import _lib
from ._lib import ModelInfo, ModelTensor, check
from .device import HIP, MATMUL_PRECISE
from .formats import DT_BF16, DT_F16, DT_F32

DTYPES = {"bfloat16": DT_BF16, "float16": DT_F16, "float32": DT_F32}


class Model:
    """One resident model and the one sequence it holds."""

    def __init__(self, handle: C.c_void_p):
        self._h = handle
        info = ModelInfo()
        check(_lib.load().litenn_hip_model_get_info(handle, C.byref(info)))
        self.architecture = info.architecture.decode()
        self.vocab_size = info.vocab_size
        self.context_length = info.context_length
        self.dtype = info.dtype

    def close(self) -> None:
        if self._h:
            _lib.load().litenn_hip_model_free(self._h)
            self._h = C.c_void_p()

    def __enter__(self):
        return self

    def __exit__(self, *exc):
        self.close()

    def __del__(self):
        try:
            self.close()
        except Exception:
            pass

    @property
    def past(self) -> int:
        """Tokens of the sequence so far."""
        return _lib.load().litenn_hip_model_past(self._h)

    def reset(self) -> None:
        check(_lib.load().litenn_hip_model_reset(self._h))

    def eval(self, tokens, want=None, precise: bool = False) -> np.ndarray:
        """Feeds the tokens behind the sequence so far; logits [len(want), vocab] at the wanted places among
        them, or of all of them when want is None."""
        t = np.ascontiguousarray(tokens, np.int32).reshape(-1)
        flags = MATMUL_PRECISE if precise else 0
        if want is None:
            out = np.empty((t.size, self.vocab_size), np.float32)
            check(_lib.load().litenn_hip_model_eval(self._h, t.ctypes.data, t.size, None, 0, out.ctypes.data, flags))
            return out
        w = np.ascontiguousarray(want, np.int32).reshape(-1)
        out = np.empty((w.size, self.vocab_size), np.float32)
        check(_lib.load().litenn_hip_model_eval(self._h, t.ctypes.data, t.size, w.ctypes.data, w.size, out.ctypes.data,
                                                flags))
        return out

    def generate(self, prompt, n_new: int, precise: bool = False):
        """Greedy decode on the device; returns (tokens, prefill_ms, decode_ms)."""
        t = np.ascontiguousarray(prompt, np.int32).reshape(-1)
        out = np.empty((n_new,), np.int32)
        pre, dec = C.c_double(), C.c_double()
        check(_lib.load().litenn_hip_model_generate(self._h, t.ctypes.data, t.size, n_new, out.ctypes.data,
                                                    MATMUL_PRECISE if precise else 0, C.byref(pre), C.byref(dec)))
        return out, pre.value, dec.value


def load_model(path, dtype="bfloat16", context_length: int = 0, device: HIP = HIP()) -> Model:
    """dtype: "bfloat16" (the precisions the model is served with) or "float32" (every operand and cache)."""
    h = C.c_void_p()
    check(_lib.load().litenn_hip_model_load(device.deviceIndex, str(path).encode(), DTYPES[dtype], context_length,
                                            C.byref(h)))
    return Model(h)


def to_bfloat16(x) -> np.ndarray:
    """Float32 values as the bits of the nearest bfloat16 (ties to even)."""
    b = np.ascontiguousarray(x, np.float32).view(np.uint32)
    return ((b + 0x7FFF + ((b >> 16) & 1)) >> 16).astype(np.uint16)


def from_bfloat16(bits) -> np.ndarray:
    return (np.ascontiguousarray(bits, np.uint16).astype(np.uint32) << 16).view(np.float32)


def create_model(config: dict, tensors, dtype="bfloat16", context_length: int = 0, device: HIP = HIP()) -> Model:
    """tensors: {name: uint16 array of bfloat16 bits, or float32 array (vectors only)}."""
    keep, descs = [], (ModelTensor * len(tensors))()
    for d, (name, a) in zip(descs, tensors.items()):
        a = np.ascontiguousarray(a)
        if a.dtype not in (np.uint16, np.float32):
            raise ValueError(f"tensor {name!r} is neither bfloat16 bits nor float32")
        keep.append((name.encode(), a))
        d.name = keep[-1][0]
        d.dtype = DT_BF16 if a.dtype == np.uint16 else DT_F32
        d.rank = a.ndim
        d.shape[:a.ndim] = a.shape
        d.data = a.ctypes.data
    h = C.c_void_p()
    check(_lib.load().litenn_hip_model_create(device.deviceIndex, json.dumps(config).encode(), descs, len(tensors),
                                              DTYPES[dtype], context_length, C.byref(h)))
    return Model(h)
