"""Host mirror of the model-folder reader in ``libwick_rocm.so`` (``include/wick_safetensors.h``), and a writer of such folders
(random-weight models of the tests and the benchmark)."""
from __future__ import annotations

import ctypes as C
import json
import os
from typing import Dict, List, Tuple

import numpy as np

from . import rocm

_P = C.c_void_p
BF16, F32, I32 = 0, 1, 2

_SIGNATURES = {
    "wick_safetensors_last_error": (C.c_char_p, []),
    "wick_safetensors_open": (C.c_int, [C.c_char_p, C.POINTER(_P)]),
    "wick_safetensors_close": (None, [_P]),
    "wick_safetensors_architecture": (C.c_char_p, [_P]),
    "wick_safetensors_config": (C.c_char_p, [_P, C.POINTER(C.c_size_t)]),
    "wick_safetensors_tensor_count": (C.c_uint64, [_P]),
    "wick_safetensors_tensor_name": (C.c_char_p, [_P, C.c_uint64]),
    "wick_safetensors_tensor": (C.c_int, [_P, C.c_char_p, C.POINTER(C.c_int), C.POINTER(C.c_uint32), C.POINTER(C.c_uint64), C.POINTER(_P),
                                          C.POINTER(C.c_size_t)]),
}
_bound = False


class CheckpointError(RuntimeError):
    def __init__(self, status: int, message: str):
        self.status = status
        super().__init__(f"wick_safetensors status {status}: {message}")


def _lib() -> C.CDLL:
    global _bound
    lib = rocm.load_library()
    if not _bound:
        for name, (res, args) in _SIGNATURES.items():
            fn = getattr(lib, name)
            fn.restype, fn.argtypes = res, args
        _bound = True
    return lib


def to_bf16(a) -> np.ndarray:
    """f32 values -> bfloat16 bit patterns (uint16), round to nearest even."""
    u = np.ascontiguousarray(a, np.float32).view(np.uint32)
    return ((u + np.uint32(0x7FFF) + ((u >> np.uint32(16)) & np.uint32(1))) >> np.uint32(16)).astype(np.uint16)


def from_bf16(b) -> np.ndarray:
    return (np.asarray(b, np.uint16).astype(np.uint32) << np.uint32(16)).view(np.float32)


def write_folder(path: str, config: dict, tensors: Dict[str, np.ndarray]) -> None:
    """config.json and model.safetensors.  uint16 arrays are bfloat16 bit patterns, int32 integers, floats are rounded to bfloat16."""
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(config, f)
    header, blobs, at = {}, [], 0
    for name, a in tensors.items():
        a = np.asarray(a)
        if a.dtype.kind == "f":
            a = to_bf16(a).reshape(a.shape)
        dtype = {"uint16": "BF16", "int32": "I32"}[a.dtype.name]
        header[name] = {"dtype": dtype, "shape": list(a.shape), "data_offsets": [at, at + a.nbytes]}
        at += a.nbytes
        blobs.append(a)
    text = json.dumps(header).encode()
    text += b" " * (-len(text) % 8)
    with open(os.path.join(path, "model.safetensors"), "wb") as f:
        f.write(len(text).to_bytes(8, "little"))
        f.write(text)
        for a in blobs:
            f.write(np.ascontiguousarray(a).tobytes())


class ModelFolder:
    """An open model folder."""

    def __init__(self, path: str):
        self._l = _lib()
        h = _P()
        self._check(self._l.wick_safetensors_open(os.fsencode(path), C.byref(h)))
        self.handle = h.value

    def _check(self, rc: int) -> None:
        if rc != 0:
            raise CheckpointError(rc, self._l.wick_safetensors_last_error().decode("utf-8", "replace"))

    def close(self) -> None:
        if self.handle:
            self._l.wick_safetensors_close(self.handle)
            self.handle = None

    def __enter__(self):
        return self

    def __exit__(self, *exc):
        self.close()

    @property
    def architecture(self) -> str:
        return self._l.wick_safetensors_architecture(self.handle).decode()

    @property
    def config(self) -> dict:
        n = C.c_size_t()
        return json.loads(self._l.wick_safetensors_config(self.handle, C.byref(n)).decode())

    def names(self) -> List[str]:
        return [self._l.wick_safetensors_tensor_name(self.handle, i).decode() for i in range(self._l.wick_safetensors_tensor_count(self.handle))]

    def tensor(self, name: str) -> Tuple[int, np.ndarray]:
        """(dtype, values): bfloat16 as uint16 bit patterns."""
        dtype, nd, dims, data, n = C.c_int(), C.c_uint32(), (C.c_uint64 * 8)(), _P(), C.c_size_t()
        self._check(self._l.wick_safetensors_tensor(self.handle, name.encode(), C.byref(dtype), C.byref(nd), dims, C.byref(data), C.byref(n)))
        np_type = {BF16: np.uint16, F32: np.float32, I32: np.int32}[dtype.value]
        raw = C.string_at(data.value, n.value) if n.value else b""
        return dtype.value, np.frombuffer(raw, np_type).reshape([dims[i] for i in range(nd.value)])
