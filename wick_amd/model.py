"""Host mirror of ``include/wick_rocm_model.h``: one handle over every model the library knows, chosen by what the file says it
is, with the step calls of the reference's ``trait Model`` (wick/src/model/mod.rs:72-323), and the loop of a generation over it."""
from __future__ import annotations

import ctypes as C
import os
from typing import Callable, List, Optional, Sequence

import numpy as np

from . import rocm
from .rocm import RocmContext

_P, _U32 = C.c_void_p, C.c_uint32
NATIVE, F32 = 0, 1  # what a model computes in


class ModelInfo(C.Structure):
    _fields_ = [("architecture", C.c_char * 32), ("vocab_size", _U32), ("hidden_size", _U32), ("max_seq_len", _U32), ("layer_runs", _U32),
                ("dtype", C.c_int)]


_SIGNATURES = {
    "wick_rocm_model_folder_architecture": (C.c_char_p, [_U32]),
    "wick_rocm_model_from_folder": (C.c_int, [_P, _P, C.c_int, _U32, C.POINTER(_P)]),
    "wick_rocm_model_from_gguf": (C.c_int, [_P, _P, C.c_int, _U32, C.POINTER(_P)]),
    "wick_rocm_model_load": (C.c_int, [_P, C.c_char_p, C.c_int, _U32, C.POINTER(_P)]),
    "wick_rocm_model_free": (C.c_int, [_P, _P]),
    "wick_rocm_model_get_info": (C.c_int, [_P, C.POINTER(ModelInfo)]),
    "wick_rocm_model_gpu_memory_bytes": (C.c_size_t, [_P]),
    "wick_rocm_model_set_graph_replay": (C.c_int, [_P, C.c_int]),
    "wick_rocm_model_reset": (C.c_int, [_P, _P]),
    "wick_rocm_model_forward": (C.c_int, [_P, _P, _P, _U32, _U32, _P, _U32, _P]),
    "wick_rocm_model_forward_layers": (C.c_int, [_P, _P, _P, _U32, _U32, _P]),
    "wick_rocm_model_prefill_chunked": (C.c_int, [_P, _P, _P, _U32, _U32, _U32, _P, C.POINTER(_U32), _P]),
    "wick_rocm_model_generate_greedy": (C.c_int, [_P, _P, _U32, _U32, _U32, _P]),
    "wick_rocm_model_state_bytes": (C.c_size_t, [_P, _U32]),
    "wick_rocm_model_snapshot_state": (C.c_int, [_P, _P, _U32, _P, C.c_size_t]),
    "wick_rocm_model_restore_state": (C.c_int, [_P, _P, _U32, _P, C.c_size_t]),
}
_bound = False


def _lib() -> C.CDLL:
    global _bound
    lib = rocm.load_library()
    if not _bound:
        for name, (res, args) in _SIGNATURES.items():
            fn = getattr(lib, name)
            fn.restype, fn.argtypes = res, args
        _bound = True
    return lib


def folder_architectures() -> List[str]:
    """The architectures a model folder's config.json may name."""
    out, i = [], 0
    while True:
        name = _lib().wick_rocm_model_folder_architecture(i)
        if name is None:
            return out
        out.append(name.decode())
        i += 1


class RocmModel:
    """A model folder or GGUF file on the GPU; holds one sequence's state."""

    def __init__(self, ctx: RocmContext, source, context_size: int, dtype: int = NATIVE):
        """source: a path, an open ``ModelFolder`` or an open ``GgufFile``."""
        from .checkpoint import ModelFolder

        self.ctx, self._l = ctx, _lib()
        h = _P()
        if isinstance(source, ModelFolder):
            rc = self._l.wick_rocm_model_from_folder(ctx._h, source.handle, dtype, context_size, C.byref(h))
        elif isinstance(source, (str, os.PathLike)):
            rc = self._l.wick_rocm_model_load(ctx._h, os.fsencode(source), dtype, context_size, C.byref(h))
        else:
            rc = self._l.wick_rocm_model_from_gguf(ctx._h, source.handle, dtype, context_size, C.byref(h))
        ctx._check(rc)
        self._h = h.value
        info = ModelInfo()
        ctx._check(self._l.wick_rocm_model_get_info(self._h, C.byref(info)))
        self.architecture = info.architecture.decode()
        self.vocab_size, self.hidden_size, self.max_seq_len, self.layer_runs = info.vocab_size, info.hidden_size, info.max_seq_len, info.layer_runs

    def free(self) -> None:
        if self._h:
            self.ctx._check(self._l.wick_rocm_model_free(self.ctx._h, self._h))
            self._h = None

    def __enter__(self):
        return self

    def __exit__(self, *exc):
        self.free()

    def gpu_memory_bytes(self) -> int:
        return int(self._l.wick_rocm_model_gpu_memory_bytes(self._h))

    def set_graph_replay(self, enabled: bool) -> None:
        self.ctx._check(self._l.wick_rocm_model_set_graph_replay(self._h, int(enabled)))

    def reset(self) -> None:
        self.ctx._check(self._l.wick_rocm_model_reset(self.ctx._h, self._h))

    def forward(self, tokens: Sequence[int], start_pos: int, want: Optional[Sequence[int]] = None) -> np.ndarray:
        """Logits [len(want)][vocab] of the wanted places (default: the last token's)."""
        t = np.ascontiguousarray(tokens, np.uint32)
        w = np.ascontiguousarray([t.size - 1] if want is None else want, np.uint32)
        out = np.empty((w.size, self.vocab_size), np.float32)
        self.ctx._check(self._l.wick_rocm_model_forward(self.ctx._h, self._h, t.ctypes.data, t.size, start_pos, w.ctypes.data, w.size, out.ctypes.data))
        return out

    def forward_layers(self, tokens: Sequence[int], start_pos: int) -> np.ndarray:
        """The residual stream after every layer run, [layer_runs][n][hidden]."""
        t = np.ascontiguousarray(tokens, np.uint32)
        out = np.empty((self.layer_runs, t.size, self.hidden_size), np.float32)
        self.ctx._check(self._l.wick_rocm_model_forward_layers(self.ctx._h, self._h, t.ctypes.data, t.size, start_pos, out.ctypes.data))
        return out

    def prefill_chunked(self, tokens: Sequence[int], start_pos: int, ubatch: int = 0, cancel=None):
        """Model::forward_prefill_chunked: (tokens consumed, logits of the last processed chunk or None)."""
        t = np.ascontiguousarray(tokens, np.uint32)
        logits, consumed = np.empty(self.vocab_size, np.float32), _U32()
        self.ctx._check(self._l.wick_rocm_model_prefill_chunked(self.ctx._h, self._h, t.ctypes.data, t.size, start_pos, ubatch,
                                                                C.addressof(cancel) if cancel is not None else None, C.byref(consumed), logits.ctypes.data))
        return consumed.value, (logits if consumed.value else None)

    def generate_greedy(self, token: int, pos: int, n: int) -> np.ndarray:
        out = np.empty(n, np.uint32)
        self.ctx._check(self._l.wick_rocm_model_generate_greedy(self.ctx._h, self._h, token, pos, n, out.ctypes.data))
        return out

    def snapshot_state(self, seq_len: int) -> np.ndarray:
        out = np.empty(int(self._l.wick_rocm_model_state_bytes(self._h, seq_len)), np.uint8)
        self.ctx._check(self._l.wick_rocm_model_snapshot_state(self.ctx._h, self._h, seq_len, out.ctypes.data, out.size))
        return out

    def restore_state(self, snapshot, seq_len: int) -> None:
        b = np.ascontiguousarray(snapshot, np.uint8)
        self.ctx._check(self._l.wick_rocm_model_restore_state(self.ctx._h, self._h, seq_len, b.ctypes.data, b.size))


def greedy_pick(logits: np.ndarray) -> int:
    """cpu_argmax (wick/src/sampler.rs:7-19): NaN counts as -inf, the last of equal maxima wins."""
    x = np.where(np.isnan(logits), -np.inf, logits)
    return int(x.size - 1 - np.argmax(x[::-1]))


def generate(model: RocmModel, prompt: Sequence[int], max_new: int, stop: Sequence[int] = (), ubatch: int = 0,
             sample: Optional[Callable[[np.ndarray], int]] = None, start_pos: int = 0) -> List[int]:
    """The tokens that follow `prompt`.  Greedy picks (sample None) are made on the GPU in bursts; `sample` gets every step's logits."""
    prompt = list(prompt)
    if max_new <= 0 or not prompt:
        return []
    _, logits = model.prefill_chunked(prompt, start_pos, ubatch)
    pos = start_pos + len(prompt)
    out = [greedy_pick(logits) if sample is None else int(sample(logits))]
    stops = {int(s) for s in stop}
    while len(out) < max_new and out[-1] not in stops and pos < model.max_seq_len:
        if sample is None:
            burst = [int(t) for t in model.generate_greedy(out[-1], pos, min(max_new - len(out), 32, model.max_seq_len - pos))]
            hit = next((i for i, t in enumerate(burst) if t in stops), len(burst) - 1)
            out += burst[:hit + 1]
            pos += hit + 1
        else:
            out.append(int(sample(model.forward([out[-1]], pos)[0])))
            pos += 1
    return out
