"""ctypes face of layered runtimes built without a model directory (measurement and tests; a model directory goes through
engine.RealModelInferenceEngine) and of their measurement calls."""
from __future__ import annotations

import ctypes as C
import json

import numpy as np

from . import _lib, llama

KERNEL_CLASSES = ("in", "retention", "latent", "out", "head", "norm", "attention", "mamba2")


class LayeredRuntime(llama.LlamaRuntime):
    """A runtime of `config` (the content of a config.json) with seeded random weights."""

    def __init__(self, config: dict, max_seq: int, float32: bool = False, max_sequences: int = 1, seed: int = 1, std: float = 0.02):
        self._L, self._h = _lib.load_library(), None
        layers = config["layers"]
        self.config = config
        self.cfg = llama.MultiModelConfig(n_layer=len(layers), n_head=layers[0]["mixer"]["heads"], n_kv_head=layers[0]["mixer"]["heads"],
                                          d_model=config["width"], head_dim=layers[0]["mixer"].get("dim", layers[0]["mixer"]["vdim"]),
                                          hidden_dim=max((l["mlp"] or {}).get("ff", 0) for l in layers), vocab=config["vocab"], max_seq=max_seq,
                                          name=config["architecture"], architecture="layered")
        self._L.esp_layered_create_synthetic.restype = C.c_void_p
        self._L.esp_layered_create_synthetic.argtypes = [C.c_char_p, C.c_int, C.c_int, C.c_int, C.c_uint64, C.c_float]
        self._h = self._L.esp_layered_create_synthetic(json.dumps(config).encode(), int(float32), max_seq, max_sequences, seed, std)
        if not self._h:
            raise _lib.EspressoError(-1, _lib.last_error())


def set_min_block_rows(rt: llama.LlamaRuntime, rows: int) -> None:
    rt._L.esp_layered_set_min_block_rows.argtypes = [C.c_void_p, C.c_int]
    _lib.check(rt._L.esp_layered_set_min_block_rows(rt._h, rows))


def trace_layers(rt: llama.LlamaRuntime, tokens, sequence: int = 0) -> np.ndarray:
    """Appends `tokens` as one block; the residual stream after every layer, [layers, tokens, width]."""
    t = np.ascontiguousarray(tokens, dtype=np.uint32)
    out = np.empty((rt.cfg.n_layer, t.size, rt.cfg.d_model), dtype=np.float32)
    rt._L.esp_layered_trace_layers.argtypes = [C.c_void_p, C.c_int, C.c_void_p, C.c_int, C.c_void_p]
    _lib.check(rt._L.esp_layered_trace_layers(rt._h, sequence, t.ctypes.data_as(C.c_void_p), t.size, out.ctypes.data_as(C.c_void_p)))
    return out


def sequence_bytes(rt: llama.LlamaRuntime) -> int:
    rt._L.esp_layered_sequence_bytes.restype = C.c_longlong
    rt._L.esp_layered_sequence_bytes.argtypes = [C.c_void_p]
    return int(rt._L.esp_layered_sequence_bytes(rt._h))


def set_kernel_timing(rt: llama.LlamaRuntime, enabled: bool) -> None:
    rt._L.esp_layered_set_kernel_timing.argtypes = [C.c_void_p, C.c_int]
    _lib.check(rt._L.esp_layered_set_kernel_timing(rt._h, int(enabled)))


def kernel_times(rt: llama.LlamaRuntime, reset: bool = True) -> dict:
    """{class: {"total_us", "brackets", "step_bytes"}} from HIP events; a bracket holds a layer's launches of the class."""
    n = len(KERNEL_CLASSES)
    us, launches, nbytes = np.zeros(n), np.zeros(n, dtype=np.int64), np.zeros(n, dtype=np.uint64)
    rt._L.esp_layered_kernel_times.argtypes = [C.c_void_p] * 4 + [C.c_int]
    _lib.check(rt._L.esp_layered_kernel_times(rt._h, us.ctypes.data_as(C.c_void_p), launches.ctypes.data_as(C.c_void_p), nbytes.ctypes.data_as(C.c_void_p), int(reset)))
    return {k: {"total_us": float(us[i]), "brackets": int(launches[i]), "step_bytes": int(nbytes[i])} for i, k in enumerate(KERNEL_CLASSES)}
