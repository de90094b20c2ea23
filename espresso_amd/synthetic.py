"""Seeded random-init llama models in packed GGUF formats, built on the GPU (ops.synth_weights).

One stream id per tensor: stream = seed * 1000 + layer * 16 + tensor index, so a model is a pure
function of (config, seed, format)."""
from __future__ import annotations

import numpy as np

from . import _lib, llama, ops

_TENSORS = ("wq", "wk", "wv", "wo", "w1", "w2", "w3")


def matrix_shapes(cfg: llama.MultiModelConfig) -> dict:
    ad, kd, d, hd = cfg.attention_dim, cfg.kv_dim, cfg.d_model, cfg.hidden_dim
    return {"wq": (ad, d), "wk": (kd, d), "wv": (kd, d), "wo": (d, ad), "w1": (hd, d), "w3": (hd, d), "w2": (d, hd)}


def build_runtime(cfg: llama.MultiModelConfig, matrix_format: int, seed: int, std: float = 0.02,
                  kv_format: int = _lib.FORMAT_F32, max_sequences: int = 1, keep_packed: bool = False,
                  head_format: int | None = None, zero_upper_outputs: bool = False):
    """Random-init model: every linear ~N(0, std) in `matrix_format`, embedding fp16 ~N(0, std), norm weights 1.
    Returns (runtime, packed) where packed holds the GGUF-layout bytes when keep_packed is set.  Tensor seeds do not depend
    on the layer count, so a model built with fewer layers from the same seed is a prefix of the deeper one.
    zero_upper_outputs: wo and w2 of every layer above the first are all-zero blocks, i.e. those layers cost what they
    always cost and add nothing to the residual stream: the model's tokens are those of its first layer alone."""
    rt = llama.LlamaRuntime(cfg, kv_format=kv_format, max_sequences=max_sequences)
    shapes = matrix_shapes(cfg)
    head_format = matrix_format if head_format is None else head_format
    packed = {"layers": []} if keep_packed else None
    ones = np.ones(cfg.d_model, dtype=np.float16)

    def put(layer, name, slot, fmt, data):
        rt.set_weight(layer, slot, fmt, data)
        if packed is not None:
            (packed["layers"][layer] if layer >= 0 and name in llama.LAYER_SLOTS else packed)[name] = data

    base = seed * 1000
    emb = ops.synth_weights(_lib.FORMAT_F16, base + 1, std, cfg.vocab * cfg.d_model)
    put(-1, "embedding", llama.SLOT_TOKEN_EMBEDDING, _lib.FORMAT_F16, emb)
    put(-1, "final_norm", llama.SLOT_FINAL_NORM, _lib.FORMAT_F16, ones.view(np.uint8))
    head = ops.synth_weights(head_format, base + 2, std, cfg.vocab * cfg.d_model)
    put(-1, "lm_head", llama.SLOT_LM_HEAD, head_format, head)
    del emb, head
    for l in range(cfg.n_layer):
        if packed is not None:
            packed["layers"].append({})
        put(l, "rms_att", llama.SLOT_RMS_ATT, _lib.FORMAT_F16, ones.view(np.uint8))
        put(l, "rms_ffn", llama.SLOT_RMS_FFN, _lib.FORMAT_F16, ones.view(np.uint8))
        for i, name in enumerate(_TENSORS):
            r, c = shapes[name]
            if zero_upper_outputs and l >= 1 and name in ("wo", "w2"):
                data = np.zeros(ops.format_bytes(matrix_format, r * c), dtype=np.uint8)
            else:
                data = ops.synth_weights(matrix_format, base + 16 * (l + 1) + i, std, r * c)
            put(l, name, llama.LAYER_SLOTS[name], matrix_format, data)
    rt.finalize()
    return rt, packed


STORIES_6L = dict(n_layer=6, n_head=12, n_kv_head=12, d_model=768, head_dim=64, hidden_dim=2048, vocab=32000,
                  max_seq=256, norm_eps=1e-5, rope_theta=10000.0, name="stories-6l-d768")
LLAMA3_8B = dict(n_layer=32, n_head=32, n_kv_head=8, d_model=4096, head_dim=128, hidden_dim=14336, vocab=128256,
                 max_seq=1024, norm_eps=1e-5, rope_theta=500000.0, name="llama3-8b-arch")


def layered_config(width: int, ff: int, vocab: int, attention: dict, retention: dict, layers: int = 6, window: int = 1024) -> dict:
    """A config.json of a layered model: latent attention, two retention layers, latent attention over the first one's latents, two
    retention layers, and so on."""
    out = []
    for i in range(layers):
        mlp = {"kind": "dense", "ff": ff}
        if i % 3:
            heads = retention["heads"]
            decay = [1.0 - 2.0 ** -(5.0 + 7.0 * h / max(heads - 1, 1)) for h in range(heads)]
            out.append({"type": "retention", "mlp": mlp, "mixer": dict(retention, decay=decay, rot={"base": 1000000.0, "dims": retention["dim"]})})
        else:
            m = dict(attention, scale=(attention["dim"] + attention["rot_dim"]) ** -0.5, mask={"size": window},
                     rot={"base": 10000.0, "dims": attention["rot_dim"], "scaling": {"factor": 4.0, "original": 4096, "fast": 32.0, "slow": 1.0}})
            if i % 6 == 3:
                m["kv_from"] = i - 3
            out.append({"type": "latent_attention", "mlp": mlp, "mixer": m})
    return {"architecture": "Ranavik", "vocab": vocab, "width": width, "residual_mult": 0.5, "logit_softcap": 30.0, "norm": {"eps": 1e-6}, "layers": out}


# Layers of the size of real models, six of them, and the llama model of equal width, feed-forward, vocabulary and depth.
LAYERED_SIZES = {
    "d768": (layered_config(768, 2048, 32000, dict(heads=12, dim=64, vdim=64, rot_dim=32, kv_rank=256), dict(heads=6, dim=128, vdim=128)),
             dict(n_layer=6, n_head=12, n_kv_head=12, d_model=768, head_dim=64, hidden_dim=2048, vocab=32000, max_seq=1024)),
    "d2048": (layered_config(2048, 8192, 32000, dict(heads=16, dim=128, vdim=128, rot_dim=64, kv_rank=512), dict(heads=8, dim=256, vdim=256)),
              dict(n_layer=6, n_head=32, n_kv_head=8, d_model=2048, head_dim=64, hidden_dim=8192, vocab=32000, max_seq=1024)),
    "d4096": (layered_config(4096, 14336, 32000, dict(heads=32, dim=128, vdim=128, rot_dim=64, kv_rank=512), dict(heads=16, dim=256, vdim=256)),
              dict(n_layer=6, n_head=32, n_kv_head=8, d_model=4096, head_dim=128, hidden_dim=14336, vocab=32000, max_seq=1024)),
}


def sequential_config(width: int, ff: int, vocab: int, attention: dict, mamba2: dict, mamba2_2: dict, layers: int = 6, window: int = 1024) -> dict:
    """A config.json of a layered model of the other design: an attention layer with a feed-forward and two Mamba-2 layers of different
    sizes, again and again; every second attention layer reads the keys and values of the one before."""
    out = []
    for i in range(layers):
        if i % 3:
            out.append({"type": ("mamba2", "mamba2_2")[i % 3 - 1], "mlp": None, "mixer": dict((mamba2, mamba2_2)[i % 3 - 1])})
        else:
            m = dict(attention, scale=attention["dim"] ** -0.5, mask={"size": window}, rot={"base": 500000.0, "dims": attention["dim"] // 2, "scaling": {"factor": 2.0}})
            if i % 6 == 3:
                m["kv_from"] = i - 3
            out.append({"type": "attention", "mlp": {"kind": "dense", "ff": ff}, "mixer": m})
    return {"architecture": "Forovik", "vocab": vocab, "width": width, "norm": {"eps": 1e-6}, "layers": out}


def _mamba2(heads: int, vdim: int, state: int, groups: int, conv: int = 4) -> dict:
    return {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": conv, "norm_groups": groups}


# The same widths and feed-forwards: (configuration, the size in LAYERED_SIZES to measure beside it).
SEQUENTIAL_SIZES = {
    "forovik-d768": (sequential_config(768, 2048, 32000, dict(heads=12, kv_heads=4, dim=64, vdim=64), _mamba2(24, 64, 128, 1), _mamba2(12, 128, 64, 2, 3)), "d768"),
    "forovik-d2048": (sequential_config(2048, 8192, 32000, dict(heads=16, kv_heads=4, dim=128, vdim=128), _mamba2(64, 64, 128, 8), _mamba2(32, 128, 64, 4, 3)), "d2048"),
    "forovik-d4096": (sequential_config(4096, 14336, 32000, dict(heads=32, kv_heads=8, dim=128, vdim=128), _mamba2(128, 64, 128, 8), _mamba2(64, 128, 64, 8, 3)), "d4096"),
}
