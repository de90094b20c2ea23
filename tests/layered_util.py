"""Small layered models for tests: configurations, seeded weights, model directories, and comparisons with the plain statement."""
import json
import os

import numpy as np

import layered_ref as ref


def rotary(dims, base=10000.0, scaling=None):
    r = {"dims": dims, "base": base}
    if scaling:
        r["scaling"] = scaling
    return r


YARN = {"factor": 4.0, "original": 256, "fast": 16.0, "slow": 1.0}


def retention(heads=2, dim=16, vdim=16, dims=None, base=50000.0, decay=None, ff=48):
    decay = [1.0 - 2.0 ** -(3.0 + h) for h in range(heads)] if decay is None else decay
    return {"type": "retention", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay, "rot": rotary(dim if dims is None else dims, base)},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def latent(heads=3, dim=16, vdim=24, kv_rank=40, rot_dim=8, window=20, scale=None, scaling=YARN, base=10000.0, kv_from=None, ff=48):
    m = {"heads": heads, "dim": dim, "vdim": vdim, "kv_rank": kv_rank, "rot_dim": rot_dim, "scale": (dim + rot_dim) ** -0.5 if scale is None else scale,
         "mask": {"size": window}, "rot": rotary(rot_dim, base, scaling)}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m, "mlp": {"kind": "dense", "ff": ff} if ff else None}


def attention(heads=4, kv_heads=2, dim=16, vdim=24, dims=8, window=20, scale=None, base=10000.0, factor=None, kv_from=None, ff=48):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": dim ** -0.5 if scale is None else scale, "mask": {"size": window},
         "rot": rotary(dims, base, None if factor is None else {"factor": factor})}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "attention", "mixer": m, "mlp": {"kind": "dense", "ff": ff} if ff else None}


def mamba2(heads=4, vdim=16, state=24, groups=2, conv=4, norm_groups=2, ff=0, kind="mamba2"):
    return {"type": kind, "mixer": {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": conv, "norm_groups": norm_groups},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def sequential(layers, vocab=96, width=56, eps=1e-5):
    return {"architecture": "Forovik", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}


def config(layers, vocab=96, width=56, residual_mult=0.7, softcap=25.0, eps=1e-5):
    return {"architecture": "Ranavik", "vocab": vocab, "width": width, "residual_mult": residual_mult, "logit_softcap": softcap, "norm": {"eps": eps},
            "layers": layers}


def tensor_shapes(cfg):
    d, out = cfg["width"], {"embed": (cfg["vocab"], cfg["width"]), "final.norm": (cfg["width"],)}
    if cfg["architecture"] == "Ranavik":
        out.update({"embed.norm": (d,), "head": (cfg["vocab"], d)})
    for i, layer in enumerate(cfg["layers"]):
        m, p = layer["mixer"], f"l{i}."
        out[p + "norm1"] = (d,)
        if layer["type"] == "retention":
            qk, v = m["heads"] * m["dim"], m["heads"] * m["vdim"]
            out.update({p + "mix.q": (qk, d), p + "mix.k": (qk, d), p + "mix.v": (v, d), p + "mix.g": (v, d), p + "mix.o": (d, v)})
        elif layer["type"].startswith("mamba2"):
            h, inner, shared = m["heads"], m["heads"] * m["vdim"], m["groups"] * m["state"]
            out.update({p + "mix.in": (2 * inner + 2 * shared + h, d), p + "mix.conv": (inner + 2 * shared, m["conv"]), p + "mix.conv.b": (inner + 2 * shared,),
                        p + "mix.dt_bias": (h,), p + "mix.A_log": (h,), p + "mix.D": (h,), p + "mix.norm": (inner,), p + "mix.o": (d, inner)})
        elif layer["type"] == "attention":
            q, k = m["heads"] * m["dim"], m["kv_heads"] * m["dim"]
            out.update({p + "mix.q": (q, d), p + "mix.q.norm": (q,), p + "mix.o": (d, m["heads"] * m["vdim"])})
            if m.get("kv_from") is None:
                out.update({p + "mix.k": (k, d), p + "mix.k.norm": (k,), p + "mix.v": (m["kv_heads"] * m["vdim"], d)})
        else:
            h = m["heads"]
            out.update({p + "mix.q": (h * (m["dim"] + m["rot_dim"]), d), p + "mix.uk": (h * m["dim"], m["kv_rank"]), p + "mix.uv": (h * m["vdim"], m["kv_rank"]),
                        p + "mix.sink": (h,), p + "mix.g": (h, d), p + "mix.o": (d, h * m["vdim"])})
            if m.get("kv_from") is None:
                out.update({p + "mix.dkv": (m["kv_rank"] + m["rot_dim"], d), p + "mix.dkv.norm": (m["kv_rank"],)})
        if layer["mlp"]:
            ff = layer["mlp"]["ff"]
            out.update({p + "norm2": (d,), p + "mlp.gate": (ff, d), p + "mlp.up": (ff, d), p + "mlp.down": (d, ff)})
    return out


def to_bf16(x):
    """fp32 -> the nearest bf16 value, as fp32."""
    b = np.ascontiguousarray(x, dtype=np.float32).view(np.uint32)
    return ((b + 0x7FFF + ((b >> 16) & 1)) & 0xFFFF0000).astype(np.uint32).view(np.float32)


def random_weights(cfg, seed, gain=1.0, sink=None):
    """Linears ~N(0, gain / sqrt(inputs)), norms around 1, sinks ~N(0, 1) (or the given value), decays from a few tokens to hundreds; every
    value is a bf16 number."""
    rng = np.random.default_rng(seed)
    w = {}
    for name, shape in sorted(tensor_shapes(cfg).items()):
        if name.endswith("sink"):
            a = rng.normal(0, 1, shape) if sink is None else np.full(shape, sink)
        elif name.endswith("A_log"):
            a = rng.uniform(-3.0, 1.0, shape)
        elif name.endswith("dt_bias"):
            a = rng.uniform(-3.0, 1.0, shape)
        elif name.endswith("conv.b"):
            a = rng.normal(0, 0.3, shape)
        elif len(shape) == 1:
            a = rng.uniform(0.6, 1.4, shape)
        else:
            a = rng.normal(0, 1.0 if name == "embed" else gain / np.sqrt(shape[1]), shape)
        w[name] = to_bf16(a)
    return w


def write_model(path, cfg, weights):
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    header, blobs, at = {}, [], 0
    for name, a in weights.items():
        raw = (np.ascontiguousarray(a, dtype=np.float32).view(np.uint32) >> 16).astype("<u2").tobytes()
        header[name] = {"dtype": "BF16", "shape": list(a.shape), "data_offsets": [at, at + len(raw)]}
        blobs.append(raw)
        at += len(raw)
    h = json.dumps(header).encode()
    with open(os.path.join(path, "model.safetensors"), "wb") as f:
        f.write(len(h).to_bytes(8, "little") + h + b"".join(blobs))
    return str(path)


class Model:
    """One model in a directory, its plain statement, and engines over it."""

    def __init__(self, tmp_path, cfg, seed=0, gain=1.0, sink=None):
        self.cfg = cfg
        self.weights = random_weights(cfg, seed, gain, sink)
        self.dir = write_model(str(tmp_path), cfg, self.weights)

    def engine(self, precision="f32", max_seq=256, sequences=4, eos=None):
        import espresso_amd.engine as eng
        c = eng.load_model_config(self.dir, max_seq)
        if eos is not None:
            c.eos_token = eos
        return eng.RealModelInferenceEngine(c, self.dir, environment={"ESPRESSO_HIP_PRECISION": precision, "ESPRESSO_HIP_MAX_SEQUENCES": str(sequences)})

    def runtime(self, precision="f32", max_seq=256, sequences=4):
        return self.engine(precision, max_seq, sequences).runtime()

    def logits(self, tokens, layers_out=None):
        return ref.forward(self.cfg, self.weights, tokens, layers_out)

    def greedy(self, prompt, count):
        tokens = list(prompt)
        for _ in range(count):
            tokens.append(int(np.argmax(self.logits(tokens)[-1])))
        return tokens[len(prompt):]


def tokens(cfg, count, seed=0):
    return np.random.default_rng(1000 + seed).integers(0, cfg["vocab"], count).tolist()


def error(got, want):
    """The worst position's root mean square difference, over the spread of the expected values."""
    d = np.asarray(got, dtype=np.float64) - want
    return float(np.sqrt((d * d).mean(axis=-1)).max() / np.std(want))


F32_LIMIT, BF16_LIMIT = 3e-5, 8e-2


def limit(precision):
    return F32_LIMIT if precision == "f32" else BF16_LIMIT


def feed(rt, seq_tokens, portions, sequence=0):
    """All logits of a sequence fed in the given portions (the last one repeats)."""
    out, at, i = [], 0, 0
    while at < len(seq_tokens):
        n = min(portions[min(i, len(portions) - 1)], len(seq_tokens) - at)
        out.append(rt.append(seq_tokens[at:at + n], list(range(n)), sequence=sequence))
        at += n
        i += 1
    return np.concatenate(out)
