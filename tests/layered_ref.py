"""Plain numpy statement of the layered decoder models (architectures "Ranavik" and "Forovik"), one function per mechanism.

Everything is float64 and written token by token where the mechanism is a recurrence, with no tiles, chunks, caches or
absorbed products, and nothing here is shared with the product.  `weights` maps tensor names to arrays ([out, in] for
linears); `config` is the parsed config.json.
"""
from __future__ import annotations

import math

import numpy as np


# ---- single mechanisms ---------------------------------------------------------------------------
def rms(x, eps):
    """x over its root mean square along the last axis."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def rms_norm(x, weight, eps):
    return rms(x, eps) * weight


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def rotary_frequencies(rot):
    """(frequencies [dims / 2], factor on cos and sin)."""
    dims, base = rot["dims"], rot["base"]
    f = np.array([base ** (-2.0 * i / dims) for i in range(dims // 2)])
    s = rot.get("scaling")
    if s is None:
        return f, 1.0
    if "original" not in s:      # linear: every frequency over the factor
        return f / s["factor"], 1.0

    def turns_at(t):   # the (fractional) pair index whose wave makes t turns over the original context
        return dims * math.log(s["original"] / (2.0 * math.pi * t)) / (2.0 * math.log(base))

    lo = max(math.floor(turns_at(s["fast"])), 0)
    hi = min(math.ceil(turns_at(s["slow"])), dims - 1)
    ramp = np.clip((np.arange(dims // 2) - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    return f / s["factor"] * ramp + f * (1.0 - ramp), 0.1 * math.log(s["factor"]) + 1.0


def rotate(x, positions, rot, interleaved):
    """x [tokens, heads, size]; the first rot.dims of each head turn with the token's position."""
    dims = rot["dims"]
    f, factor = rotary_frequencies(rot)
    a = np.asarray(positions, dtype=np.float64)[:, None] * f[None, :]
    c, s = (np.cos(a) * factor)[:, None, :], (np.sin(a) * factor)[:, None, :]
    out = np.array(x, dtype=np.float64)
    first, second = (slice(0, dims, 2), slice(1, dims, 2)) if interleaved else (slice(0, dims // 2), slice(dims // 2, dims))
    u, v = x[..., first], x[..., second]
    out[..., first] = u * c - v * s
    out[..., second] = v * c + u * s
    return out


def retention_recurrence(q, k, v, decay, state=None):
    """q, k [tokens, heads, dim], v [tokens, heads, vdim]; returns (o [tokens, heads, vdim], state [heads, dim, vdim])."""
    heads, dim, vdim = q.shape[1], q.shape[2], v.shape[2]
    state = np.zeros((heads, dim, vdim)) if state is None else state.copy()
    decay = np.asarray(decay, dtype=np.float64)[:, None, None]
    out = np.zeros((q.shape[0], heads, vdim))
    for t in range(q.shape[0]):
        state = decay * state + k[t][:, :, None] * v[t][:, None, :]
        out[t] = np.einsum("hdv,hd->hv", state, q[t])
    return out, state


def window_softmax_with_sink(scores, positions, key_positions, size, sink):
    """scores [heads, queries, keys] -> weights; a query sees itself and the size - 1 positions before it, and exp(sink) of
    its head joins the denominator."""
    distance = np.asarray(positions)[:, None] - np.asarray(key_positions)[None, :]
    seen = (distance >= 0) & (distance < size)
    s = np.where(seen[None], scores, -np.inf)
    top = np.maximum(s.max(axis=-1), sink[:, None])
    e = np.exp(s - top[..., None])
    return e / (e.sum(axis=-1) + np.exp(sink[:, None] - top))[..., None]


def window_softmax(scores, positions, key_positions, size):
    """scores [heads, queries, keys] -> weights over the keys a query sees: itself and the size - 1 positions before it (None: all)."""
    distance = np.asarray(positions)[:, None] - np.asarray(key_positions)[None, :]
    seen = (distance >= 0) & (distance < (np.inf if size is None else size))
    s = np.where(seen[None], scores, -np.inf)
    e = np.exp(s - s.max(axis=-1, keepdims=True))
    return e / e.sum(axis=-1, keepdims=True)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(np.sqrt(2.0 / np.pi) * (z + 0.044715 * z ** 3)))


def softplus(z):
    return np.logaddexp(0.0, z)


def causal_convolution(x, weight, bias, before=None):
    """Per channel over time: x [tokens, channels], weight [channels, taps] with the current token's tap last; before: the inputs ahead
    of the first token, [taps - 1, channels] (zeros at the start of a sequence)."""
    taps = weight.shape[1]
    before = np.zeros((taps - 1, x.shape[1])) if before is None else before
    padded = np.concatenate([before, x])
    return np.stack([(padded[t:t + taps] * weight.T).sum(axis=0) + bias for t in range(x.shape[0])])


def selective_recurrence(x, b, c, dt, rate, state=None):
    """x [tokens, heads, vdim], b and c [tokens, heads, state] (repeated for the heads of a group), dt [tokens, heads], rate [heads]:
    S <- exp(-rate dt) S + dt b x^T, y = S^T c.  Returns (y, S [heads, state, vdim])."""
    heads, n, vdim = x.shape[1], b.shape[2], x.shape[2]
    state = np.zeros((heads, n, vdim)) if state is None else state.copy()
    y = np.zeros(x.shape)
    for t in range(x.shape[0]):
        keep = np.exp(-rate * dt[t])[:, None, None]
        state = keep * state + dt[t][:, None, None] * b[t][:, :, None] * x[t][:, None, :]
        y[t] = np.einsum("hnv,hn->hv", state, c[t])
    return y, state


def grouped_rms_norm(x, weight, groups, eps):
    """The last axis in `groups` equal parts, each over its own root mean square."""
    return rms(x.reshape(x.shape[0], groups, -1), eps).reshape(x.shape) * weight


def softcap(logits, cap):
    return logits if not cap else cap * np.tanh(logits / cap)


# ---- mixers and feed-forward ----------------------------------------------------------------------
def retention(h, mix, w, prefix, eps, positions):
    n, heads, dim, vdim = h.shape[0], mix["heads"], mix["dim"], mix["vdim"]
    q = rotate((h @ w[prefix + "q"].T).reshape(n, heads, dim), positions, mix["rot"], interleaved=False)
    k = rotate((h @ w[prefix + "k"].T).reshape(n, heads, dim), positions, mix["rot"], interleaved=False) * dim ** -0.5
    v = (h @ w[prefix + "v"].T).reshape(n, heads, vdim)
    o, _ = retention_recurrence(q, k, v, mix["decay"])
    return (rms(o, eps).reshape(n, heads * vdim) * silu(h @ w[prefix + "g"].T)) @ w[prefix + "o"].T


def latent_of(h, mix, w, prefix, eps, positions):
    """(latent [tokens, kv_rank], rotated key part [tokens, rot_dim]): what a cache has to hold."""
    both = h @ w[prefix + "dkv"].T
    c = rms_norm(both[:, :mix["kv_rank"]], w[prefix + "dkv.norm"], eps)
    r = rotate(both[:, None, mix["kv_rank"]:], positions, mix["rot"], interleaved=True)[:, 0]
    return c, r


def latent_attention(h, mix, w, prefix, positions, c, key_rot):
    n, heads, dim, rd, vdim = h.shape[0], mix["heads"], mix["dim"], mix["rot_dim"], mix["vdim"]
    q = (h @ w[prefix + "q"].T).reshape(n, heads, dim + rd)
    q_rot = rotate(q[..., dim:], positions, mix["rot"], interleaved=True)
    k = (c @ w[prefix + "uk"].T).reshape(n, heads, dim)
    v = (c @ w[prefix + "uv"].T).reshape(n, heads, vdim)
    scores = (np.einsum("qhd,khd->hqk", q[..., :dim], k) + np.einsum("qhd,kd->hqk", q_rot, key_rot)) * mix["scale"]
    p = window_softmax_with_sink(scores, positions, positions, mix["mask"]["size"], w[prefix + "sink"])
    o = np.einsum("hqk,khv->qhv", p, v) * sigmoid(h @ w[prefix + "g"].T)[..., None]
    return o.reshape(n, heads * vdim) @ w[prefix + "o"].T


def keys_and_values(h, mix, w, prefix, eps, positions):
    """(keys [tokens, kv_heads, dim] after norm and rotation, values [tokens, kv_heads, vdim]): what a cache has to hold."""
    n, g = h.shape[0], mix["kv_heads"]
    k = rms_norm(h @ w[prefix + "k"].T, w[prefix + "k.norm"], eps).reshape(n, g, mix["dim"])
    return rotate(k, positions, mix["rot"], interleaved=False), (h @ w[prefix + "v"].T).reshape(n, g, mix["vdim"])


def attention(h, mix, w, prefix, eps, positions, k, v):
    n, heads = h.shape[0], mix["heads"]
    q = rms_norm(h @ w[prefix + "q"].T, w[prefix + "q.norm"], eps).reshape(n, heads, mix["dim"])
    q = rotate(q, positions, mix["rot"], interleaved=False)
    share = heads // mix["kv_heads"]
    k, v = np.repeat(k, share, axis=1), np.repeat(v, share, axis=1)
    p = window_softmax(np.einsum("qhd,khd->hqk", q, k) * mix["scale"], positions, positions, (mix.get("mask") or {}).get("size"))
    return np.einsum("hqk,khv->qhv", p, v).reshape(n, -1) @ w[prefix + "o"].T


def mamba2(h, mix, w, prefix, eps):
    n, heads, vdim, state, groups = h.shape[0], mix["heads"], mix["vdim"], mix["state"], mix["groups"]
    inner = heads * vdim
    z, xbc, dt = np.split(h @ w[prefix + "in"].T, [inner, 2 * inner + 2 * groups * state], axis=1)
    xbc = silu(causal_convolution(xbc, w[prefix + "conv"], w[prefix + "conv.b"]))
    x, b, c = np.split(xbc, [inner, inner + groups * state], axis=1)
    x = x.reshape(n, heads, vdim)
    b, c = (np.repeat(a.reshape(n, groups, state), heads // groups, axis=1) for a in (b, c))
    y, _ = selective_recurrence(x, b, c, softplus(dt + w[prefix + "dt_bias"]), np.exp(w[prefix + "A_log"]))
    y = (y + w[prefix + "D"][:, None] * x).reshape(n, inner) * silu(z)
    return grouped_rms_norm(y, w[prefix + "norm"], mix["norm_groups"], eps) @ w[prefix + "o"].T


def feed_forward(h, w, prefix, activation=silu):
    return (activation(h @ w[prefix + "gate"].T) * (h @ w[prefix + "up"].T)) @ w[prefix + "down"].T


# ---- the model --------------------------------------------------------------------------------------
def forward(config, weights, tokens, layers_out=None):
    """Logits [tokens, vocab] of one whole sequence; layers_out receives the residual stream after every layer."""
    w = {k: np.asarray(v, dtype=np.float64) for k, v in weights.items()}
    return {"Ranavik": forward_ranavik, "Forovik": forward_forovik}[config["architecture"]](config, w, tokens, layers_out)


def forward_forovik(config, w, tokens, layers_out):
    """Branches one after the other, each normed before it joins the stream; the head is the embedding table."""
    eps, positions = config["norm"]["eps"], np.arange(len(tokens))
    x = w["embed"][np.asarray(tokens)]
    cached = {}
    for i, layer in enumerate(config["layers"]):
        p, mix = f"l{i}.", layer["mixer"]
        if layer["type"].startswith("mamba2"):
            branch = mamba2(x, mix, w, p + "mix.", eps)
        else:
            source = mix.get("kv_from")
            if source is None:
                cached[i] = keys_and_values(x, mix, w, p + "mix.", eps, positions)
            branch = attention(x, mix, w, p + "mix.", eps, positions, *cached[i if source is None else source])
        x = x + rms_norm(branch, w[p + "norm1"], eps)
        if layer["mlp"] is not None:
            x = x + rms_norm(feed_forward(x, w, p + "mlp.", gelu_tanh), w[p + "norm2"], eps)
        if layers_out is not None:
            layers_out.append(x.copy())
    return rms_norm(x, w["final.norm"], eps) @ w["embed"].T


def forward_ranavik(config, w, tokens, layers_out):
    eps, m = config["norm"]["eps"], config["residual_mult"]
    positions = np.arange(len(tokens))
    x = rms_norm(w["embed"][np.asarray(tokens)], w["embed.norm"], eps)
    latents = {}
    for i, layer in enumerate(config["layers"]):
        p, mix = f"l{i}.", layer["mixer"]
        h = rms_norm(x, w[p + "norm1"], eps)
        if layer["type"] == "retention":
            branch = retention(h, mix, w, p + "mix.", eps, positions)
        else:
            source = mix.get("kv_from")
            if source is None:
                latents[i] = latent_of(h, mix, w, p + "mix.", eps, positions)
            branch = latent_attention(h, mix, w, p + "mix.", positions, *latents[i if source is None else source])
        if layer["mlp"] is not None:
            branch = branch + feed_forward(rms_norm(x, w[p + "norm2"], eps), w, p + "mlp.")
        x = x + m * branch
        if layers_out is not None:
            layers_out.append(x.copy())
    return softcap(rms_norm(x, w["final.norm"], eps) @ w["head"].T, config.get("logit_softcap"))
