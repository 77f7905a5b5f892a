"""Ranudra, the plain way: numpy float64, whole sequences, no cache, one function per
mechanism.  It shares nothing with the product: the tests hold the engine to it.

``config`` is the parsed config.json; ``weights`` maps tensor names to float64 arrays.
"""
from __future__ import annotations

import math

import numpy as np


def sigmoid(z):
    return np.where(z >= 0, 1.0 / (1.0 + np.exp(-np.abs(z))), np.exp(-np.abs(z)) / (1.0 + np.exp(-np.abs(z))))


def silu(z):
    return z * sigmoid(z)


def rms_norm(x: np.ndarray, w, eps: float) -> np.ndarray:
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * w


def layer_norm(x: np.ndarray, w, eps: float) -> np.ndarray:
    centred = x - x.mean(axis=-1, keepdims=True)
    return centred / np.sqrt(np.mean(centred * centred, axis=-1, keepdims=True) + eps) * w


def rotary_frequencies(rot: dict) -> tuple:
    """``(frequencies of the dims/2 pairs, what cosine and sine are multiplied by)``; with
    ``scaling`` slow pairs turn ``factor`` times slower, fast ones as they are, a ramp over the
    pair's index between."""
    dims, base = rot["dims"], rot["base"]
    i = np.arange(dims // 2, dtype=np.float64)
    f = base ** (-2.0 * i / dims)
    sc = rot.get("scaling")
    if sc is None:
        return f, 1.0

    def where(turns):  # the (fractional) pair that makes `turns` turns over the original length
        return dims * math.log(sc["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

    lo = max(math.floor(where(sc["fast"])), 0)
    hi = min(math.ceil(where(sc["slow"])), dims - 1)
    ramp = np.clip((i - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    return f / sc["factor"] * ramp + f * (1.0 - ramp), 0.1 * math.log(sc["factor"]) + 1.0


def rotate(x: np.ndarray, rot: dict, first: int = 0) -> np.ndarray:
    """x: [tokens, ..., dims] of the tokens at positions first, first + 1, ...: element 2i turns
    together with element 2i + 1 by position times frequency i."""
    f, mult = rotary_frequencies(rot)
    angle = (first + np.arange(x.shape[0], dtype=np.float64))[:, None] * f[None, :]
    shape = (x.shape[0],) + (1,) * (x.ndim - 2) + (len(f),)
    c, s = (np.cos(angle) * mult).reshape(shape), (np.sin(angle) * mult).reshape(shape)
    out = np.empty_like(x)
    u, v = x[..., 0::2], x[..., 1::2]
    out[..., 0::2] = u * c - v * s
    out[..., 1::2] = v * c + u * s
    return out


def visible(n: int, size) -> np.ndarray:
    """[query, key]: the query's own position and the size - 1 before it (None: all before it)."""
    i, j = np.arange(n)[:, None], np.arange(n)[None, :]
    seen = j <= i
    return seen if size is None else seen & (i - j < size)


def softmax_attention(q, k, v, scale, mask, sink=None) -> np.ndarray:
    """q, k [n, H, size], v [n, H, vdim] -> [n, H, vdim].  ``sink`` [H]: one more term exp(sink) in
    every denominator, with no value."""
    n, heads, _ = q.shape
    out = np.zeros((n, heads, v.shape[2]))
    for h in range(heads):
        s = np.where(mask, (q[:, h] @ k[:, h].T) * scale, -np.inf)
        top = s.max(axis=-1, keepdims=True)
        if sink is not None:
            top = np.maximum(top, sink[h])
        e = np.exp(s - top)
        denom = e.sum(axis=-1, keepdims=True)
        if sink is not None:
            denom = denom + np.exp(sink[h] - top)
        out[:, h] = (e / denom) @ v[:, h]
    return out


def latent_keys_values(h, m: dict, w: dict, pre: str, eps: float):
    """Keys [n, H, dim + rot_dim] and values [n, H, vdim] of all heads, made out in full."""
    n, H, rank = h.shape[0], m["heads"], m["kv_rank"]
    both = h @ w[pre + "dkv"].T
    c = rms_norm(both[:, :rank], w[pre + "dkv.norm"], eps)
    shared = both[:, rank:]
    if m.get("rot") is not None:
        shared = rotate(shared, m["rot"])
    plain_part = (c @ w[pre + "uk"].T).reshape(n, H, m["dim"])
    k = np.concatenate([plain_part, np.repeat(shared[:, None, :], H, axis=1)], axis=2)
    return k, (c @ w[pre + "uv"].T).reshape(n, H, m["vdim"])


def latent_mixer(h, m: dict, w: dict, pre: str, eps: float, *, gate: str) -> np.ndarray:
    n, H, dim, rot_dim = h.shape[0], m["heads"], m["dim"], m["rot_dim"]
    q = (h @ w[pre + "q"].T).reshape(n, H, dim + rot_dim)
    if m.get("rot") is not None:
        q = np.concatenate([q[..., :dim], rotate(q[..., dim:], m["rot"])], axis=2)
    k, v = latent_keys_values(h, m, w, pre, eps)
    size = m["mask"]["size"] if m.get("mask") else None
    o = softmax_attention(q, k, v, m["scale"], visible(n, size), w.get(pre + "sink"))
    g = sigmoid(h @ w[pre + "g"].T)
    o = o * g[:, :, None] if gate == "head" else o * g.reshape(o.shape)
    return o.reshape(n, -1) @ w[pre + "o"].T


def gated_linear_attention(q, k, v, decay) -> np.ndarray:
    """q, k, decay [n, H, dim], v [n, H, vdim] -> [n, H, vdim]; row d of a head's state fades by decay[t, h, d]."""
    n, heads, dim = q.shape
    out = np.zeros_like(v)
    for h in range(heads):
        S = np.zeros((dim, v.shape[2]))
        for t in range(n):
            S = decay[t, h][:, None] * S + np.outer(k[t, h], v[t, h])
            out[t, h] = S.T @ q[t, h]
    return out


def gla_mixer(h, m: dict, w: dict, pre: str, eps: float) -> np.ndarray:
    n, H, dim, vdim = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = (h @ w[pre + "q"].T).reshape(n, H, dim) * dim ** -0.5
    k = (h @ w[pre + "k"].T).reshape(n, H, dim)
    v = (h @ w[pre + "v"].T).reshape(n, H, vdim)
    z = (h @ w[pre + "a1"].T) @ w[pre + "a2"].T + w[pre + "a2.b"]
    decay = (sigmoid(z) ** (1.0 / m["tau"])).reshape(n, H, dim)
    o = rms_norm(gated_linear_attention(q, k, v, decay), w[pre + "norm"], eps)
    return (o.reshape(n, H * vdim) * silu(h @ w[pre + "g"].T)) @ w[pre + "o"].T


def mixer(kind: str, h, m: dict, w: dict, pre: str, eps: float) -> np.ndarray:
    if kind == "latent_attention":
        return latent_mixer(h, m, w, pre, eps, gate="head")
    if kind == "latent_attention_2":
        return latent_mixer(h, m, w, pre, eps, gate="element")
    assert kind == "gla", kind
    return gla_mixer(h, m, w, pre, eps)


def feed_forward(h, w: dict, pre: str) -> np.ndarray:
    return np.maximum(h @ w[pre + "up"].T, 0.0) ** 2 @ w[pre + "down"].T


def hyper_step(xs, sublayer, w: dict, pre: str) -> np.ndarray:
    """xs [streams, n, width]: the sublayer reads a weighted sum of the streams; its output, weighted per
    stream, joins a remix of what the streams held before."""
    u = np.einsum("s,snd->nd", w[pre + "in"], xs)
    y = sublayer(u)
    return np.einsum("st,snd->tnd", w[pre + "mix"], xs) + w[pre + "out"][:, None, None] * y


def run_order(config: dict) -> list:
    count = len(config["layers"])
    loop = config.get("loop")
    if not loop:
        return list(range(count))
    middle = list(range(loop["start"], loop["stop"]))
    return list(range(loop["start"])) + middle * loop["times"] + list(range(loop["stop"], count))


def forward(config: dict, weights: dict, tokens, streams=None) -> np.ndarray:
    """Logits [n, vocab] of a whole sequence.  ``streams``: a list that receives the sum of the
    streams after every layer run."""
    eps = config["norm"]["eps"]
    x = weights["embed"][np.asarray(tokens)] * config["embedding"]["scale"]
    xs = np.repeat(x[None], config["streams"], axis=0)
    for i in run_order(config):
        layer, pre = config["layers"][i], f"l{i}."
        xs = hyper_step(xs, lambda u: mixer(layer["type"], layer_norm(u, weights[pre + "norm1"], eps), layer["mixer"],
                                            weights, pre + "mix.", eps), weights, pre + "hc1.")
        if layer.get("mlp") is not None:
            xs = hyper_step(xs, lambda u: feed_forward(layer_norm(u, weights[pre + "norm2"], eps), weights, pre + "mlp."),
                            weights, pre + "hc2.")
        if streams is not None:
            streams.append(xs.sum(axis=0))
    return layer_norm(xs.sum(axis=0), weights["final.norm"], eps) @ weights["embed"].T
