"""Farorax, the plain way: numpy float64, whole sequences, no cache, one function per
mechanism.  It shares nothing with the product: the tests hold the engine to it.

``config`` is the parsed config.json; ``weights`` maps tensor names to float64 arrays.
"""
from __future__ import annotations

import math

import numpy as np


def norm(x, w, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * w


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def frequencies(rot):
    """One frequency per pair: those with a wavelength above ``original / low`` are divided by the
    factor, those below ``original / high`` stay, the ones between are blended."""
    plain = [rot["base"] ** (-2.0 * i / rot["dims"]) for i in range(rot["dims"] // 2)]
    scaling = rot.get("scaling")
    if not scaling:
        return np.array(plain)
    out = []
    for f in plain:
        length = 2.0 * math.pi / f
        if length < scaling["original"] / scaling["high"]:
            out.append(f)
        elif length > scaling["original"] / scaling["low"]:
            out.append(f / scaling["factor"])
        else:
            s = (scaling["original"] / length - scaling["low"]) / (scaling["high"] - scaling["low"])
            out.append((1.0 - s) * f / scaling["factor"] + s * f)
    return np.array(out)


def rotate_pairs(x, rot):
    """``x``: [tokens, heads, dim]; neighbours (2i, 2i+1) of the first ``dims`` elements turn."""
    if not rot:
        return x
    dims = rot["dims"]
    angle = np.arange(x.shape[0], dtype=np.float64)[:, None, None] * frequencies(rot)[None, None, :]
    out = x.copy()
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    out[..., 0:dims:2] = u * np.cos(angle) - v * np.sin(angle)
    out[..., 1:dims:2] = v * np.cos(angle) + u * np.sin(angle)
    return out


def window_mask(n, size):
    i, j = np.arange(n)[:, None], np.arange(n)[None, :]
    seen = j <= i
    return seen if size is None else seen & (i - j < size)


def softmax_with_sink(scores, visible, sink):
    """Rows of weights; ``exp(sink)`` is one more term of the denominator."""
    s = np.where(visible, scores, -np.inf)
    top = np.maximum(s.max(axis=-1, keepdims=True), sink)
    e = np.where(visible, np.exp(s - top), 0.0)
    return e / (e.sum(axis=-1, keepdims=True) + np.exp(sink - top))


def attention(h, w, prefix, m, eps):
    n, heads, groups, dim, vdim = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rotate_pairs((h @ w[prefix + "q"].T).reshape(n, heads, dim), m.get("rot"))
    k = rotate_pairs((h @ w[prefix + "k"].T).reshape(n, groups, dim), m.get("rot"))
    v = (h @ w[prefix + "v"].T).reshape(n, groups, vdim)
    visible = window_mask(n, m["mask"]["size"] if m.get("mask") else None)
    out = np.zeros((n, heads, vdim))
    for head in range(heads):
        g = head // (heads // groups)
        p = softmax_with_sink(q[:, head] @ k[:, g].T * m["scale"], visible, w[prefix + "sink"][head])
        out[:, head] = p @ v[:, g]
    return out.reshape(n, heads * vdim) @ w[prefix + "o"].T


def decayed_state(q, k, v, decay):
    """[tokens, heads, vdim]: the state of a head fades by its number, takes in ``k v^T`` and is read
    with q, the token's own write included."""
    n, heads, dim = q.shape
    out = np.zeros(v.shape)
    for head in range(heads):
        state = np.zeros((dim, v.shape[2]))
        for t in range(n):
            state = decay[head] * state + np.outer(k[t, head], v[t, head])
            out[t, head] = state.T @ q[t, head]
    return out


def lightning(h, w, prefix, m, eps):
    n, heads, dim, vdim = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = silu(h @ w[prefix + "q"].T).reshape(n, heads, dim)
    k = silu(h @ w[prefix + "k"].T).reshape(n, heads, dim)
    v = silu(h @ w[prefix + "v"].T).reshape(n, heads, vdim)
    o = decayed_state(q, k, v, m["decay"]).reshape(n, heads * vdim)
    o = norm(o, w[prefix + "norm"], eps) * sigmoid(h @ w[prefix + "g"].T)
    return o @ w[prefix + "o"].T


def gated(h, w, prefix, act):
    return (act(h @ w[prefix + "gate"].T) * (h @ w[prefix + "up"].T)) @ w[prefix + "down"].T


def route(h, w, prefix, router, margins=None):
    """(experts [tokens, top], weights [tokens, top]).  ``margins`` (a list) receives, per token, how
    close the choice was: the least lead, in scores, of a chosen expert over one that was left out
    among the kept groups and of a kept group over one that was not."""
    scores = sigmoid(h @ w[prefix + "router"].T)
    n, count, top = len(scores), scores.shape[1], router["top"]
    groups = router.get("groups")
    allowed = np.ones((n, count), dtype=bool)
    margin = np.full(n, np.inf)
    if groups:
        blocks = scores.reshape(n, groups["count"], count // groups["count"])
        value = np.sort(blocks, axis=-1)[..., -2:].sum(axis=-1)
        order = np.argsort(-value, axis=-1, kind="stable")
        keep = groups["keep"]
        kept = np.zeros(value.shape, dtype=bool)
        np.put_along_axis(kept, order[:, :keep], True, axis=-1)
        allowed = np.repeat(kept, count // groups["count"], axis=-1)
        if keep < groups["count"]:
            ranked = -np.sort(-value, axis=-1)
            margin = np.minimum(margin, ranked[:, keep - 1] - ranked[:, keep])
    choice = np.where(allowed, scores, -np.inf)
    order = np.argsort(-choice, axis=-1, kind="stable")
    if top < count:
        ranked = np.take_along_axis(choice, order, axis=-1)
        margin = np.minimum(margin, ranked[:, top - 1] - ranked[:, top])
    if margins is not None:
        margins.append(margin)
    experts = order[:, :top]
    chosen = np.take_along_axis(scores, experts, axis=-1)
    return experts, chosen / (chosen.sum(axis=-1, keepdims=True) + 1e-20)


def mixture(h, w, prefix, mlp, margins=None):
    experts, weights = route(h, w, prefix, mlp["router"], margins)
    out = np.zeros((h.shape[0], w[prefix + "e0.down"].shape[0]))
    for t in range(h.shape[0]):
        for e, p in zip(experts[t], weights[t]):
            out[t] += p * gated(h[t:t + 1], w, f"{prefix}e{e}.", silu)[0]
    if mlp.get("shared"):
        out += gated(h, w, prefix + "shared.", silu)
    return out


def feed_forward(h, w, prefix, mlp, margins=None):
    if mlp["kind"] == "dense":
        return gated(h, w, prefix, gelu_tanh)
    return mixture(h, w, prefix, mlp, margins)


def layer_runs(config):
    """(layer, number of the pass that starts right before it, or None) in running order."""
    count, loop = len(config["layers"]), config.get("loop")
    if not loop:
        return [(i, None) for i in range(count)]
    runs = [(i, None) for i in range(loop["start"])]
    for t in range(loop["times"]):
        runs += [(i, t if i == loop["start"] else None) for i in range(loop["start"], loop["stop"])]
    return runs + [(i, None) for i in range(loop["stop"], count)]


def enter_pass(x, embedded, w, t):
    """What comes ahead of a pass: the stream and the embedded tokens through one map, and the pass's
    own vector."""
    return np.concatenate([x, embedded], axis=-1) @ w["loop.in"].T + w["loop.step"][t]


def forward(config, w, tokens, *, keep_layers=False, margins=None):
    """Logits [tokens, vocab] of one whole sequence (and the stream after every layer run)."""
    eps, m = config["norm"]["eps"], config["residual_mult"]
    x = embedded = w["embed"][np.asarray(tokens)]
    kept = []
    for index, t in layer_runs(config):
        layer = config["layers"][index]
        if t is not None:
            x = enter_pass(x, embedded, w, t)
        mixer = {"attention": attention, "lightning": lightning}[layer["type"]]
        x = x + m * mixer(norm(x, w[f"l{index}.norm1"], eps), w, f"l{index}.mix.", layer["mixer"], eps)
        if layer.get("mlp"):
            h = norm(x, w[f"l{index}.norm2"], eps)
            x = x + m * feed_forward(h, w, f"l{index}.mlp.", layer["mlp"], margins)
        kept.append(x)
    logits = norm(x, w["final.norm"], eps) @ w["head"].T
    cap = config.get("logit_softcap")
    if cap:
        logits = cap * np.tanh(logits / cap)
    return (logits, np.stack(kept)) if keep_layers else logits
