"""Plain float64 restatement of the Vokelix decoder, for tests only (numpy, no batching, no cache).

One function per mechanism; ``forward`` strings them together over one whole sequence and returns the logits
at every position and the residual stream after every layer.  Pieces that other designs have too come from
their oracle.  Nothing here is shared with the product path.

``config`` is the parsed ``config.json``; ``weights`` maps tensor names to float arrays."""
from __future__ import annotations

import numpy as np

from oracle.merilorn_ref import rms_norm, rotate_interleaved, sigmoid, silu, yarn_frequencies


def zero_centred_norm(x, weight, eps):
    """The norm of the residual stream: its weight is stored as the distance from one."""
    return rms_norm(x, 1.0 + weight, eps)


def rotate_halves(x, positions, freq, magnitude=1.0):
    """Rotates entry i with entry i + len(freq) of the first ``2 * len(freq)`` entries of the last axis;
    ``x`` is [tokens, ..., n]."""
    n = len(freq)
    angle = np.asarray(positions, dtype=np.float64)[:, None] * freq
    shape = (len(x),) + (1,) * (x.ndim - 2) + (n,)
    c, s = (np.cos(angle) * magnitude).reshape(shape), (np.sin(angle) * magnitude).reshape(shape)
    u, v = x[..., :n], x[..., n:2 * n]
    out = x.copy()
    out[..., :n] = u * c - v * s
    out[..., n:2 * n] = v * c + u * s
    return out


# ------------------------------------------------------------------ attention
def sink_attention(q, k, v, scale, sink):
    """``q`` [tokens, heads, n], ``k`` [tokens, kv_heads, n], ``v`` [tokens, kv_heads, m]; consecutive query heads share a
    key head.  ``sink`` [heads] enters the denominator beside the scores of the visible keys."""
    t, heads = q.shape[:2]
    group = heads // k.shape[1]
    out = np.zeros((t, heads, v.shape[2]))
    for h in range(heads):
        s = q[:, h] @ k[:, h // group].T * scale
        s = np.where(np.tril(np.ones((t, t), dtype=bool)), s, -np.inf)
        top = np.maximum(s.max(-1, keepdims=True), sink[h])
        p = np.exp(s - top)
        out[:, h] = p @ v[:, h // group] / (p.sum(-1, keepdims=True) + np.exp(sink[h] - top))
    return out


def attention_keys(h, m, w, eps):
    """Keys (normed over all heads at once, then rotated) and values of a layer that has its own."""
    t = len(h)
    freq, magnitude = yarn_frequencies(m["rot"]["dims"], m["rot"]["base"], m["rot"].get("scaling"))
    k = rms_norm(h @ w("k").T + w("k.b"), w("k.norm"), eps).reshape(t, m["kv_heads"], m["dim"])
    v = (h @ w("v").T + w("v.b")).reshape(t, m["kv_heads"], m["vdim"])
    return rotate_interleaved(k, np.arange(t), freq, magnitude), v


def attention(h, m, w, eps, keys):
    t = len(h)
    freq, magnitude = yarn_frequencies(m["rot"]["dims"], m["rot"]["base"], m["rot"].get("scaling"))
    q = rms_norm(h @ w("q").T + w("q.b"), w("q.norm"), eps).reshape(t, m["heads"], m["dim"])
    q = rotate_interleaved(q, np.arange(t), freq, magnitude)
    o = sink_attention(q, *keys, m["scale"], w("sink")) * sigmoid(h @ w("g").T)[..., None]
    return o.reshape(t, -1) @ w("o").T


# ------------------------------------------------------------------ linear attention
def decay_scan(q, k, v, decay, state=None):
    """One head of linear attention with a constant decay, token by token.  ``q``/``k`` [tokens, dim], ``v`` [tokens, vdim].
    Returns the outputs and the final [dim, vdim] state."""
    s = np.zeros((q.shape[1], v.shape[1])) if state is None else state.copy()
    out = np.zeros((len(q), v.shape[1]))
    for t in range(len(q)):
        s = decay * s + np.outer(k[t], v[t])
        out[t] = s.T @ q[t]
    return out, s


def _scan_heads(q, k, v, decay):
    return np.stack([decay_scan(q[:, i], k[:, i], v[:, i], decay[i])[0] for i in range(q.shape[1])], axis=1)


def lightning(h, m, w, eps):
    t, heads = len(h), m["heads"]
    q = silu(h @ w("q").T).reshape(t, heads, m["dim"])
    k = silu(h @ w("k").T).reshape(t, heads, m["dim"])
    v = silu(h @ w("v").T).reshape(t, heads, m["vdim"])
    o = _scan_heads(q, k, v, m["decay"]).reshape(t, -1)
    return (rms_norm(o, w("norm"), eps) * sigmoid(h @ w("g").T)) @ w("o").T


def retention(h, m, w, eps):
    t, heads, pos = len(h), m["heads"], np.arange(len(h))
    freq, _ = yarn_frequencies(m["rot"]["dims"], m["rot"]["base"])
    q = rotate_halves((h @ w("q").T).reshape(t, heads, m["dim"]), pos, freq)
    k = rotate_halves((h @ w("k").T).reshape(t, heads, m["dim"]), pos, freq) * m["dim"] ** -0.5
    v = (h @ w("v").T).reshape(t, heads, m["vdim"])
    o = rms_norm(_scan_heads(q, k, v, m["decay"]), 1.0, eps).reshape(t, -1)
    return (o * silu(h @ w("g").T)) @ w("o").T


def dense_mlp(h, w):
    return (silu(h @ w("gate").T) * (h @ w("up").T)) @ w("down").T


# ------------------------------------------------------------------ the model
def forward(config, weights, tokens, cast=lambda a: a):
    """Logits [tokens, vocab] and the residual stream after every layer [layers, tokens, width].  ``cast`` is applied to
    what goes into and comes out of every sublayer: with a rounding function it shows what rounding alone does."""
    eps, alpha = config["norm"]["eps"], config["postln_alpha"]
    x = weights["embed"][np.asarray(tokens)]
    stream, kept = [], {}
    for i, layer in enumerate(config["layers"]):
        m, name = layer["mixer"], f"l{i}."

        def mix(key):
            return weights[name + "mix." + key]

        def mlp(key):
            return weights[name + "mlp." + key]

        h = cast(x)
        if layer["type"] == "attention":
            if m.get("kv_from") is None:
                kept[i] = attention_keys(h, m, mix, eps)
            y = attention(h, m, mix, eps, kept[i if m.get("kv_from") is None else m["kv_from"]])
        else:
            y = {"lightning": lightning, "retention": retention}[layer["type"]](h, m, mix, eps)
        x = zero_centred_norm(alpha * x + cast(y), weights[name + "norm1"], eps)
        if layer["mlp"] is not None:
            assert layer["mlp"]["kind"] == "dense"
            x = zero_centred_norm(alpha * x + cast(dense_mlp(cast(x), mlp)), weights[name + "norm2"], eps)
        stream.append(x)
    return cast(zero_centred_norm(x, weights["final.norm"], eps)) @ weights["head"].T, np.stack(stream)
