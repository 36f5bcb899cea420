"""Plain float64 restatement of the Merilorn decoder, for tests only (numpy, no batching, no cache).

One function per mechanism; ``forward`` strings them together over one whole sequence and returns the logits
at every position and the residual stream after every layer.  Nothing here is shared with the product path.

``config`` is the parsed ``config.json``; ``weights`` maps tensor names to float arrays."""
from __future__ import annotations

import math

import numpy as np


# ------------------------------------------------------------------ small pieces
def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.logaddexp(0.0, z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def rms_norm(x, weight, eps):
    """Rows of ``x`` over their root mean square (eps inside the root), times ``weight``."""
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps) * weight


def unit_norm(x, eps=1e-6):
    """Rows of ``x`` over their length (eps inside the root)."""
    return x / np.sqrt((x * x).sum(-1, keepdims=True) + eps)


# ------------------------------------------------------------------ rotary positions
def yarn_frequencies(dims, base, scaling=None):
    """Angle per position of every rotated pair and the factor on cos and sin."""
    i = np.arange(dims // 2)
    freq = base ** (-2.0 * i / dims)
    if not scaling:
        return freq, 1.0

    def pair_turning(times):          # the (fractional) pair that turns ``times`` times within the original length
        return dims * math.log(scaling["original"] / (2.0 * math.pi * times)) / (2.0 * math.log(base))

    lo = max(math.floor(pair_turning(scaling["fast"])), 0)
    hi = min(math.ceil(pair_turning(scaling["slow"])), dims - 1)
    slow_share = np.clip((i - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    freq = freq / scaling["factor"] * slow_share + freq * (1.0 - slow_share)
    return freq, 0.1 * math.log(scaling["factor"]) + 1.0


def rotate_interleaved(x, positions, freq, magnitude=1.0):
    """Rotates the pairs (0, 1), (2, 3), ... of the first ``2 * len(freq)`` entries of the last axis;
    ``x`` is [tokens, ..., n]."""
    n = 2 * len(freq)
    angle = np.asarray(positions, dtype=np.float64)[:, None] * freq
    shape = (len(x),) + (1,) * (x.ndim - 2) + (len(freq),)
    c, s = (np.cos(angle) * magnitude).reshape(shape), (np.sin(angle) * magnitude).reshape(shape)
    u, v = x[..., 0:n:2], x[..., 1:n:2]
    out = x.copy()
    out[..., 0:n:2] = u * c - v * s
    out[..., 1:n:2] = v * c + u * s
    return out


# ------------------------------------------------------------------ mixers
def causal_attention(q, k, v, scale):
    """``q``/``k`` [tokens, heads, n], ``v`` [tokens, heads, m]; every query sees itself and what came before."""
    t = len(q)
    scores = np.einsum("ihd,jhd->hij", q, k) * scale
    scores = np.where(np.tril(np.ones((t, t), dtype=bool)), scores, -np.inf)
    p = np.exp(scores - scores.max(-1, keepdims=True))
    p /= p.sum(-1, keepdims=True)
    return np.einsum("hij,jhd->ihd", p, v)


def latent_attention(h, m, w, eps):
    """``m`` is the mixer entry of the configuration, ``w(name)`` its tensor ``mix.<name>``."""
    t, heads = len(h), m["heads"]
    dim, rot_dim, vdim, rank = m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    freq, magnitude = yarn_frequencies(m["rot"]["dims"], m["rot"]["base"], m["rot"].get("scaling"))
    pos = np.arange(t)
    q = (h @ w("q").T).reshape(t, heads, dim + rot_dim)
    down = h @ w("dkv").T
    c = rms_norm(down[:, :rank], w("dkv.norm"), eps)
    k_rot = rotate_interleaved(down[:, None, rank:], pos, freq, magnitude)
    q_rot = rotate_interleaved(q[..., dim:], pos, freq, magnitude)
    k_plain = (c @ w("uk").T).reshape(t, heads, dim)
    v = (c @ w("uv").T).reshape(t, heads, vdim)
    qs = np.concatenate([q[..., :dim], q_rot], -1)
    ks = np.concatenate([k_plain, np.broadcast_to(k_rot, (t, heads, rot_dim))], -1)
    o = causal_attention(qs, ks, v, m["scale"])
    o = o * sigmoid(h @ w("g").T)[..., None]
    return o.reshape(t, heads * vdim) @ w("o").T


def causal_conv(x, taps):
    """``x`` [tokens, channels], ``taps`` [channels, n]; the last tap meets the current token."""
    n = taps.shape[1]
    padded = np.concatenate([np.zeros((n - 1, x.shape[1])), x])
    return sum(padded[j:j + len(x)] * taps[:, j] for j in range(n))


def delta_scan(q, k, v, log_decay, beta, state=None):
    """The gated delta rule of one head, token by token.  ``q``/``k``/``log_decay`` [tokens, dim],
    ``v`` [tokens, vdim], ``beta`` [tokens].  Returns the outputs and the final [dim, vdim] state."""
    s = np.zeros((q.shape[1], v.shape[1])) if state is None else state.copy()
    out = np.zeros((len(q), v.shape[1]))
    for t in range(len(q)):
        s = np.exp(log_decay[t])[:, None] * s
        u = beta[t] * (v[t] - s.T @ k[t])
        s = s + np.outer(k[t], u)
        out[t] = s.T @ q[t]
    return out, s


def channel_delta(h, m, w, eps):
    t, heads, kv_heads, dim, vdim = len(h), m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = silu(causal_conv(h @ w("q").T, w("q.conv"))).reshape(t, kv_heads, dim)
    k = silu(causal_conv(h @ w("k").T, w("k.conv"))).reshape(t, kv_heads, dim)
    v = silu(causal_conv(h @ w("v").T, w("v.conv"))).reshape(t, heads, vdim)
    q, k = unit_norm(q) * dim ** -0.5, unit_norm(k)
    beta = sigmoid(h @ w("b").T)
    step = softplus(h @ w("a1").T @ w("a2").T + w("dt_bias")).reshape(t, heads, dim)
    log_decay = -np.exp(w("A_log"))[None, :, None] * step
    gate = sigmoid(h @ w("g1").T @ w("g2").T).reshape(t, heads, vdim)
    o = np.zeros((t, heads, vdim))
    for i in range(heads):
        j = i // (heads // kv_heads)
        o[:, i], _ = delta_scan(q[:, j], k[:, j], v[:, i], log_decay[:, i], beta[:, i])
    o = rms_norm(o, w("norm"), eps) * gate
    return o.reshape(t, heads * vdim) @ w("o").T


def dense_mlp(h, w):
    return (gelu_tanh(h @ w("gate").T) * (h @ w("up").T)) @ w("down").T


MIXERS = {"latent_attention": latent_attention, "channel_delta": channel_delta}


# ------------------------------------------------------------------ the model
def forward(config, weights, tokens, cast=lambda a: a):
    """Logits [tokens, vocab] and the residual stream after every layer [layers, tokens, width].  ``cast`` is applied to
    what goes into and comes out of every sublayer: with a rounding function it shows what rounding alone does."""
    eps = config["norm"]["eps"]
    x = weights["embed"][np.asarray(tokens)] * config["embedding"]["scale"]
    stream = []
    for i, layer in enumerate(config["layers"]):
        owner = layer.get("weights_of", i)
        name = f"l{owner}."

        def mix(key):
            return weights[name + "mix." + key]

        def mlp(key):
            return weights[name + "mlp." + key]

        y = MIXERS[layer["type"]](cast(rms_norm(x, weights[name + "norm1"], eps)), layer["mixer"], mix, eps)
        x = x + rms_norm(cast(y), weights[name + "norm1b"], eps)
        if layer["mlp"] is not None:
            assert layer["mlp"]["kind"] == "dense"
            y = dense_mlp(cast(rms_norm(x, weights[name + "norm2"], eps)), mlp)
            x = x + rms_norm(cast(y), weights[name + "norm2b"], eps)
        stream.append(x)
    logits = cast(rms_norm(x, weights["final.norm"], eps)) @ weights["head"].T
    return logits, np.stack(stream)
