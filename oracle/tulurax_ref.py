"""Plain float64 restatement of the Tulurax decoder, for tests only (numpy, no batching, no cache).

One function per mechanism; ``forward`` strings them together over one whole sequence and returns the logits
at every position and the residual stream after every layer.  Pieces that other designs have too come from
their oracle.  Nothing here is shared with the product path.

``config`` is the parsed ``config.json``; ``weights`` maps tensor names to float arrays."""
from __future__ import annotations

import numpy as np

from oracle.dogetar_ref import softplus
from oracle.merilorn_ref import rms_norm, silu


def tanh_norm(x, alpha, weight, bias):
    """A norm without statistics: every entry is squashed on its own."""
    return np.tanh(alpha * x) * weight + bias


# ------------------------------------------------------------------ attention
def query_temperature(positions, coef, every):
    return 1.0 + coef * np.log(np.floor((np.asarray(positions) + 1.0) / every) + 1.0)


def sink_weights(q, k, scale):
    """Weights [heads, queries, keys] of a causal softmax whose denominator has one more term, a score of zero that stands for no
    key.  ``q`` [tokens, heads, n], ``k`` [tokens, kv_heads, n]; consecutive query heads share a key head."""
    t, heads = q.shape[:2]
    group = heads // k.shape[1]
    out = np.zeros((heads, t, t))
    for h in range(heads):
        s = np.where(np.tril(np.ones((t, t), dtype=bool)), q[:, h] @ k[:, h // group].T * scale, -np.inf)
        top = np.maximum(s.max(-1, keepdims=True), 0.0)
        p = np.exp(s - top)
        out[h] = p / (p.sum(-1, keepdims=True) + np.exp(-top))
    return out


def mix_heads(weights, talk):
    """Row h of ``talk`` says how much of every head's weights goes into those of head h."""
    return np.einsum("hg,gij->hij", talk, weights)


def apply_weights(weights, v):
    """``v`` [tokens, kv_heads, m]: every head's weights meet the values of its own key/value head."""
    heads, group = len(weights), len(weights) // v.shape[1]
    return np.stack([weights[h] @ v[:, h // group] for h in range(heads)], axis=1)


def talking_attention(h, m, w, eps, cast=lambda a: a):
    t, heads, kv = len(h), m["heads"], m["kv_heads"]
    q = rms_norm(cast(h @ w("q").T).reshape(t, heads, m["dim"]), 1.0, eps)
    k = cast(rms_norm(cast(h @ w("k").T).reshape(t, kv, m["dim"]), 1.0, eps))
    v = cast(rms_norm(cast(h @ w("v").T).reshape(t, kv, m["vdim"]), 1.0, eps))
    temp = m.get("q_temp")
    if temp:
        q = q * query_temperature(np.arange(t), temp["coef"], temp["every"])[:, None, None]
    o = apply_weights(mix_heads(sink_weights(cast(q), k, m["scale"]), w("talk")), v)
    return cast(o.reshape(t, -1)) @ w("o").T


# ------------------------------------------------------------------ retention
def retention_scan(q, k, v, decay, state=None):
    """One head, token by token.  Returns the outputs and the final [dim, vdim] state."""
    s = np.zeros((k.shape[1], v.shape[1])) if state is None else state.copy()
    out = np.zeros(v.shape)
    for t in range(len(v)):
        s = decay * s + np.outer(k[t], v[t])
        out[t] = s.T @ q[t]
    return out, s


def retention(h, m, w, eps, cast=lambda a: a):
    t, heads, dim, vdim = len(h), m["heads"], m["dim"], m["vdim"]
    q = cast(h @ w("q").T).reshape(t, heads, dim)
    k = cast(h @ w("k").T).reshape(t, heads, dim) * dim ** -0.5
    v = cast(h @ w("v").T).reshape(t, heads, vdim)
    o = np.stack([retention_scan(q[:, i], k[:, i], v[:, i], m["decay"][i])[0] for i in range(heads)], axis=1)
    return cast(rms_norm(o, 1.0, eps).reshape(t, -1) * silu(cast(h @ w("g").T))) @ w("o").T


# ------------------------------------------------------------------ feed-forward
def xielu(z, p, q):
    low = np.minimum(z, 0.0)
    return np.where(z > 0, softplus(p) * z * z, (0.5 + softplus(q)) * (np.expm1(low) - low)) + 0.5 * z


def plain_mlp(h, w, cast=lambda a: a):
    return cast(xielu(cast(h @ w("up").T) + w("up.b"), *w("act"))) @ w("down").T + w("down.b")


# ------------------------------------------------------------------ the model
def forward(config, weights, tokens, cast=lambda a: a):
    """Logits [tokens, vocab] and the residual stream after every layer [layers, tokens, width].  ``cast`` is applied to what goes
    into and comes out of every product: with a rounding function it shows what rounding alone does."""
    eps = config["norm"]["eps"]

    def norm(x, name):
        return tanh_norm(x, weights[name + ".alpha"], weights[name], weights[name + ".b"])

    x = norm(weights["embed"][np.asarray(tokens)] * config["embedding"]["scale"], "embed.norm")
    stream = []
    for i, layer in enumerate(config["layers"]):
        name, m = f"l{i}.", layer["mixer"]
        h = cast(norm(x, name + "norm1"))
        x = x + cast(m["left_scale"] * talking_attention(h, m["left"], lambda key: weights[name + "mix.left." + key], eps, cast)
                     + m["right_scale"] * retention(h, m["right"], lambda key: weights[name + "mix.right." + key], eps, cast))
        if layer["mlp"] is not None:
            x = x + cast(plain_mlp(cast(norm(x, name + "norm2")), lambda key: weights[name + "mlp." + key], cast))
        stream.append(x)
    logits = cast(norm(x, "final.norm")) @ weights["head"].T * config.get("logit_scale", 1.0)
    cap = config.get("logit_softcap")
    return cap * np.tanh(logits / cap) if cap else logits, np.stack(stream)
