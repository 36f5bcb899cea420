"""Plain float64 restatement of the Dogetar decoder, for tests only (numpy, no batching, no cache).

One function per mechanism; ``forward`` strings them together over one whole sequence and returns the logits
at every position and the residual stream after every run of a layer.  Pieces that other designs have too come from
their oracle.  Nothing here is shared with the product path.

``config`` is the parsed ``config.json``; ``weights`` maps tensor names to float arrays."""
from __future__ import annotations

import numpy as np

from oracle.merilorn_ref import rms_norm, sigmoid, silu
from oracle.vokelix_ref import rotate_halves


def softplus(z):
    return np.logaddexp(0.0, z)


# ------------------------------------------------------------------ embedding
def bigram_rows(tokens, buckets, mul_prev, mul_cur):
    """The row of the second table that each token adds; the first token of a sequence has the last row."""
    rows = [buckets]
    for prev, cur in zip(tokens[:-1], tokens[1:]):
        rows.append((int(prev) * mul_prev + int(cur) * mul_cur) % buckets)
    return np.asarray(rows[:len(tokens)])


# ------------------------------------------------------------------ attention
def chunk_mask(t, size):
    at = np.arange(t)
    return (at[None, :] <= at[:, None]) & (at[None, :] // size == at[:, None] // size)


def window_mask(t, size):
    back = np.arange(t)[:, None] - np.arange(t)[None, :]
    return (back >= 0) & (back < size)


def masked_attention(q, k, v, scale, mask, sink=None, slopes=None):
    """``q`` [tokens, heads, n], ``k`` [tokens, kv_heads, n], ``v`` [tokens, kv_heads, m]; consecutive query heads share a
    key head.  ``sink`` [heads]: a score of its own in the denominator; ``slopes`` [heads]: what a score loses per token of
    distance."""
    t, heads = q.shape[:2]
    group = heads // k.shape[1]
    back = np.arange(t)[:, None] - np.arange(t)[None, :]
    out = np.zeros((t, heads, v.shape[2]))
    for h in range(heads):
        s = q[:, h] @ k[:, h // group].T * scale
        if slopes is not None:
            s = s - slopes[h] * back
        s = np.where(mask, s, -np.inf)
        top = s.max(-1, keepdims=True)
        if sink is not None:
            top = np.maximum(top, sink[h])
        p = np.exp(s - top)
        z = p.sum(-1, keepdims=True)
        if sink is not None:
            z = z + np.exp(sink[h] - top)
        out[:, h] = p @ v[:, h // group] / z
    return out


def distance_slopes(heads):
    return 2.0 ** (-8.0 * np.arange(1, heads + 1) / heads)


def scaled_frequencies(rot):
    """Angles per position.  With ``scaling``, waves longer than the original length allows are slowed down by a factor,
    short ones kept, and those in between interpolated."""
    i = np.arange(rot["dims"] // 2)
    freq = float(rot["base"]) ** (-2.0 * i / rot["dims"])
    s = rot.get("scaling")
    if not s:
        return freq
    out = []
    for f in freq:
        wave = 2.0 * np.pi / f
        if wave < s["original"] / s["high"]:
            out.append(f)
        elif wave > s["original"] / s["low"]:
            out.append(f / s["factor"])
        else:
            mix = (s["original"] / wave - s["low"]) / (s["high"] - s["low"])
            out.append((1.0 - mix) * f / s["factor"] + mix * f)
    return np.asarray(out)


def two_map_lambda(w, diff):
    return np.exp(np.sum(w("lq1") * w("lk1"))) - np.exp(np.sum(w("lq2") * w("lk2"))) + diff


def two_map_attention(h, m, w, eps):
    """The difference of two attentions over the same values, normed per head and gated."""
    t, heads, kv, dim, vdim = len(h), m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    freq, pos = scaled_frequencies(m["rot"]), np.arange(t)
    q = rotate_halves((h @ w("q").T).reshape(t, heads, 2, dim), pos, freq)
    k = rotate_halves((h @ w("k").T).reshape(t, kv, 2, dim), pos, freq)
    v = (h @ w("v").T).reshape(t, kv, vdim)
    mask = chunk_mask(t, m["mask"]["size"])
    a1, a2 = (masked_attention(q[:, :, i], k[:, :, i], v, m["scale"], mask) for i in range(2))
    o = rms_norm(a1 - two_map_lambda(w, m["diff"]) * a2, 1.0, eps) * (1.0 - m["diff"])
    o = o * sigmoid(h @ w("g").T)[..., None]
    return o.reshape(t, -1) @ w("o").T


def window_attention(h, m, w, eps):
    t, heads, kv, dim, vdim = len(h), m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    freq, pos = scaled_frequencies(m["rot"]), np.arange(t)
    q = rms_norm((h @ w("q").T + w("q.b")).reshape(t, heads, dim), w("q.norm"), eps)
    k = rms_norm((h @ w("k").T + w("k.b")).reshape(t, kv, dim), w("k.norm"), eps)
    v = (h @ w("v").T + w("v.b")).reshape(t, kv, vdim)
    o = masked_attention(rotate_halves(q, pos, freq), rotate_halves(k, pos, freq), v, m["scale"], window_mask(t, m["mask"]["size"]))
    return o.reshape(t, -1) @ w("o").T


def biased_attention(h, m, w):
    """No rotation: a bias that grows with the distance, and a sink."""
    t, heads, kv, dim, vdim = len(h), m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k = (h @ w("q").T).reshape(t, heads, dim), (h @ w("k").T).reshape(t, kv, dim)
    v = (h @ w("v").T).reshape(t, kv, vdim)
    o = masked_attention(q, k, v, m["scale"], chunk_mask(t, m["mask"]["size"]), w("sink"), distance_slopes(heads))
    return o.reshape(t, -1) @ w("o").T


# ------------------------------------------------------------------ state space
def causal_conv(x, taps, bias):
    """``x`` [tokens, channels], ``taps`` [channels, n]: the last column meets the current token, zeros before the start."""
    n = taps.shape[1]
    padded = np.concatenate((np.zeros((n - 1, x.shape[1])), x))
    return sum(padded[i:i + len(x)] * taps[:, i] for i in range(n)) + bias


def state_space_scan(x, b, c, dt, a, d, state=None):
    """One head, token by token: ``x`` [tokens, vdim], ``b``/``c`` [tokens, state], ``dt`` [tokens], ``a`` (negative) and ``d``
    numbers.  Returns the outputs and the final [state, vdim] state."""
    s = np.zeros((b.shape[1], x.shape[1])) if state is None else state.copy()
    out = np.zeros(x.shape)
    for t in range(len(x)):
        s = np.exp(a * dt[t]) * s + dt[t] * np.outer(b[t], x[t])
        out[t] = s.T @ c[t] + d * x[t]
    return out, s


def gated_part_norm(y, z, parts, weight, eps):
    t, inner = y.shape
    g = (y * silu(z)).reshape(t, parts, inner // parts)
    return rms_norm(g, 1.0, eps).reshape(t, inner) * weight


def state_space(h, m, w, eps):
    t, heads, vdim, n, groups = len(h), m["heads"], m["vdim"], m["state"], m["groups"]
    inner = heads * vdim
    proj = h @ w("in").T
    z, xbc, dt = proj[:, :inner], proj[:, inner:2 * inner + 2 * groups * n], proj[:, 2 * inner + 2 * groups * n:]
    xbc = silu(causal_conv(xbc, w("conv"), w("conv.b")))
    x = xbc[:, :inner].reshape(t, heads, vdim)
    b = xbc[:, inner:inner + groups * n].reshape(t, groups, n)
    c = xbc[:, inner + groups * n:].reshape(t, groups, n)
    dt = softplus(dt + w("dt_bias"))
    y = np.zeros((t, heads, vdim))
    for i in range(heads):
        g = i // (heads // groups)
        y[:, i] = state_space_scan(x[:, i], b[:, g], c[:, g], dt[:, i], -np.exp(w("A_log")[i]), w("D")[i])[0]
    return gated_part_norm(y.reshape(t, inner), z, m["norm_groups"], w("norm"), eps) @ w("o").T


# ------------------------------------------------------------------ feed-forward
def clamped_mlp(h, w, limit):
    g = np.minimum(h @ w("gate").T, limit)
    u = np.clip(h @ w("up").T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ w("down").T


def expert_mlp(h, w):
    return (silu(h @ w("gate").T) * (h @ w("up").T)) @ w("down").T


def route(z, correction, top, groups, scale):
    """Chosen experts [tokens, top] and their weights for router logits ``z`` [tokens, experts]."""
    p = np.exp(z - z.max(-1, keepdims=True))
    p /= p.sum(-1, keepdims=True)
    choice = p + correction
    if groups:
        count, keep = groups["count"], groups["keep"]
        size = z.shape[1] // count
        best = np.argsort(-choice.reshape(len(z), count, size).max(-1), axis=-1, kind="stable")[:, :keep]
        open_ = np.zeros((len(z), count), dtype=bool)
        np.put_along_axis(open_, best, True, axis=1)
        choice = np.where(np.repeat(open_, size, axis=1), choice, -np.inf)
    chosen = np.argsort(-choice, axis=-1, kind="stable")[:, :top]
    return chosen, np.take_along_axis(p, chosen, axis=1) * scale


def mixture(h, m, w):
    r = m["router"]
    chosen, weight = route(h @ w("router").T, w("correction"), r["top"], r.get("groups"), r["scale"])
    out = np.zeros_like(h)
    for e in range(r["experts"] + r.get("identity", 0)):
        rows, place = np.nonzero(chosen == e)
        if len(rows) == 0:
            continue
        y = h[rows] if e >= r["experts"] else expert_mlp(h[rows], lambda key, e=e: w(f"e{e}.{key}"))
        out[rows] += weight[rows, place][:, None] * y
    if m.get("shared"):
        out = out + expert_mlp(h, lambda key: w("shared." + key))
    return out


# ------------------------------------------------------------------ the model
def run_order(config):
    """(layer, pass or None) in the order of execution."""
    n, loop = len(config["layers"]), config.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    body = [(i, t) for t in range(loop["times"]) for i in range(loop["start"], loop["stop"])]
    return [(i, None) for i in range(loop["start"])] + body + [(i, None) for i in range(loop["stop"], n)]


def embed(config, weights, tokens):
    x = weights["embed"][np.asarray(tokens)]
    b = config["embedding"].get("bigram")
    if b:
        x = x + weights["bigram"][bigram_rows(tokens, b["buckets"], b["mul_prev"], b["mul_cur"])]
    return x


def forward(config, weights, tokens, cast=lambda a: a):
    """Logits [tokens, vocab] and the residual stream after every run of a layer [runs, tokens, width].  ``cast`` is applied
    to what goes into and comes out of every sublayer: with a rounding function it shows what rounding alone does."""
    eps = config["norm"]["eps"]
    x = embed(config, weights, tokens)
    first, stream = x, []
    for i, t in run_order(config):
        layer, name = config["layers"][i], f"l{i}."
        m = layer["mixer"]
        if t is not None and i == config["loop"]["start"]:
            x = (x + first if t else x) + weights["loop.step"][t]

        def mix(key, at=""):
            return weights[name + "mix." + at + key]

        h = cast(rms_norm(x, weights[name + "norm1"], eps))
        if layer["type"] == "attention":
            y = two_map_attention(h, m, mix, eps)
        elif layer["type"] == "attention_2":
            y = window_attention(h, m, mix, eps)
        else:
            y = m["left_scale"] * biased_attention(h, m["left"], lambda key: mix(key, "left.")) \
                + m["right_scale"] * state_space(h, m["right"], lambda key: mix(key, "right."), eps)
        x = x + cast(y) * weights[name + "ls1"]
        mlp = layer["mlp"]
        if mlp is not None:
            h = cast(rms_norm(x, weights[name + "norm2"], eps))
            y = clamped_mlp(h, lambda key: weights[name + "mlp." + key], mlp["limit"]) if mlp["kind"] == "dense" \
                else mixture(h, mlp, lambda key: weights[name + "mlp." + key])
            x = x + cast(y) * weights[name + "ls2"]
        stream.append(x)
    logits = cast(rms_norm(x, weights["final.norm"], eps)) @ weights["head"].T
    cap = config.get("logit_softcap")
    return cap * np.tanh(logits / cap) if cap else logits, np.stack(stream)
