"""Small random Dogetar models for the tests: configurations, bf16-exact weights."""
import json

import numpy as np
import torch

SCALING = {"factor": 5.0, "low": 1.5, "high": 6.0, "original": 160}


def dense(ff=56, limit=0.9):
    return {"kind": "dense", "ff": ff, "limit": limit}


def moe(ff=24, experts=5, identity=1, top=2, count=3, keep=2, scale=1.3, shared=40):
    router = {"experts": experts, "top": top, "identity": identity, "scale": scale, "groups": {"count": count, "keep": keep}}
    return {"kind": "moe", "expert": {"ff": ff}, "router": router, **({"shared": {"ff": shared}} if shared else {})}


def chunked(heads=6, kv_heads=2, dim=16, vdim=24, size=40, scale=0.3, diff=0.45, rot_dims=12, base=9000.0, mlp=None):
    return {"type": "attention", "mlp": mlp, "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "diff": diff, "scale": scale,
                                                       "mask": {"size": size}, "rot": {"base": base, "dims": rot_dims}}}


def windowed(heads=4, kv_heads=2, dim=24, vdim=16, size=37, scale=0.4, rot_dims=16, base=700.0, scaling=SCALING, mlp=None):
    rot = {"base": base, "dims": rot_dims, **({"scaling": dict(scaling)} if scaling else {})}
    return {"type": "attention_2", "mlp": mlp, "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale,
                                                         "mask": {"size": size}, "rot": rot}}


def parallel(heads=3, kv_heads=1, dim=20, vdim=16, size=50, scale=0.25, ssm=(4, 12, 16, 2, 4, 3), left=0.7, right=1.2, mlp=None):
    """``ssm``: heads, vdim, state, groups, taps, parts of the norm."""
    h, v, n, groups, taps, parts = ssm
    return {"type": "parallel", "mlp": mlp, "mixer": {
        "left": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "mask": {"size": size}}, "left_scale": left,
        "right": {"heads": h, "vdim": v, "state": n, "groups": groups, "conv": taps, "norm_groups": parts}, "right_scale": right}}


def make_config(layers, width=72, vocab=131, eps=1e-4, cap=12.0, loop=None, bigram=(53, 7, 11)):
    return {"architecture": "Dogetar", "vocab": vocab, "width": width, "norm": {"eps": eps}, "logit_softcap": cap, "layers": layers,
            "loop": dict(zip(("start", "stop", "times"), loop)) if loop else None,
            "embedding": {"bigram": dict(zip(("buckets", "mul_prev", "mul_cur"), bigram))} if bigram else {}}


def small_config():
    """Every kind of layer and feed-forward, a loop that starts behind the first layer, sizes that differ from layer to layer."""
    return make_config([parallel(mlp=dense()), chunked(mlp=moe()), windowed(), parallel(2, 2, 32, 32, 33, ssm=(6, 8, 24, 3, 3, 1), mlp=moe(
        ff=17, experts=6, identity=2, top=3, count=2, keep=1, shared=None)), chunked(2, 1, 24, 40, 64, 0.2, 0.2, 24, mlp=dense(33, 2.0))],
        loop=(1, 4, 2))


def make_weights(config, seed=0):
    """name -> float64 array whose values are exact in bf16."""
    rng = np.random.default_rng(seed)
    w, width = {}, config["width"]

    def put(name, *shape, scale=None):
        w[name] = rng.standard_normal(shape) * (shape[-1] ** -0.5 if scale is None else scale)

    def norm(name, n):
        w[name] = 1.0 + 0.2 * rng.standard_normal(n)

    def attention(p, m, maps=1):
        for name, n in (("q", m["heads"] * maps * m["dim"]), ("k", m["kv_heads"] * maps * m["dim"]), ("v", m["kv_heads"] * m["vdim"])):
            put(p + name, n, width)
        put(p + "o", width, m["heads"] * m["vdim"])

    def gated(p, ff):
        put(p + "gate", ff, width)
        put(p + "up", ff, width)
        put(p + "down", width, ff)

    put("embed", config["vocab"], width, scale=1.0)
    if config["embedding"].get("bigram"):
        put("bigram", config["embedding"]["bigram"]["buckets"] + 1, width, scale=0.7)
    if config["loop"]:
        put("loop.step", config["loop"]["times"], width, scale=0.5)
    for i, layer in enumerate(config["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        norm(p + "norm1", width)
        w[p + "ls1"] = 0.6 + 0.2 * rng.standard_normal(width)
        if layer["type"] == "attention":
            attention(p + "mix.", m, 2)
            put(p + "mix.g", m["heads"], width)
            for name in ("lq1", "lk1", "lq2", "lk2"):
                put(p + "mix." + name, m["dim"], scale=0.3)
        elif layer["type"] == "attention_2":
            attention(p + "mix.", m)
            for name, n in (("q", m["heads"] * m["dim"]), ("k", m["kv_heads"] * m["dim"]), ("v", m["kv_heads"] * m["vdim"])):
                put(p + f"mix.{name}.b", n, scale=0.3)
                if name != "v":
                    norm(p + f"mix.{name}.norm", m["dim"])
        else:
            attention(p + "mix.left.", m["left"])
            put(p + "mix.left.sink", m["left"]["heads"], scale=1.5)
            r, p2 = m["right"], p + "mix.right."
            inner, channels = r["heads"] * r["vdim"], r["heads"] * r["vdim"] + 2 * r["groups"] * r["state"]
            put(p2 + "in", inner + channels + r["heads"], width)
            put(p2 + "conv", channels, r["conv"])
            put(p2 + "conv.b", channels, scale=0.3)
            put(p2 + "dt_bias", r["heads"], scale=1.0)
            w[p2 + "A_log"] = rng.uniform(-5.0, 1.5, r["heads"])
            put(p2 + "D", r["heads"], scale=1.0)
            norm(p2 + "norm", inner)
            put(p2 + "o", width, inner)
        mlp = layer["mlp"]
        if mlp:
            norm(p + "norm2", width)
            w[p + "ls2"] = 0.6 + 0.2 * rng.standard_normal(width)
            if mlp["kind"] == "dense":
                gated(p + "mlp.", mlp["ff"])
            else:
                every = mlp["router"]["experts"] + mlp["router"]["identity"]
                put(p + "mlp.router", every, width, scale=2.0 * width ** -0.5)
                put(p + "mlp.correction", every, scale=0.3)
                for e in range(mlp["router"]["experts"]):
                    gated(p + f"mlp.e{e}.", mlp["expert"]["ff"])
                if mlp.get("shared"):
                    gated(p + "mlp.shared.", mlp["shared"]["ff"])
    norm("final.norm", width)
    put("head", config["vocab"], width, scale=4.0 * width ** -0.5)
    return {k: torch.from_numpy(np.asarray(v)).to(torch.bfloat16).double().numpy() for k, v in w.items()}


def copy(entry):
    return json.loads(json.dumps(entry))
