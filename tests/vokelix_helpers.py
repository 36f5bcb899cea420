"""Small random Vokelix models for the tests: a configuration, bf16-exact weights."""
import json

import numpy as np
import torch

SCALING = {"factor": 2.5, "original": 256, "fast": 16.0, "slow": 2.0}


def _mlp(ff):
    return {"kind": "dense", "ff": ff} if ff else None


def attention(heads=6, kv_heads=2, dim=24, vdim=16, scale=0.27, ff=56, kv_from=None, rot_dims=16, base=9000.0, scaling=SCALING):
    rot = {"base": base, "dims": rot_dims, **({"scaling": dict(scaling)} if scaling else {})}
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "rot": rot}
    return {"type": "attention", "mlp": _mlp(ff), "mixer": m if kv_from is None else {**m, "kv_from": kv_from}}


def lightning(decay=(0.4, 0.93, 0.997), dim=16, vdim=24, ff=None):
    return {"type": "lightning", "mlp": _mlp(ff), "mixer": {"heads": len(decay), "dim": dim, "vdim": vdim, "decay": list(decay)}}


def retention(decay=(0.9, 0.9975), dim=48, vdim=40, ff=40, rot_dims=32, base=400.0):
    return {"type": "retention", "mlp": _mlp(ff),
            "mixer": {"heads": len(decay), "dim": dim, "vdim": vdim, "decay": list(decay), "rot": {"base": base, "dims": rot_dims}}}


def make_config(layers, width=72, vocab=131, eps=1e-4, alpha=1.7):
    return {"architecture": "Vokelix", "vocab": vocab, "width": width, "norm": {"eps": eps}, "postln_alpha": alpha, "layers": layers}


def small_config():
    """Every kind of layer, shared keys near and far, with and without feed-forward, sizes that differ from layer to layer."""
    a = attention()
    return make_config([lightning(), a, retention(), {**json.loads(json.dumps(a)), "mlp": None}, lightning((0.99, 0.8), 32, 16, ff=48),
                        attention(kv_from=1, ff=None), retention((0.5, 0.98, 0.9995), 16, 16, ff=None, rot_dims=16),
                        attention(kv_from=3, scale=0.4)])


def make_weights(config, seed=0):
    """name -> float64 array whose values are exact in bf16."""
    rng = np.random.default_rng(seed)
    w, width = {}, config["width"]

    def put(name, *shape, scale=None):
        w[name] = rng.standard_normal(shape) * (shape[-1] ** -0.5 if scale is None else scale)

    def norm(name, n, centre=1.0):
        w[name] = centre + 0.2 * rng.standard_normal(n)

    put("embed", config["vocab"], width, scale=1.0)
    for i, layer in enumerate(config["layers"]):
        p, m, heads = f"l{i}.", layer["mixer"], layer["mixer"]["heads"]
        norm(p + "norm1", width, 0.0)
        qk, v = heads * m["dim"], heads * m["vdim"]
        put(p + "mix.q", qk, width)
        if layer["type"] == "attention":
            names = [("q", qk)]
            if m.get("kv_from") is None:
                names += [("k", m["kv_heads"] * m["dim"]), ("v", m["kv_heads"] * m["vdim"])]
            for name, n in names:
                put(p + "mix." + name, n, width)
                put(p + f"mix.{name}.b", n, scale=0.3)
                if name != "v":
                    norm(p + f"mix.{name}.norm", n)
            put(p + "mix.sink", heads, scale=1.5)
            put(p + "mix.g", heads, width)
        else:
            put(p + "mix.k", qk, width)
            put(p + "mix.v", v, width)
            put(p + "mix.g", v, width)
            if layer["type"] == "lightning":
                norm(p + "mix.norm", v)
        put(p + "mix.o", width, v)
        if layer["mlp"]:
            norm(p + "norm2", width, 0.0)
            put(p + "mlp.gate", layer["mlp"]["ff"], width)
            put(p + "mlp.up", layer["mlp"]["ff"], width)
            put(p + "mlp.down", width, layer["mlp"]["ff"])
    norm("final.norm", width, 0.0)
    put("head", config["vocab"], width, scale=4.0 * width ** -0.5)
    return {k: torch.from_numpy(np.asarray(v)).to(torch.bfloat16).double().numpy() for k, v in w.items()}
