"""Small random Tulurax models for the tests: configurations, bf16-exact weights."""
import json

import numpy as np
import torch


def layer(heads=6, kv_heads=2, dim=24, vdim=16, scale=0.35, temp=(0.6, 20), decay=(0.9, 0.999, 0.5), rdim=16, rvdim=24, left=0.7, right=1.3,
          ff=56):
    m = {"left": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale,
                  "q_temp": {"coef": temp[0], "every": temp[1]} if temp else None}, "left_scale": left,
         "right": {"heads": len(decay), "dim": rdim, "vdim": rvdim, "decay": list(decay)}, "right_scale": right}
    return {"type": "parallel", "mixer": m, "mlp": {"kind": "dense", "ff": ff} if ff else None}


def make_config(layers, width=72, vocab=131, eps=1e-4, embed_scale=2.5, logit_scale=1.5, cap=15.0):
    return {"architecture": "Tulurax", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": embed_scale},
            "layers": layers, "logit_scale": logit_scale, "logit_softcap": cap}


def small_config():
    """Grouped and ungrouped heads, layers without a feed-forward, sizes and constants that differ from layer to layer."""
    return make_config([layer(), layer(5, 5, 16, 40, 0.5, (1.0, 33), (0.97,), 32, 16, 1.1, 0.6, None),
                        layer(4, 1, 40, 24, 0.2, None, (0.8, 1.0 - 2.0 ** -9), 24, 40, 0.4, 0.9, 40)])


def make_weights(config, seed=0):
    """name -> float64 array whose values are exact in bf16."""
    rng = np.random.default_rng(seed)
    w, width = {}, config["width"]

    def put(name, *shape, scale=None):
        w[name] = rng.standard_normal(shape) * (shape[-1] ** -0.5 if scale is None else scale)

    def norm(name):
        w[name + ".alpha"] = np.asarray(rng.uniform(0.3, 0.8))
        w[name] = 1.0 + 0.2 * rng.standard_normal(width)
        put(name + ".b", width, scale=0.2)

    put("embed", config["vocab"], width, scale=1.0 / config["embedding"]["scale"])
    norm("embed.norm")
    for i, entry in enumerate(config["layers"]):
        p, m = f"l{i}.", entry["mixer"]
        norm(p + "norm1")
        a, r = m["left"], m["right"]
        for name, n in (("q", a["heads"] * a["dim"]), ("k", a["kv_heads"] * a["dim"]), ("v", a["kv_heads"] * a["vdim"])):
            put(p + "mix.left." + name, n, width)
        w[p + "mix.left.talk"] = np.eye(a["heads"]) + 0.4 * rng.standard_normal((a["heads"], a["heads"]))
        put(p + "mix.left.o", width, a["heads"] * a["vdim"])
        for name, n in (("q", r["heads"] * r["dim"]), ("k", r["heads"] * r["dim"]), ("v", r["heads"] * r["vdim"]), ("g", r["heads"] * r["vdim"])):
            put(p + "mix.right." + name, n, width)
        put(p + "mix.right.o", width, r["heads"] * r["vdim"])
        if entry["mlp"]:
            ff = entry["mlp"]["ff"]
            norm(p + "norm2")
            put(p + "mlp.up", ff, width)
            put(p + "mlp.up.b", ff, scale=0.3)
            put(p + "mlp.down", width, ff, scale=0.5 * ff ** -0.5)
            put(p + "mlp.down.b", width, scale=0.3)
            put(p + "mlp.act", 2, scale=0.7)
    norm("final.norm")
    put("head", config["vocab"], width, scale=4.0 * width ** -0.5)
    return {k: torch.from_numpy(np.asarray(v)).to(torch.bfloat16).double().numpy() for k, v in w.items()}


def copy(entry):
    return json.loads(json.dumps(entry))
