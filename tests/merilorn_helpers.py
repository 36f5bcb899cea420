"""Small random Merilorn models for the tests: a configuration, bf16-exact weights, a model folder on disk."""
import json
import os

import numpy as np
import torch

ROT = {"base": 10000.0, "scaling": {"factor": 2.5, "original": 256, "fast": 16.0, "slow": 2.0}}


def latent(heads=3, dim=16, rot_dim=8, vdim=24, kv_rank=40, scale=0.21, ff=56, **rot):
    r = {"dims": rot_dim, **ROT, **rot}
    return {"type": "latent_attention", "mlp": {"kind": "dense", "ff": ff} if ff else None,
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "scale": scale, "rot": r}}


def delta(heads=4, kv_heads=2, dim=24, vdim=16, conv=4, ff=None):
    return {"type": "channel_delta", "mlp": {"kind": "dense", "ff": ff} if ff else None,
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}}


def shared(entry, owner):
    return {**json.loads(json.dumps(entry)), "weights_of": owner}


def make_config(layers, width=72, vocab=131, eps=1e-5, embed_scale=3.0):
    return {"architecture": "Merilorn", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": embed_scale},
            "layers": layers}


def small_config():
    """Both kinds of layers, with and without feed-forward, shared weights, sizes that differ from layer to layer."""
    a, d1, d2 = latent(), delta(), delta(heads=3, kv_heads=1, dim=16, vdim=40, conv=3, ff=48)
    b = latent(heads=2, dim=32, rot_dim=16, vdim=32, kv_rank=64, scale=0.15, ff=None)
    return make_config([d1, a, d2, shared(a, 1), b, shared(d1, 0), shared(d2, 2)])


def make_weights(config, seed=0, ranks=(12, 20)):
    """name -> float64 array whose values are exact in bf16."""
    rng = np.random.default_rng(seed)
    w, width = {}, config["width"]

    def put(name, *shape, scale=None):
        std = shape[-1] ** -0.5 if scale is None else scale
        t = torch.from_numpy(rng.standard_normal(shape) * std).to(torch.bfloat16)
        w[name] = t.double().numpy()

    def norm(name, n):
        w[name] = torch.from_numpy(1.0 + 0.2 * rng.standard_normal(n)).to(torch.bfloat16).double().numpy()

    put("embed", config["vocab"], width, scale=1.0 / config["embedding"]["scale"])
    for i, layer in enumerate(config["layers"]):
        if layer.get("weights_of", i) != i:
            continue
        p, m = f"l{i}.", layer["mixer"]
        norm(p + "norm1", width)
        norm(p + "norm1b", width)
        if layer["type"] == "latent_attention":
            put(p + "mix.q", m["heads"] * (m["dim"] + m["rot_dim"]), width, scale=2.0 * width ** -0.5)
            put(p + "mix.dkv", m["kv_rank"] + m["rot_dim"], width)
            norm(p + "mix.dkv.norm", m["kv_rank"])
            put(p + "mix.uk", m["heads"] * m["dim"], m["kv_rank"])
            put(p + "mix.uv", m["heads"] * m["vdim"], m["kv_rank"])
            put(p + "mix.g", m["heads"], width)
            put(p + "mix.o", width, m["heads"] * m["vdim"])
        else:
            qk, v = m["kv_heads"] * m["dim"], m["heads"] * m["vdim"]
            for name, n in (("q", qk), ("k", qk), ("v", v)):
                put(p + f"mix.{name}", n, width)
                put(p + f"mix.{name}.conv", n, m["conv"], scale=0.6)
            put(p + "mix.b", m["heads"], width)
            put(p + "mix.A_log", m["heads"], scale=1.0)
            put(p + "mix.dt_bias", m["heads"] * m["dim"], scale=1.0)
            w[p + "mix.dt_bias"] -= 3.0                     # long memory
            norm(p + "mix.norm", m["vdim"])
            put(p + "mix.a1", ranks[0], width)
            put(p + "mix.a2", m["heads"] * m["dim"], ranks[0])
            put(p + "mix.g1", ranks[1], width)
            put(p + "mix.g2", v, ranks[1])
            put(p + "mix.o", width, v)
        if layer["mlp"]:
            norm(p + "norm2", width)
            norm(p + "norm2b", width)
            put(p + "mlp.gate", layer["mlp"]["ff"], width)
            put(p + "mlp.up", layer["mlp"]["ff"], width)
            put(p + "mlp.down", width, layer["mlp"]["ff"])
    norm("final.norm", width)
    put("head", config["vocab"], width, scale=4.0 * width ** -0.5)
    return {k: torch.from_numpy(v).to(torch.bfloat16).double().numpy() for k, v in w.items()}


def save_model(folder, config, weights):
    from safetensors.torch import save_file
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(config, f)
    save_file({k: torch.from_numpy(v).to(torch.bfloat16) for k, v in weights.items()}, os.path.join(folder, "model.safetensors"))
    return str(folder)


def tokens(n, config, seed=0):
    return [int(t) for t in np.random.default_rng(seed).integers(0, config["vocab"], n)]


def row_errors(got, want):
    """Root mean square of the difference of every row (mean taken off) over that of the wanted row."""
    d = np.asarray(got, np.float64) - want
    d = d - d.mean(-1, keepdims=True)
    w = want - want.mean(-1, keepdims=True)
    return np.sqrt((d * d).mean(-1) / (w * w).mean(-1))


def bf16(a):
    return torch.from_numpy(np.asarray(a)).to(torch.bfloat16).double().numpy()
