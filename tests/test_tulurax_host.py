"""Tulurax without a GPU: the oracle against other ways to compute the same, configuration and loading, storage, and the index arithmetic
of the prompt kernel's LDS records."""
import json
import math

import numpy as np
import pytest
import torch

from infer_amd.cache import LayeredLayout
from infer_amd.config import Config, TuluraxConfig, load_model_config
from infer_amd.layers import XieluMLP
from infer_amd.registry import model_class
from infer_amd.tulurax import TuluraxForCausalLM
from infer_amd.weight_loader import load_model
from oracle import tulurax_ref as ref
from tests import merilorn_helpers as mh, tulurax_helpers as th


# ------------------------------------------------------------------ the oracle
def test_tanh_norm_by_hand():
    x = np.array([[0.5, -2.0]])
    want = [[math.tanh(0.25) * 2 + 0.1, math.tanh(-1.0) * 3 - 0.2]]
    assert np.allclose(ref.tanh_norm(x, 0.5, np.array([2.0, 3.0]), np.array([0.1, -0.2])), want)


def test_temperature_grows_in_steps():
    t = ref.query_temperature(np.arange(10), 0.5, 4)
    assert np.allclose(t[:3], 1.0) and np.allclose(t[3:7], 1 + 0.5 * math.log(2)) and np.allclose(t[7:], 1 + 0.5 * math.log(3))


def test_sink_takes_its_share_of_a_lonely_key():
    q, k = np.array([[[2.0]], [[1.0]]]), np.array([[[3.0]], [[-1.0]]])
    w = ref.sink_weights(q, k, 0.5)
    assert np.allclose(w[0, 0], [math.exp(3) / (1 + math.exp(3)), 0.0])
    z = 1 + math.exp(1.5) + math.exp(-0.5)
    assert np.allclose(w[0, 1], [math.exp(1.5) / z, math.exp(-0.5) / z])
    far = ref.sink_weights(q * 1000.0, k, 1.0)
    assert np.isfinite(far).all() and np.allclose(far[0, 0, 0], 1.0)


def test_mixing_weights_is_mixing_outputs_of_every_head_over_every_value():
    """What a head would give with the values of another head's group, mixed: the same numbers in another order."""
    rng = np.random.default_rng(1)
    t, heads, kv = 7, 6, 3
    q, k, v = rng.standard_normal((t, heads, 4)), rng.standard_normal((t, kv, 4)), rng.standard_normal((t, kv, 5))
    talk, w = rng.standard_normal((heads, heads)), ref.sink_weights(q, k, 0.7)
    got = ref.apply_weights(ref.mix_heads(w, talk), v)
    cross = np.stack([[w[g] @ v[:, c] for c in range(kv)] for g in range(heads)])         # [heads, kv, t, 5]
    want = np.stack([sum(talk[h, g] * cross[g, h // 2] for g in range(heads)) for h in range(heads)], axis=1)
    assert np.allclose(got, want) and not np.allclose(got, ref.apply_weights(w, v))
    assert np.allclose(ref.apply_weights(ref.mix_heads(w, np.eye(heads)), v), ref.apply_weights(w, v))


def test_retention_equals_its_closed_form():
    rng = np.random.default_rng(2)
    t, d = 9, 0.8
    q, k, v = rng.standard_normal((t, 3)), rng.standard_normal((t, 3)), rng.standard_normal((t, 4))
    i, j = np.arange(t)[:, None], np.arange(t)[None, :]
    want = np.where(j <= i, d ** np.maximum(i - j, 0), 0.0) * (q @ k.T) @ v
    got, state = ref.retention_scan(q, k, v, d)
    assert np.allclose(got, want)
    head, s = ref.retention_scan(q[:4], k[:4], v[:4], d)
    tail, s = ref.retention_scan(q[4:], k[4:], v[4:], d, s)
    assert np.allclose(np.concatenate([head, tail]), want) and np.allclose(s, state)


def test_xielu_is_smooth_at_zero_and_linear_far_below():
    p, q = 0.4, -0.3
    z = np.array([-1e-6, 0.0, 1e-6])
    assert np.allclose(ref.xielu(z, p, q), z / 2, atol=1e-11)
    a, b = ref.xielu(np.array([-60.0, -50.0]), p, q)
    assert np.isclose((b - a) / 10, 0.5 - (0.5 + math.log1p(math.exp(q))))
    assert np.isclose(ref.xielu(np.array(2.0), p, q), 4 * math.log1p(math.exp(p)) + 1.0)


def test_streams_and_caps_by_hand():
    """Sublayers that give nothing but the bias of the last product."""
    config = th.make_config([th.layer(), th.layer(ff=None)], width=24)
    w = th.make_weights(config)
    for name in w:
        if name.endswith((".o", ".down")):
            w[name] = np.zeros_like(w[name])
    logits, stream = ref.forward(config, w, [5, 6])
    x0 = np.tanh(w["embed.norm.alpha"] * 2.5 * w["embed"][[5, 6]]) * w["embed.norm"] + w["embed.norm.b"]
    assert np.allclose(stream, np.stack([x0 + w["l0.mlp.down.b"]] * 2))
    raw = (np.tanh(w["final.norm.alpha"] * stream[-1]) * w["final.norm"] + w["final.norm.b"]) @ w["head"].T
    assert np.allclose(logits, 15 * np.tanh(1.5 * raw / 15))
    assert np.allclose(ref.forward({**config, "logit_softcap": None}, w, [5, 6])[0], 1.5 * raw)


# ------------------------------------------------------------------ configuration and weights
def test_config_and_registry(tmp_path):
    config = th.small_config()
    folder = mh.save_model(tmp_path / "m", config, th.make_weights(config))
    cfg = load_model_config(folder)
    assert isinstance(cfg, TuluraxConfig) and model_class(cfg) is TuluraxForCausalLM and cfg.num_hidden_layers == 3
    assert (cfg.logit_scale, cfg.logit_softcap, cfg.embedding_scale, cfg.norm_eps, cfg.vocab_size, cfg.hidden_size) == (1.5, 15.0, 2.5, 1e-4, 131, 72)
    assert [s.ff for s in cfg.layers] == [56, None, 40] and cfg.layers[1].mixer["right"]["decay"] == [0.97]
    assert Config(folder, kvcache_block_size=64, dtype="float32").hf_config.torch_dtype == torch.float32
    with pytest.raises(AssertionError):
        Config(folder, kvcache_block_size=48)
    model = TuluraxForCausalLM.build(cfg, "cpu")
    left, right = model.blocks[0].mixer.parts["left"].shape, model.blocks[0].mixer.parts["right"].shape
    assert (left.heads, left.kv_heads, left.dim, left.vdim, left.scale, left.out_scale, left.eps) == (6, 2, 24, 16, 0.35, 0.7, 1e-4)
    assert (left.temp_coef, left.temp_every, left.norm_values, left.key_pad, left.vdim_pad) == (0.6, 20, True, 32, 32)
    assert model.blocks[2].mixer.parts["left"].shape.temp_every == 0
    assert (right.heads, right.dim, right.vdim, right.scale, right.norm_per_head, right.gate_silu, right.silu, right.rot_dims) == (
        3, 16, 24, 0.25, True, True, False, 0)
    assert model.blocks[0].mixer.parts["right"].out_scale == 1.3 and model.blocks[0].mixer.parts["right"].out_norm is None
    for change, error in ((lambda c: c["layers"][0]["mlp"].update(kind="other"), "other"), (lambda c: c["layers"][1].update(type="none"), "none"),
                          (lambda c: c["layers"][0]["mixer"]["left"].update(kv_heads=4), "share"),
                          (lambda c: c["layers"][0]["mixer"]["right"].update(heads=4), "decays"),
                          (lambda c: c["layers"][0]["mixer"]["left"]["q_temp"].update(every=0), "temperature")):
        broken = th.copy(config)
        change(broken)
        (tmp_path / "m" / "config.json").write_text(json.dumps(broken))
        with pytest.raises(ValueError, match=error):
            TuluraxForCausalLM.build(load_model_config(folder), "cpu")


def test_every_tensor_lands_in_its_place(tmp_path):
    config = th.small_config()
    weights = th.make_weights(config)
    folder = mh.save_model(tmp_path / "m", config, weights)
    cfg = load_model_config(folder)
    model = TuluraxForCausalLM.build(cfg, "cpu")
    assert load_model(model, folder) == len(weights)

    def same(tensor, name):
        assert np.array_equal(tensor.double().numpy(), weights[name]), name

    for i, block in enumerate(model.blocks):
        mixer = block.mixer
        for part, keys in (("left", "qkv"), ("right", "qkvg")):
            for key in keys:
                same(mixer.in_proj.piece(mixer.in_proj.weight.data.T, f"{part}.{key}").T, f"l{i}.mix.{part}.{key}")
            at = mixer.o_proj.offset[part]
            same(mixer.o_proj.weight[:, at:at + mixer.o_proj.sizes[part]], f"l{i}.mix.{part}.o")
        same(mixer.parts["left"].talk, f"l{i}.mix.left.talk")
    for module, name in ((model.embed_norm, "embed.norm"), (model.final_norm, "final.norm"), (model.blocks[1].norm1, "l1.norm1"),
                         (model.blocks[2].norm2, "l2.norm2")):
        same(module.weight, name)
        same(module.bias, name + ".b")
        same(module.alpha, name + ".alpha")
        module.finish_loading()
        assert module.norm.alpha == weights[name + ".alpha"] and module.weight.dtype == torch.float32
    mlp = model.blocks[0].mlp
    for tensor, name in ((mlp.up_proj.weight, "up"), (mlp.up_bias, "up.b"), (mlp.down_proj.weight, "down"), (mlp.down_bias, "down.b"), (mlp.act, "act")):
        same(tensor, "l0.mlp." + name)
    same(model.embed_tokens.weight, "embed")
    same(model.lm_head.weight, "head")
    assert model.blocks[1].mlp is None and isinstance(mlp, XieluMLP)
    mlp.finish_loading()
    p, q = weights["l0.mlp.act"]
    assert np.allclose(mlp.constants, (ref.softplus(p), 0.5 + ref.softplus(q)), rtol=1e-12)
    for name, change, error in (("l1.mix.left.talk", None, KeyError), ("l0.mlp.up.b", None, KeyError), ("embed.norm.alpha", None, KeyError),
                                ("l2.norm2.b", None, KeyError), ("l1.norm2", np.zeros(72), KeyError), ("l1.mlp.act", np.zeros(2), KeyError),
                                ("l0.mix.left.g", np.zeros((6, 72)), KeyError), ("l0.mix.q", np.zeros((6, 72)), KeyError),
                                ("l0.mix.right.talk", np.zeros((3, 3)), KeyError), ("l0.norm3", np.zeros(72), KeyError), ("l0.norm1.c", np.zeros(72), KeyError),
                                ("l9.norm1", np.zeros(72), KeyError), ("l0.mix.left.talk", np.zeros((6, 5)), ValueError),
                                ("l0.mix.right.o", np.zeros((72, 71)), ValueError), ("final.norm.alpha", np.zeros(72), ValueError)):
        w = dict(weights)
        if change is None:
            del w[name]
        else:
            w[name] = change
        broken = mh.save_model(tmp_path / name.replace(".", "_"), config, w)
        with pytest.raises(error):
            load_model(TuluraxForCausalLM.build(cfg, "cpu"), broken)


def test_random_weights_leave_no_parameter_unset():
    cfg = TuluraxConfig(40, 24, embedding_scale=2.0)
    from infer_amd.config import LayerSpec
    cfg.layers = [LayerSpec(e["type"], e["mixer"], 16, i) for i, e in enumerate(th.small_config()["layers"])]
    model = TuluraxForCausalLM(cfg)
    for p in model.parameters():
        p.data.fill_(float("nan"))
    model.init_random_weights(1)
    assert all(p.isfinite().all() for p in model.parameters())


# ------------------------------------------------------------------ storage
def test_a_layer_keeps_pages_of_keys_pages_of_values_and_a_state(tmp_path):
    config = th.small_config()
    cfg = load_model_config(mh.save_model(tmp_path / "m", config, th.make_weights(config)))
    layout = TuluraxForCausalLM(cfg).cache_layout(64)
    assert isinstance(layout, LayeredLayout) and len(layout.layers) == 3
    storage = layout.allocate(5, 2, "cpu")
    assert storage[0]["left"]["keys"].shape == (5, 2, 2, 4, 32, 8) and storage[0]["left"]["values"].shape == (5, 2, 2, 2, 4, 16, 8)
    assert storage[1]["left"]["keys"].shape == (5, 5, 2, 4, 32, 8) and storage[1]["left"]["values"].shape == (5, 5, 2, 4, 4, 16, 8)
    assert storage[2]["left"]["keys"].shape == (5, 1, 2, 8, 32, 8) and storage[2]["left"]["values"].dtype == torch.bfloat16
    assert storage[0]["right"]["state"].shape == (2, 3, 32, 32) and storage[0]["right"]["state"].dtype == torch.float32
    assert layout.block_bytes == sum(t.numel() * 2 for s in storage for t in s["left"].values()) // 5
    assert layout.slot_bytes == sum(s["right"]["state"].numel() * 4 for s in storage) // 2


# ------------------------------------------------------------------ index arithmetic of the kernels
def row_token(r, x):
    return 8 * (r >> 2) + 4 * x + (r & 3)


def key_entry(token, d):
    return (d >> 3) * 256 + ((token >> 2 & 1) * 16 + (token >> 3) * 4 + (token & 3)) * 8 + (d & 7)


def value_entry(token, v):
    return (v >> 4) * 512 + (token >> 3) * 128 + (v & 15) * 8 + (token & 7)


def test_tiles_hold_every_entry_and_operands_lie_in_a_row():
    for entry in (key_entry, value_entry):
        assert sorted(entry(t, d) for t in range(32) for d in range(64)) == list(range(2048))
        assert all(entry(t, d) == entry(t, 0) + entry(0, d) for t in range(32) for d in range(64))
    for x in range(2):                                           # lane (g, n): row n, entries 8 g + e of a k-step
        lanes = [key_entry(row_token(n, x), 8 * g) for g in range(4) for n in range(16)]
        assert lanes == [256 * g + 128 * x + 8 * n for g in range(4) for n in range(16)]
    assert [value_entry(8 * g, n) for g in range(4) for n in range(16)] == [8 * i for i in range(64)]
    for g in range(4):
        assert [row_token(r, x) for x in range(2) for r in range(4 * g, 4 * g + 4)] == list(range(8 * g, 8 * g + 8))


def record_place(rec, q, token, at):
    low = (token & 3) | (token >> 1 & 4) if rec == 128 else (token >> 1 & 1) | (token >> 2 & 2) if rec == 64 else token >> 3 & 1
    return ((q * 32 + token) * rec + at) ^ (low << 4) ^ ((q & 15) << 4) ^ (q & 8)


@pytest.mark.parametrize("per_wave,tiles", [(1, 2), (1, 4), (2, 1), (2, 2), (4, 1)])
def test_records_of_the_prompt_kernel_have_places_of_their_own(per_wave, tiles):
    """Every (query, key, head) has one word, written once and read back at the same address; the mixed weights likewise."""
    heads, queries = 8 * per_wave, 16 * tiles
    rec, words = 4 * heads, {}
    for q in range(queries):
        for key in range(32):
            for wave in range(8):
                for u in range(per_wave):                        # as the kernel puts the address together
                    fixed = record_place(rec, q % 16, key // 8 * 8, wave * per_wave * 4)
                    words[(fixed ^ record_place(rec, 0, key % 8, 4 * u)) + q // 16 * (16 * 32 * rec)] = (q, key, wave * per_wave + u)
    assert len(words) == queries * 32 * heads and max(words) + 4 == queries * 32 * rec
    for q in range(queries):
        for key in range(32):
            for unit in range(rec // 16):                        # a 16-byte read holds four heads, two by two in either order
                base = record_place(rec, q, key, 16 * unit ^ (q & 8))
                assert base % 16 == 0
                order = (2, 3, 0, 1) if q & 8 else (0, 1, 2, 3)
                assert [words[base + 4 * i] for i in range(4)] == [(q, key, 4 * unit + i) for i in order]
    for wave in range(8):                                        # the queries that a wavefront mixes have one order
        assert len({q & 8 for q in range(2 * tiles * wave, 2 * tiles * (wave + 1))}) == 1
    places = {(q * heads + (h ^ (q & (heads - 1)))) * 64 + 16 * (g ^ (q >> 2 & 3)) for q in range(queries) for h in range(heads) for g in range(4)}
    assert len(places) == queries * heads * 4 and max(places) + 16 == queries * heads * 64


@pytest.mark.parametrize("per_wave", [1, 2, 4])
def test_lanes_meet_all_banks(per_wave):
    """128 bytes a clock: writes of 16 lanes (one key, 16 queries), reads of eight lanes (eight keys, one query)."""
    rec = 32 * per_wave
    size = 8 if per_wave > 1 else 4
    for key in range(32):
        banks = [(record_place(rec, q, key, 0) + b) % 128 // 4 for q in range(16) for b in range(0, size, 4)]
        assert len(set(banks)) == len(banks)
    for q in range(16):
        for x in range(2):
            for r0 in (0, 8):
                units = {record_place(rec, q, row_token(r, x), q & 8) % 128 // 16 for r in range(r0, r0 + 8)}
                assert len(units) == 8
