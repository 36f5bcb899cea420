"""Dogetar without a GPU: the oracle against other ways to compute the same, configuration and loading, the order of layer runs,
storage, the step plan."""
import json
import math

import numpy as np
import pytest
import torch

from infer_amd.cache import LayeredLayout
from infer_amd.config import Config, DogetarConfig, load_model_config
from infer_amd.dogetar import DogetarForCausalLM
from infer_amd.layers import ColumnPackedLinear, banded_rotary_table
from infer_amd.registry import model_class
from infer_amd.sequence import Sequence
from infer_amd.step_plan import build
from infer_amd.weight_loader import load_model
from oracle import dogetar_ref as ref
from tests import dogetar_helpers as dh, merilorn_helpers as mh


# ------------------------------------------------------------------ the oracle
def test_pairs_address_rows_and_a_first_token_has_the_last():
    assert ref.bigram_rows([3, 4, 0, 9], 10, 7, 5).tolist() == [10, (21 + 20) % 10, 28 % 10, 45 % 10]
    assert ref.bigram_rows([3], 10, 7, 5).tolist() == [10]


def test_masks_by_hand():
    assert ref.chunk_mask(5, 2).astype(int).tolist() == [[1, 0, 0, 0, 0], [1, 1, 0, 0, 0], [0, 0, 1, 0, 0], [0, 0, 1, 1, 0], [0, 0, 0, 0, 1]]
    assert ref.window_mask(4, 2).astype(int).tolist() == [[1, 0, 0, 0], [1, 1, 0, 0], [0, 1, 1, 0], [0, 0, 1, 1]]


def test_distance_bias_with_a_sink_is_no_shift_of_the_keys():
    rng = np.random.default_rng(1)
    t, heads = 6, 3
    q, k, v = rng.standard_normal((t, heads, 4)), rng.standard_normal((t, 1, 4)), rng.standard_normal((t, 1, 5))
    sink, slopes = rng.standard_normal(heads), ref.distance_slopes(heads)
    assert np.allclose(slopes, [2 ** (-8 / 3), 2 ** (-16 / 3), 2 ** -8])
    mask = ref.chunk_mask(t, 4)
    got = ref.masked_attention(q, k, v, 0.5, mask, sink, slopes)
    for i in range(t):
        for h in range(heads):
            at = np.flatnonzero(mask[i])
            s = np.append(k[at, 0] @ q[i, h] * 0.5 - slopes[h] * (i - at), sink[h])
            p = np.exp(s) / np.exp(s).sum()
            assert np.allclose(got[i, h], p[:-1] @ v[at, 0])
            shifted = np.append(k[at, 0] @ q[i, h] * 0.5 + slopes[h] * at, sink[h])      # equal but for the sink
            p = np.exp(shifted) / np.exp(shifted).sum()
            assert i == 0 or not np.allclose(got[i, h], p[:-1] @ v[at, 0])


def test_scaled_frequencies_keep_short_waves_and_slow_long_ones():
    rot = {"base": 1000.0, "dims": 24, "scaling": {"factor": 5.0, "low": 1.0, "high": 4.0, "original": 300}}
    plain, scaled = ref.scaled_frequencies({**rot, "scaling": None}), ref.scaled_frequencies(rot)
    wave = 2 * math.pi / plain
    short, long_ = wave < 75, wave > 300
    assert short.any() and long_.any() and (~short & ~long_).any()
    assert np.array_equal(scaled[short], plain[short]) and np.allclose(scaled[long_], plain[long_] / 5)
    between = scaled[~short & ~long_] / plain[~short & ~long_]
    assert ((between > 0.2) & (between < 1.0)).all() and (np.diff(between) < 0).all()
    table = banded_rotary_table(24, 500, 1000.0, rot["scaling"], "cpu").double().numpy()
    angle = np.arange(500)[:, None] * scaled
    assert np.abs(table - np.stack((np.cos(angle), np.sin(angle)), -1)).max() < 1e-6


def test_state_space_scan_equals_its_chunk_form_and_its_halves():
    """The algebra of the chunked kernel and of its segments, in numpy."""
    rng = np.random.default_rng(2)
    n, state, vdim, a, d = 13, 6, 5, -0.7, 0.3
    x, b, c = rng.standard_normal((n, vdim)), rng.standard_normal((n, state)), rng.standard_normal((n, state))
    dt, s0 = rng.random(n), rng.standard_normal((state, vdim))
    want, s_want = ref.state_space_scan(x, b, c, dt, a, d, s0)
    sums = np.cumsum(a * dt)
    inside = np.tril(np.exp(np.minimum(sums[:, None] - sums, 0.0)) * (c @ b.T) * dt)
    assert np.allclose(np.exp(sums)[:, None] * (c @ s0) + inside @ x + d * x, want)
    assert np.allclose(np.exp(sums[-1]) * s0 + b.T @ (np.exp(sums[-1] - sums)[:, None] * dt[:, None] * x), s_want)
    half, s_half = ref.state_space_scan(x[:7], b[:7], c[:7], dt[:7], a, d, s0)
    rest, s_rest = ref.state_space_scan(x[7:], b[7:], c[7:], dt[7:], a, d, s_half)
    assert np.allclose(np.concatenate([half, rest]), want) and np.allclose(s_rest, s_want)
    added = ref.state_space_scan(x[7:], b[7:], c[7:], dt[7:], a, d)[1]
    assert np.allclose(np.exp(a * dt[7:].sum()) * s_half + added, s_want)


def test_convolution_by_hand():
    x = np.array([[1.0], [2.0], [3.0]])
    assert np.allclose(ref.causal_conv(x, np.array([[10.0, 1.0]]), np.array([0.5])), [[1.5], [12.5], [23.5]])


def test_a_group_is_as_good_as_its_best_and_negative_choices_count():
    z = np.log(np.array([[0.5, 0.05, 0.2, 0.25]]))
    chosen, weight = ref.route(z, np.zeros(4), 2, {"count": 2, "keep": 1}, 2.0)
    assert chosen.tolist() == [[0, 1]] and np.allclose(weight, [[1.0, 0.1]])             # not 3: its group is closed
    chosen, weight = ref.route(z, np.array([-1.0, -1.0, -1.0, -1.0]), 3, None, 1.0)
    assert chosen.tolist() == [[0, 3, 2]] and np.allclose(weight, [[0.5, 0.25, 0.2]])     # scores without the correction
    chosen, _ = ref.route(z, np.array([-1.0, -1.0, 0.0, 0.0]), 2, {"count": 2, "keep": 1}, 1.0)
    assert chosen.tolist() == [[3, 2]]
    chosen, _ = ref.route(z, np.array([-2.0, -2.0, -1.0, -1.5]), 2, {"count": 2, "keep": 1}, 1.0)
    assert chosen.tolist() == [[2, 3]]                                                    # closed entries are not zeros


def test_identity_experts_return_their_input():
    h = np.random.default_rng(3).standard_normal((2, 4))
    router = np.zeros((3, 4))
    w = {"router": router, "correction": np.array([0.0, 0.0, 5.0]), "e0.gate": None}
    m = {"router": {"experts": 2, "identity": 1, "top": 1, "scale": 3.0}}
    assert np.allclose(ref.mixture(h, m, w.get), h)                                       # a third of a three-fold


def test_layer_loop_by_hand():
    """Sublayers that give nothing: the stream is the embedding, once more in front of every pass but the first, and the steps."""
    config = dh.make_config([dh.windowed(), dh.chunked(), dh.windowed(mlp=dh.dense())], loop=(1, 3, 3), width=24)
    w = dh.make_weights(config)
    for name in w:
        if name.endswith((".o", ".down")):
            w[name] = np.zeros_like(w[name])
    x0 = ref.embed(config, w, [5, 6])
    assert ref.run_order(config) == [(0, None)] + [(i, t) for t in range(3) for i in (1, 2)]
    stream = ref.forward(config, w, [5, 6])[1]
    step = w["loop.step"]
    assert np.allclose(stream[0], x0) and np.allclose(stream[2], x0 + step[0]) and np.allclose(stream[-1], 3 * x0 + step.sum(0))


# ------------------------------------------------------------------ configuration and weights
def test_config_and_registry(tmp_path):
    config = dh.small_config()
    folder = mh.save_model(tmp_path / "m", config, dh.make_weights(config))
    cfg = load_model_config(folder)
    assert isinstance(cfg, DogetarConfig) and model_class(cfg) is DogetarForCausalLM
    assert [s.kind for s in cfg.layers] == [e["type"] for e in config["layers"]]
    assert cfg.runs() == ref.run_order(config)
    assert (cfg.logit_softcap, cfg.norm_eps, cfg.vocab_size, cfg.hidden_size) == (12.0, 1e-4, 131, 72)
    assert cfg.bigram == {"buckets": 53, "mul_prev": 7, "mul_cur": 11} and cfg.layers[2].mlp is None
    assert Config(folder, kvcache_block_size=64, dtype="float32").hf_config.torch_dtype == torch.float32
    for change, error in ((lambda c: c["layers"][1]["mlp"].update(kind="other"), "other"), (lambda c: c["layers"][1].update(type="none"), "none"),
                          (lambda c: c["loop"].update(stop=9), "cannot run"), (lambda c: c["layers"][1]["mlp"]["router"].update(top=5), "cannot be chosen")):
        broken = dh.copy(config)
        change(broken)
        (tmp_path / "m" / "config.json").write_text(json.dumps(broken))
        with pytest.raises(ValueError, match=error):
            DogetarForCausalLM.build(load_model_config(folder), "cpu")


def test_every_tensor_lands_in_its_place(tmp_path):
    config = dh.small_config()
    weights = dh.make_weights(config)
    folder = mh.save_model(tmp_path / "m", config, weights)
    cfg = load_model_config(folder)
    model = DogetarForCausalLM.build(cfg, "cpu")
    assert load_model(model, folder) == len(weights)

    def same(tensor, name):
        assert np.array_equal(tensor.double().numpy(), weights[name]), name

    for layer, part, names in ((0, "left.", "qkv"), (1, "", "qkvg"), (2, "", "qkv")):
        mixer = model.blocks[layer].mixer
        for key in names:
            same(mixer.in_proj.piece(mixer.in_proj.weight.data.T, part + key).T, f"l{layer}.mix.{part}{key}")
    mixer = model.blocks[0].mixer
    same(mixer.in_proj.piece(mixer.in_proj.weight.data.T, "right.in").T, "l0.mix.right.in")
    off = mixer.o_proj.offset
    same(mixer.o_proj.weight[:, off["left"]:off["left"] + 48], "l0.mix.left.o")
    same(mixer.o_proj.weight[:, off["right"]:off["right"] + 48], "l0.mix.right.o")
    same(mixer.parts["left"].sink, "l0.mix.left.sink")
    for key, name in (("conv", "conv"), ("conv.b", "conv_bias"), ("A_log", "a_log"), ("D", "d"), ("norm", "out_norm"), ("dt_bias", "dt_bias")):
        same(getattr(mixer.parts["right"], name), "l0.mix.right." + key)
    bias = model.blocks[2].mixer.bias
    for key in "qkv":
        same(bias.weight[bias.offset[key]:bias.offset[key] + bias.sizes[key]], f"l2.mix.{key}.b")
    moe = model.blocks[1].mlp
    for e in range(5):
        same(moe.gate_up.weight[e, :24], f"l1.mlp.e{e}.gate")
        same(moe.gate_up.weight[e, 24:], f"l1.mlp.e{e}.up")
        same(moe.down.weight[e, :, :24], f"l1.mlp.e{e}.down")
    same(moe.router, "l1.mlp.router")
    same(moe.correction, "l1.mlp.correction")
    same(moe.shared.down_proj.weight, "l1.mlp.shared.down")
    odd = model.blocks[3].mlp
    assert odd.down.weight.shape == (6, 72, 24) and not odd.down.weight[..., 17:].any() and odd.shared is None
    same(odd.down.weight[2, :, :17], "l3.mlp.e2.down")
    same(model.bigram.weight, "bigram")
    same(model.loop_step, "loop.step")
    same(model.blocks[4].ls2, "l4.ls2")
    assert model.loop_step.dtype == model.blocks[4].norm1.dtype == mixer.parts["left"].sink.dtype == torch.float32
    for name, change, error in (("l1.mix.lq1", None, KeyError), ("l2.mix.q.b", None, KeyError), ("bigram", None, KeyError),
                                ("l0.mix.sink", np.zeros(3), KeyError), ("l2.norm2", np.zeros(72), KeyError), ("l3.mlp.shared.up", np.zeros((4, 72)), KeyError),
                                ("l1.mlp.e5.up", np.zeros((24, 72)), KeyError), ("l9.norm1", np.zeros(72), KeyError), ("l1.mlp.e4.up", np.zeros((24, 71)), ValueError),
                                ("l0.mix.left.o", np.zeros((72, 47)), ValueError)):
        w = dict(weights)
        if change is None:
            del w[name]
        else:
            w[name] = change
        broken = mh.save_model(tmp_path / name.replace(".", "_"), config, w)
        with pytest.raises(error):
            load_model(DogetarForCausalLM.build(cfg, "cpu"), broken)


def test_inputs_side_by_side_meet_their_columns():
    lin = ColumnPackedLinear({"a": 6, "b": 8}, 3, torch.float32)
    a, b = torch.randn(3, 6), torch.randn(3, 8)
    lin.weight_loader(lin.weight, a, "a")
    lin.weight_loader(lin.weight, b, "b")
    x, y = torch.randn(5, 6), torch.randn(5, 8)
    both = torch.zeros(5, lin.in_features)
    both[:, :6], both[:, lin.offset["b"]:lin.offset["b"] + 8] = x, y
    assert lin.padded and torch.allclose(lin(both), x @ a.T + y @ b.T, atol=1e-5)


# ------------------------------------------------------------------ storage and step plan
def test_every_pass_has_a_storage_of_its_own():
    config = dh.make_config([dh.windowed(), dh.parallel(mlp=dh.dense())], loop=(1, 2, 3))
    cfg = DogetarConfig(131, 72, bigram=None)
    from infer_amd.config import LayerLoop, LayerSpec
    cfg.layers = [LayerSpec(e["type"], e["mixer"], None, i, e["mlp"]) for i, e in enumerate(config["layers"])]
    cfg.loop = LayerLoop(1, 2, 3)
    layout = DogetarForCausalLM(cfg).cache_layout(32)
    assert isinstance(layout, LayeredLayout) and len(layout.layers) == 4
    storage = layout.allocate(5, 2, "cpu")
    states = [s["right"]["state"] for s in storage[1:]]
    assert len({t.data_ptr() for t in states}) == 3 and all(t.shape == (2, 4, 16, 12) and t.dtype == torch.float32 for t in states)
    assert layout.slot_bytes == 3 * (4 * 16 * 12 * 4 + 4 * (48 + 2 * 2 * 16) * 2)
    assert layout.block_bytes == 32 * 2 * (2 * (32 + 32) + 3 * (32 + 32))


def test_previous_tokens_of_a_step():
    bs, portions = 32, []
    for slot, (lo, n) in enumerate([(40, 1), (0, 1), (0, 3), (17, 2)]):
        seq = Sequence(list(range(100 * slot, 100 * slot + lo + n)), block_size=bs)
        seq.num_computed_tokens, seq.state_slot, seq.block_table = lo, slot, [2 * slot, 2 * slot + 1]
        portions.append((seq, n))
    plan, _ = build(portions, bs, 4, 4, 16, "cpu")
    before = dict(zip(plan.input_ids.tolist(), plan.prev_ids.tolist()))
    assert before == {40: 39, 100: -1, 200: -1, 201: 200, 202: 201, 317: 316, 318: 317}
