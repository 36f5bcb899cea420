"""Vokelix without a GPU: the oracle against other ways to compute the same, configuration and loading, shared storage,
the step plan."""
import json

import numpy as np
import pytest
import torch

from infer_amd import hybrid_ops
from infer_amd.cache import GroupedPages, LayeredLayout, SharedStorage, StateSlots
from infer_amd.config import Config, VokelixConfig, load_model_config
from infer_amd.layers import PackedBias, PackedLinear
from infer_amd.registry import model_class
from infer_amd.sequence import Sequence
from infer_amd.step_plan import build
from infer_amd.vokelix import VokelixForCausalLM
from infer_amd.weight_loader import load_model
from oracle import vokelix_ref as ref
from tests import merilorn_helpers as mh, vokelix_helpers as vh


# ------------------------------------------------------------------ the oracle
def test_rotation_of_halves_depends_on_distance_only_and_leaves_the_rest_alone():
    rng = np.random.default_rng(0)
    q, k = rng.standard_normal((2, 13))
    freq, _ = ref.yarn_frequencies(8, 50.0)
    for a, b in ((3, 1), (40, 38)):
        x = ref.rotate_halves(np.stack([q, k]), [a, b], freq)
        assert np.isclose(x[0] @ x[1], ref.rotate_halves(np.stack([q, k]), [2, 0], freq)[0] @ k)
        assert np.array_equal(x[:, 8:], np.stack([q, k])[:, 8:])
    one = ref.rotate_halves(np.array([[1.0, 0.0, 0.0, 2.0]]), [1], np.array([0.5, 0.25]))
    assert np.allclose(one, [[np.cos(.5), -2 * np.sin(.25), np.sin(.5), 2 * np.cos(.25)]])


def test_a_sink_is_a_key_without_value():
    rng = np.random.default_rng(1)
    t, heads, kv = 7, 4, 2
    q, k, v = rng.standard_normal((t, heads, 6)), rng.standard_normal((t, kv, 6)), rng.standard_normal((t, kv, 5))
    sink = rng.standard_normal(heads) * 3
    got = ref.sink_attention(q, k, v, 0.7, sink)
    for i in range(t):
        for h in range(heads):
            s = np.append(k[:i + 1, h // 2] @ q[i, h] * 0.7, sink[h])
            p = np.exp(s - s.max())
            p /= p.sum()
            assert np.allclose(got[i, h], p[:-1] @ v[:i + 1, h // 2])


def test_decay_scan_equals_its_chunk_form_and_its_halves():
    """The algebra of the chunked kernel and of its segments, in numpy."""
    rng = np.random.default_rng(1)
    n, dim, vdim, d = 13, 6, 5, 0.8
    q, k, v, s0 = (rng.standard_normal(s) for s in ((n, dim), (n, dim), (n, vdim), (dim, vdim)))
    want, s_want = ref.decay_scan(q, k, v, d, s0)
    i = np.arange(n)
    inside = np.tril(d ** np.maximum(i[:, None] - i, 0)) * (q @ k.T) @ v
    assert np.allclose(inside + d ** (i + 1.0)[:, None] * (q @ s0), want)
    assert np.allclose(d ** n * s0 + k.T @ (d ** (n - 1.0 - i)[:, None] * v), s_want)
    half, s_half = ref.decay_scan(q[:7], k[:7], v[:7], d, s0)
    rest, s_rest = ref.decay_scan(q[7:], k[7:], v[7:], d, s_half)
    assert np.allclose(np.concatenate([half, rest]), want) and np.allclose(s_rest, s_want)
    added = ref.decay_scan(q[7:], k[7:], v[7:], d)[1]
    assert np.allclose(d ** 6 * s_half + added, s_want)


def test_post_norm_stream_by_hand():
    """Two layers whose sublayers give nothing: the stream is normed twice per layer with a feed-forward, once without."""
    config = vh.make_config([vh.lightning(ff=8), vh.lightning()], width=12, eps=0.1, alpha=3.0)
    w = vh.make_weights(config)
    for name in w:
        if name.endswith((".o", ".down")):
            w[name] = np.zeros_like(w[name])
    x = w["embed"][[5, 6]]
    for name in ("l0.norm1", "l0.norm2", "l1.norm1"):
        x = 3.0 * x / np.sqrt((9.0 * x * x).mean(-1, keepdims=True) + 0.1) * (1.0 + w[name])
    assert np.allclose(ref.forward(config, w, [5, 6])[1][-1], x)


def test_three_pieces_hold_a_float_exactly():
    """What the chunked kernel relies on: the leading 8 bits, the next 8 and the rest are bf16 numbers whose sum is x."""
    rng = np.random.default_rng(2)
    x = (rng.standard_normal(10000) * 10.0 ** rng.uniform(-20, 20, 10000)).astype(np.float32)

    def head(a):
        return (a.view(np.uint32) & np.uint32(0xffff0000)).view(np.float32)
    hi = head(x)
    mid = head(x - hi)
    lo = x - hi - mid
    assert np.array_equal(lo, head(lo)) and np.array_equal(hi.astype(np.float64) + mid + lo, x.astype(np.float64))


def test_decay_constants_keep_what_float_loses():
    d = [0.9, 1.0 - 2.0 ** -20, 1.0 / 3.0, 1.0]
    c = hybrid_ops.decay_constants(d, "cpu").double().numpy()
    assert np.abs(c[0] + c[1] - d).max() < 1e-15 and np.allclose(c[2], np.log2(d), rtol=1e-7, atol=1e-12)
    assert hybrid_ops.decay_constants([0.0], "cpu")[2, 0] == -1e4             # finite: its zeroth power is one


# ------------------------------------------------------------------ configuration and weights
def test_config_and_registry(tmp_path):
    config = vh.small_config()
    folder = mh.save_model(tmp_path / "m", config, vh.make_weights(config))
    cfg = load_model_config(folder)
    assert isinstance(cfg, VokelixConfig) and model_class(cfg) is VokelixForCausalLM
    assert [s.kind for s in cfg.layers] == [e["type"] for e in config["layers"]]
    assert [s.ff for s in cfg.layers] == [None, 56, 40, None, 48, None, None, 56]
    assert (cfg.residual_alpha, cfg.norm_eps, cfg.vocab_size, cfg.hidden_size) == (1.7, 1e-4, 131, 72)
    assert Config(folder, kvcache_block_size=64, dtype="float32").hf_config.torch_dtype == torch.float32
    config["layers"][1]["mlp"]["kind"] = "other"
    (tmp_path / "m" / "config.json").write_text(json.dumps(config))
    with pytest.raises(ValueError, match="other"):
        load_model_config(folder)


def test_every_tensor_lands_in_its_place(tmp_path):
    config = vh.small_config()
    weights = vh.make_weights(config)
    folder = mh.save_model(tmp_path / "m", config, weights)
    cfg = load_model_config(folder)
    model = VokelixForCausalLM.build(cfg, "cpu")
    assert load_model(model, folder) == len(weights)
    mixer = model.blocks[1].mixer
    for name in "qkvg":
        assert np.array_equal(mixer.in_proj.piece(mixer.in_proj.weight.data.T, name).T.double().numpy(), weights[f"l1.mix.{name}"])
    off = mixer.in_proj.offset
    assert np.array_equal(mixer.bias.weight[off["v"]:off["v"] + 32].double().numpy(), weights["l1.mix.v.b"])
    assert np.array_equal(mixer.k_norm.double().numpy(), weights["l1.mix.k.norm"]) and mixer.sink.dtype == torch.float32
    assert set(model.blocks[5].mixer.in_proj.sizes) == {"q", "g"} and model.blocks[5].mixer.k_norm is None
    norm = model.blocks[4].norm2
    norm.finish_loading()
    assert np.allclose(norm.gain.double().numpy(), 1.0 + weights["l4.norm2"], rtol=1e-7)
    for name, change, error in (("l1.mix.sink", None, KeyError), ("l1.mix.q.b", None, KeyError), ("l0.mix.norm", np.zeros(5), ValueError),
                                ("l5.mix.k", np.zeros((48, 72)), KeyError), ("l2.mix.norm", np.zeros(80), KeyError),
                                ("l9.norm1", np.zeros(72), KeyError), ("l6.norm2", np.zeros(72), KeyError)):
        w = dict(weights)
        if change is None:
            del w[name]
        else:
            w[name] = change
        broken = mh.save_model(tmp_path / name.replace(".", "_"), config, w)
        with pytest.raises(error):
            load_model(VokelixForCausalLM.build(cfg, "cpu"), broken)


@pytest.mark.parametrize("owner,other", [(0, {}), (5, {}), (2, {}), (1, dict(dim=32)), (1, dict(heads=3, kv_heads=3)), (1, dict(vdim=8))])
def test_keys_are_shared_only_with_an_earlier_attention_layer_of_equal_shape(owner, other):
    """Layer 0 is no attention, layer 2 has no keys of its own, layer 5 does not come first."""
    layers = [vh.lightning(), vh.attention(), vh.attention(kv_from=1), vh.attention(kv_from=owner, **other)]
    raw = vh.make_config(layers)
    from infer_amd.config import LayerSpec
    cfg = VokelixConfig(131, 72, [LayerSpec(e["type"], e["mixer"], 8, i) for i, e in enumerate(raw["layers"])])
    with pytest.raises(ValueError, match="layer 3"):
        VokelixForCausalLM(cfg)


def test_packed_bias_lies_where_its_projection_does():
    lin = PackedLinear(4, {"q": 6, "k": 3, "g": 2}, torch.float32)
    bias = PackedBias(lin, ("q", "k"))
    bias.weight_loader(bias.weight, torch.ones(3), "k")
    assert bias.weight.nonzero().flatten().tolist() == [8, 9, 10] and set(bias.sizes) == {"q", "k"}
    with pytest.raises(ValueError):
        bias.weight_loader(bias.weight, torch.ones(4), "q")


# ------------------------------------------------------------------ storage and step plan
def test_shared_storage_takes_no_memory_and_is_the_owners():
    pages, slots = GroupedPages(2, 64, torch.bfloat16), StateSlots(state=((3, 32, 32), torch.float32))
    layout = LayeredLayout([slots, pages, SharedStorage(1), GroupedPages(1, 32, torch.float32)], 32)
    assert layout.block_bytes == 32 * 2 * 64 * 2 + 32 * 32 * 4 and layout.slot_bytes == 3 * 32 * 32 * 4
    storage = layout.allocate(5, 2, "cpu")
    assert storage[2] is storage[1] and storage[1].shape == (5, 2, 32, 64) and storage[0]["state"].shape == (2, 3, 32, 32)


def test_spans_cover_the_rows_behind_the_decoded_tokens():
    bs, portions = 32, []
    for slot, (lo, n) in enumerate([(40, 1), (0, 70), (17, 2), (33, 33)]):
        seq = Sequence(list(range(lo + n)), block_size=bs)
        seq.num_computed_tokens, seq.state_slot, seq.block_table = lo, slot, list(range(4 * slot, 4 * slot + 4))
        portions.append((seq, n))
    plan, first = build(portions, bs, 4, 4, 16, "cpu")
    assert plan.decode_rows == 1 and plan.max_span == 70
    assert plan.spans.tolist() == [[first[2], 2, 2, 17], [first[3], 33, 3, 33], [first[1], 70, 1, 0]]
    alone, _ = build(portions[:1], bs, 4, 4, 16, "cpu")
    assert alone.spans.shape == (0, 4) and alone.max_span == 0


def requested_rows(count, dim):
    """The rows of a span of ``count`` tokens that the chunk kernel of constant-decay attention requests for q and k: its
    index arithmetic, for every thread and every chunk, the request behind the last chunk included."""
    per_thread, units = max(1, dim // 128 if dim <= 128 else 2), dim // 16
    u = np.arange(256)[:, None] + 256 * np.arange(per_thread)
    tok = np.where(u < 32 * units, u // units, 0)
    rows = []
    for c in range(-(-count // 32) + 1):
        last = count - c * 32 - 1
        rows.append(tok + 32 * c - np.maximum(tok - last, 0))
    return np.concatenate(rows)


@pytest.mark.parametrize("dim", [16, 32, 48, 64, 80, 96, 112, 128, 192, 256])
def test_requests_of_the_chunk_kernel_stay_inside_the_span(dim):
    for count in (2, 3, 31, 32, 33, 63, 64, 65, 96, 100, 128, 512):
        rows = requested_rows(count, dim)
        assert rows.min() == 0 and rows.max() == count - 1
