"""Dogetar decoder: pre-norm layers of masked attention (windowed with normed heads, the difference of two maps in chunks, or biased
by distance beside a state space), dense feed-forwards and mixtures of experts with a learned scale behind every sublayer, a run of
layers that is repeated, a second embedding of token pairs, a float32 residual stream.

The scale behind a sublayer, the sum of its experts, the residual sum, what enters at the start of a pass and the norm in front of
the next sublayer are one kernel.  A repeated layer has a cache and a state for every pass."""
from __future__ import annotations

import torch
from torch import nn

from . import hybrid_ops
from .cache import LayeredLayout
from .context import get_context
from .layers import Embedding, GatedMLP, Linear
from .masked_attention import MaskedAttention
from .mixer import MAIN, Mixer
from .moe import MixtureOfExperts
from .state_space import StateSpace


def _vector(width: int) -> nn.Parameter:
    return nn.Parameter(torch.ones(width), requires_grad=False)


def _mixer(config, spec) -> Mixer:
    m, dtype, eps = spec.mixer, config.torch_dtype, config.norm_eps

    def attention(m, mask, **named):
        return MaskedAttention(m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["scale"], eps, dtype, mask=mask,
                               mask_size=m["mask"]["size"], rot=m.get("rot"), **named)
    if spec.kind == "attention":
        parts = {MAIN: attention(m, "chunk", diff=m["diff"], gate=True)}
    elif spec.kind == "attention_2":
        parts = {MAIN: attention(m, "window", bias=True, head_norm=True)}
    elif spec.kind == "parallel":
        r = m["right"]
        parts = {"left": attention(m["left"], "chunk", distance_bias=True, sink=True, out_scale=m["left_scale"]),
                 "right": StateSpace(r["heads"], r["vdim"], r["state"], r["groups"], r["conv"], r["norm_groups"], eps, dtype,
                                     out_scale=m["right_scale"])}
    else:
        raise ValueError(f"no mixer of kind {spec.kind!r}")
    return Mixer(config.hidden_size, parts, dtype)


def _feed_forward(config, mlp: dict) -> nn.Module:
    width, dtype = config.hidden_size, config.torch_dtype
    if mlp["kind"] == "dense":
        return GatedMLP(width, mlp["ff"], dtype, act="clamped", limit=mlp["limit"])
    r, shared = mlp["router"], mlp.get("shared")
    groups = r.get("groups") or {"count": 1, "keep": 1}
    return MixtureOfExperts(width, mlp["expert"]["ff"], r["experts"], r["top"], dtype, identity=r.get("identity") or 0,
                            groups=groups["count"], keep=groups["keep"], scale=r["scale"], shared_ff=shared["ff"] if shared else None)


class DogetarBlock(nn.Module):
    """The weights of a layer."""

    def __init__(self, config, spec):
        super().__init__()
        width = config.hidden_size
        self.mixer = _mixer(config, spec)
        self.norm1, self.ls1 = _vector(width), _vector(width)
        self.mlp = None
        if spec.mlp is not None:
            self.mlp = _feed_forward(config, spec.mlp)
            self.norm2, self.ls2 = _vector(width), _vector(width)


class DogetarForCausalLM(nn.Module):
    mixed_steps = True            # a step is a batch of portions (``PortionScheduler``, ``StepPlan``)

    _STATE = {"conv": "conv", "conv.b": "conv_bias", "dt_bias": "dt_bias", "A_log": "a_log", "D": "d", "norm": "out_norm"}
    _ATTENTION = {"q.norm": "q_norm", "k.norm": "k_norm", "sink": "sink", "lq1": "lq1", "lk1": "lk1", "lq2": "lq2", "lk2": "lk2"}

    def __init__(self, config):
        super().__init__()
        self.config = config
        dtype, width = config.torch_dtype, config.hidden_size
        self.runs = config.runs()
        self.embed_tokens = Embedding(config.vocab_size, width, dtype)
        self.bigram = Embedding(config.bigram["buckets"] + 1, width, dtype) if config.bigram else None
        self.loop_step = nn.Parameter(torch.zeros(config.loop.times, width), requires_grad=False) if config.loop else None
        self.blocks = nn.ModuleList([DogetarBlock(config, spec) for spec in config.layers])
        self.final_norm = _vector(width)
        self.lm_head = Linear(width, config.vocab_size, dtype=dtype)
        self.caches: list = [None] * len(self.runs)

    @classmethod
    def build(cls, config, device) -> "DogetarForCausalLM":
        return cls(config).to(device)                 # parameters have their types already: norms stay float32

    # ------------------------------------------------------------------ weights
    def checkpoint_target(self, name: str) -> tuple[str, object]:
        whole = {"embed": "embed_tokens.weight", "bigram": "bigram.weight", "loop.step": "loop_step", "head": "lm_head.weight",
                 "final.norm": "final_norm"}
        if name in whole:
            return whole[name], None
        layer, _, rest = name.partition(".")
        index = layer[1:]
        if layer[:1] != "l" or not index.isdecimal() or int(index) >= len(self.blocks):
            raise KeyError(f"checkpoint tensor {name} belongs to no layer of the model")
        block = self.blocks[int(index)]
        group, _, key = rest.partition(".")
        target = None
        if rest in ("norm1", "norm2", "ls1", "ls2"):
            target = rest, None
        elif group == "mix":
            target = self._mixer_target(block.mixer, key)
        elif group == "mlp" and block.mlp is not None:
            target = self._mlp_target(block.mlp, key)
        if target is None:
            raise KeyError(f"checkpoint tensor {name} has no place in its layer")
        return f"blocks.{int(index)}.{target[0]}", target[1]

    @classmethod
    def _mixer_target(cls, mixer: Mixer, key: str):
        part = MAIN
        if MAIN not in mixer.parts:
            part, _, key = key.partition(".")
            if part not in mixer.parts:
                return None
        module = mixer.parts[part]
        if key in module.pieces():
            return "mixer.in_proj.weight", mixer.piece(part, key)
        if key == "o":
            return "mixer.o_proj.weight", part
        if key.endswith(".b") and key[:-2] in module.biased_pieces:
            return "mixer.bias.weight", mixer.piece(part, key[:-2])
        name = (cls._STATE if isinstance(module, StateSpace) else cls._ATTENTION).get(key)
        return None if name is None else (f"mixer.parts.{part}.{name}", None)

    @staticmethod
    def _mlp_target(mlp: nn.Module, key: str):
        dense = {"gate": ("gate_up_proj.weight", 0), "up": ("gate_up_proj.weight", 1), "down": ("down_proj.weight", None)}
        if isinstance(mlp, GatedMLP):
            return ("mlp." + dense[key][0], dense[key][1]) if key in dense else None
        if key in ("router", "correction"):
            return f"mlp.{key}", None
        owner, _, key = key.partition(".")
        if owner == "shared" and key in dense and mlp.shared is not None:
            return "mlp.shared." + dense[key][0], dense[key][1]
        if owner[:1] == "e" and owner[1:].isdecimal() and int(owner[1:]) < mlp.shape.experts and key in dense:
            return ("mlp.down.weight", (int(owner[1:]), 0)) if key == "down" else ("mlp.gate_up.weight", (int(owner[1:]), dense[key][1]))
        return None

    def init_random_weights(self, seed: int = 0) -> None:
        """Weights that keep activations of the order of one: the stand-in for a checkpoint."""
        gen = torch.Generator(device=self.final_norm.device).manual_seed(seed)
        for name, p in self.named_parameters():
            leaf = name.rpartition(".")[2]
            if leaf.endswith("norm") or leaf in ("norm1", "norm2", "d"):
                p.data.fill_(1.0)
            elif leaf in ("ls1", "ls2"):
                p.data.fill_(0.5)
            elif leaf in ("sink", "conv_bias", "lq1", "lk1", "lq2", "lk2", "loop_step", "correction") or name.endswith("bias.weight"):
                p.data.zero_()
            elif leaf in ("a_log", "dt_bias"):
                p.data.uniform_(-2.0, 1.0, generator=gen)
            elif name in ("embed_tokens.weight", "bigram.weight"):
                p.data.normal_(0.0, 1.0, generator=gen)
            else:
                p.data.normal_(0.0, p.shape[-1] ** -0.5, generator=gen)

    def finish_loading(self, max_position: int) -> None:
        for block in self.blocks:
            block.mixer.finish_loading(max_position)

    # ------------------------------------------------------------------ cache
    def cache_layout(self, block_size: int) -> LayeredLayout:
        return LayeredLayout([self.blocks[i].mixer.cache_spec() for i, _ in self.runs], block_size)

    def bind_cache(self, storage: list) -> None:
        assert len(storage) == len(self.caches)
        self.caches = storage

    def prepare_decode(self, device, max_batch: int) -> None:
        pass                                          # every workspace of a step comes from torch's allocator

    # ------------------------------------------------------------------ the step
    def forward(self, input_ids: torch.Tensor, positions: torch.Tensor) -> torch.Tensor:
        """Final hidden states of the step in ``get_context().step``."""
        cfg, plan = self.config, get_context().step
        n = input_ids.numel()
        x = torch.empty((n, cfg.hidden_size), dtype=torch.float32, device=input_ids.device)
        first = torch.empty_like(x) if cfg.loop and cfg.loop.times > 1 else None
        # (sublayer, scale behind it) in order; (norm, what is added in front of it) of each, and the final norm
        sublayers, before = [], []
        for (i, turn), cache in zip(self.runs, self.caches):
            block, enter = self.blocks[i], {}
            if turn is not None and i == cfg.loop.start:
                enter = dict(step=self.loop_step[turn], first=first if turn else None)
            sublayers.append((lambda h, m=block.mixer, c=cache: m(h, c), block.ls1))
            before.append((block.norm1, enter))
            if block.mlp is not None:
                sublayers.append((block.mlp, block.ls2))
                before.append((block.norm2, {}))
        before.append((self.final_norm, {}))
        common = dict(eps=cfg.norm_eps, dtype=cfg.torch_dtype)
        pair = dict(prev=plan.prev_ids, bigram=self.bigram.weight,
                    multipliers=(cfg.bigram["mul_prev"], cfg.bigram["mul_cur"])) if self.bigram is not None else {}
        h = hybrid_ops.pre_norm(x, before[0][0], tokens=input_ids, embed=self.embed_tokens.weight, **pair, **common,
                                **{**before[0][1], "first": first})
        for (run, scale), (norm, enter) in zip(sublayers, before[1:]):
            h = hybrid_ops.pre_norm(x, norm, y=run(h), scale=scale, **enter, **common)
        return h

    def compute_logits(self, hidden_states: torch.Tensor) -> torch.Tensor:
        logits = self.lm_head(hidden_states)
        return hybrid_ops.softcap(logits, self.config.logit_softcap) if self.config.logit_softcap else logits
