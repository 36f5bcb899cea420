"""Vokelix decoder: layers of grouped attention and of linear attention with a constant decay (lightning, retention) in
the order the configuration gives, a norm behind every residual sum, a float32 residual stream.

The residual sum, the norm behind it and, after the last sublayer, the model's final norm are one kernel."""
from __future__ import annotations

import torch
from torch import nn

from . import hybrid_ops
from .cache import LayeredLayout, SharedStorage
from .decay_attention import DecayAttention
from .grouped_attention import GroupedAttention
from .layers import Embedding, GatedMLP, Linear, ZeroCentredNorm


class VokelixBlock(nn.Module):
    """The weights of a layer."""

    def __init__(self, config, spec):
        super().__init__()
        m, width, dtype, eps = spec.mixer, config.hidden_size, config.torch_dtype, config.norm_eps
        if spec.kind == "attention":
            self.mixer = GroupedAttention(width, m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["scale"], m["rot"], eps, dtype,
                                          own_keys=m.get("kv_from") is None)
        elif spec.kind == "lightning":
            self.mixer = DecayAttention(width, m["heads"], m["dim"], m["vdim"], m["decay"], eps, dtype, silu=True)
        elif spec.kind == "retention":
            self.mixer = DecayAttention(width, m["heads"], m["dim"], m["vdim"], m["decay"], eps, dtype, rot=m["rot"],
                                        scale=m["dim"] ** -0.5, norm_per_head=True, norm_weight=False, gate_silu=True)
        else:
            raise ValueError(f"no mixer of kind {spec.kind!r}")
        self.norm1 = ZeroCentredNorm(width)
        self.mlp = None
        if spec.ff is not None:
            self.mlp = GatedMLP(width, spec.ff, dtype, act="silu")
            self.norm2 = ZeroCentredNorm(width)


class VokelixForCausalLM(nn.Module):
    mixed_steps = True            # a step is a batch of portions (``PortionScheduler``, ``StepPlan``)

    # checkpoint names behind 'l<i>.' -> parameter of the block, shard
    _TARGETS = {
        "attention": {
            **{f"mix.{n}": ("mixer.in_proj.weight", n) for n in "qkvg"}, **{f"mix.{n}.b": ("mixer.bias.weight", n) for n in "qkv"},
            "mix.q.norm": ("mixer.q_norm", None), "mix.k.norm": ("mixer.k_norm", None), "mix.sink": ("mixer.sink", None),
            "mix.o": ("mixer.o_proj.weight", None),
        },
        "lightning": {
            **{f"mix.{n}": ("mixer.in_proj.weight", n) for n in "qkvg"}, "mix.norm": ("mixer.out_norm", None),
            "mix.o": ("mixer.o_proj.weight", None),
        },
        "retention": {
            **{f"mix.{n}": ("mixer.in_proj.weight", n) for n in "qkvg"}, "mix.o": ("mixer.o_proj.weight", None),
        },
    }
    _COMMON = {
        "norm1": ("norm1.weight", None), "norm2": ("norm2.weight", None),
        "mlp.gate": ("mlp.gate_up_proj.weight", 0), "mlp.up": ("mlp.gate_up_proj.weight", 1),
        "mlp.down": ("mlp.down_proj.weight", None),
    }

    def __init__(self, config):
        super().__init__()
        self.config = config
        dtype, width = config.torch_dtype, config.hidden_size
        self.embed_tokens = Embedding(config.vocab_size, width, dtype)
        self.blocks = nn.ModuleList([VokelixBlock(config, spec) for spec in config.layers])
        for i, spec in enumerate(config.layers):
            owner = spec.mixer.get("kv_from") if spec.kind == "attention" else None
            if owner is not None and not self._can_share(i, owner):
                raise ValueError(f"layer {i} cannot use the keys and values of layer {owner}")
        self.final_norm = ZeroCentredNorm(width)
        self.lm_head = Linear(width, config.vocab_size, dtype=dtype)
        self.caches: list = [None] * len(config.layers)

    def _can_share(self, i: int, owner: int) -> bool:
        if not 0 <= owner < i or self.config.layers[owner].kind != "attention":
            return False
        a, b = self.blocks[owner].mixer, self.blocks[i].mixer
        return a.own_keys and (a.kv_heads, a.dim, a.vdim) == (b.kv_heads, b.dim, b.vdim)

    @classmethod
    def build(cls, config, device) -> "VokelixForCausalLM":
        return cls(config).to(device)                 # parameters have their types already: norms stay float32

    # ------------------------------------------------------------------ weights
    def checkpoint_target(self, name: str) -> tuple[str, str | int | None]:
        whole = {"embed": "embed_tokens.weight", "head": "lm_head.weight", "final.norm": "final_norm.weight"}
        if name in whole:
            return whole[name], None
        layer, _, rest = name.partition(".")
        index = layer[1:]
        if layer[:1] != "l" or not index.isdecimal() or int(index) >= len(self.blocks):
            raise KeyError(f"checkpoint tensor {name} belongs to no layer of the model")
        target = self._TARGETS[self.config.layers[int(index)].kind].get(rest) or self._COMMON.get(rest)
        if target is None:
            raise KeyError(f"checkpoint tensor {name} has no place in its layer")
        return f"blocks.{int(index)}.{target[0]}", target[1]

    def init_random_weights(self, seed: int = 0) -> None:
        """Weights that keep activations of the order of one: the stand-in for a checkpoint."""
        gen = torch.Generator(device=self.lm_head.weight.device).manual_seed(seed)
        for name, p in self.named_parameters():
            if name.endswith(("q_norm", "k_norm", "out_norm")):
                p.data.fill_(1.0)
            elif name.endswith(("norm.weight", "norm1.weight", "norm2.weight", "bias.weight", "sink")):
                p.data.zero_()
            elif name.endswith("embed_tokens.weight"):
                p.data.normal_(0.0, 1.0, generator=gen)
            else:
                p.data.normal_(0.0, p.shape[-1] ** -0.5, generator=gen)

    def finish_loading(self, max_position: int) -> None:
        for block in self.blocks:
            block.mixer.finish_loading(max_position)
        for module in self.modules():
            if isinstance(module, ZeroCentredNorm):
                module.finish_loading()

    # ------------------------------------------------------------------ cache
    def cache_layout(self, block_size: int) -> LayeredLayout:
        owners = [s.mixer.get("kv_from") if s.kind == "attention" else None for s in self.config.layers]
        return LayeredLayout([b.mixer.cache_spec() if o is None else SharedStorage(o) for b, o in zip(self.blocks, owners)], block_size)

    def bind_cache(self, storage: list) -> None:
        assert len(storage) == len(self.caches)
        self.caches = storage

    def prepare_decode(self, device, max_batch: int) -> None:
        pass                                          # every workspace of a step comes from torch's allocator

    # ------------------------------------------------------------------ the step
    def forward(self, input_ids: torch.Tensor, positions: torch.Tensor) -> torch.Tensor:
        """Final hidden states of the step in ``get_context().step``."""
        cfg = self.config
        sublayers = []                                # (sublayer, norm behind its residual sum) in order
        for block, cache in zip(self.blocks, self.caches):
            sublayers.append((lambda h, m=block.mixer, c=cache: m(h, c), block.norm1))
            if block.mlp is not None:
                sublayers.append((block.mlp, block.norm2))
        x = torch.empty((input_ids.numel(), cfg.hidden_size), dtype=torch.float32, device=input_ids.device)
        common = dict(eps=cfg.norm_eps, dtype=cfg.torch_dtype)
        h = hybrid_ops.post_norm(x, tokens=input_ids, embed=self.embed_tokens.weight, **common)
        for i, (run, norm) in enumerate(sublayers):
            last = self.final_norm.gain if i + 1 == len(sublayers) else None
            h = hybrid_ops.post_norm(x, y=run(h), w_post=norm.gain, alpha=cfg.residual_alpha, w_last=last, **common)
        return h

    def compute_logits(self, hidden_states: torch.Tensor) -> torch.Tensor:
        return self.lm_head(hidden_states)
