"""Merilorn decoder: layers of latent attention and of gated delta rule in the order the configuration gives,
norms before and after every sublayer, a float32 residual stream.

A layer may use another layer's weights (``LayerSpec.owner``); every layer has a cache or state of its own.
The norm behind a sublayer, the residual sum and the norm in front of the next sublayer are one kernel."""
from __future__ import annotations

import torch
from torch import nn

from . import hybrid_ops
from .cache import LayeredLayout
from .delta_rule import ChannelDelta
from .latent_attention import LatentAttention
from .layers import Embedding, GatedMLP, Linear


def _norm_weight(width: int) -> nn.Parameter:
    return nn.Parameter(torch.ones(width), requires_grad=False)


class MerilornBlock(nn.Module):
    """The weights of a layer."""

    def __init__(self, config, spec):
        super().__init__()
        m, width, dtype = spec.mixer, config.hidden_size, config.torch_dtype
        if spec.kind == "latent_attention":
            self.mixer = LatentAttention(width, m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"], m["scale"], m["rot"],
                                         config.norm_eps, dtype)
        elif spec.kind == "channel_delta":
            self.mixer = ChannelDelta(width, m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"], m["decay_rank"],
                                      m["gate_rank"], config.norm_eps, dtype)
        else:
            raise ValueError(f"no mixer of kind {spec.kind!r}")
        self.norm1, self.norm1b = _norm_weight(width), _norm_weight(width)
        self.mlp = None
        if spec.ff is not None:
            self.mlp = GatedMLP(width, spec.ff, dtype)
            self.norm2, self.norm2b = _norm_weight(width), _norm_weight(width)


class MerilornForCausalLM(nn.Module):
    mixed_steps = True            # a step is a batch of portions (``PortionScheduler``, ``StepPlan``)

    # checkpoint names behind 'l<i>.' -> parameter of the block, shard
    _TARGETS = {
        "latent_attention": {
            "mix.q": ("mixer.in_proj.weight", "q"), "mix.dkv": ("mixer.in_proj.weight", "dkv"),
            "mix.g": ("mixer.in_proj.weight", "g"), "mix.dkv.norm": ("mixer.latent_norm", None),
            "mix.uk": ("mixer.k_up", None), "mix.uv": ("mixer.v_up", None), "mix.o": ("mixer.o_proj.weight", None),
        },
        "channel_delta": {
            "mix.q": ("mixer.in_proj.weight", "q"), "mix.k": ("mixer.in_proj.weight", "k"),
            "mix.v": ("mixer.in_proj.weight", "v"), "mix.b": ("mixer.in_proj.weight", "b"),
            "mix.a1": ("mixer.in_proj.weight", "a1"), "mix.g1": ("mixer.in_proj.weight", "g1"),
            "mix.q.conv": ("mixer.conv.weight", "q"), "mix.k.conv": ("mixer.conv.weight", "k"),
            "mix.v.conv": ("mixer.conv.weight", "v"), "mix.a2": ("mixer.decay_up.weight", None),
            "mix.g2": ("mixer.gate_up.weight", None), "mix.A_log": ("mixer.a_log", None),
            "mix.dt_bias": ("mixer.dt_bias", None), "mix.norm": ("mixer.out_norm", None),
            "mix.o": ("mixer.o_proj.weight", None),
        },
    }
    _COMMON = {
        "norm1": ("norm1", None), "norm1b": ("norm1b", None), "norm2": ("norm2", None), "norm2b": ("norm2b", None),
        "mlp.gate": ("mlp.gate_up_proj.weight", 0), "mlp.up": ("mlp.gate_up_proj.weight", 1),
        "mlp.down": ("mlp.down_proj.weight", None),
    }

    def __init__(self, config):
        super().__init__()
        self.config = config
        dtype, width = config.torch_dtype, config.hidden_size
        self.embed_tokens = Embedding(config.vocab_size, width, dtype)
        self.blocks = nn.ModuleDict()
        for i, spec in enumerate(config.layers):
            if spec.owner == i:
                self.blocks[str(i)] = MerilornBlock(config, spec)
        for i, spec in enumerate(config.layers):
            owner = config.layers[spec.owner]
            if owner.owner != spec.owner or owner.kind != spec.kind:
                raise ValueError(f"layer {i} cannot use the weights of layer {spec.owner}")
        self.final_norm = _norm_weight(width)
        self.lm_head = Linear(width, config.vocab_size, dtype=dtype)
        self.caches: list = [None] * len(config.layers)

    @classmethod
    def build(cls, config, device) -> "MerilornForCausalLM":
        return cls(config).to(device)                 # parameters have their types already: norms stay float32

    # ------------------------------------------------------------------ weights
    def checkpoint_target(self, name: str) -> tuple[str, str | int | None]:
        whole = {"embed": "embed_tokens.weight", "head": "lm_head.weight", "final.norm": "final_norm"}
        if name in whole:
            return whole[name], None
        layer, _, rest = name.partition(".")
        index = layer[1:]
        if layer[:1] != "l" or index not in self.blocks:
            raise KeyError(f"checkpoint tensor {name} belongs to no layer of the model")
        table = self._TARGETS[self.config.layers[int(index)].kind]
        target = table.get(rest) or self._COMMON.get(rest)
        if target is None:
            raise KeyError(f"checkpoint tensor {name} has no place in its layer")
        return f"blocks.{index}.{target[0]}", target[1]

    def init_random_weights(self, seed: int = 0) -> None:
        """Weights that keep activations of the order of one: the stand-in for a checkpoint."""
        gen = torch.Generator(device=self.final_norm.device).manual_seed(seed)
        for name, p in self.named_parameters():
            if name.endswith(("norm", "norm1", "norm1b", "norm2", "norm2b")):
                p.data.fill_(1.0)
            elif name.endswith(("a_log", "dt_bias")):
                p.data.uniform_(-2.0, 1.0, generator=gen)
            elif name.endswith("embed_tokens.weight"):
                p.data.normal_(0.0, 1.0 / self.config.embedding_scale, generator=gen)
            else:
                p.data.normal_(0.0, p.shape[-1] ** -0.5, generator=gen)

    def finish_loading(self, max_position: int) -> None:
        for block in self.blocks.values():
            block.mixer.finish_loading(max_position)

    # ------------------------------------------------------------------ cache
    def cache_layout(self, block_size: int) -> LayeredLayout:
        return LayeredLayout([self.blocks[str(s.owner)].mixer.cache_spec() for s in self.config.layers], block_size)

    def bind_cache(self, storage: list) -> None:
        assert len(storage) == len(self.caches)
        self.caches = storage

    def prepare_decode(self, device, max_batch: int) -> None:
        pass                                          # every workspace of a step comes from torch's allocator

    # ------------------------------------------------------------------ the step
    def forward(self, input_ids: torch.Tensor, positions: torch.Tensor) -> torch.Tensor:
        """Final hidden states of the step in ``get_context().step``."""
        cfg = self.config
        dtype, eps = cfg.torch_dtype, cfg.norm_eps
        # (sublayer, norm in front of it, norm behind it) in order
        sublayers = []
        for spec, cache in zip(cfg.layers, self.caches):
            block = self.blocks[str(spec.owner)]
            sublayers.append((lambda h, m=block.mixer, c=cache: m(h, c), block.norm1, block.norm1b))
            if block.mlp is not None:
                sublayers.append((block.mlp, block.norm2, block.norm2b))
        before = [pre for _, pre, _ in sublayers] + [self.final_norm]
        x = torch.empty((input_ids.numel(), cfg.hidden_size), dtype=torch.float32, device=input_ids.device)
        h = hybrid_ops.residual_norm(x, eps, tokens=input_ids, embed=self.embed_tokens.weight,
                                     embed_scale=cfg.embedding_scale, w_pre=before[0], dtype=dtype)
        for (run, _, post), pre in zip(sublayers, before[1:]):
            h = hybrid_ops.residual_norm(x, eps, y=run(h), w_post=post, w_pre=pre, dtype=dtype)
        return h

    def compute_logits(self, hidden_states: torch.Tensor) -> torch.Tensor:
        return self.lm_head(hidden_states)
