"""Tulurax decoder: pre-norm layers of talking-heads attention beside retention, feed-forwards with a learned activation, a norm that
squashes instead of measuring, a float32 residual stream, logits that are scaled and capped.

The bias behind a sublayer, the residual sum and the norm in front of the next sublayer are one kernel."""
from __future__ import annotations

import torch
from torch import nn

from . import hybrid_ops
from .cache import LayeredLayout
from .decay_attention import DecayHeads
from .layers import DynamicTanh, Embedding, Linear, XieluMLP
from .mixer import Mixer
from .talking_attention import TalkingAttention


def _mixer(config, spec) -> Mixer:
    if spec.kind != "parallel":
        raise ValueError(f"no mixer of kind {spec.kind!r}")
    m, dtype, eps = spec.mixer, config.torch_dtype, config.norm_eps
    a, r = m["left"], m["right"]
    return Mixer(config.hidden_size, {
        "left": TalkingAttention(a["heads"], a["kv_heads"], a["dim"], a["vdim"], a["scale"], eps, dtype, temperature=a.get("q_temp"),
                                 out_scale=m["left_scale"]),
        "right": DecayHeads(r["heads"], r["dim"], r["vdim"], r["decay"], eps, dtype, scale=r["dim"] ** -0.5, norm_per_head=True,
                            norm_weight=False, gate_silu=True, out_scale=m["right_scale"])}, dtype)


class TuluraxBlock(nn.Module):
    """The weights of a layer."""

    def __init__(self, config, spec):
        super().__init__()
        width = config.hidden_size
        self.mixer, self.norm1, self.mlp = _mixer(config, spec), DynamicTanh(width), None
        if spec.ff is not None:
            self.mlp, self.norm2 = XieluMLP(width, spec.ff, config.torch_dtype), DynamicTanh(width)


class TuluraxForCausalLM(nn.Module):
    mixed_steps = True            # a step is a batch of portions (``PortionScheduler``, ``StepPlan``)

    _NORMS = {"": "weight", ".b": "bias", ".alpha": "alpha"}
    _MLP = {"up": "up_proj.weight", "up.b": "up_bias", "down": "down_proj.weight", "down.b": "down_bias", "act": "act"}

    def __init__(self, config):
        super().__init__()
        self.config = config
        dtype, width = config.torch_dtype, config.hidden_size
        self.embed_tokens = Embedding(config.vocab_size, width, dtype)
        self.embed_norm, self.final_norm = DynamicTanh(width), DynamicTanh(width)
        self.blocks = nn.ModuleList([TuluraxBlock(config, spec) for spec in config.layers])
        self.lm_head = Linear(width, config.vocab_size, dtype=dtype)
        self.caches: list = [None] * len(config.layers)

    @classmethod
    def build(cls, config, device) -> "TuluraxForCausalLM":
        return cls(config).to(device)                 # parameters have their types already: norms stay float32

    # ------------------------------------------------------------------ weights
    def checkpoint_target(self, name: str) -> tuple[str, str | None]:
        whole = {"embed": "embed_tokens.weight", "head": "lm_head.weight"}
        if name in whole:
            return whole[name], None
        norm = self._norm_target(name, {"embed.norm": "embed_norm", "final.norm": "final_norm"})
        if norm is not None:
            return norm, None
        layer, _, rest = name.partition(".")
        index = layer[1:]
        if layer[:1] != "l" or not index.isdecimal() or int(index) >= len(self.blocks):
            raise KeyError(f"checkpoint tensor {name} belongs to no layer of the model")
        block = self.blocks[int(index)]
        group, _, key = rest.partition(".")
        target = self._norm_target(rest, {"norm1": "norm1", "norm2": "norm2"} if block.mlp is not None else {"norm1": "norm1"}), None
        if group == "mix":
            target = self._mixer_target(block.mixer, *key.partition(".")[::2])
        elif group == "mlp" and block.mlp is not None and key in self._MLP:
            target = "mlp." + self._MLP[key], None
        if target[0] is None:
            raise KeyError(f"checkpoint tensor {name} has no place in its layer")
        return f"blocks.{int(index)}.{target[0]}", target[1]

    @classmethod
    def _norm_target(cls, name: str, norms: dict) -> str | None:
        for stored, module in norms.items():
            if name.startswith(stored) and name[len(stored):] in cls._NORMS:
                return f"{module}.{cls._NORMS[name[len(stored):]]}"
        return None

    @staticmethod
    def _mixer_target(mixer: Mixer, part: str, key: str) -> tuple[str | None, str | None]:
        if part not in mixer.parts:
            return None, None
        if key in mixer.parts[part].pieces():
            return "mixer.in_proj.weight", mixer.piece(part, key)
        if key == "o":
            return "mixer.o_proj.weight", part
        return ("mixer.parts.left.talk", None) if (part, key) == ("left", "talk") else (None, None)

    def init_random_weights(self, seed: int = 0) -> None:
        """Weights that keep activations of the order of one: the stand-in for a checkpoint."""
        gen = torch.Generator(device=self.lm_head.weight.device).manual_seed(seed)
        for name, p in self.named_parameters():
            leaf = name.rpartition(".")[2]
            if p.dim() < 2:
                p.data.fill_({"alpha": 0.5, "weight": 1.0}.get(leaf, 0.0))
            elif leaf == "talk":
                p.data.normal_(0.0, 0.3 * p.shape[-1] ** -0.5, generator=gen)
                p.data += torch.eye(len(p), dtype=p.dtype, device=p.device)
            elif name == "embed_tokens.weight":
                p.data.normal_(0.0, 1.0 / self.config.embedding_scale, generator=gen)
            else:
                p.data.normal_(0.0, p.shape[-1] ** -0.5, generator=gen)

    def finish_loading(self, max_position: int) -> None:
        for block in self.blocks:
            block.mixer.finish_loading(max_position)
        for module in self.modules():
            if isinstance(module, (DynamicTanh, XieluMLP)):
                module.finish_loading()

    # ------------------------------------------------------------------ cache
    def cache_layout(self, block_size: int) -> LayeredLayout:
        return LayeredLayout([block.mixer.cache_spec() for block in self.blocks], block_size)

    def bind_cache(self, storage: list) -> None:
        assert len(storage) == len(self.caches)
        self.caches = storage

    def prepare_decode(self, device, max_batch: int) -> None:
        pass                                          # every workspace of a step comes from torch's allocator

    # ------------------------------------------------------------------ the step
    def forward(self, input_ids: torch.Tensor, positions: torch.Tensor) -> torch.Tensor:
        """Final hidden states of the step in ``get_context().step``."""
        cfg = self.config
        sublayers, norms = [], []                     # (sublayer, bias behind it) in order; the norm in front of each, and the final one
        for block, cache in zip(self.blocks, self.caches):
            sublayers.append((lambda h, m=block.mixer, c=cache: m(h, c), None))
            norms.append(block.norm1.norm)
            if block.mlp is not None:
                sublayers.append((block.mlp, block.mlp.down_bias))
                norms.append(block.norm2.norm)
        norms.append(self.final_norm.norm)
        x = torch.empty((input_ids.numel(), cfg.hidden_size), dtype=torch.float32, device=input_ids.device)
        h = hybrid_ops.tanh_norm(x, norms[0], tokens=input_ids, embed=self.embed_tokens.weight, embed_scale=cfg.embedding_scale,
                                 embed_norm=self.embed_norm.norm, dtype=cfg.torch_dtype)
        for (run, bias), norm in zip(sublayers, norms[1:]):
            h = hybrid_ops.tanh_norm(x, norm, y=run(h), bias=bias, dtype=cfg.torch_dtype)
        return h

    def compute_logits(self, hidden_states: torch.Tensor) -> torch.Tensor:
        cfg, logits = self.config, self.lm_head(hidden_states)
        if cfg.logit_softcap:
            return hybrid_ops.softcap(logits, cfg.logit_softcap, cfg.logit_scale)
        return logits if cfg.logit_scale == 1.0 else logits.float() * cfg.logit_scale
