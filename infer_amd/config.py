"""Engine configuration (mirror of ``infer/config.py:5-27``) and the model configurations behind it.

The reference reads the model geometry with ``transformers.AutoConfig`` from a checkpoint
directory.  Here ``hf_config`` may also be handed in directly (a ``ModelConfig`` or any object with
the same attributes), which is how a random-initialised model of a published shape is built where
no checkpoint exists; with a directory, its ``config.json`` is parsed."""
from __future__ import annotations

import json
import os
import struct
from dataclasses import dataclass, field

import torch


@dataclass
class ModelConfig:
    """The attributes of a Qwen3 ``config.json`` that the engine reads."""
    vocab_size: int = 151936
    hidden_size: int = 4096
    intermediate_size: int = 12288
    num_hidden_layers: int = 36
    num_attention_heads: int = 32
    num_key_value_heads: int = 8
    head_dim: int = 128
    max_position_embeddings: int = 40960
    rms_norm_eps: float = 1e-6
    rope_theta: float = 1e6
    tie_word_embeddings: bool = False
    torch_dtype: torch.dtype = torch.bfloat16

    block_multiple = 256          # the paged K/V kernels take blocks of a multiple of this many tokens
    dtypes = (torch.bfloat16,)

    @classmethod
    def from_json(cls, path: str) -> "ModelConfig":
        with open(path) as f:
            raw = json.load(f)
        known = {k: raw[k] for k in cls.__dataclass_fields__ if k in raw and k != "torch_dtype"}
        cfg = cls(**known)
        if "head_dim" not in raw:
            cfg.head_dim = cfg.hidden_size // cfg.num_attention_heads
        dtype = raw.get("torch_dtype", raw.get("dtype", "bfloat16"))
        cfg.torch_dtype = getattr(torch, dtype) if isinstance(dtype, str) else dtype
        return cfg


def qwen3_8b() -> ModelConfig:
    return ModelConfig()


def qwen3_0_6b() -> ModelConfig:
    return ModelConfig(hidden_size=1024, intermediate_size=3072, num_hidden_layers=28, num_attention_heads=16,
                       num_key_value_heads=8, tie_word_embeddings=True)


def qwen3_32b() -> ModelConfig:
    return ModelConfig(hidden_size=5120, intermediate_size=25600, num_hidden_layers=64, num_attention_heads=64,
                       num_key_value_heads=8)


def checkpoint_shapes(directory: str) -> dict[str, tuple[int, ...]]:
    """Tensor shapes of the ``*.safetensors`` files of a directory, from their headers alone."""
    shapes = {}
    for name in sorted(os.listdir(directory)):
        if not name.endswith(".safetensors"):
            continue
        with open(os.path.join(directory, name), "rb") as f:
            (length,) = struct.unpack("<Q", f.read(8))
            header = json.loads(f.read(length))
        shapes.update({k: tuple(v["shape"]) for k, v in header.items() if k != "__metadata__"})
    return shapes


@dataclass
class LayerSpec:
    """One layer of a model whose layers differ: the kind of its mixer, the mixer's sizes and constants, the
    width of its feed-forward (None: it has none) and the layer whose weights it uses (its own index unless
    weights are shared).  ``mlp`` is the whole description of a feed-forward that is more than a width."""
    kind: str
    mixer: dict
    ff: int | None
    owner: int
    mlp: dict | None = None


def dense_width(entry: dict, index: int) -> int | None:
    """The width of a layer's dense feed-forward, None if it has none."""
    mlp = entry.get("mlp")
    if mlp is None:
        return None
    if mlp["kind"] != "dense":
        raise ValueError(f"layer {index}: feed-forward kind {mlp['kind']!r} is not known")
    return mlp["ff"]


@dataclass
class MerilornConfig:
    """Merilorn: ``layers`` in order, each latent attention or a gated delta rule, norms on both sides of every
    sublayer.  The ranks of the low-rank projections of a delta layer (``decay_rank``, ``gate_rank`` of its mixer)
    are not in ``config.json``; they are read off the checkpoint's tensors."""
    vocab_size: int
    hidden_size: int
    layers: list[LayerSpec] = field(default_factory=list)
    norm_eps: float = 1e-6
    embedding_scale: float = 1.0
    max_position_embeddings: int = 1 << 20          # the design sets no bound; ``max_model_len`` does
    torch_dtype: torch.dtype = torch.bfloat16

    block_multiple = 32
    dtypes = (torch.bfloat16, torch.float32)

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)

    @classmethod
    def from_json(cls, path: str) -> "MerilornConfig":
        with open(path) as f:
            raw = json.load(f)
        shapes = checkpoint_shapes(os.path.dirname(os.path.abspath(path)))
        layers = []
        for i, entry in enumerate(raw["layers"]):
            owner = entry.get("weights_of", i)
            owner = i if owner is None else int(owner)
            mixer = dict(entry["mixer"])
            if entry["type"] == "channel_delta":
                for key, tensor in (("decay_rank", "a1"), ("gate_rank", "g1")):
                    name = f"l{owner}.mix.{tensor}"
                    if name in shapes:
                        mixer[key] = shapes[name][0]
            layers.append(LayerSpec(entry["type"], mixer, dense_width(entry, i), owner))
        return cls(vocab_size=raw["vocab"], hidden_size=raw["width"], layers=layers, norm_eps=raw["norm"]["eps"],
                   embedding_scale=raw["embedding"]["scale"])


@dataclass
class VokelixConfig:
    """Vokelix: ``layers`` in order, each grouped attention, lightning or retention, and a norm behind every residual sum
    ``residual_alpha * x + sublayer(x)``.  The mixer of an attention layer with ``kv_from`` reads the keys and values of
    that earlier layer."""
    vocab_size: int
    hidden_size: int
    layers: list[LayerSpec] = field(default_factory=list)
    norm_eps: float = 1e-6
    residual_alpha: float = 1.0
    max_position_embeddings: int = 1 << 20          # the design sets no bound; ``max_model_len`` does
    torch_dtype: torch.dtype = torch.bfloat16

    block_multiple = 32
    dtypes = (torch.bfloat16, torch.float32)

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)

    @classmethod
    def from_json(cls, path: str) -> "VokelixConfig":
        with open(path) as f:
            raw = json.load(f)
        layers = [LayerSpec(e["type"], dict(e["mixer"]), dense_width(e, i), i) for i, e in enumerate(raw["layers"])]
        return cls(vocab_size=raw["vocab"], hidden_size=raw["width"], layers=layers, norm_eps=raw["norm"]["eps"],
                   residual_alpha=raw["postln_alpha"])


@dataclass
class LayerLoop:
    """Layers ``start`` .. ``stop - 1`` run ``times`` times in a row with the same weights."""
    start: int
    stop: int
    times: int


@dataclass
class DogetarConfig:
    """Dogetar: ``layers`` in order, each masked attention or masked attention beside a state space, with a dense feed-forward, a
    mixture of experts or none; ``loop`` repeats some of them.  ``bigram`` (``mul_prev``, ``mul_cur``, ``buckets``) adds a second
    embedding."""
    vocab_size: int
    hidden_size: int
    layers: list[LayerSpec] = field(default_factory=list)
    norm_eps: float = 1e-6
    bigram: dict | None = None
    loop: LayerLoop | None = None
    logit_softcap: float | None = None
    max_position_embeddings: int = 1 << 20          # the design sets no bound; ``max_model_len`` does
    torch_dtype: torch.dtype = torch.bfloat16

    block_multiple = 32
    dtypes = (torch.bfloat16, torch.float32)

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)

    def runs(self) -> list[tuple[int, int | None]]:
        """(layer, number of the pass or None) in the order of execution."""
        n = len(self.layers)
        if self.loop is None:
            return [(i, None) for i in range(n)]
        a, b = self.loop.start, self.loop.stop
        if not (0 <= a < b <= n and self.loop.times >= 1):
            raise ValueError(f"layers {a} .. {b - 1} of {n} cannot run {self.loop.times} times")
        return [(i, None) for i in range(a)] + [(i, t) for t in range(self.loop.times) for i in range(a, b)] + [(i, None) for i in range(b, n)]

    @classmethod
    def from_json(cls, path: str) -> "DogetarConfig":
        with open(path) as f:
            raw = json.load(f)
        layers = []
        for i, e in enumerate(raw["layers"]):
            mlp = e.get("mlp")
            if mlp is not None and mlp["kind"] not in ("dense", "moe"):
                raise ValueError(f"layer {i}: feed-forward kind {mlp['kind']!r} is not known")
            layers.append(LayerSpec(e["type"], dict(e["mixer"]), mlp["ff"] if mlp is not None and mlp["kind"] == "dense" else None, i, mlp))
        loop = raw.get("loop")
        return cls(vocab_size=raw["vocab"], hidden_size=raw["width"], layers=layers, norm_eps=raw["norm"]["eps"],
                   bigram=(raw.get("embedding") or {}).get("bigram"),
                   loop=LayerLoop(loop["start"], loop["stop"], loop["times"]) if loop else None, logit_softcap=raw.get("logit_softcap"))


@dataclass
class TuluraxConfig:
    """Tulurax: ``layers`` in order, each talking-heads attention beside retention, with a dense feed-forward or none."""
    vocab_size: int
    hidden_size: int
    layers: list[LayerSpec] = field(default_factory=list)
    norm_eps: float = 1e-6
    embedding_scale: float = 1.0
    logit_scale: float = 1.0
    logit_softcap: float | None = None
    max_position_embeddings: int = 1 << 20          # the design sets no bound; ``max_model_len`` does
    torch_dtype: torch.dtype = torch.bfloat16

    block_multiple = 32
    dtypes = (torch.bfloat16, torch.float32)

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)

    @classmethod
    def from_json(cls, path: str) -> "TuluraxConfig":
        with open(path) as f:
            raw = json.load(f)
        layers = [LayerSpec(e["type"], dict(e["mixer"]), dense_width(e, i), i) for i, e in enumerate(raw["layers"])]
        return cls(vocab_size=raw["vocab"], hidden_size=raw["width"], layers=layers, norm_eps=raw["norm"]["eps"],
                   embedding_scale=raw["embedding"]["scale"], logit_scale=raw["logit_scale"], logit_softcap=raw.get("logit_softcap"))


def load_model_config(directory: str):
    """The configuration of the model in a directory, of the class its ``config.json`` names (``architecture``, or the
    ``architectures`` list of the transformers layout; without either it is read as Qwen3)."""
    path = os.path.join(directory, "config.json")
    with open(path) as f:
        raw = json.load(f)
    names = [raw["architecture"]] if "architecture" in raw else raw.get("architectures") or ["Qwen3ForCausalLM"]
    for name in names:
        if name in CONFIG_CLASSES:
            return CONFIG_CLASSES[name].from_json(path)
    raise ValueError(f"no model of this package serves {names}; known: {sorted(CONFIG_CLASSES)}")


CONFIG_CLASSES = {"Qwen3ForCausalLM": ModelConfig, "Merilorn": MerilornConfig, "Vokelix": VokelixConfig,
                  "Dogetar": DogetarConfig, "Tulurax": TuluraxConfig}


@dataclass
class Config:
    model: str = ""
    max_num_batched_tokens: int = 16384
    max_num_seqs: int = 512
    max_model_len: int = 4096
    gpu_memory_utilization: float = 0.9
    tensor_parallel_size: int = 1
    enforce_eager: bool = False
    hf_config: ModelConfig | MerilornConfig | VokelixConfig | DogetarConfig | TuluraxConfig | None = None
    eos: int = -1
    kvcache_block_size: int = 256
    num_kvcache_blocks: int = -1
    # Decode tokens are fed position len(seq) by the reference (``model_runner.py:117``) while its
    # prefill positions are zero-based (``:84``); 1 reproduces that, 0 makes both zero-based.
    # (Models that run portions of prompts beside decoded tokens have one position per token, zero-based.)
    decode_position_offset: int = 1
    seed: int = 0
    dtype: str | None = None      # element type of weights and activations; None: the model's

    def __post_init__(self):
        if self.hf_config is None:
            assert os.path.isdir(self.model)
            self.hf_config = load_model_config(self.model)
        if self.dtype is not None:
            self.hf_config.torch_dtype = getattr(torch, self.dtype)
        if self.hf_config.torch_dtype not in self.hf_config.dtypes:
            raise ValueError(f"{type(self.hf_config).__name__} does not run in {self.hf_config.torch_dtype}")
        assert self.kvcache_block_size > 0 and self.kvcache_block_size % self.hf_config.block_multiple == 0
        assert 1 <= self.tensor_parallel_size <= 8
        self.max_model_len = min(self.max_model_len, self.hf_config.max_position_embeddings)
        assert self.max_num_batched_tokens >= self.max_model_len
