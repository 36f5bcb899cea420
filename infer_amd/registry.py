"""Which model class serves which configuration."""
from __future__ import annotations

from .config import DogetarConfig, MerilornConfig, ModelConfig, TuluraxConfig, VokelixConfig
from .dogetar import DogetarForCausalLM
from .merilorn import MerilornForCausalLM
from .qwen3 import QwenForCausalLM
from .tulurax import TuluraxForCausalLM
from .vokelix import VokelixForCausalLM

MODELS = {ModelConfig: QwenForCausalLM, MerilornConfig: MerilornForCausalLM, VokelixConfig: VokelixForCausalLM,
          DogetarConfig: DogetarForCausalLM, TuluraxConfig: TuluraxForCausalLM}


def model_class(config):
    """The model class of a configuration (any object with Qwen3's attributes counts as Qwen3's)."""
    return MODELS.get(type(config), QwenForCausalLM)
