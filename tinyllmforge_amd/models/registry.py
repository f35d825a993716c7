"""Configuration class -> model class."""
from ..config import GigopelConfig, GitopelConfig, ModelConfig, ZuzunexConfig
from .gigopel import GigopelForCausalLM
from .gitopel import GitopelForCausalLM
from .qwen3 import Qwen3ForCausalLM
from .zuzunex import ZuzunexForCausalLM

MODELS = {ModelConfig: Qwen3ForCausalLM, GitopelConfig: GitopelForCausalLM, GigopelConfig: GigopelForCausalLM,
          ZuzunexConfig: ZuzunexForCausalLM}


def model_class(config):
    return MODELS[type(config)]
