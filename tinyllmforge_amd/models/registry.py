"""Configuration class -> model class."""
from ..config import GigopelConfig, GitopelConfig, ModelConfig, TibenexConfig, ZuzunexConfig
from .gigopel import GigopelForCausalLM
from .gitopel import GitopelForCausalLM
from .qwen3 import Qwen3ForCausalLM
from .tibenex import TibenexForCausalLM
from .zuzunex import ZuzunexForCausalLM

MODELS = {ModelConfig: Qwen3ForCausalLM, GitopelConfig: GitopelForCausalLM, GigopelConfig: GigopelForCausalLM,
          ZuzunexConfig: ZuzunexForCausalLM, TibenexConfig: TibenexForCausalLM}


def model_class(config):
    return MODELS[type(config)]
