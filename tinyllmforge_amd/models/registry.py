"""Configuration class -> model class."""
from ..config import GitopelConfig, ModelConfig
from .gitopel import GitopelForCausalLM
from .qwen3 import Qwen3ForCausalLM

MODELS = {ModelConfig: Qwen3ForCausalLM, GitopelConfig: GitopelForCausalLM}


def model_class(config):
    return MODELS[type(config)]
