"""Configuration class -> model class."""
from ..config import GigopelConfig, GitopelConfig, ModelConfig
from .gigopel import GigopelForCausalLM
from .gitopel import GitopelForCausalLM
from .qwen3 import Qwen3ForCausalLM

MODELS = {ModelConfig: Qwen3ForCausalLM, GitopelConfig: GitopelForCausalLM, GigopelConfig: GigopelForCausalLM}


def model_class(config):
    return MODELS[type(config)]
