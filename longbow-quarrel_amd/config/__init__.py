"""Typed configurations read from a model folder's config.json."""
from .base import ConfigError, ModelConfig, read_config_json
from .llama import LlamaConfig, RopeScaling
from .mifidra import MifidraConfig
from .puzonex import PuzonexConfig
from .sofinex import SofinexConfig
from .tukedra import TukedraConfig
from .vafodra import VafodraConfig
from .vupelorn import VupelornConfig

__all__ = ["ConfigError", "ModelConfig", "read_config_json", "LlamaConfig", "MifidraConfig", "PuzonexConfig", "RopeScaling", "SofinexConfig", "TukedraConfig", "VafodraConfig", "VupelornConfig"]
