"""Typed model configurations read from config.json."""

from .base import ConfigError, ModelConfig, read_config_json
from .botulorn import BotulornConfig
from .fiterax import FiteraxConfig
from .gilozen import GilozenConfig
from .nenizen import NenizenConfig
from .qwen2 import Qwen2Config
from .romepel import RomepelConfig

__all__ = ["BotulornConfig", "ConfigError", "FiteraxConfig", "GilozenConfig", "ModelConfig", "NenizenConfig", "Qwen2Config",
           "RomepelConfig", "read_config_json"]
