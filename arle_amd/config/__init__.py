from .base import ConfigError
from .gufasun import GufasunConfig
from .nafezen import NafezenConfig
from .pozirax import PoziraxConfig
from .qwen3 import Qwen3Config
from .retudra import RetudraConfig
from .sovutar import SovutarConfig
from .tazitar import TazitarConfig
from .registry import (Architecture, detect_architecture, known_architectures, load_model_config,
                       register_architecture)

__all__ = ["ConfigError", "Qwen3Config", "GufasunConfig", "SovutarConfig", "TazitarConfig", "RetudraConfig", "NafezenConfig",
           "PoziraxConfig", "Architecture", "detect_architecture", "known_architectures", "load_model_config",
           "register_architecture"]
