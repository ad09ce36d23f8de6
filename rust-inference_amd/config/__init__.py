from .base import ModelConfig, read_config_json
from .qwen3 import Qwen3Config
from .zidepel import ZidepelConfig
from .pisulorn import PisulornConfig
from .zakelorn import ZakelornConfig
from .dagezen import DagezenConfig
from .notadra import NotadraConfig
from .kisepel import KisepelConfig
from .registry import (Architecture, config_from_dict, known_architectures, load_config,
                       register_architecture, resolve_architecture)

__all__ = ["ModelConfig", "Qwen3Config", "ZidepelConfig", "PisulornConfig", "ZakelornConfig", "DagezenConfig", "NotadraConfig", "KisepelConfig", "Architecture", "read_config_json", "config_from_dict",
           "known_architectures", "load_config", "register_architecture", "resolve_architecture"]
