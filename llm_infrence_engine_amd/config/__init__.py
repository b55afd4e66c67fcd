from .engine_config import EngineConfig
from .registry import (ConfigError, build_spec, config_class, config_from_dict, known_architectures,
                       load_config, register_architecture)
from .spec import LayerSpec, ModelSpec, PartSpec, Run, layer
from .qwen2 import Qwen2Config
from .gemadra import GemadraConfig
from .gidurax import GiduraxConfig
from .kuvazen import KuvazenConfig
from .silizen import SilizenConfig
from .gositar import GositarConfig
from .kisusun import KisusunConfig
from .presets import PRESETS, preset

__all__ = ["EngineConfig", "ConfigError", "build_spec", "config_class", "config_from_dict",
           "known_architectures", "load_config", "register_architecture", "LayerSpec", "ModelSpec",
           "PartSpec", "Run", "layer", "Qwen2Config", "GemadraConfig", "GiduraxConfig", "KuvazenConfig", "SilizenConfig", "GositarConfig",
           "KisusunConfig", "PRESETS", "preset"]
