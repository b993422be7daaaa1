from .llama import ConfigError, LlamaConfig, RopeScaling
from .registry import (config_from_dict, config_from_folder, register_architecture, registered_architectures,
                       unregister_architecture)
from .bovozen import BovozenConfig
from .gedunex import GedunexConfig
from .gemepel import GemepelConfig
from .rekirax import RekiraxConfig
from .situlorn import SitulornConfig
from .spec import LayerSpec, ModelSpec, PartSpec, ScheduleEntry
from .zebivik import ZebivikConfig

__all__ = ["BovozenConfig", "ConfigError", "GedunexConfig", "GemepelConfig", "LlamaConfig", "RekiraxConfig", "RopeScaling", "SitulornConfig", "ZebivikConfig", "config_from_dict", "config_from_folder",
           "register_architecture", "registered_architectures", "unregister_architecture", "LayerSpec", "ModelSpec",
           "PartSpec", "ScheduleEntry"]
