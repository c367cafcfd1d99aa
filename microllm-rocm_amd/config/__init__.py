from .fields import ConfigError
from .gupitar import GupitarConfig
from .kalevik import KalevikConfig
from .mapedra import MapedraConfig
from .qwen2 import Qwen2Config
from .siditar import SiditarConfig
from .zabozen import ZabozenConfig
from .zuluvik import ZuluvikConfig
from .registry import (Architecture, architecture_named, architecture_of, load_config,
                       register_architecture, registered_architectures, unregister_architecture)

__all__ = ["ConfigError", "GupitarConfig", "KalevikConfig", "MapedraConfig", "Qwen2Config", "SiditarConfig", "ZabozenConfig", "ZuluvikConfig", "Architecture", "architecture_named", "architecture_of",
           "load_config", "register_architecture", "registered_architectures", "unregister_architecture"]
