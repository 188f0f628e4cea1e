"""Architectures this engine knows. Importing the package registers them."""
from ..config.registry import register_architecture
from .lalepel import LalepelConfig
from .ludelorn import LudelornConfig
from .nodopel import NodopelConfig
from .qwen2 import Qwen2Config
from .rerupel import RerupelConfig
from .retotar import RetotarConfig
from .tugalix import TugalixConfig

register_architecture(Qwen2Config.architecture, Qwen2Config)
register_architecture(TugalixConfig.architecture, TugalixConfig)
register_architecture(RerupelConfig.architecture, RerupelConfig)
register_architecture(RetotarConfig.architecture, RetotarConfig)
register_architecture(LudelornConfig.architecture, LudelornConfig)
register_architecture(LalepelConfig.architecture, LalepelConfig)
register_architecture(NodopelConfig.architecture, NodopelConfig)

__all__ = ["LalepelConfig", "LudelornConfig", "NodopelConfig", "Qwen2Config", "RerupelConfig", "RetotarConfig", "TugalixConfig"]
