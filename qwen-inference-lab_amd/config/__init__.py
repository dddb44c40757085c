"""Typed configurations.  One class per architecture; ``registry`` maps names to them."""
from .base import ConfigError, read_config_json
from .qwen3 import Qwen3Config
from .fubapel import FubapelConfig
from .gerivik import GerivikConfig
from .zinesun import ZinesunConfig
from .dogozen import DogozenConfig
from .tinuzen import TinuzenConfig
from .kebudra import KebudraConfig

__all__ = ['ConfigError', 'read_config_json', 'Qwen3Config', 'FubapelConfig', 'GerivikConfig', 'ZinesunConfig', 'DogozenConfig',
           'TinuzenConfig', 'KebudraConfig']
