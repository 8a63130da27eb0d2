from .base import ConfigError, KeyReader, read_json
from .bubetar import BubetarConfig
from .karesun import KaresunConfig
from .kezolix import KezolixConfig
from .nebanex import NebanexConfig
from .pekasun import PekasunConfig
from .qwen2 import Qwen2Config
from .tipezen import TipezenConfig
from .registry import (
    Architecture,
    UnknownArchitectureError,
    load_model_config,
    register_architecture,
    registered_architectures,
    resolve_architecture,
    unregister_architecture,
)

__all__ = [
    "Architecture",
    "BubetarConfig",
    "ConfigError",
    "KeyReader",
    "KaresunConfig",
    "KezolixConfig",
    "NebanexConfig",
    "PekasunConfig",
    "Qwen2Config",
    "TipezenConfig",
    "UnknownArchitectureError",
    "load_model_config",
    "read_json",
    "register_architecture",
    "registered_architectures",
    "resolve_architecture",
    "unregister_architecture",
]
