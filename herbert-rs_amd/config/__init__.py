"""Typed configurations and the architecture registry."""
from .base import read_config_json
from .registry import (Architecture, ChatFormat, load_config, register_architecture,
                       registered_architectures, resolve_architecture)
from .qwen3 import Qwen3Config
from .vipalorn import VipalornConfig
from .modasun import ModasunConfig
from .mefatar import MefatarConfig
from .bozasun import BozasunConfig
from .mutedra import MutedraConfig
from .figalorn import FigalornConfig

__all__ = ["Architecture", "BozasunConfig", "ChatFormat", "FigalornConfig", "MefatarConfig", "ModasunConfig", "MutedraConfig", "Qwen3Config", "VipalornConfig", "load_config", "read_config_json",
           "register_architecture", "registered_architectures", "resolve_architecture"]
