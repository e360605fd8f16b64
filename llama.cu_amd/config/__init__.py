"""Typed configurations, read from a model folder's config.json, and the registry
that maps an architecture's name to its configuration class and its model."""
from .base import ConfigError, read_config_json
from .llama import LlamaConfig
from .divasun import DivasunConfig
from .lozezen import LozezenConfig
from .ralepel import RalepelConfig
from .mufotar import MufotarConfig
from .gefudra import GefudraConfig
from .lapunex import LapunexConfig
from .registry import (Architecture, architecture_of, register_architecture, registered_architectures, load_config,
                       load_plugins, load_plugins_from_env, PLUGINS_ENV)

__all__ = ["ConfigError", "read_config_json", "LlamaConfig", "DivasunConfig", "LozezenConfig", "RalepelConfig", "MufotarConfig", "GefudraConfig", "LapunexConfig", "Architecture", "architecture_of",
           "register_architecture", "registered_architectures", "load_config", "load_plugins", "load_plugins_from_env",
           "PLUGINS_ENV"]
