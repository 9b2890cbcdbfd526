from .layout import LayerSpec, ModelLayout, PartSpec, RunEntry
from .model_args import ConfigError, ModelArgs, RopeArgs, architecture_name, read_config_json
from .registry import (
    Architecture,
    get_architecture,
    register_architecture,
    registered_architectures,
    unregister_architecture,
)
from . import llama as _llama  # registers LlamaForCausalLM
from . import buderax as _buderax  # registers Buderax
from . import gisodra as _gisodra  # registers Gisodra
from . import zudisun as _zudisun  # registers Zudisun
from . import sodotar as _sodotar  # registers Sodotar
from . import ropelix as _ropelix  # registers Ropelix
from . import poselorn as _poselorn  # registers Poselorn

__all__ = [
    "Architecture",
    "ConfigError",
    "LayerSpec",
    "ModelArgs",
    "ModelLayout",
    "PartSpec",
    "RopeArgs",
    "RunEntry",
    "architecture_name",
    "get_architecture",
    "read_config_json",
    "register_architecture",
    "registered_architectures",
    "unregister_architecture",
]
