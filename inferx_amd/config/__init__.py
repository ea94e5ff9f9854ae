"""Typed configurations and the architecture registry."""
from .registry import (ConfigError, config_class_for, config_from_dict, config_from_directory,
                       config_from_json, known_architectures, register_architecture)
from .spec import LayerSpec, ModelSpec, PartSpec, ScheduleEntry, linear_head, token_embedding
from . import qwen2_moe  # registers Qwen2MoeForCausalLM
from .qwen2_moe import Qwen2MoeConfig
from . import pelalix  # registers Pelalix
from .pelalix import PelalixConfig
from . import dezudra  # registers Dezudra
from .dezudra import DezudraConfig
from . import bibevik  # registers Bibevik
from .bibevik import BibevikConfig
from . import gosuvik  # registers Gosuvik
from .gosuvik import GosuvikConfig
from . import setopel  # registers Setopel
from .setopel import SetopelConfig
from . import zevivik  # registers Zevivik
from .zevivik import ZevivikConfig

__all__ = [
    "ConfigError", "config_class_for", "config_from_dict", "config_from_directory", "config_from_json",
    "known_architectures", "register_architecture", "LayerSpec", "ModelSpec", "PartSpec", "ScheduleEntry", "linear_head", "token_embedding",
    "Qwen2MoeConfig", "PelalixConfig", "DezudraConfig", "BibevikConfig", "GosuvikConfig", "SetopelConfig", "ZevivikConfig",
]
