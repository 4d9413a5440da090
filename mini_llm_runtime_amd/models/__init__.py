"""Architectures: each module registers one name with its configuration and builder."""

from . import bubitar, fedolorn, goguzen, pepulix, qwen2, rofetar, vobisun  # noqa: F401  (each registers its architecture)
from .registry import (
    ARCHITECTURES,
    Architecture,
    architecture_of,
    build_model,
    build_spec,
    config_from_dict,
    load_config,
    register_architecture,
    unregister_architecture,
)

__all__ = [
    "ARCHITECTURES",
    "Architecture",
    "architecture_of",
    "build_model",
    "build_spec",
    "config_from_dict",
    "load_config",
    "register_architecture",
    "unregister_architecture",
]
