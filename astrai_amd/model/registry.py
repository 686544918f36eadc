"""Which classes a model directory's config.json stands for.

``config.json`` names its design under ``architecture``; a file without that key is the dense
decoder, whose checkpoints never had one.
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import Callable, Dict

from astrai_amd.model.decoder import AutoRegressiveLM, AutoRegressiveLMConfig
from astrai_amd.model.lugitar import LugitarConfig, LugitarLM

DEFAULT_ARCHITECTURE = "AutoRegressiveLM"


@dataclass(frozen=True)
class Architecture:
    make_config: Callable[[dict], object]   # the parsed config.json -> configuration
    model_class: type


_ARCHITECTURES: Dict[str, Architecture] = {}


def register_architecture(name: str, make_config: Callable[[dict], object], model_class: type) -> None:
    _ARCHITECTURES[name] = Architecture(make_config, model_class)


def architectures():
    return sorted(_ARCHITECTURES)


def architecture_of(config: dict) -> Architecture:
    name = config.get("architecture", DEFAULT_ARCHITECTURE)
    if name not in _ARCHITECTURES:
        raise ValueError(f"unknown architecture {name!r} (known: {', '.join(architectures())})")
    return _ARCHITECTURES[name]


register_architecture(
    DEFAULT_ARCHITECTURE,
    lambda d: AutoRegressiveLMConfig(**{k: v for k, v in d.items() if k != "architecture"}), AutoRegressiveLM)
register_architecture("Lugitar", LugitarConfig.from_dict, LugitarLM)
