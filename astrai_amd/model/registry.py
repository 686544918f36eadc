"""Which classes a model directory's config.json stands for.

``config.json`` names its design under ``architecture``; a file without that key is the dense
decoder, whose checkpoints never had one.
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import Callable, Dict, Optional

from astrai_amd.model.decoder import AutoRegressiveLM, AutoRegressiveLMConfig
from astrai_amd.model.lugitar import LugitarConfig, LugitarLM
from astrai_amd.model.sarulix import SarulixConfig, SarulixLM

DEFAULT_ARCHITECTURE = "AutoRegressiveLM"


@dataclass(frozen=True)
class Architecture:
    make_config: Callable[[dict], object]   # the parsed config.json -> configuration
    model_class: type
    # (configuration, stored tensors) -> configuration, for sizes that only the tensors' shapes tell
    complete: Optional[Callable[[object, dict], object]] = None

    def configure(self, config: dict, tensors: dict):
        made = self.make_config(config)
        return made if self.complete is None else self.complete(made, tensors)


_ARCHITECTURES: Dict[str, Architecture] = {}


def register_architecture(name: str, make_config: Callable[[dict], object], model_class: type,
                          complete: Optional[Callable[[object, dict], object]] = None) -> None:
    _ARCHITECTURES[name] = Architecture(make_config, model_class, complete)


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
register_architecture("Sarulix", SarulixConfig.from_dict, SarulixLM, SarulixConfig.with_tensors)
