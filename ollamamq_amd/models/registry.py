"""Model registry: named configurations, architectures, checkpoint folders.

A model is found by name among the presets and the registered checkpoint
folders; a folder's config.json names its architecture.  The worker, the
bench and the trace runner all build models and caches through here.
"""
from __future__ import annotations

import os
from typing import Dict, NamedTuple, Optional

from .checkpoint import read_config
from .kavedra import KAVEDRA_PRESETS, KavedraConfig, KavedraModel
from .llama import PRESETS, LlamaConfig, LlamaModel
from .pemidra import PEMIDRA_PRESETS, PemidraConfig, PemidraModel
from .revitar import REVITAR_PRESETS, RevitarConfig, RevitarModel
from .rinitar import RINITAR_PRESETS, RinitarConfig, RinitarModel


class Architecture(NamedTuple):
    config: type
    model: type


ARCHITECTURES: Dict[str, Architecture] = {
    "Llama": Architecture(LlamaConfig, LlamaModel),
    "Rinitar": Architecture(RinitarConfig, RinitarModel),
    "Revitar": Architecture(RevitarConfig, RevitarModel),
    "Kavedra": Architecture(KavedraConfig, KavedraModel),
    "Pemidra": Architecture(PemidraConfig, PemidraModel),
}
PRESETS.update(RINITAR_PRESETS)
PRESETS.update(REVITAR_PRESETS)
PRESETS.update(KAVEDRA_PRESETS)
PRESETS.update(PEMIDRA_PRESETS)


def config_from_folder(path: str, name: Optional[str] = None):
    """The configuration of a checkpoint folder."""
    d = read_config(path)
    arch = ARCHITECTURES.get(d.get("architecture"))
    if arch is None or not hasattr(arch.config, "from_json"):
        raise ValueError(f"{path}: unknown architecture "
                         f"{d.get('architecture')!r}")
    name = name or os.path.basename(os.path.normpath(path)).lower()
    return arch.config.from_json(d, name=name, checkpoint=path)


def register_checkpoint(spec: str) -> str:
    """Make a folder available under a name; spec is NAME=DIR."""
    name, _, path = spec.partition("=")
    if not name or not path:
        raise ValueError(f"expected NAME=DIR, got {spec!r}")
    PRESETS[name] = config_from_folder(path, name)
    return name


def model_class(cfg) -> type:
    for arch in ARCHITECTURES.values():
        if isinstance(cfg, arch.config):
            return arch.model
    raise TypeError(f"no model class for {type(cfg).__name__}")


def build_model(cfg, **kw):
    """Instantiate the model a configuration describes."""
    return model_class(cfg)(cfg, **kw)
