from .kavedra import KavedraConfig, KavedraModel
from .llama import LlamaConfig, LlamaModel, PRESETS
from .pemidra import PemidraConfig, PemidraModel
from .revitar import RevitarConfig, RevitarModel
from .rinitar import RinitarConfig, RinitarModel
from .registry import (build_model, config_from_folder, model_class,
                       register_checkpoint)

__all__ = ["KavedraConfig", "KavedraModel", "LlamaConfig", "LlamaModel",
           "PemidraConfig", "PemidraModel", "RevitarConfig", "RevitarModel", "RinitarConfig", "RinitarModel",
           "PRESETS", "build_model", "config_from_folder", "model_class",
           "register_checkpoint"]
