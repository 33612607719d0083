"""Registry of the model designs a checkpoint folder can hold.

A folder checkpoint is `config.json` + `model.safetensors`; its `architecture` names the entry here that
reads the configuration into a `ModelConfig` and maps tensor names to the engine's.  (A GGUF file
carries its own architecture and names: `ModelConfig.from_gguf`.)
"""
from __future__ import annotations

import dataclasses
import importlib
import json
import os
from typing import Callable, Dict, Tuple

from ..runtime.safetensors import SafetensorsReader
from .config import ModelConfig


@dataclasses.dataclass(frozen=True)
class Architecture:
    # (config.json, model name, {tensor name: shape}) -> ModelConfig; the shapes give sizes that config.json does not name
    parse: Callable[[dict, str, Dict[str, Tuple[int, ...]]], ModelConfig]
    tensor_names: Callable[[dict], Dict[str, str]]    # config.json -> {checkpoint name: engine name}


# architecture -> module under aios_amd.models that defines ARCHITECTURE
_MODULES = {"gefazen": "gefazen", "movalorn": "movalorn", "sinisun": "sinisun", "seledra": "seledra"}


def architectures():
    return sorted(_MODULES)


def get(name: str) -> Architecture:
    mod = _MODULES.get(str(name).lower())
    if mod is None:
        raise ValueError(f"unknown model architecture {name!r}; have {architectures()}")
    return importlib.import_module(f"{__package__}.{mod}").ARCHITECTURE


def is_checkpoint_dir(path: str) -> bool:
    """Whether `path` is a folder checkpoint of a registered architecture."""
    f = os.path.join(path, "config.json")
    if not (os.path.isfile(f) and os.path.isfile(os.path.join(path, "model.safetensors"))):
        return False
    try:
        with open(f) as fh:
            return str(json.load(fh).get("architecture", "")).lower() in _MODULES
    except (OSError, ValueError, AttributeError):
        return False


def load_config(path: str, name: str = "") -> Tuple[ModelConfig, dict, Architecture]:
    """(ModelConfig, raw config.json, architecture) of a folder checkpoint."""
    with open(os.path.join(path, "config.json")) as f:
        raw = json.load(f)
    arch = get(raw.get("architecture", ""))
    shapes = {k: t.shape for k, t in SafetensorsReader(os.path.join(path, "model.safetensors")).tensors.items()}
    return arch.parse(raw, name or os.path.basename(os.path.normpath(path)), shapes), raw, arch
