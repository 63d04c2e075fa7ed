"""Which class serves which model: presets by name, checkpoints by their
config.json."""

from __future__ import annotations

import json
import os
from typing import Optional

from .bolatar import BOLATAR_PRESETS, BolatarConfig, BolatarForCausalLM
from .fimunex import FIMUNEX_PRESETS, FimunexConfig, FimunexForCausalLM
from .llama import MODEL_PRESETS, LlamaConfig, LlamaForCausalLM
from .mixed import MixedModel
from .nesizen import NESIZEN_PRESETS, NesizenConfig, NesizenForCausalLM
from .riruzen import RIRUZEN_PRESETS, RiruzenConfig, RiruzenForCausalLM

# config.json 'architecture' -> (configuration, model)
ARCHITECTURES = {"Bolatar": (BolatarConfig, BolatarForCausalLM),
                 "Fimunex": (FimunexConfig, FimunexForCausalLM),
                 "Nesizen": (NesizenConfig, NesizenForCausalLM),
                 "Riruzen": (RiruzenConfig, RiruzenForCausalLM)}
_MODELS = {LlamaConfig: LlamaForCausalLM, **dict(ARCHITECTURES.values())}
# presets that are made when asked for
_MADE_PRESETS = {**BOLATAR_PRESETS, **FIMUNEX_PRESETS, **NESIZEN_PRESETS,
                 **RIRUZEN_PRESETS}


def model_names() -> list:
    return sorted([*MODEL_PRESETS, *_MADE_PRESETS])


def checkpoint_architecture(path: Optional[str]) -> Optional[str]:
    """The 'architecture' a checkpoint directory names, if it names one
    that is registered here."""
    file = os.path.join(path, "config.json") if path else None
    if not file or not os.path.isfile(file):
        return None
    with open(file) as f:
        arch = json.load(f).get("architecture")
    return arch if arch in ARCHITECTURES else None


def get_config(name: str, weights: Optional[str] = None):
    """The configuration of preset ``name``, or of the checkpoint
    directory ``weights`` (or ``name`` itself) when that says what it is."""
    for path in (weights, name):
        arch = checkpoint_architecture(path)
        if arch is not None:
            return ARCHITECTURES[arch][0].from_dir(path)
    if name in MODEL_PRESETS:
        return MODEL_PRESETS[name]
    if name in _MADE_PRESETS:
        return _MADE_PRESETS[name]()
    raise KeyError(f"unknown model {name!r}; have {model_names()}")


def get_model_class(name: str, weights: Optional[str] = None):
    return _MODELS[type(get_config(name, weights))]


def build_model(config, weights: Optional[str] = None, **kw):
    """The model of ``config``; with ``weights``, loaded from there."""
    cls = _MODELS[type(config)]
    if issubclass(cls, MixedModel):
        return cls(config, weights=weights, **kw)
    model = cls(config, **kw)
    if weights:
        model.load_safetensors(weights)
    return model
