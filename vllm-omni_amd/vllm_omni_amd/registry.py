"""Which model class serves which configuration.

``config_from_dir`` / ``config_from_hf`` turn a checkpoint folder's ``config.json`` (or an ``hf_config`` object) into the
configuration class of the architecture it names; ``model_class_for`` gives the class the runner builds for it.  Model
modules are imported on first use.
"""
from __future__ import annotations

import importlib
import json
import os
from typing import Any

from .compat import _get

# architecture name -> (module, configuration class, model class)
ARCHITECTURES = {
    "Qwen2_5OmniTalkerForConditionalGeneration": ("talker", "TalkerConfig", "Qwen2_5OmniTalkerForConditionalGeneration"),
    "Dogulorn": ("dogulorn", "DogulornConfig", "DogulornForCausalLM"),
    "Bodopel": ("bodopel", "BodopelConfig", "BodopelForCausalLM"),
    "Lifuzen": ("lifuzen", "LifuzenConfig", "LifuzenForCausalLM"),
    "Pupopel": ("pupopel", "PupopelConfig", "PupopelForCausalLM"),
}
DEFAULT_ARCHITECTURE = "Qwen2_5OmniTalkerForConditionalGeneration"


def _load(arch: str, which: int):
    entry = ARCHITECTURES[arch]
    return getattr(importlib.import_module("." + entry[0], __package__), entry[which])


def architecture_of(cfg: Any) -> str:
    """Name from ``architecture`` or ``architectures[0]``; configurations that name none of the table are talkers (their
    variants differ in ``model_type`` only)."""
    names = [_get(cfg, "architecture")] + list(_get(cfg, "architectures") or [])
    for n in names:
        if n in ARCHITECTURES:
            return n
    if names[0] is not None:
        raise ValueError(f"unknown architecture {names[0]!r} (known: {', '.join(ARCHITECTURES)})")
    return DEFAULT_ARCHITECTURE


def config_from_hf(hf: Any):
    """``hf_config`` (object or dict), or an already built configuration, -> configuration of its architecture"""
    for arch in ARCHITECTURES:
        if isinstance(hf, _load(arch, 1)):
            return hf
    arch = architecture_of(hf)
    if arch == DEFAULT_ARCHITECTURE:
        from .compat import talker_config_from_hf

        return talker_config_from_hf(hf)
    return _load(arch, 1).from_dict(hf if isinstance(hf, dict) else hf.to_dict())


def checkpoint_shapes(path: str) -> dict[str, tuple[int, ...]]:
    """name -> shape of every tensor in a folder's ``*.safetensors`` files (headers only)"""
    from safetensors import safe_open

    out = {}
    for name in sorted(f for f in os.listdir(path) if f.endswith(".safetensors")):
        with safe_open(os.path.join(path, name), framework="pt") as f:
            out.update((key, tuple(f.get_slice(key).get_shape())) for key in f.keys())
    return out


def config_from_dir(path: str):
    """Configuration of a checkpoint folder.  A class with ``from_checkpoint`` also sees the tensors' shapes: its
    ``config.json`` does not give every size."""
    with open(os.path.join(path, "config.json")) as f:
        d = json.load(f)
    cls = _load(architecture_of(d), 1)
    if hasattr(cls, "from_checkpoint"):
        return cls.from_checkpoint(d, checkpoint_shapes(path))
    return config_from_hf(d)


def model_class_for(config: Any):
    for arch in ARCHITECTURES:
        if isinstance(config, _load(arch, 1)):
            return _load(arch, 2)
    raise TypeError(f"no registered model has a configuration of type {type(config).__name__}")
