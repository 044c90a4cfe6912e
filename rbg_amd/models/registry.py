"""Model families: configuration by name or folder, model class by config."""
from __future__ import annotations

import json
import os
from typing import Callable, Dict

from ..engine.config import ModelConfig
from . import bitatar, danipel, gogalix, llama, notadra

# architecture -> model class
MODELS: Dict[str, type] = {
    "llama": llama.LlamaForCausalLM,        # Llama and Qwen3 shapes
    "Bitatar": bitatar.BitatarForCausalLM,
    "Notadra": notadra.NotadraForCausalLM,
    "Gogalix": gogalix.GogalixForCausalLM,
    "Danipel": danipel.DanipelForCausalLM,
}

# architecture of a config.json -> its reader
CONFIG_READERS: Dict[str, Callable[..., ModelConfig]] = {
    "Bitatar": bitatar.BitatarConfig.from_json,
    "Notadra": notadra.NotadraConfig.from_json,
    "Gogalix": gogalix.GogalixConfig.from_json,
    "Danipel": danipel.DanipelConfig.from_json,
}


def load_config(folder: str) -> ModelConfig:
    """Configuration of a model folder (config.json + model.safetensors)."""
    with open(os.path.join(folder, "config.json")) as f:
        d = json.load(f)
    arch = d.get("architecture")
    if arch not in CONFIG_READERS:
        raise ValueError(f"{folder}: unknown architecture {arch!r}; known: "
                         f"{sorted(CONFIG_READERS)}")
    return CONFIG_READERS[arch](
        d, name=os.path.basename(os.path.abspath(folder)),
        weights_path=os.path.abspath(folder))


def resolve_model(name: str) -> ModelConfig:
    """A preset's name, or a model folder."""
    if os.path.isdir(name):
        return load_config(name)
    for family in (bitatar, notadra, gogalix, danipel):
        cfg = family.preset(name)
        if cfg is not None:
            return cfg
    return ModelConfig.preset(name)


def build_model(cfg: ModelConfig, device, tp=None, pp=None):
    return MODELS[cfg.architecture](cfg, device, tp, pp=pp)
