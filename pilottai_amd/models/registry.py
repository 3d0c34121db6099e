"""The model families the engine serves: configuration lookup and model construction.

A model is named by a preset ("llama-3-8b", "mudepel-base", ...), by a folder with a config.json
(its "architecture" entry selects the family; the folder's weights are loaded) or by a
configuration object. A family is a configuration class with `from_dict`, its presets, and a model
class with the interface the models share: forward, make_cache, cache_bytes_per_block,
state_bytes_per_slot, attention_items, attention_workspace, health_words, weight_bytes.
"""
from __future__ import annotations

import json
import os
from typing import Dict, Optional

from pilottai_amd.models import bozupel, llama, mudepel, pusunex, salipel

CONFIG_CLASSES: Dict[str, type] = {"Bozupel": bozupel.BozupelConfig, "Mudepel": mudepel.MudepelConfig,
                                  "Salipel": salipel.SalipelConfig, "Pusunex": pusunex.PusunexConfig}
MODEL_CLASSES: Dict[type, type] = {llama.LlamaConfig: llama.LlamaModel, bozupel.BozupelConfig: bozupel.BozupelModel,
                                   mudepel.MudepelConfig: mudepel.MudepelModel,
                                   salipel.SalipelConfig: salipel.SalipelModel, pusunex.PusunexConfig: pusunex.PusunexModel}
PRESETS = {**llama.PRESETS, **bozupel.PRESETS, **mudepel.PRESETS, **salipel.PRESETS, **pusunex.PRESETS}


def is_folder(name) -> bool:
    return isinstance(name, (str, os.PathLike)) and os.path.isfile(os.path.join(name, "config.json"))


def load_config(folder: str):
    with open(os.path.join(folder, "config.json")) as f:
        d = json.load(f)
    arch = d.get("architecture")
    if arch not in CONFIG_CLASSES:
        raise ValueError(f"{folder}: unknown architecture {arch!r}; known: {sorted(CONFIG_CLASSES)}")
    return CONFIG_CLASSES[arch].from_dict(d, name=os.path.basename(os.path.abspath(folder)))


def get_config(name_or_cfg):
    if type(name_or_cfg) in MODEL_CLASSES:
        return name_or_cfg
    key = str(name_or_cfg).lower()
    if key in PRESETS:
        return PRESETS[key]
    if is_folder(name_or_cfg):
        return load_config(str(name_or_cfg))
    raise ValueError(f"unknown model {name_or_cfg!r}; known: {sorted(PRESETS)}, or a folder with a config.json")


def default_weights(name_or_cfg) -> Optional[str]:
    """The checkpoint folder a model name stands for (None: random weights)."""
    return str(name_or_cfg) if is_folder(name_or_cfg) and str(name_or_cfg).lower() not in PRESETS else None


def model_class(cfg) -> type:
    return MODEL_CLASSES[type(cfg)]
