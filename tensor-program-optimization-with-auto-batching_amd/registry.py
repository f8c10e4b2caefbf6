"""Models by the architecture that a folder's config.json names, and loading of such a folder.

A folder holds config.json and model.safetensors (or the shards that model.safetensors.index.json lists).
"""
from __future__ import annotations

import importlib
import json
import os

import torch
from safetensors import safe_open

MODELS = {                    # architecture -> (module, class)
    "LlamaForCausalLM": ("llama", "LlamaForCausalLM"),
    "Safolorn": ("safolorn", "SafolornForCausalLM"),
    "Dinasun": ("dinasun", "DinasunForCausalLM"),
}


def read_config(folder: str) -> dict:
    with open(os.path.join(folder, "config.json")) as f:
        return json.load(f)


def architecture(config: dict) -> str:
    arch = config.get("architecture") or next(iter(config.get("architectures") or ()), None)
    if arch not in MODELS:
        raise ValueError(f"unknown architecture {arch!r} (known: {sorted(MODELS)})")
    return arch


def model_class(config: dict):
    module, name = MODELS[architecture(config)]
    return getattr(importlib.import_module("." + module, __package__), name)


class Tensors:
    """tensors(name) reads one tensor of a folder's safetensors files."""

    def __init__(self, folder: str):
        index = os.path.join(folder, "model.safetensors.index.json")
        files = ["model.safetensors"]
        if os.path.exists(index):
            with open(index) as f:
                files = sorted(set(json.load(f)["weight_map"].values()))
        self._file_of = {}
        for name in files:
            f = safe_open(os.path.join(folder, name), "pt")
            self._file_of.update({k: f for k in f.keys()})

    def __contains__(self, name: str) -> bool:
        return name in self._file_of

    def __call__(self, name: str) -> torch.Tensor:
        if name not in self._file_of:
            raise KeyError(f"tensor {name!r} is not in the model's files")
        return self._file_of[name].get_tensor(name)


def load_model(folder: str, dtype: str = None, device="cuda:0"):
    """The model of a folder in one of its element types (default: its first)."""
    config = read_config(folder)
    cls = model_class(config)
    dtype = dtype or cls.dtypes[0]
    if dtype not in cls.dtypes:
        raise ValueError(f"{cls.__name__} runs in {cls.dtypes}, not in {dtype}")
    return cls.from_weights(config, Tensors(folder), getattr(torch, dtype), device)
