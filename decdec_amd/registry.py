"""Checkpoints by architecture (models with random weights go by name: ``model.ModelArgs.from_name``).

A checkpoint is a folder with ``config.json`` (whose "architecture" names the design) and ``model.safetensors``."""
from __future__ import annotations

import json
import os

import torch

from .hybrid import HybridDecoder, PreNormDecoder

# architectures a checkpoint's config.json may name
ARCHITECTURES = {"Fivitar": HybridDecoder, "Fekulix": PreNormDecoder}


def model_class(config: dict):
    name = config.get("architecture")
    if name not in ARCHITECTURES:
        raise KeyError(f"Unknown architecture: {name}, available: {sorted(ARCHITECTURES)}")
    return ARCHITECTURES[name]


def is_checkpoint(path: str) -> bool:
    return os.path.isfile(os.path.join(path, "config.json"))


def read_config(path: str) -> dict:
    with open(os.path.join(path, "config.json")) as f:
        return json.load(f)


def load_model(path: str, dtype=torch.bfloat16, device="cuda"):
    """The model of a checkpoint folder, ready for setup_caches."""
    from safetensors.torch import load_file
    cfg = read_config(path)
    model = model_class(cfg).from_config(cfg, dtype, device=device)
    model.load_weights(load_file(os.path.join(path, "model.safetensors")))
    return model.eval()

