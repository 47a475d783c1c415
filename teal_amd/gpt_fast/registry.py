"""Which model class a checkpoint or a name belongs to: the uniform Llama stack (model.Transformer: named architectures, model.pth)
or a layered design (layered.LayeredTransformer: config.json + model.safetensors, or a named synthetic configuration)."""
from __future__ import annotations

import json
from pathlib import Path

import torch

from . import layered


def load_model(path, device, dtype: torch.dtype):
    """the model in `path`, a folder with config.json or a checkpoint file"""
    path = Path(path)
    folder = path if path.is_dir() else path.parent
    if layered.is_layered_checkpoint(folder):
        return layered.load_layered_checkpoint(folder, device, dtype)
    if (folder / "config.json").is_file() and not path.is_file():
        with open(folder / "config.json") as f:
            raise ValueError(f"{folder}: no model class for architecture {json.load(f).get('architecture')!r} (known: {sorted(layered.DESIGNS)})")
    from .generate import load_checkpoint_model
    return load_checkpoint_model(path, device, dtype)


def build_model(name: str, device, dtype: torch.dtype, n_layer=None, shard=None):
    """random weights of a named architecture"""
    if layered.is_layered_name(name):
        if shard is not None:
            raise ValueError("layered designs are not sharded")
        return layered.build_layered_model(layered.LayeredArgs.from_name(name, n_layer), device, dtype)
    from .generate import build_synthetic_model
    return build_synthetic_model(name, device, dtype, n_layer=n_layer, shard=shard)
