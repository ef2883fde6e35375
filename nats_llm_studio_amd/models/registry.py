"""Which model class runs a checkpoint: GGUF files by their architecture key (models/config.py), folders with a
config.json by its `architecture` (models/stack_config.py)."""
from __future__ import annotations

import json
import os

from .config import SUPPORTED_ARCHS
from .stack_config import DESIGNS, is_stack_dir


def checkpoint_kind(path: str) -> str:
    """'gguf' or 'stack'; raises for anything else."""
    if os.path.isfile(path):
        if os.path.basename(path) == "config.json" and is_stack_dir(os.path.dirname(path)):
            return "stack"
        return "gguf"
    if is_stack_dir(path):
        return "stack"
    raise FileNotFoundError(f"{path}: neither a GGUF file nor a folder with config.json and model.safetensors")


def stack_arch(path: str):
    """The design a checkpoint folder names, or None when its config.json is not one of ours."""
    try:
        with open(os.path.join(path, "config.json")) as f:
            a = json.load(f).get("architecture")
    except (OSError, ValueError, AttributeError):
        return None
    return a if a in DESIGNS else None


def supported_architectures():
    return tuple(SUPPORTED_ARCHS) + tuple(DESIGNS)


def load_model(path: str, device, shard=None, comm=None, dtype=None, ctx=None):
    """The model of a checkpoint on `device`. dtype / ctx: stack models only (default bfloat16)."""
    from .llama import LlamaModel, ShardSpec
    shard = shard or ShardSpec()
    if checkpoint_kind(path) == "gguf":
        from ..gguf.reader import GGUFReader
        return LlamaModel(GGUFReader(path), device, shard, comm)
    import torch
    from .stack import StackModel
    if os.path.isfile(path):
        path = os.path.dirname(path)
    return StackModel(path, device, dtype or torch.bfloat16, shard, comm, ctx)
