"""Which configuration and model class serve a checkpoint, from its ``config.json``.

``model_type`` names the quantised families of mlx_lm layout (``ModelConfig`` / ``ShardModel``);
``architecture`` names a layer-list design (``StackConfig`` / ``StackModel``).
"""

from __future__ import annotations

import json
from pathlib import Path

from .config import ModelConfig
from .stack_config import READERS, StackConfig


def config_from_dict(d: dict) -> ModelConfig | StackConfig:
    if d.get("architecture") in READERS:
        return StackConfig.from_dict(d)
    if "model_type" in d:
        return ModelConfig.from_dict(d)
    return StackConfig.from_dict(d)  # raises with the designs it knows


def load_config(model_dir: str | Path) -> ModelConfig | StackConfig:
    with open(Path(model_dir) / "config.json") as f:
        return config_from_dict(json.load(f))


def build_model(cfg, weights, start_layer: int = 0, end_layer: int | None = None, device="cuda:0", dtype=None):
    """The model class of ``cfg`` over the shard's tensors.  ``dtype`` (layer-list designs only):
    torch.bfloat16 (default) or torch.float32."""
    if isinstance(cfg, StackConfig):
        from .stack_model import StackModel
        kw = {} if dtype is None else {"dtype": dtype}
        return StackModel(cfg, weights, start_layer, end_layer, device, **kw)
    import torch
    if dtype not in (None, torch.bfloat16):
        raise ValueError(f"{cfg.model_type}: only bfloat16 activations, got {dtype}")
    from .model import ShardModel
    return ShardModel(cfg, weights, start_layer, end_layer, device)


def load_model(model_dir: str | Path, device="cuda:0", dtype=None):
    """Whole model of a checkpoint directory."""
    from .loader import load_shard_weights
    cfg = load_config(model_dir)
    it = load_shard_weights(model_dir, cfg, 0, cfg.num_hidden_layers, device)
    try:
        while True:
            next(it)
    except StopIteration as stop:
        return build_model(cfg, stop.value, device=device, dtype=dtype)
