"""Model registry: names and checkpoint folders -> configs -> runners.

A served model is either a registered name (random-init weights) or a folder
with config.json and model.safetensors; config.json's "architecture" chooses
the reader and the runner.
"""
import json
import os
from typing import Union

import torch

from . import checkpoint, configs, rururax, sezazen
from .configs import LayeredConfig, ModelConfig

AnyConfig = Union[ModelConfig, LayeredConfig]

MODELS = {c.name: c for c in (
    configs.LLAMA_3_8B, configs.QWEN3_32B, configs.LLAVA_1_5_7B_TEXT,
    configs.TINY_LLAMA, configs.TINY_QWEN, configs.TINY_LLAVA,
    configs.RURURAX_8B, configs.TINY_RURURAX, configs.SEZAZEN_8B,
    configs.TINY_SEZAZEN)}

# config.json "architecture" (LayeredConfig.architecture) -> module with the
# design's read_config, tensor_shapes and random_tensor
DESIGNS = {d.ARCHITECTURE: d for d in (rururax, sezazen)}


def resolve(model: str) -> AnyConfig:
    """A registered name or a checkpoint folder -> its config."""
    if model in MODELS:
        return MODELS[model]
    path = os.path.join(model, "config.json")
    if not os.path.isfile(path):
        raise ValueError(f"unknown model {model!r}: neither a folder with "
                         f"config.json nor one of {sorted(MODELS)}")
    with open(path) as f:
        raw = json.load(f)
    arch = raw.get("architecture")
    if arch not in DESIGNS:
        raise ValueError(f"{path}: unknown architecture {arch!r}")
    return DESIGNS[arch].read_config(raw, model)


def build_runner(config: AnyConfig, device: torch.device,
                 dtype: torch.dtype, seed: int = 0,
                 max_model_len: int = 8192):
    if isinstance(config, ModelConfig):
        from .llama import LlamaRunner
        return LlamaRunner(config, device, dtype, seed=seed)
    from .layered import LayeredRunner
    design = DESIGNS[config.architecture]
    take = checkpoint.weights(config.weights_dir,
                              design.tensor_shapes(config),
                              design.random_tensor, device, seed)
    return LayeredRunner(config, take, device, dtype,
                         max_model_len=max_model_len)
