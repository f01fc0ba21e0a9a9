"""Which model a checkpoint directory holds, and how to load it: one entry per model family, chosen by config.json."""
from __future__ import annotations

import json
import os
from dataclasses import dataclass
from typing import Callable


def read_config(model_dir: str) -> dict:
    with open(os.path.join(model_dir, "config.json")) as f:
        return json.load(f)


@dataclass
class Family:
    name: str
    matches: Callable[[dict], bool]
    load: Callable             # (model_dir, capacity, act) -> (config, weights)
    runtime: Callable          # (config, weights) -> runtime
    acts: tuple = (16,)        # activation widths it runs in (32: everything in fp32)
    kv_bits: bool = False      # takes a quantised KV cache


def _load_layer(model_dir, capacity, act):
    from .checkpoint import load_layer_checkpoint
    return load_layer_checkpoint(model_dir, act, capacity)


def _layer_runtime(cfg, w):
    from .layer_decoder import LayerRuntime
    return LayerRuntime(cfg, w)


def _load_moe(model_dir, capacity, act):
    from .checkpoint import load_moe_checkpoint
    return load_moe_checkpoint(model_dir, capacity=capacity)


def _moe_runtime(cfg, w):
    from .moe_decoder import MoeRuntime
    return MoeRuntime(cfg, w)


def _load_dense(model_dir, capacity, act):
    from .checkpoint import load_mlx_checkpoint
    return load_mlx_checkpoint(model_dir, capacity=capacity)


def _dense_runtime(cfg, w):
    from .decoder import DecoderRuntime
    return DecoderRuntime(cfg, w)


FAMILIES = [
    Family("layer-list", lambda c: c.get("architecture") in ("Pusavik", "Fumotar"), _load_layer, _layer_runtime, acts=(16, 32)),
    Family("moe", lambda c: c.get("model_type", "").startswith("deepseek"), _load_moe, _moe_runtime),
    Family("dense", lambda c: "hidden_size" in c.get("text_config", c), _load_dense, _dense_runtime, kv_bits=True),
]


def family_of(config: dict) -> Family:
    for f in FAMILIES:
        if f.matches(config):
            return f
    raise ValueError("config.json describes no model of this library (architecture %r, model_type %r)"
                     % (config.get("architecture"), config.get("model_type")))


def vocab_of(config: dict) -> int:
    c = config.get("text_config", config)
    return int(c["vocab_size"] if "vocab_size" in c else c["vocab"])
