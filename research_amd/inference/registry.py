"""Model registry: from a local checkpoint folder to a model on its backend.

A folder holds ``config.json`` and ``*.safetensors``; the first entry whose
``matches`` accepts the config builds the model.  A design is added with
``register`` and from then on is served by everything that loads a folder: the
engine, the command line and the trace runner.
"""

from __future__ import annotations

import json
import os
from dataclasses import dataclass
from typing import Callable, Dict, List, Optional

import torch
from torch import Tensor, nn

from .attention import CacheConfig, HipPagedAttentionBackend
from .hybrid import HybridConfig, HybridDecoder, loluzen_config, lotozen_config, tevirax_config, vusalix_config
from .model import ModelConfig, PagedLlama

DTYPES = {"bfloat16": torch.bfloat16, "float32": torch.float32}


@dataclass(frozen=True)
class LoadOptions:
    """What the caller fixes: the cache's sizes and the type of activations and products."""

    num_blocks: int
    block_size: int
    num_state_slots: int
    max_positions: int
    dtype: torch.dtype = torch.bfloat16
    device: str = "cuda"


@dataclass(frozen=True)
class ModelEntry:
    name: str
    matches: Callable[[dict], bool]
    build: Callable[[str, dict, LoadOptions], nn.Module]
    positions: Callable[[dict], Optional[int]] = lambda config: None  # positions the design ends at, None: any


_ENTRIES: List[ModelEntry] = []


def register(entry: ModelEntry) -> None:
    if any(e.name == entry.name for e in _ENTRIES):
        raise ValueError(f"model {entry.name!r} is registered already")
    _ENTRIES.append(entry)


def find(config: dict) -> ModelEntry:
    for entry in _ENTRIES:
        if entry.matches(config):
            return entry
    raise ValueError(f"no registered model for this config.json (known: {[e.name for e in _ENTRIES]})")


def read_config(path: str) -> dict:
    with open(os.path.join(path, "config.json")) as fh:
        return json.load(fh)


def read_weights(path: str) -> Dict[str, Tensor]:
    from safetensors.torch import load_file

    state: Dict[str, Tensor] = {}
    for name in sorted(os.listdir(path)):
        if name.endswith(".safetensors"):
            state.update(load_file(os.path.join(path, name)))
    if not state:
        raise FileNotFoundError(f"no .safetensors files in {path}")
    return state


def load_model(path: str, options: LoadOptions) -> nn.Module:
    config = read_config(path)
    return find(config).build(path, config, options)


def model_len(path: str, wanted: int) -> int:
    """``wanted``, or what the design of the folder has positions for."""
    config = read_config(path)
    limit = find(config).positions(config)
    return wanted if limit is None else min(wanted, limit)


# ------------------------------------------------------------------ entries


Weights = Dict[str, Tensor]


def _hybrid(reader: Callable[[dict, Weights], HybridConfig]) -> Callable[[str, dict, LoadOptions], nn.Module]:
    def build(path: str, config: dict, o: LoadOptions) -> nn.Module:
        weights = read_weights(path)
        cfg = reader(config, weights)
        backend = HipPagedAttentionBackend(cfg.cache_config(o.num_blocks, o.block_size, o.num_state_slots, o.dtype, o.device))
        model = HybridDecoder(cfg, backend, o.max_positions, o.dtype)
        model.load_state_dict(weights, strict=False)
        return model.eval()
    return build


def _vusalix(config: dict, weights: Weights) -> HybridConfig:
    return vusalix_config(config, lambda i: weights[f"l{i}.mix.rel"].shape[0])


def _build_llama(path: str, config: dict, o: LoadOptions) -> nn.Module:
    def backend_for(cfg: ModelConfig) -> HipPagedAttentionBackend:
        return HipPagedAttentionBackend(CacheConfig(
            num_layers=cfg.num_layers, num_kv_heads=cfg.num_kv_heads, head_dim=cfg.head_dim, num_blocks=o.num_blocks,
            block_size=o.block_size, device=o.device, dtype=o.dtype))
    return PagedLlama.from_local(path, backend_for, dtype=o.dtype, device=o.device)


register(ModelEntry("lotozen", lambda c: c.get("architecture") == "Lotozen", _hybrid(lambda c, w: lotozen_config(c))))
register(ModelEntry("tevirax", lambda c: c.get("architecture") == "Tevirax", _hybrid(lambda c, w: tevirax_config(c)),
                    lambda c: int(c["max_positions"])))
register(ModelEntry("vusalix", lambda c: c.get("architecture") == "Vusalix", _hybrid(_vusalix)))
register(ModelEntry("loluzen", lambda c: c.get("architecture") == "Loluzen", _hybrid(lambda c, w: loluzen_config(c))))
register(ModelEntry("llama", lambda c: "num_attention_heads" in c, _build_llama,
                    lambda c: c.get("max_position_embeddings")))
