"""Dimensions of the paged KV pool.

Same fields, defaults, derived properties and hashing rule as the reference's
``CacheConfig`` (rollouts/rollouts/inference/attention/config.py:8-58), plus
optional fields: the fp8-e4m3 pool layout, layers of different shapes, and
slots for per-sequence recurrent state.
"""

from __future__ import annotations

from dataclasses import dataclass, fields
from typing import Optional, Tuple

import torch


_EXTENSIONS = {"kv_format": None, "layer_kv": None, "num_state_slots": 0}


@dataclass(frozen=True)
class CacheConfig:
    num_layers: int
    num_kv_heads: int
    head_dim: int
    num_blocks: int = 1024
    block_size: int = 16
    sliding_window: Optional[int] = None
    dtype: torch.dtype = torch.bfloat16
    device: str = "cuda"
    # Extension: "fp8_e4m3" keeps K/V as one byte per element with one fp32
    # scale per (block, kv head); ``dtype`` then names the q / output type.
    kv_format: Optional[str] = None
    # Extension: one (kv heads, head size) per layer, or (kv heads, key size, value size), where value size 0 stands for a
    # layer without a value pool; None for a layer that keeps no keys.  ``num_kv_heads`` and ``head_dim`` then only
    # describe the layer the caller considers typical.
    layer_kv: Optional[Tuple[Optional[Tuple[int, ...]], ...]] = None
    # Extension: sequences that can hold recurrent state at a time (0: the model keeps none).
    num_state_slots: int = 0

    def kv_shape(self, layer_idx: int) -> Optional[Tuple[int, ...]]:
        """(kv heads, head size), or (kv heads, key size, value size), of a layer's pool, None when it has none."""
        return (self.num_kv_heads, self.head_dim) if self.layer_kv is None else self.layer_kv[layer_idx]

    @property
    def total_slots(self) -> int:
        # config.py:38-40 of the reference
        return self.block_size * self.num_blocks

    @property
    def cache_shape(self) -> Tuple[int, int, int, int]:
        # config.py:43-45 of the reference: layer-major, then slot, head, dim
        return (self.num_layers, self.total_slots, self.num_kv_heads, self.head_dim)

    def __hash__(self) -> int:
        # torch dtypes are hashed through their name, as the reference does
        # (config.py:47-58); the extension fields are appended only when set so
        # that reference-shaped configs hash to the reference's value.
        key = tuple(
            str(getattr(self, f.name)) if f.name == "dtype" else getattr(self, f.name)
            for f in fields(self)
            if f.name not in _EXTENSIONS
        )
        for name, default in _EXTENSIONS.items():
            if getattr(self, name) != default:
                key = key + (getattr(self, name),)
        return hash(key)
