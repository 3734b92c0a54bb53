"""Hybrid decoder: window attention and linear-attention layers in any order over one packed batch.

``HybridDecoder`` is the block structure: a 32-bit residual, pre-norm mixer and
feed-forward, optionally a per-layer token input.  The residual sums are fused
with the norms that read them (``pa_residual_norm``).  It runs packed rows: a
batch is one run of tokens, sequences one after the other, single decoded
tokens beside portions of prompts, and the context says which rows belong to
whom (``InferenceContext.q_lens``).

Designs on top of it are a function from their ``config.json`` to a
``HybridConfig`` and a table of checkpoint names.  Lotozen is one: layer norms
with biases, unit-RMS q and k behind three-way short convolutions, value mixing,
per-head output gates, lightning attention, per-layer token inputs.
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import Dict, Iterable, List, Optional, Tuple, Union

import torch
import torch.nn.functional as F
from torch import Tensor, nn

from .. import ops
from .attention import CacheConfig, HipPagedAttentionBackend
from .mixers import (AttentionSpec, ConvAttention, GatedMLP, LightningMixer, LightningSpec, RotaryTables, StepRows,
                     TokenSide, _param, fill)
from .types import InferenceContext


@dataclass(frozen=True)
class LayerSpec:
    mixer: Union[AttentionSpec, LightningSpec]
    ff: Optional[int]  # inner width of the feed-forward, None: the layer has none


@dataclass(frozen=True)
class HybridConfig:
    vocab_size: int
    width: int
    layers: Tuple[LayerSpec, ...]
    norm_eps: float
    side_dim: int = 0  # columns per layer of the second embedding, 0: no per-layer token input

    def __post_init__(self) -> None:
        mixed = {(l.mixer.kv_heads, l.mixer.vdim) for l in self.layers if isinstance(l.mixer, AttentionSpec) and l.mixer.v_mix}
        if len(mixed) > 1:
            raise ValueError(f"layers that mix values differ in their value heads: {sorted(mixed)}")

    def v_roles(self) -> List[Optional[str]]:
        """Per layer: "first" for the first that mixes values, "mix" for the others that do."""
        roles: List[Optional[str]] = []
        for layer in self.layers:
            mixes = isinstance(layer.mixer, AttentionSpec) and layer.mixer.v_mix
            roles.append(("mix" if "first" in roles else "first") if mixes else None)
        return roles

    def cache_config(self, num_blocks: int, block_size: int, num_state_slots: int, dtype: torch.dtype,
                     device: str) -> CacheConfig:
        shapes = tuple((l.mixer.kv_heads, l.mixer.pool_dim) if isinstance(l.mixer, AttentionSpec) else None
                       for l in self.layers)
        typical = next((s for s in shapes if s is not None), (1, 8))
        return CacheConfig(num_layers=len(shapes), num_kv_heads=typical[0], head_dim=typical[1], num_blocks=num_blocks,
                           block_size=block_size, dtype=dtype, device=device, layer_kv=shapes,
                           num_state_slots=num_state_slots)


def lotozen_config(d: dict) -> HybridConfig:
    """From the fields of a Lotozen ``config.json``.  Anything it does not know it refuses."""
    def only(what: str, got: dict, *keys: str) -> None:
        extra = sorted(set(got) - set(keys))
        if extra:
            raise ValueError(f"{what}: unknown fields {extra}")

    layers = []
    for i, layer in enumerate(d["layers"]):
        m, mlp = layer["mixer"], layer.get("mlp")
        only(f"layer {i}", layer, "type", "mixer", "mlp")
        if layer["type"] == "attention":
            only(f"layer {i} mixer", m, "heads", "kv_heads", "dim", "vdim", "conv", "rot", "scale", "mask", "v_mix")
            rot, mask = m.get("rot") or {}, m.get("mask") or {}
            only(f"layer {i} rot", rot, "base", "dims", "scaling")
            only(f"layer {i} mask", mask, "size")
            scaling = rot.get("scaling") or {}
            only(f"layer {i} rot.scaling", scaling, "factor")
            mixer: Union[AttentionSpec, LightningSpec] = AttentionSpec(
                heads=int(m["heads"]), kv_heads=int(m["kv_heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]),
                scale=float(m["scale"]), window=int(mask["size"]) if mask.get("size") is not None else None,
                taps=int(m.get("conv") or 0), rot_dims=int(rot.get("dims", 0)), rot_base=float(rot.get("base", 1.0)),
                rot_factor=float(scaling.get("factor", 1.0)), v_mix=bool(m.get("v_mix", False)))
        elif layer["type"] == "lightning":
            only(f"layer {i} mixer", m, "heads", "dim", "vdim", "decay")
            mixer = LightningSpec(heads=int(m["heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]),
                                  decay=tuple(float(x) for x in m["decay"]))
        else:
            raise ValueError(f"layer {i}: unknown mixer {layer['type']!r}")
        if mlp is not None:
            only(f"layer {i} mlp", mlp, "kind", "ff")
            if mlp["kind"] != "dense":
                raise ValueError(f"layer {i}: unknown feed-forward {mlp['kind']!r}")
        layers.append(LayerSpec(mixer, int(mlp["ff"]) if mlp is not None else None))
    only("norm", d["norm"], "eps")
    side = d.get("token_side") or {}
    only("token_side", side, "dim")
    return HybridConfig(vocab_size=int(d["vocab"]), width=int(d["width"]), layers=tuple(layers),
                        norm_eps=float(d["norm"]["eps"]), side_dim=int(side.get("dim", 0)))


class _Norm(nn.Module):
    """Weights of a layer norm; the arithmetic is fused into the residual sums."""

    def __init__(self, width: int, device) -> None:
        super().__init__()
        self.w = _param(width, dtype=torch.float32, device=device)
        self.b = _param(width, dtype=torch.float32, device=device)

    def load(self, get, name: str) -> None:
        fill(self.w, get(name), name)
        fill(self.b, get(name + ".b"), name + ".b")


class _HybridLayer(nn.Module):
    def __init__(self, cfg: HybridConfig, i: int, backend: HipPagedAttentionBackend, rotary: RotaryTables,
                 v_role: Optional[str], dtype: torch.dtype, device) -> None:
        super().__init__()
        spec = cfg.layers[i]
        self.norm1 = _Norm(cfg.width, device)
        if isinstance(spec.mixer, AttentionSpec):
            self.mixer = ConvAttention(spec.mixer, cfg.width, cfg.norm_eps, i, backend, rotary, v_role, dtype, device)
        else:
            self.mixer = LightningMixer(spec.mixer, cfg.width, cfg.norm_eps, i, backend, dtype, device)
        self.norm2 = self.mlp = self.side = None
        if spec.ff is not None:
            self.norm2 = _Norm(cfg.width, device)
            self.mlp = GatedMLP(cfg.width, spec.ff, dtype, device)
        if cfg.side_dim:
            self.side = TokenSide(cfg.width, cfg.side_dim, i, dtype, device)

    def load(self, get, prefix: str) -> None:
        self.norm1.load(get, prefix + "norm1")
        self.mixer.load(get, prefix + "mix.")
        if self.mlp is not None:
            self.norm2.load(get, prefix + "norm2")
            self.mlp.load(get, prefix + "mlp.")
        if self.side is not None:
            self.side.load(get, prefix + "side.")


class HybridDecoder(nn.Module):
    """``forward(input_ids, positions, ctx)`` -> float32 residual rows in the shape of ``input_ids`` plus the width;
    ``logits(rows)`` applies the final norm and the output projection.  Positions are those of the context."""

    packed = True  # runs packed batches (InferenceContext.q_lens)
    recurrent = True  # keeps per-sequence state: no sharing of prefixes

    def __init__(self, cfg: HybridConfig, backend: HipPagedAttentionBackend, max_positions: int,
                 dtype: torch.dtype = torch.bfloat16) -> None:
        super().__init__()
        device = backend.config.device
        self.cfg, self.backend, self.dtype = cfg, backend, dtype
        self.max_positions = max_positions
        self.rotary = RotaryTables(max_positions, device)
        self.embed = _param(cfg.vocab_size, cfg.width, dtype=dtype, device=device)
        self.side_embed = None
        if cfg.side_dim:
            self.side_embed = _param(cfg.vocab_size, cfg.side_dim * len(cfg.layers), dtype=dtype, device=device)
        self.layers = nn.ModuleList(_HybridLayer(cfg, i, backend, self.rotary, role, dtype, device)
                                    for i, role in enumerate(cfg.v_roles()))
        self.norm = _Norm(cfg.width, device)
        self.head = _param(cfg.vocab_size, cfg.width, dtype=dtype, device=device)

    # ------------------------------------------------------------------ weights
    def load_state_dict(self, state: Dict[str, Tensor], strict: bool = True, assign: bool = False):
        """Checkpoint tensors under their checkpoint names, copied in place (captured graphs keep reading them).
        Missing or, with ``strict``, unknown tensors raise."""
        used = set()

        def get(name: str) -> Tensor:
            if name not in state:
                raise KeyError(f"checkpoint lacks {name}")
            used.add(name)
            return state[name]

        with torch.no_grad():
            fill(self.embed, get("embed"), "embed")
            if self.side_embed is not None:
                fill(self.side_embed, get("side.embed"), "side.embed")
            for i, layer in enumerate(self.layers):
                layer.load(get, f"l{i}.")
            self.norm.load(get, "final.norm")
            fill(self.head, get("head"), "head")
        # (the first mixing layer carries a weight it has no use for)
        unknown = sorted(n for n in state if n not in used and not n.endswith(".mix.vmix"))
        if strict and unknown:
            raise KeyError(f"checkpoint has tensors this model does not know: {unknown[:5]}")

    # ------------------------------------------------------------------ forward
    def forward(self, input_ids: Tensor, positions: Optional[Tensor], ctx: InferenceContext,
                trace: Optional[List[Tensor]] = None) -> Tensor:
        """``trace`` collects a copy of the residual after every layer."""
        ids = input_ids.reshape(-1)
        packed = self.backend.packed_step(ctx)
        if packed.num_rows != ids.numel():
            raise ValueError(f"{ids.numel()} tokens for a context of {packed.num_rows} rows")
        step = StepRows(packed, ids)
        eps, dtype = self.cfg.norm_eps, self.dtype
        x = torch.empty((ids.numel(), self.cfg.width), dtype=torch.float32, device=ids.device)
        # what the next residual sum adds: nothing but the embedding at first, then the last branch's output
        pending: dict = {"ids": ids, "table": self.embed}
        for layer in self.layers:
            h = ops.residual_norm(x, dtype, **pending, norm="layer", weight=layer.norm1.w, bias=layer.norm1.b, eps=eps)
            pending = {"y": layer.mixer(h, step)}
            if layer.mlp is not None:
                h = ops.residual_norm(x, dtype, **pending, norm="layer", weight=layer.norm2.w, bias=layer.norm2.b, eps=eps)
                pending = {"y": layer.mlp(h)}
            if layer.side is not None:
                h = ops.residual_norm(x, dtype, **pending)
                pending = {"y": layer.side(h, ids, self.side_embed), "y_weight": layer.side.norm, "y_eps": eps}
            if trace is not None:
                ops.residual_norm(x, dtype, **pending, want_out=False)
                pending = {}
                trace.append(x.clone())
        if pending:
            ops.residual_norm(x, dtype, **pending, want_out=False)
        return x.view(*input_ids.shape, self.cfg.width)

    def logits(self, hidden_rows: Tensor) -> Tensor:
        h = ops.residual_norm(hidden_rows.contiguous(), self.dtype, norm="layer", weight=self.norm.w, bias=self.norm.b,
                              eps=self.cfg.norm_eps)
        return F.linear(h, self.head)
