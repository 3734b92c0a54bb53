"""Hybrid decoder: attention and recurrent layers in any order over one packed batch.

``HybridDecoder`` is the block structure: a 32-bit residual, mixer and
feed-forward with norms ahead of or behind them, optionally a per-layer token
input and learned positions.  The residual sums are fused with the norms around
them (``pa_residual_norm``).  It runs packed rows: a
batch is one run of tokens, sequences one after the other, single decoded
tokens beside portions of prompts, and the context says which rows belong to
whom (``InferenceContext.q_lens``).

Designs on top of it are a function from their ``config.json`` to a
``HybridConfig`` and a table of checkpoint names.  Lotozen is one: layer norms
with biases, unit-RMS q and k behind three-way short convolutions, value mixing,
per-head output gates, lightning attention, per-layer token inputs.  Tevirax is
another: RMS norms on the sublayers' outputs, chunk attention beside a matrix
memory in one layer, Mamba-2 layers, mixtures of experts, capped logits.  Vusalix:
several residual streams with learned mixing, latent attention, attention with
distance biases and sinks, the gated delta rule, experts beside identity experts.
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import Callable, Dict, Iterable, List, Optional, Tuple, Union

import torch
import torch.nn.functional as F
from torch import Tensor, nn

from .. import ops
from .attention import CacheConfig, HipPagedAttentionBackend
from .mixers import (AttentionSpec, BiasedAttention, BiasedAttentionSpec, ConvAttention, DeltaMixer, DeltaSpec, GatedMLP,
                     LatentAttention, LatentSpec, LightningMixer, LightningSpec, Mamba2Mixer, Mamba2Spec, MlstmSpec,
                     ParallelMixer, ParallelSpec, RotaryTables, StepRows, TokenSide, YarnScaling, _param, fill)
from .moe import MoE, MoESpec
from .types import InferenceContext


MixerSpec = Union[AttentionSpec, BiasedAttentionSpec, LatentSpec, LightningSpec, Mamba2Spec, DeltaSpec, ParallelSpec]


@dataclass(frozen=True)
class LayerSpec:
    mixer: MixerSpec
    ff: Union[int, MoESpec, None]  # inner width of a dense feed-forward, experts, None: the layer has none

    @property
    def kv_pool(self) -> Optional[Tuple[int, ...]]:
        """What the layer keeps per token (an entry of ``CacheConfig.layer_kv``), None for a layer without keys."""
        mixer = self.mixer.left if isinstance(self.mixer, ParallelSpec) else self.mixer
        return getattr(mixer, "kv_pool", None)


@dataclass(frozen=True)
class HybridConfig:
    vocab_size: int
    width: int
    layers: Tuple[LayerSpec, ...]
    norm_eps: float
    side_dim: int = 0  # columns per layer of the second embedding, 0: no per-layer token input
    norm: str = "layer"  # "layer" (with biases) | "rms"
    post_norm: bool = False  # the norms are on the sublayers' outputs ("rms"), which read the residual itself
    embed_scale: float = 1.0
    positions: int = 0  # rows of a learned position table that the embedding adds, 0: none
    logit_softcap: Optional[float] = None
    streams: int = 0  # residual streams with learned mixing around every sublayer, 0: one plain residual

    def __post_init__(self) -> None:
        if self.streams and (self.norm != "rms" or self.post_norm or self.side_dim or self.positions or self.embed_scale != 1.0):
            raise ValueError("residual streams are for RMS norms ahead of the sublayers and a plain embedding")
        if not 0 <= self.streams <= 16:
            raise ValueError(f"streams={self.streams} not in 1 .. 16")
        if not self.streams and any(isinstance(l.ff, MoESpec) and l.ff.identity for l in self.layers):
            raise ValueError("identity experts are for residual streams")
        if self.post_norm and (self.norm != "rms" or self.side_dim):
            raise ValueError("norms behind the sublayers are RMS norms, without a per-layer token input")
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
        shapes = tuple(l.kv_pool for l in self.layers)
        typical = next((s for s in shapes if s is not None), (1, 8))
        return CacheConfig(num_layers=len(shapes), num_kv_heads=typical[0], head_dim=typical[1], num_blocks=num_blocks,
                           block_size=block_size, dtype=dtype, device=device, layer_kv=shapes,
                           num_state_slots=num_state_slots)


def _only(what: str, got: dict, *keys: str) -> None:
    extra = sorted(set(got) - set(keys))
    if extra:
        raise ValueError(f"{what}: unknown fields {extra}")


def _yarn(where: str, scaling: Optional[dict]) -> Optional[YarnScaling]:
    if scaling is None:
        return None
    _only(where, scaling, "factor", "original", "fast", "slow")
    return YarnScaling(**{key: float(scaling[key]) for key in ("factor", "original", "fast", "slow")})


def lotozen_config(d: dict) -> HybridConfig:
    """From the fields of a Lotozen ``config.json``.  Anything it does not know it refuses."""
    only = _only
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


def _tevirax_ff(where: str, mlp: Optional[dict]) -> Union[int, MoESpec, None]:
    if mlp is None:
        return None
    if mlp["kind"] == "dense":
        _only(where, mlp, "kind", "ff")
        return int(mlp["ff"])
    if mlp["kind"] != "moe":
        raise ValueError(f"{where}: unknown feed-forward {mlp['kind']!r}")
    _only(where, mlp, "kind", "expert", "router", "shared")
    expert, router, shared = mlp["expert"], mlp["router"], mlp.get("shared")
    groups = router.get("groups") or {"count": 1, "keep": 1}
    _only(f"{where} expert", expert, "ff")
    _only(f"{where} router", router, "experts", "top", "groups")
    _only(f"{where} router.groups", groups, "count", "keep")
    if shared is not None:
        _only(f"{where} shared", shared, "ff")
    return MoESpec(experts=int(router["experts"]), ff=int(expert["ff"]), top=int(router["top"]), groups=int(groups["count"]),
                   keep=int(groups["keep"]), shared=int(shared["ff"]) if shared is not None else None)


def tevirax_config(d: dict) -> HybridConfig:
    """From the fields of a Tevirax ``config.json``.  Anything it does not know it refuses."""
    layers = []
    for i, layer in enumerate(d["layers"]):
        m, at = layer["mixer"], f"layer {i} mixer"
        _only(f"layer {i}", layer, "type", "mixer", "mlp")
        if layer["type"] == "mamba2":
            _only(at, m, "heads", "vdim", "state", "groups", "conv", "norm_groups")
            mixer: MixerSpec = Mamba2Spec(heads=int(m["heads"]), vdim=int(m["vdim"]), state=int(m["state"]), groups=int(m["groups"]),
                                          taps=int(m["conv"]), norm_groups=int(m["norm_groups"]))
        elif layer["type"] == "parallel":
            _only(at, m, "left", "right", "left_scale", "right_scale")
            left, right = m["left"], m["right"]
            _only(at + ".left", left, "heads", "kv_heads", "dim", "vdim", "rot", "scale", "mask")
            _only(at + ".right", right, "heads", "dim", "vdim", "gate_cap")
            rot, mask = left.get("rot") or {}, left.get("mask") or {}
            _only(at + ".left.rot", rot, "base", "dims", "scaling")
            _only(at + ".left.mask", mask, "size")
            scaling = _yarn(at + ".left.rot.scaling", rot.get("scaling"))
            mixer = ParallelSpec(
                left=AttentionSpec(heads=int(left["heads"]), kv_heads=int(left["kv_heads"]), dim=int(left["dim"]), vdim=int(left["vdim"]),
                                   scale=float(left["scale"]), window=None, taps=0, rot_dims=int(rot.get("dims", 0)),
                                   rot_base=float(rot.get("base", 1.0)), chunk=int(mask["size"]) if mask.get("size") is not None else None,
                                   rot_yarn=scaling, rot_halves=True, qk_weights=True, gates=False),
                right=MlstmSpec(heads=int(right["heads"]), dim=int(right["dim"]), vdim=int(right["vdim"]), gate_cap=float(right["gate_cap"])),
                left_scale=float(m["left_scale"]), right_scale=float(m["right_scale"]))
        else:
            raise ValueError(f"layer {i}: unknown mixer {layer['type']!r}")
        layers.append(LayerSpec(mixer, _tevirax_ff(f"layer {i} mlp", layer.get("mlp"))))
    _only("norm", d["norm"], "eps")
    _only("embedding", d["embedding"], "scale")
    cap = d.get("logit_softcap")
    return HybridConfig(vocab_size=int(d["vocab"]), width=int(d["width"]), layers=tuple(layers), norm_eps=float(d["norm"]["eps"]),
                        norm="rms", post_norm=True, embed_scale=float(d["embedding"]["scale"]), positions=int(d["max_positions"]),
                        logit_softcap=float(cap) if cap else None)


def _window(where: str, m: dict) -> Optional[int]:
    mask = m.get("mask") or {}
    _only(f"{where}.mask", mask, "size")
    return int(mask["size"]) if mask.get("size") is not None else None


def vusalix_config(d: dict, buckets: Callable[[int], int]) -> HybridConfig:
    """From the fields of a Vusalix ``config.json``; ``buckets``: how many distance buckets layer i's table has (the length of
    a checkpoint tensor).  Anything it does not know it refuses."""
    layers = []
    for i, layer in enumerate(d["layers"]):
        m, mlp, at = layer["mixer"], layer.get("mlp"), f"layer {i} mixer"
        _only(f"layer {i}", layer, "type", "mixer", "mlp")
        if layer["type"] == "delta":
            _only(at, m, "heads", "kv_heads", "dim", "vdim", "conv")
            mixer: MixerSpec = DeltaSpec(heads=int(m["heads"]), kv_heads=int(m["kv_heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]),
                                         taps=int(m["conv"]))
        elif layer["type"] == "latent_attention":
            _only(at, m, "heads", "dim", "rot_dim", "vdim", "kv_rank", "rot", "scale", "mask")
            rot = m.get("rot") or {}
            _only(at + ".rot", rot, "base", "dims", "scaling")
            if int(rot.get("dims", m["rot_dim"])) != int(m["rot_dim"]):
                raise ValueError(f"{at}: rot.dims={rot['dims']} is not rot_dim={m['rot_dim']}")
            mixer = LatentSpec(heads=int(m["heads"]), dim=int(m["dim"]), rot_dim=int(m["rot_dim"]), vdim=int(m["vdim"]),
                               kv_rank=int(m["kv_rank"]), scale=float(m["scale"]), window=_window(at, m),
                               rot_base=float(rot.get("base", 1.0)), rot_yarn=_yarn(at + ".rot.scaling", rot.get("scaling")))
        elif layer["type"] == "attention":
            _only(at, m, "heads", "kv_heads", "dim", "vdim", "scale", "softcap", "bias_max", "mask")
            cap = m.get("softcap")
            mixer = BiasedAttentionSpec(heads=int(m["heads"]), kv_heads=int(m["kv_heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]),
                                        scale=float(m["scale"]), window=_window(at, m), softcap=float(cap) if cap else None,
                                        buckets=buckets(i), bias_max=int(m["bias_max"]))
        else:
            raise ValueError(f"layer {i}: unknown mixer {layer['type']!r}")
        layers.append(LayerSpec(mixer, _vusalix_ff(f"layer {i} mlp", mlp)))
    _only("norm", d["norm"], "eps")
    return HybridConfig(vocab_size=int(d["vocab"]), width=int(d["width"]), layers=tuple(layers), norm_eps=float(d["norm"]["eps"]),
                        norm="rms", streams=int(d["streams"]))


def _vusalix_ff(where: str, mlp: Optional[dict]) -> Optional[MoESpec]:
    if mlp is None:
        return None
    if mlp["kind"] != "moe":
        raise ValueError(f"{where}: unknown feed-forward {mlp['kind']!r}")
    _only(where, mlp, "kind", "expert", "router", "shared")
    router, shared = mlp["router"], mlp.get("shared")
    groups = router.get("groups") or {"count": 1, "keep": 1}
    _only(f"{where} expert", mlp["expert"], "ff")
    _only(f"{where} router", router, "experts", "identity", "top", "groups")
    _only(f"{where} router.groups", groups, "count", "keep")
    if shared is not None:
        _only(f"{where} shared", shared, "ff")
    return MoESpec(experts=int(router["experts"]), ff=int(mlp["expert"]["ff"]), top=int(router["top"]), groups=int(groups["count"]),
                   keep=int(groups["keep"]), shared=int(shared["ff"]) if shared is not None else None, shared_gate=False,
                   identity=int(router.get("identity") or 0), scores="softmax", group_top=1, correction=True, renormalize=False)


class _Norm(nn.Module):
    """Weights of a norm; the arithmetic is fused into the residual sums.  ``args`` as ``pa_residual_norm`` takes them."""

    def __init__(self, cfg: HybridConfig, device) -> None:
        super().__init__()
        self.w = _param(cfg.width, dtype=torch.float32, device=device)
        self.b = _param(cfg.width, dtype=torch.float32, device=device) if cfg.norm == "layer" else None
        self.args = dict(norm=cfg.norm, weight=self.w, bias=self.b, eps=cfg.norm_eps)

    def load(self, get, name: str) -> None:
        fill(self.w, get(name), name)
        if self.b is not None:
            fill(self.b, get(name + ".b"), name + ".b")


class _Streams(nn.Module):
    """Weights of the residual streams around one sublayer; the arithmetic is one kernel (``pa_hyper_norm``)."""

    def __init__(self, streams: int, device) -> None:
        super().__init__()
        kw = dict(dtype=torch.float32, device=device)
        self.weights = _param(streams, **kw)
        self.between = _param(streams, streams, **kw)
        self.into = _param(streams, **kw)

    def load(self, get, prefix: str) -> None:
        fill(self.weights, get(prefix + "in"), prefix + "in")
        fill(self.between, get(prefix + "mix"), prefix + "mix")
        fill(self.into, get(prefix + "out"), prefix + "out")


class _HybridLayer(nn.Module):
    def __init__(self, cfg: HybridConfig, i: int, backend: HipPagedAttentionBackend, rotary: RotaryTables,
                 v_role: Optional[str], dtype: torch.dtype, device) -> None:
        super().__init__()
        spec = cfg.layers[i]
        self.norm1 = _Norm(cfg, device)
        if isinstance(spec.mixer, AttentionSpec):
            self.mixer = ConvAttention(spec.mixer, cfg.width, cfg.norm_eps, i, backend, rotary, v_role, dtype, device)
        elif isinstance(spec.mixer, ParallelSpec):
            self.mixer = ParallelMixer(spec.mixer, cfg.width, cfg.norm_eps, i, backend, rotary, dtype, device)
        elif isinstance(spec.mixer, BiasedAttentionSpec):
            self.mixer = BiasedAttention(spec.mixer, cfg.width, i, backend, dtype, device)
        elif isinstance(spec.mixer, LatentSpec):
            self.mixer = LatentAttention(spec.mixer, cfg.width, cfg.norm_eps, i, backend, rotary, dtype, device)
        elif isinstance(spec.mixer, DeltaSpec):
            self.mixer = DeltaMixer(spec.mixer, cfg.width, cfg.norm_eps, i, backend, dtype, device)
        elif isinstance(spec.mixer, Mamba2Spec):
            self.mixer = Mamba2Mixer(spec.mixer, cfg.width, cfg.norm_eps, i, backend, dtype, device)
        else:
            self.mixer = LightningMixer(spec.mixer, cfg.width, cfg.norm_eps, i, backend, dtype, device)
        self.norm2 = self.mlp = self.side = self.streams1 = self.streams2 = None
        if cfg.streams:
            self.streams1 = _Streams(cfg.streams, device)
            self.streams2 = _Streams(cfg.streams, device) if spec.ff is not None else None
        if spec.ff is not None:
            self.norm2 = _Norm(cfg, device)
            self.mlp = (MoE(spec.ff, cfg.width, dtype, device) if isinstance(spec.ff, MoESpec)
                        else GatedMLP(cfg.width, spec.ff, dtype, device))
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
        for streams, name in ((self.streams1, "hc1."), (self.streams2, "hc2.")):
            if streams is not None:
                streams.load(get, prefix + name)


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
        self.max_positions = min(max_positions, cfg.positions) if cfg.positions else max_positions
        self.rotary = RotaryTables(max_positions, device)
        self.embed = _param(cfg.vocab_size, cfg.width, dtype=dtype, device=device)
        self.pos_embed = _param(cfg.positions, cfg.width, dtype=dtype, device=device) if cfg.positions else None
        self.side_embed = None
        if cfg.side_dim:
            self.side_embed = _param(cfg.vocab_size, cfg.side_dim * len(cfg.layers), dtype=dtype, device=device)
        self.layers = nn.ModuleList(_HybridLayer(cfg, i, backend, self.rotary, role, dtype, device)
                                    for i, role in enumerate(cfg.v_roles()))
        self.norm = _Norm(cfg, device)
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
            if self.pos_embed is not None:
                fill(self.pos_embed, get("pos"), "pos")
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
        if self.cfg.streams:
            return self._forward_streams(step, trace).view(*input_ids.shape, self.cfg.width)
        cfg, eps, dtype = self.cfg, self.cfg.norm_eps, self.dtype
        x = torch.empty((ids.numel(), self.cfg.width), dtype=torch.float32, device=ids.device)
        # what the next residual sum adds: nothing but the embedding at first, then the last branch's output
        pending: dict = {"ids": ids, "table": self.embed, "table_scale": cfg.embed_scale}
        if self.pos_embed is not None:
            if positions is None:
                raise ValueError("learned positions need the rows' positions")
            pending.update(positions=positions.reshape(-1), pos_table=self.pos_embed)
        # a norm's weights either with the sum that a sublayer reads, or with the sublayer's output as it is added
        ahead = (lambda norm: {}) if cfg.post_norm else (lambda norm: norm.args)
        behind = (lambda norm: {"y_weight": norm.w, "y_eps": eps}) if cfg.post_norm else (lambda norm: {})
        for layer in self.layers:
            h = ops.residual_norm(x, dtype, **pending, **ahead(layer.norm1))
            pending = {"y": layer.mixer(h, step), **behind(layer.norm1)}
            if layer.mlp is not None:
                h = ops.residual_norm(x, dtype, **pending, **ahead(layer.norm2))
                pending = {**layer.mlp.branch(h), **behind(layer.norm2)}
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

    def _forward_streams(self, step: StepRows, trace: Optional[List[Tensor]]) -> Tensor:
        """The sum of the streams ``[rows, width]`` after the last layer."""
        cfg, dtype = self.cfg, self.dtype
        x = torch.empty((step.ids.numel(), cfg.streams, cfg.width), dtype=torch.float32, device=step.ids.device)
        # what the next pass over the streams takes in: the embedding at first, then the last branch's output
        pending: dict = {"ids": step.ids, "table": self.embed}
        for layer in self.layers:
            for norm, streams, branch in ((layer.norm1, layer.streams1, lambda h: {"y": layer.mixer(h, step)}),
                                          (layer.norm2, layer.streams2, lambda h: layer.mlp.branch(h))):
                if norm is None:
                    continue
                h = ops.hyper_norm(x, dtype, **pending, sum_weight=streams.weights, weight=norm.w, eps=cfg.norm_eps)
                pending = {**branch(h), "between": streams.between, "into": streams.into}
            if trace is not None:
                trace.append(ops.hyper_norm(x, dtype, **pending, want="sum"))
        return ops.hyper_norm(x, dtype, **pending, want="sum")

    def logits(self, hidden_rows: Tensor) -> Tensor:
        h = ops.residual_norm(hidden_rows.contiguous(), self.dtype, **self.norm.args)
        y = F.linear(h, self.head)
        return y if self.cfg.logit_softcap is None else ops.softcap(y, self.cfg.logit_softcap)
