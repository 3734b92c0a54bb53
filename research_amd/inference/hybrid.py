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
Loluzen: norms ahead of and behind every sublayer, a stretch of layers that runs
several times, attention with mixed heads beside HGRN2, convolved and rotated
attention, feed-forwards without gates.
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import Callable, Dict, List, NamedTuple, Optional, Tuple, Union

import torch
import torch.nn.functional as F
from torch import Tensor, nn

from .. import ops
from .attention import CacheConfig, HipPagedAttentionBackend
from .mixers import (MIXERS, AttentionSpec, BiasedAttentionSpec, DeltaSpec, GatedMLP, Hgrn2Spec, LatentSpec, LightningSpec,
                     LlamaScaling, Mamba2Spec, MLPSpec, MlstmSpec, ParallelSpec, PlainMLP, RotaryTables, Site, StepRows, TalkingSpec,
                     TokenSide, YarnScaling, _param, fill)
from .moe import MoE, MoESpec
from .types import InferenceContext


MixerSpec = Union[AttentionSpec, BiasedAttentionSpec, LatentSpec, LightningSpec, Mamba2Spec, DeltaSpec, TalkingSpec, Hgrn2Spec,
                  ParallelSpec]


@dataclass(frozen=True)
class LayerSpec:
    mixer: MixerSpec
    ff: Union[int, MLPSpec, MoESpec, None]  # inner width of a gated feed-forward, one without gates, experts, None: none

    @property
    def kv_pool(self) -> Optional[Tuple[int, ...]]:
        """What the layer keeps per token (an entry of ``CacheConfig.layer_kv``), None for a layer without keys."""
        mixer = self.mixer.left if isinstance(self.mixer, ParallelSpec) else self.mixer
        return getattr(mixer, "kv_pool", None)


@dataclass(frozen=True)
class Loop:
    """Layers ``start .. stop - 1`` run ``times`` times in a row with the same weights, each turn with keys and state of its
    own; the embedding is added to the residual ahead of every turn but the first."""

    start: int
    stop: int
    times: int


class Run(NamedTuple):
    """One pass through a layer."""

    layer: int
    turn: int
    again: bool  # the embedding is added ahead of it


@dataclass(frozen=True)
class HybridConfig:
    vocab_size: int
    width: int
    layers: Tuple[LayerSpec, ...]
    norm_eps: float
    side_dim: int = 0  # columns per layer of the second embedding, 0: no per-layer token input
    norm: str = "layer"  # "layer" (with biases) | "rms"
    post_norm: bool = False  # the norms are on the sublayers' outputs ("rms"), which read the residual itself
    both_norms: bool = False  # norms ahead of the sublayers and on their outputs ("rms")
    norm_offset: float = 0.0  # added to the weights of these norms as they are loaded
    residual_mult: float = 1.0  # on the normed outputs of sublayers
    loop: Optional[Loop] = None
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
        if self.both_norms and (self.norm != "rms" or self.post_norm or self.side_dim or self.streams):
            raise ValueError("norms on both sides of the sublayers are RMS norms of one plain residual")
        if self.residual_mult != 1.0 and not (self.both_norms or self.post_norm):
            raise ValueError(f"residual_mult={self.residual_mult} without norms on the sublayers' outputs")
        if self.loop is not None:
            if not 0 <= self.loop.start < self.loop.stop <= len(self.layers) or self.loop.times < 1:
                raise ValueError(f"{self.loop} of {len(self.layers)} layers")
            if self.streams or self.positions or any(isinstance(l.mixer, AttentionSpec) and l.mixer.v_mix for l in self.layers):
                raise ValueError("layers that run again are for one plain residual, without learned positions and value mixing")
        mixed = {(l.mixer.kv_heads, l.mixer.vdim) for l in self.layers if isinstance(l.mixer, AttentionSpec) and l.mixer.v_mix}
        if len(mixed) > 1:
            raise ValueError(f"layers that mix values differ in their value heads: {sorted(mixed)}")

    def runs(self) -> List[Run]:
        """The layers in the order in which they run; each run has its own place in the cache."""
        loop, n = self.loop or Loop(0, len(self.layers), 1), len(self.layers)
        runs = [Run(i, 0, False) for i in range(loop.start)]
        for turn in range(loop.times):
            runs += [Run(i, turn, turn > 0 and i == loop.start) for i in range(loop.start, loop.stop)]
        return runs + [Run(i, 0, False) for i in range(loop.stop, n)]

    def v_roles(self) -> List[Optional[str]]:
        """Per layer: "first" for the first that mixes values, "mix" for the others that do."""
        roles: List[Optional[str]] = []
        for layer in self.layers:
            mixes = isinstance(layer.mixer, AttentionSpec) and layer.mixer.v_mix
            roles.append(("mix" if "first" in roles else "first") if mixes else None)
        return roles

    def cache_config(self, num_blocks: int, block_size: int, num_state_slots: int, dtype: torch.dtype,
                     device: str) -> CacheConfig:
        shapes = tuple(self.layers[run.layer].kv_pool for run in self.runs())
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


def _llama_scaling(where: str, scaling: Optional[dict]) -> Optional[LlamaScaling]:
    if scaling is None:
        return None
    _only(where, scaling, "factor", "original", "low", "high")
    return LlamaScaling(**{key: float(scaling[key]) for key in ("factor", "original", "low", "high")})


def loluzen_config(d: dict) -> HybridConfig:
    """From the fields of a Loluzen ``config.json``.  Anything it does not know it refuses."""
    layers = []
    for i, layer in enumerate(d["layers"]):
        m, mlp, at = layer["mixer"], layer.get("mlp"), f"layer {i} mixer"
        _only(f"layer {i}", layer, "type", "mixer", "mlp")
        if layer["type"] == "attention":
            _only(at, m, "heads", "kv_heads", "dim", "vdim", "conv", "rot", "scale")
            rot = m.get("rot") or {}
            _only(at + ".rot", rot, "base", "dims", "scaling")
            mixer: MixerSpec = AttentionSpec(
                heads=int(m["heads"]), kv_heads=int(m["kv_heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]), scale=float(m["scale"]),
                window=None, taps=int(m.get("conv") or 0), rot_dims=int(rot.get("dims", 0)), rot_base=float(rot.get("base", 1.0)),
                rot_llama=_llama_scaling(at + ".rot.scaling", rot.get("scaling")), qk_weights=True)
        elif layer["type"] == "parallel":
            _only(at, m, "left", "right")
            left, right = m["left"], m["right"]
            _only(at + ".left", left, "heads", "kv_heads", "dim", "vdim", "scale")
            _only(at + ".right", right, "heads", "dim", "vdim")
            mixer = ParallelSpec(
                left=TalkingSpec(heads=int(left["heads"]), kv_heads=int(left["kv_heads"]), dim=int(left["dim"]), vdim=int(left["vdim"]),
                                 scale=float(left["scale"])),
                right=Hgrn2Spec(heads=int(right["heads"]), dim=int(right["dim"]), vdim=int(right["vdim"])),
                left_scale=0.5, right_scale=0.5, norms=True)
        else:
            raise ValueError(f"layer {i}: unknown mixer {layer['type']!r}")
        if mlp is not None:
            _only(f"layer {i} mlp", mlp, "kind", "ff")
            if mlp["kind"] != "dense":
                raise ValueError(f"layer {i}: unknown feed-forward {mlp['kind']!r}")
        layers.append(LayerSpec(mixer, MLPSpec(int(mlp["ff"]), "relu2") if mlp is not None else None))
    _only("norm", d["norm"], "eps")
    embedding, loop = d.get("embedding") or {}, d.get("loop")
    _only("embedding", embedding, "scale")
    if loop is not None:
        _only("loop", loop, "start", "stop", "times")
        loop = Loop(*(int(loop[key]) for key in ("start", "stop", "times")))
    return HybridConfig(vocab_size=int(d["vocab"]), width=int(d["width"]), layers=tuple(layers), norm_eps=float(d["norm"]["eps"]),
                        norm="rms", both_norms=True, norm_offset=1.0, residual_mult=float(d.get("residual_mult", 1.0)),
                        embed_scale=float(embedding.get("scale", 1.0)), loop=loop)


class _Norm(nn.Module):
    """Weights of a norm, ``scale`` times what is loaded plus the config's offset; the arithmetic is fused into the residual
    sums.  ``args`` as ``pa_residual_norm`` takes them."""

    def __init__(self, cfg: HybridConfig, device, scale: float = 1.0) -> None:
        super().__init__()
        self.offset, self.scale = cfg.norm_offset, scale
        self.w = _param(cfg.width, dtype=torch.float32, device=device)
        self.b = _param(cfg.width, dtype=torch.float32, device=device) if cfg.norm == "layer" else None
        self.args = dict(norm=cfg.norm, weight=self.w, bias=self.b, eps=cfg.norm_eps)

    def load(self, get, name: str) -> None:
        fill(self.w, get(name), name)
        self.w.add_(self.offset).mul_(self.scale)
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
    def __init__(self, cfg: HybridConfig, i: int, site: Site) -> None:
        super().__init__()
        spec, dtype, device = cfg.layers[i], site.dtype, site.device
        behind = lambda: _Norm(cfg, device, cfg.residual_mult)
        norm = behind if cfg.post_norm else lambda: _Norm(cfg, device)
        self.norm1, self.norm1b = norm(), behind() if cfg.both_norms else None
        self.mixer = MIXERS[type(spec.mixer)](spec.mixer, site)
        self.norm2 = self.norm2b = self.mlp = self.side = self.streams1 = self.streams2 = None
        if cfg.streams:
            self.streams1 = _Streams(cfg.streams, device)
            self.streams2 = _Streams(cfg.streams, device) if spec.ff is not None else None
        if spec.ff is not None:
            self.norm2, self.norm2b = norm(), behind() if cfg.both_norms else None
            if isinstance(spec.ff, MoESpec):
                self.mlp = MoE(spec.ff, cfg.width, dtype, device)
            else:
                self.mlp = (PlainMLP if isinstance(spec.ff, MLPSpec) else GatedMLP)(cfg.width, spec.ff, dtype, device)
        if cfg.side_dim:
            self.side = TokenSide(cfg.width, cfg.side_dim, i, dtype, device)

    def load(self, get, prefix: str) -> None:
        self.norm1.load(get, prefix + "norm1")
        self.mixer.load(get, prefix + "mix.")
        if self.mlp is not None:
            self.norm2.load(get, prefix + "norm2")
            self.mlp.load(get, prefix + "mlp.")
        for behind, name in ((self.norm1b, "norm1b"), (self.norm2b, "norm2b")):
            if behind is not None:
                behind.load(get, prefix + name)
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
        self.runs = cfg.runs()
        places = lambda i: tuple(at for at, run in enumerate(self.runs) if run.layer == i)
        self.layers = nn.ModuleList(_HybridLayer(cfg, i, Site(cfg.width, cfg.norm_eps, places(i), backend, self.rotary, dtype, device, role))
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
        """``trace`` collects a copy of the residual after every run of a layer."""
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
        behind = lambda norm: {} if norm is None else {"y_weight": norm.w, "y_eps": eps}
        for i, step.turn, again in self.runs:
            layer = self.layers[i]
            if again:
                pending = {**pending, "ids": ids, "table": self.embed, "table_scale": cfg.embed_scale, "ids_add": True}
            h = ops.residual_norm(x, dtype, **pending, **ahead(layer.norm1))
            pending = {**layer.mixer.branch(h, step), **behind(layer.norm1 if cfg.post_norm else layer.norm1b)}
            if layer.mlp is not None:
                h = ops.residual_norm(x, dtype, **pending, **ahead(layer.norm2))
                pending = {**layer.mlp.branch(h), **behind(layer.norm2 if cfg.post_norm else layer.norm2b)}
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
