"""Token mixers of hybrid decoders and the feed-forward beside them.

A mixer reads packed rows ``h [rows, width]`` (the normed residual) and returns
what is added to the residual.  Sizes and constants come from its spec; keys,
values and recurrent state live in the backend, addressed by the step's block
tables and state slots.  Every mixer joins its input projections into one
product and everything between the products into one or two kernels:

* ``ConvAttention``: joint projection -> ``pa_qkv_conv_append`` (short causal
  convolution with its carried rows, rotation, unit norms, value mixing, append)
  -> paged attention -> ``pa_head_gate`` -> output projection;
* ``LightningMixer``: joint projection -> ``pa_lightning_*`` (silu, recurrence)
  -> ``pa_rms_gate`` -> output projection;
* ``MlstmMixer``: joint projection -> ``pa_gated_linear`` (gates, recurrence,
  normaliser) -> ``pa_rms_gate`` per head -> output projection;
* ``Mamba2Mixer``: joint projection -> ``pa_short_conv`` -> ``pa_gated_linear``
  -> ``pa_rms_gate`` (gate first) -> output projection;
* ``DeltaMixer``: joint projection -> ``pa_short_conv`` -> ``pa_delta`` (unit
  norms, gates, delta rule) -> ``pa_rms_gate`` per head -> output projection;
* ``BiasedAttention``: joint projection -> ``pa_qkv_conv_append`` (append) ->
  ``pa_scored_attention`` (cap, distance biases, sinks) -> output projection;
* ``LatentAttention``: joint projection -> ``pa_latent_append``; decoded tokens
  attend to the cached latents themselves (``pa_scored_attention`` between two
  products per head), portions to keys and values made again from them;
* ``TalkingAttention``: joint projection -> ``pa_qkv_conv_append`` (biases, append)
  -> ``pa_talking_attention`` (distance bias, heads' weights mixed) ->
  ``pa_head_gate`` -> output projection;
* ``Hgrn2Mixer``: joint projection -> ``pa_channel_linear`` (gates, recurrence) ->
  ``pa_rms_gate`` per head without a gate -> output projection;
* ``ParallelMixer``: two of them side by side with one joint input projection and
  one joint output projection (their scales ride on the steps before the latter)
  or, where each side's output is normed on its own, one of each side's.

A layer that runs several times with the same weights keeps keys and state per
turn: a mixer's ``Site`` names one place in the cache for each of its turns.
"""

from __future__ import annotations

import math
from dataclasses import dataclass
from typing import Callable, Dict, List, Optional, Tuple, Union

import torch
import torch.nn.functional as F
from torch import Tensor, nn

from .. import ops
from .attention.hip_backend import HipPagedAttentionBackend, PackedStep

_LN2 = math.log(2.0)
DECAY_POWERS = 65  # powers 0 .. 64 of a decay, one more than the rows of a chunk

Getter = Callable[[str], Tensor]  # checkpoint tensor by name


@dataclass(frozen=True)
class YarnScaling:
    """Rotary frequencies interpolated by parts: pairs that turn more than ``fast`` times over ``original`` positions keep
    theirs, those that turn less than ``slow`` times are divided by ``factor``, with a ramp over the pairs between."""

    factor: float
    original: float
    fast: float
    slow: float


@dataclass(frozen=True)
class LlamaScaling:
    """Rotary frequencies by their wavelength: those shorter than ``original / high`` positions keep theirs, those longer than
    ``original / low`` are divided by ``factor``, with a ramp in the number of waves between."""

    factor: float
    original: float
    low: float
    high: float


RotaryScaling = Union[YarnScaling, LlamaScaling]


@dataclass(frozen=True)
class AttentionSpec:
    """Softmax attention over a sliding window behind short convolutions.  ``window`` and ``chunk`` None: plain causal;
    ``chunk``: keys of the query's own chunk of positions; ``taps`` 0: no convolution; ``v_mix``: the layer takes part in
    value mixing; ``rot_halves``: dimension i turns with i + rot_dims / 2, else 2i with 2i + 1; ``qk_weights``: RMS norms of
    q and k with weights ahead of the rotation, else norms without weights behind it; ``gates``: a gate per head."""

    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    window: Optional[int]
    taps: int
    rot_dims: int
    rot_base: float
    rot_factor: float = 1.0
    v_mix: bool = False
    chunk: Optional[int] = None
    rot_yarn: Optional[YarnScaling] = None
    rot_halves: bool = False
    qk_weights: bool = False
    gates: bool = True
    rot_llama: Optional[LlamaScaling] = None

    def __post_init__(self) -> None:
        if self.heads % self.kv_heads != 0:
            raise ValueError(f"heads={self.heads} is not a multiple of kv_heads={self.kv_heads}")
        if self.rot_dims % 2 or not 0 <= self.rot_dims <= self.dim:
            raise ValueError(f"rot_dims={self.rot_dims} must be even and at most dim={self.dim}")
        if self.window is not None and self.window < 1:
            raise ValueError(f"window={self.window} must be positive")
        if self.chunk is not None and (self.chunk < 1 or self.window is not None):
            raise ValueError(f"chunk={self.chunk} must be positive, and no window beside it")
        if self.dim > 256:
            raise ValueError(f"dim={self.dim} above 256")
        if self.v_slices > 1 and (self.v_mix or self.gates or self.taps):
            raise ValueError(f"vdim={self.vdim} above 256 with value mixing, head gates or convolutions")

    @property
    def v_slices(self) -> int:
        """Equal slices of a value head that keep it within 256.  Each is stored and attended as a head of its own beside a
        copy of the key, with a copy of its query heads (in the order key head, slice, query head)."""
        return -(-self.vdim // 256)

    @property
    def slice_dim(self) -> int:
        return -(-self.vdim // self.v_slices)

    @property
    def pool_heads(self) -> int:
        return self.kv_heads * self.v_slices

    @property
    def pool_dim(self) -> int:
        """Head size of the layer's pool: holds a key or a value, in whole 8-element vectors."""
        return -(-max(self.dim, self.slice_dim) // 8) * 8

    @property
    def channels(self) -> int:
        return self.v_slices * ((self.heads + self.kv_heads) * self.dim + self.kv_heads * self.slice_dim)

    @property
    def mask_window(self) -> int:
        """The kernels' ``window``: positive a sliding window, negative chunks, 0 neither."""
        return self.window or -(self.chunk or 0)

    def head_order(self) -> Tensor:
        """The order in which the dimensions of q and k heads are stored: pairs that turn together side by side."""
        order = torch.arange(self.dim)
        if self.rot_halves:
            order[: self.rot_dims] = order[: self.rot_dims].view(2, -1).t().reshape(-1)
        return order


    @property
    def kv_pool(self) -> Tuple[int, ...]:
        """The layer's pool, as an entry of ``CacheConfig.layer_kv``."""
        return self.pool_heads, self.pool_dim


@dataclass(frozen=True)
class BiasedAttentionSpec:
    """Softmax attention without rotation: scores under a soft cap, a learned bias per distance bucket and head, a sink per
    head in the denominator.  ``bias_max``: the distance from which on all share the last bucket."""

    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    window: Optional[int]
    softcap: Optional[float]
    buckets: int
    bias_max: int

    def __post_init__(self) -> None:
        if self.heads % self.kv_heads != 0:
            raise ValueError(f"heads={self.heads} is not a multiple of kv_heads={self.kv_heads}")
        if self.window is not None and self.window < 1:
            raise ValueError(f"window={self.window} must be positive")
        if self.buckets < 2 or self.bias_max <= self.buckets // 2:
            raise ValueError(f"bias_max={self.bias_max} must be above half of buckets={self.buckets}")
        if max(self.dim, self.vdim) > 256:
            raise ValueError(f"dim={self.dim} or vdim={self.vdim} above 256")

    @property
    def kv_pool(self) -> Tuple[int, ...]:
        return self.kv_heads, _pad8(max(self.dim, self.vdim))

    def bucket_of(self) -> List[int]:
        """The bucket of every distance 0 .. bias_max: single distances up to half of the buckets, then equal ratios.  Bucket
        half + k starts where (n / half)^rest reaches (bias_max / half)^k, in whole numbers."""
        half, most = self.buckets // 2, self.bias_max
        rest, out = self.buckets - half, list(range(half))
        k = 0
        for n in range(half, most + 1):
            while k + 1 < rest and n ** rest * half ** (k + 1) >= most ** (k + 1) * half ** rest:
                k += 1
            out.append(half + k)
        return out


@dataclass(frozen=True)
class LatentSpec:
    """Attention whose keys and values per head are linear in one latent of ``kv_rank`` per token; beside them a rotated key
    part of ``rot_dim`` shared by all heads.  The cache keeps the latent and the rotated part."""

    heads: int
    dim: int
    rot_dim: int
    vdim: int
    kv_rank: int
    scale: float
    window: Optional[int]
    rot_base: float
    rot_yarn: Optional[YarnScaling] = None

    def __post_init__(self) -> None:
        if self.rot_dim % 2:
            raise ValueError(f"rot_dim={self.rot_dim} must be even")
        if self.window is not None and self.window < 1:
            raise ValueError(f"window={self.window} must be positive")
        if self.kv_rank > 1024 or self.kv_rank + self.rot_dim > 2048:
            raise ValueError(f"kv_rank={self.kv_rank} above 1024")

    @property
    def pool_row(self) -> int:
        return _pad8(self.kv_rank + self.rot_dim)

    @property
    def kv_pool(self) -> Tuple[int, ...]:
        return 1, self.pool_row, 0

    @property
    def made(self) -> Tuple[int, int]:
        """Sizes of a head's key and value made again from the latents: one size, as the kernels for plain attention have it,
        except where that would carry values of at most 128 in rows of 256."""
        key, value = _pad8(self.dim + self.rot_dim), _pad8(self.vdim)
        return (key, value) if 128 < key <= 192 and value <= 128 else (max(key, value),) * 2


@dataclass(frozen=True)
class DeltaSpec:
    """The gated delta rule behind short convolutions; ``heads`` value heads share ``kv_heads`` q/k heads."""

    heads: int
    kv_heads: int
    dim: int
    vdim: int
    taps: int

    def __post_init__(self) -> None:
        if self.heads % self.kv_heads != 0:
            raise ValueError(f"heads={self.heads} is not a multiple of kv_heads={self.kv_heads}")
        if self.dim > 256 or not 1 <= self.taps <= 8:
            raise ValueError(f"dim={self.dim} above 256 or taps={self.taps} not in 1 .. 8")

    @property
    def channels(self) -> int:
        return 2 * self.kv_heads * self.dim + self.heads * self.vdim


@dataclass(frozen=True)
class LightningSpec:
    """Linear attention with one constant decay per head."""

    heads: int
    dim: int
    vdim: int
    decay: Tuple[float, ...]

    def __post_init__(self) -> None:
        if len(self.decay) != self.heads:
            raise ValueError(f"{len(self.decay)} decays for {self.heads} heads")
        if self.dim > 256:
            raise ValueError(f"dim={self.dim} above 256")


@dataclass(frozen=True)
class MlstmSpec:
    """Matrix memory with exponential gates under a soft cap."""

    heads: int
    dim: int
    vdim: int
    gate_cap: float

    def __post_init__(self) -> None:
        if self.dim > 256:
            raise ValueError(f"dim={self.dim} above 256")


@dataclass(frozen=True)
class Mamba2Spec:
    """Mamba-2: a state of ``state`` x ``vdim`` per head, input and output vectors shared by the heads of a group."""

    heads: int
    vdim: int
    state: int
    groups: int
    taps: int
    norm_groups: int

    def __post_init__(self) -> None:
        if self.heads % self.groups or (self.heads * self.vdim) % self.norm_groups:
            raise ValueError(f"{self.heads} heads of {self.vdim} do not divide into groups={self.groups} / norm_groups={self.norm_groups}")
        if self.state > 256 or not 1 <= self.taps <= 8:
            raise ValueError(f"state={self.state} above 256 or taps={self.taps} not in 1 .. 8")

    @property
    def inner(self) -> int:
        return self.heads * self.vdim

    @property
    def channels(self) -> int:
        return self.inner + 2 * self.groups * self.state


@dataclass(frozen=True)
class TalkingSpec:
    """Softmax attention without rotation whose scores lose ``r1 ln(1 + r2 distance)`` per head and whose heads' weights are
    mixed by a matrix before they meet the values; biases in the projections, a gate per head."""

    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float

    def __post_init__(self) -> None:
        if self.heads % self.kv_heads != 0:
            raise ValueError(f"heads={self.heads} is not a multiple of kv_heads={self.kv_heads}")
        if max(self.dim, self.vdim) > 256 or self.heads > 128:
            raise ValueError(f"dim={self.dim} or vdim={self.vdim} above 256, or heads={self.heads} above 128")

    @property
    def kv_pool(self) -> Tuple[int, ...]:
        return self.kv_heads, _pad8(max(self.dim, self.vdim))

    @property
    def channels(self) -> int:
        return (self.heads + self.kv_heads) * self.dim + self.kv_heads * self.vdim


@dataclass(frozen=True)
class Hgrn2Spec:
    """Linear attention with a forget gate per channel, bounded from below, whose complement is the key."""

    heads: int
    dim: int
    vdim: int

    def __post_init__(self) -> None:
        if self.dim > 256:
            raise ValueError(f"dim={self.dim} above 256")


@dataclass(frozen=True)
class ParallelSpec:
    """Attention and a recurrent mixer on the same input.  Their outputs are added under two scales; ``norms``: each first
    RMS-normed with a weight of its own."""

    left: Union[AttentionSpec, TalkingSpec]
    right: Union[MlstmSpec, Hgrn2Spec]
    left_scale: float = 1.0
    right_scale: float = 1.0
    norms: bool = False


def yarn_frequencies(base: float, dims: int, yarn: YarnScaling) -> Tuple[Tensor, float]:
    """float64 frequencies of the ``dims / 2`` pairs, and the factor on cosine and sine."""
    def pair_of(turns: float) -> float:
        return dims * math.log(yarn.original / (2 * math.pi * turns)) / (2 * math.log(base))

    first, last = max(math.floor(pair_of(yarn.fast)), 0), min(math.ceil(pair_of(yarn.slow)), dims - 1)
    pairs = torch.arange(dims // 2, dtype=torch.float64)
    ramp = ((pairs - first) / max(last - first, 0.001)).clamp(0.0, 1.0)
    freq = base ** (-2.0 * pairs / dims)
    return freq / yarn.factor * ramp + freq * (1.0 - ramp), 0.1 * math.log(yarn.factor) + 1.0


def llama_frequencies(base: float, dims: int, s: LlamaScaling) -> Tensor:
    """float64 frequencies of the ``dims / 2`` pairs."""
    freq = base ** (-torch.arange(0, dims, 2, dtype=torch.float64) / dims)
    length = 2 * math.pi / freq
    part = (s.original / length - s.low) / (s.high - s.low) if s.high != s.low else torch.zeros_like(freq)
    between = (1 - part) * freq / s.factor + part * freq
    return torch.where(length < s.original / s.high, freq, torch.where(length > s.original / s.low, freq / s.factor, between))


class RotaryTables:
    """(cos, sin) per position and pair, float32 from float64 angles; one table per (base, dims, factor, scaling), shared by
    the layers that name it.  The position limit is fixed once a captured graph may hold a table's address."""

    def __init__(self, max_positions: int, device) -> None:
        self.max_positions = max_positions
        self.device = device
        self._tables: Dict[tuple, Tensor] = {}

    def get(self, base: float, dims: int, factor: float, scaling: Optional[RotaryScaling] = None) -> Optional[Tensor]:
        if dims == 0:
            return None
        key = (base, dims, factor, scaling)
        if key not in self._tables:
            freq, size = base ** (-torch.arange(0, dims, 2, dtype=torch.float64) / dims), 1.0
            if isinstance(scaling, YarnScaling):
                freq, size = yarn_frequencies(base, dims, scaling)
            elif scaling is not None:
                freq = llama_frequencies(base, dims, scaling)
            angle = torch.arange(self.max_positions, dtype=torch.float64)[:, None] * (freq / factor)[None, :]
            table = (torch.stack([angle.cos(), angle.sin()], dim=-1) * size).float()
            self._tables[key] = table.contiguous().to(self.device)
        return self._tables[key]


@dataclass
class StepRows:
    """What one forward pass shares between its layers."""

    packed: PackedStep
    ids: Tensor
    v_first: Optional[Tensor] = None
    turn: int = 0  # how often the layer has run already


@dataclass(frozen=True)
class Site:
    """Where a mixer lives: the model's width, norm constant and types, and the layer's place in the cache for each turn."""

    width: int
    eps: float
    places: Tuple[int, ...]
    backend: HipPagedAttentionBackend
    rotary: RotaryTables
    dtype: torch.dtype
    device: Union[str, torch.device]
    v_role: Optional[str] = None  # None, "first" (the layer whose values the others mix in) or "mix"

    def weight(self, *shape: int) -> nn.Parameter:
        return _param(*shape, dtype=self.dtype, device=self.device)

    def constant(self, *shape: int) -> nn.Parameter:
        return _param(*shape, dtype=torch.float32, device=self.device)

    def keep(self, name: str, shape: Tuple[int, ...], dtype: torch.dtype, when: bool = True) -> List[Optional[Tensor]]:
        """State per sequence: a tensor for each turn, or, without one, None for each."""
        return [self.backend.register_state(at, name, shape, dtype) if when else None for at in self.places]


def _param(*shape: int, dtype: torch.dtype, device) -> nn.Parameter:
    return nn.Parameter(torch.zeros(shape, dtype=dtype, device=device), requires_grad=False)


def fill(dst: Tensor, src: Tensor, name: str) -> None:
    if tuple(dst.shape) != tuple(src.shape):
        raise ValueError(f"{name}: checkpoint shape {tuple(src.shape)}, expected {tuple(dst.shape)}")
    dst.copy_(src)


def _pad8(n: int) -> int:
    return -(-n // 8) * 8


def _pad16(n: int) -> int:
    return -(-n // 16) * 16


Slices = Optional[Tuple[Tensor, Tensor]]


class Mixer(nn.Module):
    """A joint input product, ``mix`` between the products, an output product.  ``in_rows`` and ``out_cols`` are the sizes of
    the two weights; a mixer that is part of another is handed its slices of that one's weights.  ``out_scale`` multiplies
    what ``mix`` returns."""

    def __init__(self, in_rows: int, out_cols: int, site: Site, slices: Slices = None, out_scale: float = 1.0) -> None:
        super().__init__()
        self.site, self.backend, self.eps, self.out_scale = site, site.backend, site.eps, out_scale
        if slices is None:
            slices = site.weight(in_rows, site.width), site.weight(site.width, out_cols)
        self.w_in, self.w_out = slices

    def mix(self, u: Tensor, step: StepRows, out: Optional[Tensor] = None) -> Tensor:
        raise NotImplementedError

    def forward(self, h: Tensor, step: StepRows) -> Tensor:
        return F.linear(self.mix(F.linear(h, self.w_in), step), self.w_out)

    def branch(self, h: Tensor, step: StepRows) -> Dict[str, object]:
        """What the residual sum adds, as ``ops.residual_norm`` takes it."""
        return {"y": self(h, step)}


class ConvAttention(Mixer):
    @staticmethod
    def sizes(spec: AttentionSpec) -> Tuple[int, int]:
        return _pad8(spec.channels + (spec.heads if spec.gates else 0)), spec.heads * spec.v_slices * spec.slice_dim

    def __init__(self, spec: AttentionSpec, site: Site, slices: Slices = None, out_scale: float = 1.0) -> None:
        """Rows of ``w_in``: q, k, v, head gates, padding."""
        super().__init__(*self.sizes(spec), site, slices, out_scale)
        self.spec, self.v_role = spec, site.v_role
        self.q_norm = self.k_norm = None
        if spec.qk_weights:
            self.q_norm, self.k_norm = site.constant(spec.dim), site.constant(spec.dim)
        self.conv = site.constant(spec.taps, spec.channels) if spec.taps else None
        self.v_lambda = site.constant(1)
        self.conv_state = site.keep("conv", (spec.taps - 1, spec.channels), site.dtype, spec.taps > 1)

    def load(self, get: Getter, prefix: str) -> None:
        s, at = self.spec, 0
        order = s.head_order()
        if s.v_slices > 1:
            self._load_slices(get, prefix, order)
            return
        for name, n in (("q", s.heads * s.dim), ("k", s.kv_heads * s.dim), ("v", s.kv_heads * s.vdim)):
            pick = slice(None)
            if s.rot_halves and name != "v":  # (the scores do not change when q and k heads are stored in another order)
                pick = (torch.arange(0, n, s.dim)[:, None] + order).reshape(-1)
            fill(self.w_in[at: at + n], get(prefix + name)[pick], prefix + name)
            if self.conv is not None:
                fill(self.conv[:, at: at + n], get(f"{prefix}{name}.conv")[pick].t(), f"{prefix}{name}.conv")
            at += n
        if s.gates:
            fill(self.w_in[at: at + s.heads], get(prefix + "g"), prefix + "g")
        self._load_qk_norms(get, prefix, order)
        fill(self.w_out, get(prefix + "o"), prefix + "o")
        if self.v_role == "mix":
            fill(self.v_lambda, get(prefix + "vmix").reshape(1), prefix + "vmix")

    def _load_qk_norms(self, get: Getter, prefix: str, order: Tensor) -> None:
        if self.spec.qk_weights:
            fill(self.q_norm, get(prefix + "q.norm")[order], prefix + "q.norm")
            fill(self.k_norm, get(prefix + "k.norm")[order], prefix + "k.norm")

    def _load_slices(self, get: Getter, prefix: str, order: Tensor) -> None:
        """The layout of ``v_slices``: copies of the key heads and their query heads for every slice of the value head; the
        part of the last slice past the head's end is zeros."""
        s = self.spec
        n, rep, width = s.v_slices, s.heads // s.kv_heads, self.w_in.shape[1]

        def heads(name: str, count: int, dim: int) -> Tensor:
            w = get(prefix + name)
            if tuple(w.shape) != (count * dim, width):
                raise ValueError(f"{prefix}{name}: checkpoint shape {tuple(w.shape)}, expected {(count * dim, width)}")
            return w.view(s.kv_heads, -1, dim, width)

        q = heads("q", s.heads, s.dim)[:, None, :, order].expand(-1, n, -1, -1, -1)
        k = heads("k", s.kv_heads, s.dim)[:, :, order].expand(-1, n, -1, -1)
        pad = n * s.slice_dim - s.vdim
        v = F.pad(heads("v", s.kv_heads, s.vdim)[:, 0], (0, 0, 0, pad))
        at = 0
        for name, w in (("q", q), ("k", k), ("v", v)):
            w = w.reshape(-1, width)
            fill(self.w_in[at: at + w.shape[0]], w, prefix + name)
            at += w.shape[0]
        self._load_qk_norms(get, prefix, order)
        o = get(prefix + "o")
        if tuple(o.shape) != (self.w_out.shape[0], s.heads * s.vdim):
            raise ValueError(f"{prefix}o: checkpoint shape {tuple(o.shape)}")
        o = F.pad(o.view(-1, s.kv_heads, rep, s.vdim), (0, pad)).view(-1, s.kv_heads, rep, n, s.slice_dim).transpose(2, 3)
        fill(self.w_out, o.reshape(self.w_out.shape), prefix + "o")

    def mix(self, u: Tensor, step: StepRows, out: Optional[Tensor] = None) -> Tensor:
        s, packed = self.spec, step.packed
        if self.v_role == "first":
            step.v_first = torch.empty((u.shape[0], s.kv_heads * s.vdim), dtype=u.dtype, device=u.device)
        place = self.site.places[step.turn]
        kc, vc = self.backend._layer(place)
        # q carries scale * log2(e) from its 32-bit registers, so that the attention kernels' own factor is one
        q = ops.qkv_conv_append(u, packed.rows, packed.slots, kc, vc, s.heads * s.v_slices, s.dim, s.slice_dim, s.scale / _LN2, self.eps,
                                not s.qk_weights, self.site.rotary.get(s.rot_base, s.rot_dims, s.rot_factor, s.rot_yarn or s.rot_llama),
                                s.rot_dims, self.conv, self.conv_state[step.turn], self.v_role, step.v_first if self.v_role else None,
                                self.v_lambda if self.v_role == "mix" else None, q_norm=self.q_norm, k_norm=self.k_norm)
        o = self.backend.attend_packed(q, place, packed, _LN2, s.mask_window)
        gate = u[:, s.channels: s.channels + s.heads] if s.gates else None
        return ops.head_gate(o, gate, s.slice_dim, self.out_scale, out)


class LightningMixer(Mixer):
    def __init__(self, spec: LightningSpec, site: Site) -> None:
        """Rows of ``w_in``: q, k, v, output gate, padding."""
        inner = spec.heads * spec.vdim
        super().__init__(_pad8(spec.heads * 2 * spec.dim + 2 * inner), inner, site)
        self.spec = spec
        self.norm = site.constant(inner)
        self.state = site.keep("lightning", (spec.heads, _pad16(spec.dim), _pad16(spec.vdim)), torch.float32)
        powers = torch.tensor(spec.decay, dtype=torch.float64)[:, None] ** torch.arange(DECAY_POWERS, dtype=torch.float64)
        self.register_buffer("decay_powers", powers.float().to(site.device).contiguous(), persistent=False)

    def load(self, get: Getter, prefix: str) -> None:
        s, at = self.spec, 0
        for name, n in (("q", s.heads * s.dim), ("k", s.heads * s.dim), ("v", s.heads * s.vdim), ("g", s.heads * s.vdim)):
            fill(self.w_in[at: at + n], get(prefix + name), prefix + name)
            at += n
        fill(self.w_out, get(prefix + "o"), prefix + "o")
        fill(self.norm, get(prefix + "norm"), prefix + "norm")

    def mix(self, u: Tensor, step: StepRows, out: Optional[Tensor] = None) -> Tensor:
        s, packed, state = self.spec, step.packed, self.state[step.turn]
        inner = s.heads * s.vdim
        o = torch.empty((u.shape[0], inner), dtype=u.dtype, device=u.device)
        nd = packed.num_decodes
        if packed.decodes is not None:
            ops.lightning(u[:nd], packed.decodes, state, self.decay_powers, s.heads, s.dim, s.vdim, o[:nd])
        if packed.chunks is not None:
            c = packed.chunks
            need = ops.lightning_workspace_bytes(c.ctx_lens.numel(), s.heads, s.dim, s.vdim, c.max_q_len)
            ops.lightning(u, c, state, self.decay_powers, s.heads, s.dim, s.vdim, o,
                          workspace=self.backend._scratch_for(need) if need else None)
        g = 2 * s.heads * s.dim + inner
        return ops.rms_gate(o, u[:, g: g + inner], self.norm, self.eps, out=out)


def _gated_rows(kind: str, q: Tensor, k: Tensor, v: Tensor, gates, constants, step: StepRows, state: Tensor, heads: int, dim: int,
                vdim: int, backend: HipPagedAttentionBackend, **kw) -> Tensor:
    """A gated recurrence over a step's rows: single tokens, then portions."""
    packed = step.packed
    out = torch.empty((v.shape[0], heads * vdim), dtype=v.dtype, device=v.device)
    if packed.decodes is not None:
        cut = lambda t: None if t is None else t[: packed.num_decodes]
        ops.gated_linear(kind, cut(q), cut(k), cut(v), tuple(cut(g) for g in gates), constants, packed.decodes, state, heads, dim,
                         vdim, cut(out), **kw)
    if packed.chunks is not None:
        c = packed.chunks
        need = ops.gated_linear_workspace_bytes(c.ctx_lens.numel(), heads, dim, vdim, c.max_q_len)
        ops.gated_linear(kind, q, k, v, gates, constants, c, state, heads, dim, vdim, out,
                         workspace=backend._scratch_for(need) if need else None, **kw)
    return out


class MlstmMixer(Mixer):
    DEN_EPS = 1e-6

    @staticmethod
    def sizes(spec: MlstmSpec) -> Tuple[int, int]:
        inner = spec.heads * spec.vdim
        return _pad8(2 * spec.heads * spec.dim + 2 * inner + 2 * spec.heads), inner

    def __init__(self, spec: MlstmSpec, site: Site, slices: Slices = None, out_scale: float = 1.0) -> None:
        """Rows of ``w_in``: q, k, v, output gate, input gates, forget gates, padding."""
        super().__init__(*self.sizes(spec), site, slices, out_scale)
        self.spec = spec
        self.norm = site.constant(spec.heads * spec.vdim)  # times out_scale
        self.i_bias, self.f_bias = site.constant(spec.heads), site.constant(spec.heads)
        floats = ops.gated_linear_state_floats("mlstm", spec.dim, spec.vdim)
        self.state = site.keep("mlstm", (spec.heads, floats), torch.float32)

    def _parts(self) -> Tuple[Tuple[str, int], ...]:
        s = self.spec
        return (("q", s.heads * s.dim), ("k", s.heads * s.dim), ("v", s.heads * s.vdim), ("g", s.heads * s.vdim), ("i", s.heads),
                ("f", s.heads))

    def load(self, get: Getter, prefix: str) -> None:
        at = 0
        for name, n in self._parts():
            fill(self.w_in[at: at + n], get(prefix + name), prefix + name)
            at += n
        fill(self.i_bias, get(prefix + "i.b"), prefix + "i.b")
        fill(self.f_bias, get(prefix + "f.b"), prefix + "f.b")
        fill(self.norm, get(prefix + "norm"), prefix + "norm")
        self.norm.mul_(self.out_scale)
        fill(self.w_out, get(prefix + "o"), prefix + "o")

    def mix(self, u: Tensor, step: StepRows, out: Optional[Tensor] = None) -> Tensor:
        s = self.spec
        sizes = [n for _, n in self._parts()]
        q, k, v, g, i, f = u[:, : sum(sizes)].split(sizes, dim=1)
        o = _gated_rows("mlstm", q, k, v, (i, f), (self.i_bias, self.f_bias, None), step, self.state[step.turn], s.heads, s.dim, s.vdim,
                        self.backend, cap=s.gate_cap, q_scale=s.dim ** -0.5, den_eps=self.DEN_EPS)
        return ops.rms_gate(o, g, self.norm, self.eps, groups=s.heads, out=out)


class Mamba2Mixer(Mixer):
    def __init__(self, spec: Mamba2Spec, site: Site) -> None:
        """Rows of ``w_in``: gate, x, B, C, step sizes, padding."""
        super().__init__(_pad8(spec.inner + spec.channels + spec.heads), spec.inner, site)
        self.spec = spec
        self.conv, self.conv_bias = site.constant(spec.taps, spec.channels), site.constant(spec.channels)
        self.dt_bias, self.rate, self.skip = (site.constant(spec.heads) for _ in range(3))
        self.norm = site.constant(spec.inner)
        self.conv_state = site.keep("conv", (spec.taps - 1, spec.channels), site.dtype, spec.taps > 1)
        floats = ops.gated_linear_state_floats("ssd", spec.state, spec.vdim)
        self.state = site.keep("ssd", (spec.heads, floats), torch.float32)

    def load(self, get: Getter, prefix: str) -> None:
        s = self.spec
        fill(self.w_in[: s.inner + s.channels + s.heads], get(prefix + "in"), prefix + "in")
        fill(self.conv, get(prefix + "conv").t(), prefix + "conv")
        fill(self.conv_bias, get(prefix + "conv.b"), prefix + "conv.b")
        fill(self.dt_bias, get(prefix + "dt_bias"), prefix + "dt_bias")
        fill(self.rate, get(prefix + "A_log").float().exp(), prefix + "A_log")
        fill(self.skip, get(prefix + "D"), prefix + "D")
        fill(self.norm, get(prefix + "norm"), prefix + "norm")
        fill(self.w_out, get(prefix + "o"), prefix + "o")

    def mix(self, u: Tensor, step: StepRows, out: Optional[Tensor] = None) -> Tensor:
        s = self.spec
        z, x, dt = u[:, : s.inner + s.channels + s.heads].split([s.inner, s.channels, s.heads], dim=1)
        x = ops.short_conv(x, step.packed.rows, self.conv, self.conv_bias, self.conv_state[step.turn], "silu")
        n = s.groups * s.state
        x, b, c = x.split([s.inner, n, n], dim=1)
        y = _gated_rows("ssd", c, b, x, (dt, None), (self.dt_bias, self.rate, self.skip), step, self.state[step.turn], s.heads,
                        s.state, s.vdim, self.backend, heads_per_group=s.heads // s.groups)
        return ops.rms_gate(y, z, self.norm, self.eps, groups=s.norm_groups, order="silu_first", out=out)


class DeltaMixer(Mixer):
    def __init__(self, spec: DeltaSpec, site: Site) -> None:
        """Rows of ``w_in``: q, k, v, output gate, decay logits, beta logits, padding."""
        inner = spec.heads * spec.vdim
        super().__init__(_pad8(spec.channels + inner + 2 * spec.heads), inner, site)
        self.spec = spec
        self.conv = site.constant(spec.taps, spec.channels)
        self.dt_bias, self.rate = (site.constant(spec.heads) for _ in range(2))
        self.norm = site.constant(inner)  # one head's weights, for every head
        self.conv_state = site.keep("conv", (spec.taps - 1, spec.channels), site.dtype, spec.taps > 1)
        self.state = site.keep("delta", (spec.heads, _pad16(spec.dim), _pad16(spec.vdim)), torch.float32)

    def _parts(self) -> Tuple[Tuple[str, int], ...]:
        s = self.spec
        qk, inner = s.kv_heads * s.dim, s.heads * s.vdim
        return ("q", qk), ("k", qk), ("v", inner), ("g", inner), ("a", s.heads), ("b", s.heads)

    def load(self, get: Getter, prefix: str) -> None:
        s, at = self.spec, 0
        for name, n in self._parts():
            fill(self.w_in[at: at + n], get(prefix + name), prefix + name)
            if name in "qkv":
                fill(self.conv[:, at: at + n], get(f"{prefix}{name}.conv").t(), f"{prefix}{name}.conv")
            at += n
        fill(self.dt_bias, get(prefix + "dt_bias"), prefix + "dt_bias")
        fill(self.rate, get(prefix + "A_log").float().exp(), prefix + "A_log")
        fill(self.norm, get(prefix + "norm").repeat(s.heads), prefix + "norm")
        fill(self.w_out, get(prefix + "o"), prefix + "o")

    def mix(self, u: Tensor, step: StepRows, out: Optional[Tensor] = None) -> Tensor:
        s, packed = self.spec, step.packed
        x, g, a, b = u[:, : s.channels + s.heads * (s.vdim + 2)].split([s.channels, s.heads * s.vdim, s.heads, s.heads], dim=1)
        x = ops.short_conv(x, packed.rows, self.conv, None, self.conv_state[step.turn], "silu")
        q, k, v = x.split([s.kv_heads * s.dim, s.kv_heads * s.dim, s.heads * s.vdim], dim=1)
        o = torch.empty((u.shape[0], s.heads * s.vdim), dtype=u.dtype, device=u.device)
        sizes = (self.dt_bias, self.rate)
        tail = (self.state[step.turn], s.heads, s.dim, s.vdim, s.dim ** -0.5)
        kw = dict(heads_per_group=s.heads // s.kv_heads)
        if packed.decodes is not None:
            n = packed.num_decodes
            ops.delta_rule(*(t[:n] for t in (q, k, v, a, b)), *sizes, packed.decodes, *tail, o[:n], **kw)
        if packed.chunks is not None:
            c = packed.chunks
            need = ops.delta_workspace_bytes(c.ctx_lens.numel(), s.heads, s.dim, s.vdim, c.max_q_len) if u.dtype == torch.bfloat16 else 0
            ops.delta_rule(q, k, v, a, b, *sizes, c, *tail, o, workspace=self.backend._scratch_for(need) if need else None, **kw)
        return ops.rms_gate(o, g, self.norm, self.eps, groups=s.heads, order="silu_last", out=out)


class BiasedAttention(Mixer):
    def __init__(self, spec: BiasedAttentionSpec, site: Site) -> None:
        """Rows of ``w_in``: q, k, v, padding."""
        super().__init__(_pad8((spec.heads + spec.kv_heads) * spec.dim + spec.kv_heads * spec.vdim), spec.heads * spec.vdim, site)
        self.spec = spec
        self.buckets = torch.tensor(spec.bucket_of())
        self.bias = site.constant(spec.heads, len(self.buckets))  # by distance
        self.sink = site.constant(spec.heads)

    def load(self, get: Getter, prefix: str) -> None:
        s, at = self.spec, 0
        for name, n in (("q", s.heads * s.dim), ("k", s.kv_heads * s.dim), ("v", s.kv_heads * s.vdim)):
            fill(self.w_in[at: at + n], get(prefix + name), prefix + name)
            at += n
        rel = get(prefix + "rel")
        if tuple(rel.shape) != (s.buckets, s.heads):
            raise ValueError(f"{prefix}rel: checkpoint shape {tuple(rel.shape)}, expected {(s.buckets, s.heads)}")
        fill(self.bias, rel[self.buckets.to(rel.device)].t(), prefix + "rel")
        fill(self.sink, get(prefix + "sink"), prefix + "sink")
        fill(self.w_out, get(prefix + "o"), prefix + "o")

    def mix(self, u: Tensor, step: StepRows, out: Optional[Tensor] = None) -> Tensor:
        s, packed = self.spec, step.packed
        place = self.site.places[step.turn]
        kc, vc = self.backend._layer(place)
        q = ops.qkv_conv_append(u, packed.rows, packed.slots, kc, vc, s.heads, s.dim, s.vdim, 1.0, 0.0, False, None, 0, None, None)
        # (q and the pool hold zeros between dim and its next multiple of 8)
        o = self.backend.attend_scored((q[..., : _pad8(s.dim)],), place, packed, s.vdim, s.scale, s.window or 0,
                                       softcap=s.softcap or 0.0, bias=self.bias, sink=self.sink)
        o = o.view(u.shape[0], -1)
        return o if out is None else out.copy_(o)


class LatentAttention(Mixer):
    def __init__(self, spec: LatentSpec, site: Site) -> None:
        """Rows of ``w_in``: q, latent, rotated key part, padding.  The two weights on the latent are kept in two forms: per
        head, for products before and behind attention over the latents (``w_key`` transposed), and over whole pool rows,
        for keys and values made again (the rotated part passes through an identity)."""
        s = spec
        super().__init__(_pad8(s.heads * (s.dim + s.rot_dim) + s.kv_rank + s.rot_dim), s.heads * s.vdim, site)
        self.spec = spec
        pad = lambda n: -(-n // 64) * 64
        self.norm = site.constant(s.kv_rank)
        self.w_key = site.weight(s.heads, s.kv_rank, pad(s.dim))
        self.w_value = site.weight(s.heads, s.vdim, pad(s.kv_rank))
        self.remake = site.dtype == torch.bfloat16 and max(s.made) <= 256
        if self.remake:
            self.k_made, self.v_made = (site.weight(s.heads, size, s.pool_row) for size in s.made)
        self._lists: Dict[int, ops.ExpertChoice] = {}

    def load(self, get: Getter, prefix: str) -> None:
        s = self.spec
        n = s.heads * (s.dim + s.rot_dim)
        fill(self.w_in[:n], get(prefix + "q"), prefix + "q")
        fill(self.w_in[n: n + s.kv_rank + s.rot_dim], get(prefix + "dkv"), prefix + "dkv")
        fill(self.norm, get(prefix + "dkv.norm"), prefix + "dkv.norm")
        key, value = (get(prefix + name).view(s.heads, -1, s.kv_rank) for name in ("uk", "uv"))
        fill(self.w_key[:, :, : s.dim], key.transpose(1, 2), prefix + "uk")
        fill(self.w_value[:, :, : s.kv_rank], value, prefix + "uv")
        if self.remake:
            fill(self.k_made[:, : s.dim, : s.kv_rank], key, prefix + "uk")
            self.k_made[:, s.dim: s.dim + s.rot_dim, s.kv_rank: s.kv_rank + s.rot_dim] = torch.eye(s.rot_dim).to(self.k_made)
            fill(self.v_made[:, : s.vdim, : s.kv_rank], value, prefix + "uv")
        fill(self.w_out, get(prefix + "o"), prefix + "o")

    def _per_head(self, rows: int, device, keep: bool) -> ops.ExpertChoice:
        """Products per head as products per expert: every row uses every head.  (``keep``: a captured graph may hold them.)"""
        if rows in self._lists:
            return self._lists[rows]
        h = self.spec.heads
        lists = (torch.arange(rows, dtype=torch.int32, device=device)[None] * h +
                 torch.arange(h, dtype=torch.int32, device=device)[:, None]).contiguous()
        choice = ops.ExpertChoice(lists.view(rows, h), torch.empty(0, device=device),
                                  torch.full((h,), rows, dtype=torch.int32, device=device), lists)
        if keep:
            self._lists[rows] = choice
        return choice

    def _over_latents(self, q: Tensor, step: StepRows, part: str) -> Tensor:
        s, rows, packed = self.spec, q.shape[0], step.packed
        choice = self._per_head(rows, q.device, part == "decodes")
        over = ops.moe_product(q.view(rows * s.heads, -1)[:, : s.dim], choice, self.w_key, s.kv_rank, s.dim, glu=False)
        o = self.backend.attend_scored((over.view(rows, s.heads, s.kv_rank), q[..., s.dim: s.dim + s.rot_dim]),
                                       self.site.places[step.turn], packed, s.kv_rank, _LN2, s.window or 0, part=part)
        return ops.moe_product(o.view(rows * s.heads, s.kv_rank), choice, self.w_value, s.vdim, s.kv_rank, glu=False).view(rows, -1)

    def mix(self, u: Tensor, step: StepRows, out: Optional[Tensor] = None) -> Tensor:
        s, packed = self.spec, step.packed
        pool, _ = self.backend._layer(self.site.places[step.turn])
        # (q carries scale * log2(e) from its 32-bit registers)
        q = ops.latent_append(u, packed.rows, packed.slots, pool, self.norm, self.eps,
                              self.site.rotary.get(s.rot_base, s.rot_dim, 1.0, s.rot_yarn), s.heads, s.dim, s.rot_dim, s.kv_rank, s.made[0], s.scale / _LN2)
        nd = packed.num_decodes
        if packed.chunks is None:
            o = self._over_latents(q, step, "decodes")
            return o if out is None else out.copy_(o)
        if self.remake:
            stretch = self.backend.stretch(packed, s.window or 0)
            rows = ops.latent_gather(pool, stretch.slots)
            k, v = (F.linear(rows, w.view(-1, s.pool_row)).view(-1, s.heads, w.shape[1]) for w in (self.k_made, self.v_made))
            o = self.backend.attend_stretch(q, k, v, stretch, _LN2, s.window or 0, q.new_empty(u.shape[0], s.heads, v.shape[2]))
            if out is None and v.shape[2] == s.vdim:
                out = o.view(u.shape[0], -1)
            else:
                if out is None:
                    out = torch.empty((u.shape[0], s.heads * s.vdim), dtype=u.dtype, device=u.device)
                ops.head_gate(o[nd:], None, s.vdim, out=out[nd:])
        else:
            o = self._over_latents(q, step, "chunks")
            out = o if out is None else out.copy_(o)
        if nd:
            out[:nd] = self._over_latents(q[:nd], step, "decodes")
        return out


class TalkingAttention(Mixer):
    @staticmethod
    def sizes(spec: TalkingSpec) -> Tuple[int, int]:
        return _pad8(spec.channels + spec.heads), spec.heads * spec.vdim

    def __init__(self, spec: TalkingSpec, site: Site, slices: Slices = None, out_scale: float = 1.0) -> None:
        """Rows of ``w_in``: q, k, v, head gates, padding."""
        super().__init__(*self.sizes(spec), site, slices, out_scale)
        self.spec = spec
        self.bias = site.constant(spec.channels)
        self.bias_size, self.bias_rate = site.constant(spec.heads), site.constant(spec.heads)
        self.talk = site.constant(spec.heads, spec.heads)

    def load(self, get: Getter, prefix: str) -> None:
        s, at = self.spec, 0
        for name, n in (("q", s.heads * s.dim), ("k", s.kv_heads * s.dim), ("v", s.kv_heads * s.vdim)):
            fill(self.w_in[at: at + n], get(prefix + name), prefix + name)
            fill(self.bias[at: at + n], get(f"{prefix}{name}.b"), f"{prefix}{name}.b")
            at += n
        fill(self.w_in[at: at + s.heads], get(prefix + "g"), prefix + "g")
        fill(self.bias_size, get(prefix + "r1"), prefix + "r1")
        fill(self.bias_rate, get(prefix + "r2"), prefix + "r2")
        fill(self.talk, get(prefix + "talk"), prefix + "talk")
        fill(self.w_out, get(prefix + "o"), prefix + "o")

    def mix(self, u: Tensor, step: StepRows, out: Optional[Tensor] = None) -> Tensor:
        s, packed, place = self.spec, step.packed, self.site.places[step.turn]
        kc, vc = self.backend._layer(place)
        q = ops.qkv_conv_append(u, packed.rows, packed.slots, kc, vc, s.heads, s.dim, s.vdim, 1.0, 0.0, False, None, 0, None, None,
                                bias=self.bias)
        # (q and the pool hold zeros between dim and its next multiple of 8)
        o = self.backend.attend_talking(q[..., : _pad8(s.dim)], place, packed, s.vdim, s.scale, self.talk, self.bias_size, self.bias_rate)
        return ops.head_gate(o, u[:, s.channels: s.channels + s.heads], s.vdim, self.out_scale, out)


class Hgrn2Mixer(Mixer):
    @staticmethod
    def sizes(spec: Hgrn2Spec) -> Tuple[int, int]:
        inner = spec.heads * spec.vdim
        return _pad8(2 * spec.heads * spec.dim + inner), inner

    def __init__(self, spec: Hgrn2Spec, site: Site, slices: Slices = None, out_scale: float = 1.0) -> None:
        """Rows of ``w_in``: q, forget logits, v, padding."""
        super().__init__(*self.sizes(spec), site, slices, out_scale)
        self.spec = spec
        self.f_bias, self.lower = (site.constant(spec.heads * spec.dim) for _ in range(2))
        self.norm = site.constant(spec.heads * spec.vdim)  # one head's weights, for every head, times out_scale
        self.state = site.keep("hgrn2", (spec.heads, _pad16(spec.dim), _pad16(spec.vdim)), torch.float32)

    def _parts(self) -> Tuple[Tuple[str, int], ...]:
        s = self.spec
        return ("q", s.heads * s.dim), ("f", s.heads * s.dim), ("v", s.heads * s.vdim)

    def load(self, get: Getter, prefix: str) -> None:
        at = 0
        for name, n in self._parts():
            fill(self.w_in[at: at + n], get(prefix + name), prefix + name)
            at += n
        fill(self.f_bias, get(prefix + "f.b"), prefix + "f.b")
        fill(self.lower, get(prefix + "lower"), prefix + "lower")
        fill(self.norm, get(prefix + "norm").repeat(self.spec.heads), prefix + "norm")
        self.norm.mul_(self.out_scale)
        fill(self.w_out, get(prefix + "o"), prefix + "o")

    def mix(self, u: Tensor, step: StepRows, out: Optional[Tensor] = None) -> Tensor:
        s, packed = self.spec, step.packed
        sizes = [n for _, n in self._parts()]
        q, f, v = u[:, : sum(sizes)].split(sizes, dim=1)
        o = torch.empty((u.shape[0], s.heads * s.vdim), dtype=u.dtype, device=u.device)
        tail = (self.state[step.turn], s.heads, s.dim, s.vdim)
        if packed.decodes is not None:
            n = packed.num_decodes
            ops.channel_linear(q[:n], f[:n], v[:n], self.f_bias, self.lower, packed.decodes, *tail, o[:n], q_act="silu")
        if packed.chunks is not None:
            c = packed.chunks
            need = ops.channel_linear_workspace_bytes(c.ctx_lens.numel(), s.heads, s.dim, s.vdim, c.max_q_len)
            ops.channel_linear(q, f, v, self.f_bias, self.lower, c, *tail, o, q_act="silu",
                               workspace=self.backend._scratch_for(need) if need else None)
        return ops.rms_gate(o, None, self.norm, self.eps, groups=s.heads, order=None, out=out)


class ParallelMixer(Mixer):
    SIDES = {AttentionSpec: ConvAttention, TalkingSpec: TalkingAttention, MlstmSpec: MlstmMixer, Hgrn2Spec: Hgrn2Mixer}

    def __init__(self, spec: ParallelSpec, site: Site) -> None:
        left, right = (self.SIDES[type(s)] for s in (spec.left, spec.right))
        (in_l, out_l), (in_r, out_r) = left.sizes(spec.left), right.sizes(spec.right)
        slices = None
        if spec.norms:  # (each output is normed on its own: two output products)
            slices = site.weight(in_l + in_r, site.width), None
        super().__init__(in_l + in_r, out_l + out_r, site, slices)
        self.spec, self._in, self._out = spec, in_l, out_l
        scales, outs = (spec.left_scale, spec.right_scale), (None, None)
        self.left_norm = self.right_norm = None
        if spec.norms:
            scales, outs = (1.0, 1.0), (site.weight(site.width, out_l), site.weight(site.width, out_r))
            self.left_norm, self.right_norm = site.constant(site.width), site.constant(site.width)  # times the scales
        else:
            outs = self.w_out[:, :out_l], self.w_out[:, out_l:]
        self.left = left(spec.left, site, (self.w_in[:in_l], outs[0]), scales[0])
        self.right = right(spec.right, site, (self.w_in[in_l:], outs[1]), scales[1])

    def load(self, get: Getter, prefix: str) -> None:
        self.left.load(get, prefix + "left.")
        self.right.load(get, prefix + "right.")
        if self.spec.norms:
            for norm, scale, name in ((self.left_norm, self.spec.left_scale, "left.out"), (self.right_norm, self.spec.right_scale, "right.out")):
                fill(norm, get(prefix + name), prefix + name)
                norm.mul_(scale)

    def mix(self, u: Tensor, step: StepRows, out: Optional[Tensor] = None) -> Tensor:
        if out is None:
            out = torch.empty((u.shape[0], self.w_out.shape[1]), dtype=u.dtype, device=u.device)
        self.left.mix(u[:, : self._in], step, out[:, : self._out])
        self.right.mix(u[:, self._in:], step, out[:, self._out:])
        return out

    def branch(self, h: Tensor, step: StepRows) -> Dict[str, object]:
        if not self.spec.norms:
            return super().branch(h, step)
        u = F.linear(h, self.w_in)
        left = F.linear(self.left.mix(u[:, : self._in], step), self.left.w_out)
        right = F.linear(self.right.mix(u[:, self._in:], step), self.right.w_out)
        return {"y": left, "y2": (right, self.left_norm, self.right_norm), "y_eps": self.eps}


MIXERS = {AttentionSpec: ConvAttention, BiasedAttentionSpec: BiasedAttention, LatentSpec: LatentAttention, LightningSpec: LightningMixer,
          Mamba2Spec: Mamba2Mixer, DeltaSpec: DeltaMixer, TalkingSpec: TalkingAttention, Hgrn2Spec: Hgrn2Mixer, ParallelSpec: ParallelMixer}


class GatedMLP(nn.Module):
    """``down(silu(gate h) * up h)`` with gate and up in one product.  ``branch`` returns what the residual sum adds, as
    ``pa_residual_norm`` takes it."""

    def __init__(self, width: int, inner: int, dtype: torch.dtype, device) -> None:
        super().__init__()
        self.inner = inner
        self.w_in = _param(2 * inner, width, dtype=dtype, device=device)
        self.w_out = _param(width, inner, dtype=dtype, device=device)

    def load(self, get: Getter, prefix: str) -> None:
        fill(self.w_in[: self.inner], get(prefix + "gate"), prefix + "gate")
        fill(self.w_in[self.inner:], get(prefix + "up"), prefix + "up")
        fill(self.w_out, get(prefix + "down"), prefix + "down")

    def forward(self, h: Tensor) -> Tensor:
        u = F.linear(h, self.w_in)
        return F.linear(ops.glu(u[:, : self.inner], u[:, self.inner:], "silu"), self.w_out)

    def branch(self, h: Tensor) -> Dict[str, Tensor]:
        return {"y": self(h)}


@dataclass(frozen=True)
class MLPSpec:
    """A feed-forward without a gate: ``down(act(up h))``, both products with biases."""

    inner: int
    act: str


class PlainMLP(nn.Module):
    """The biases ride on the steps behind the products: the activation's, and the residual sum."""

    def __init__(self, width: int, spec: MLPSpec, dtype: torch.dtype, device) -> None:
        super().__init__()
        self.spec = spec
        self.w_in = _param(spec.inner, width, dtype=dtype, device=device)
        self.w_out = _param(width, spec.inner, dtype=dtype, device=device)
        self.in_bias = _param(spec.inner, dtype=torch.float32, device=device)
        self.out_bias = _param(width, dtype=torch.float32, device=device)

    def load(self, get: Getter, prefix: str) -> None:
        for w, bias, name in ((self.w_in, self.in_bias, "up"), (self.w_out, self.out_bias, "down")):
            fill(w, get(prefix + name), prefix + name)
            fill(bias, get(f"{prefix}{name}.b"), f"{prefix}{name}.b")

    def branch(self, h: Tensor) -> Dict[str, Tensor]:
        act = ops.bias_act(F.linear(h, self.w_in), self.in_bias, self.spec.act)
        return {"y": F.linear(act, self.w_out), "y_bias": self.out_bias}


class TokenSide(nn.Module):
    """Per-layer token input: ``proj(gelu_tanh(gate x) * e)`` with ``e`` the layer's columns of a second embedding.
    What comes back is RMS-normed with ``norm`` as it is added to the residual."""

    def __init__(self, width: int, dim: int, layer_idx: int, dtype: torch.dtype, device) -> None:
        super().__init__()
        self.dim, self.first = dim, layer_idx * dim
        self.w_in = _param(dim, width, dtype=dtype, device=device)
        self.w_out = _param(width, dim, dtype=dtype, device=device)
        self.norm = _param(width, dtype=torch.float32, device=device)

    def load(self, get: Getter, prefix: str) -> None:
        fill(self.w_in, get(prefix + "gate"), prefix + "gate")
        fill(self.w_out, get(prefix + "proj"), prefix + "proj")
        fill(self.norm, get(prefix + "norm"), prefix + "norm")

    def forward(self, x: Tensor, ids: Tensor, table: Tensor) -> Tensor:
        g = F.linear(x, self.w_in)
        return F.linear(ops.glu(g, table[:, self.first: self.first + self.dim], "gelu_tanh", ids=ids), self.w_out)
