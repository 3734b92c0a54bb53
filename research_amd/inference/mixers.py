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
  -> ``pa_rms_gate`` -> output projection.
"""

from __future__ import annotations

import math
from dataclasses import dataclass
from typing import Callable, Dict, Optional, Tuple

import torch
import torch.nn.functional as F
from torch import Tensor, nn

from .. import ops
from .attention.hip_backend import HipPagedAttentionBackend, PackedStep

_LN2 = math.log(2.0)
DECAY_POWERS = 65  # powers 0 .. 64 of a decay, one more than the rows of a chunk

Getter = Callable[[str], Tensor]  # checkpoint tensor by name


@dataclass(frozen=True)
class AttentionSpec:
    """Softmax attention over a sliding window behind short convolutions.  ``window`` None: plain causal; ``taps`` 0:
    no convolution; ``v_mix``: the layer takes part in value mixing."""

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

    def __post_init__(self) -> None:
        if self.heads % self.kv_heads != 0:
            raise ValueError(f"heads={self.heads} is not a multiple of kv_heads={self.kv_heads}")
        if self.rot_dims % 2 or not 0 <= self.rot_dims <= self.dim:
            raise ValueError(f"rot_dims={self.rot_dims} must be even and at most dim={self.dim}")
        if self.window is not None and self.window < 1:
            raise ValueError(f"window={self.window} must be positive")
        if self.pool_dim > 256:
            raise ValueError(f"head sizes {self.dim} / {self.vdim} above 256")

    @property
    def pool_dim(self) -> int:
        """Head size of the layer's pool: holds a key or a value, in whole 8-element vectors."""
        return -(-max(self.dim, self.vdim) // 8) * 8

    @property
    def channels(self) -> int:
        return (self.heads + self.kv_heads) * self.dim + self.kv_heads * self.vdim


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


class RotaryTables:
    """(cos, sin) per position and pair, float32 from float64 angles; one table per (base, dims, factor), shared by the
    layers that name it.  The position limit is fixed once a captured graph may hold a table's address."""

    def __init__(self, max_positions: int, device) -> None:
        self.max_positions = max_positions
        self.device = device
        self._tables: Dict[Tuple[float, int, float], Tensor] = {}

    def get(self, base: float, dims: int, factor: float) -> Optional[Tensor]:
        if dims == 0:
            return None
        key = (base, dims, factor)
        if key not in self._tables:
            freq = base ** (-torch.arange(0, dims, 2, dtype=torch.float64) / dims) / factor
            angle = torch.arange(self.max_positions, dtype=torch.float64)[:, None] * freq[None, :]
            table = torch.stack([angle.cos(), angle.sin()], dim=-1).float()
            self._tables[key] = table.contiguous().to(self.device)
        return self._tables[key]


@dataclass
class StepRows:
    """What one forward pass shares between its layers."""

    packed: PackedStep
    ids: Tensor
    v_first: Optional[Tensor] = None


def _param(*shape: int, dtype: torch.dtype, device) -> nn.Parameter:
    return nn.Parameter(torch.zeros(shape, dtype=dtype, device=device), requires_grad=False)


def fill(dst: Tensor, src: Tensor, name: str) -> None:
    if tuple(dst.shape) != tuple(src.shape):
        raise ValueError(f"{name}: checkpoint shape {tuple(src.shape)}, expected {tuple(dst.shape)}")
    dst.copy_(src)


class ConvAttention(nn.Module):
    def __init__(self, spec: AttentionSpec, width: int, eps: float, layer_idx: int, backend: HipPagedAttentionBackend,
                 rotary: RotaryTables, v_role: Optional[str], dtype: torch.dtype, device) -> None:
        """``v_role``: None, "first" (the layer whose values the others mix in) or "mix"."""
        super().__init__()
        self.spec, self.eps, self.layer_idx, self.backend, self.v_role = spec, eps, layer_idx, backend, v_role
        self.rotary = rotary
        rows = spec.channels + spec.heads
        self.w_in = _param(-(-rows // 8) * 8, width, dtype=dtype, device=device)  # q, k, v, head gates, padding
        self.w_out = _param(width, spec.heads * spec.vdim, dtype=dtype, device=device)
        self.conv = _param(spec.taps, spec.channels, dtype=torch.float32, device=device) if spec.taps else None
        self.v_lambda = _param(1, dtype=torch.float32, device=device)
        self.conv_state = None
        if spec.taps > 1:
            self.conv_state = backend.register_state(layer_idx, "conv", (spec.taps - 1, spec.channels), dtype)

    def load(self, get: Getter, prefix: str) -> None:
        s, at = self.spec, 0
        for name, n in (("q", s.heads * s.dim), ("k", s.kv_heads * s.dim), ("v", s.kv_heads * s.vdim)):
            fill(self.w_in[at: at + n], get(prefix + name), prefix + name)
            if self.conv is not None:
                fill(self.conv[:, at: at + n], get(f"{prefix}{name}.conv").t(), f"{prefix}{name}.conv")
            at += n
        fill(self.w_in[at: at + s.heads], get(prefix + "g"), prefix + "g")
        fill(self.w_out, get(prefix + "o"), prefix + "o")
        if self.v_role == "mix":
            fill(self.v_lambda, get(prefix + "vmix").reshape(1), prefix + "vmix")

    def forward(self, h: Tensor, step: StepRows) -> Tensor:
        s, packed = self.spec, step.packed
        u = F.linear(h, self.w_in)
        if self.v_role == "first":
            step.v_first = torch.empty((h.shape[0], s.kv_heads * s.vdim), dtype=h.dtype, device=h.device)
        kc, vc = self.backend._layer(self.layer_idx)
        # q carries scale * log2(e) from its 32-bit registers, so that the attention kernels' own factor is one
        q = ops.qkv_conv_append(u, packed.rows, packed.slots, kc, vc, s.heads, s.dim, s.vdim, s.scale / _LN2, self.eps, True,
                                self.rotary.get(s.rot_base, s.rot_dims, s.rot_factor), s.rot_dims, self.conv, self.conv_state,
                                self.v_role, step.v_first if self.v_role else None,
                                self.v_lambda if self.v_role == "mix" else None)
        o = self.backend.attend_packed(q, self.layer_idx, packed, _LN2, s.window or 0)
        o = ops.head_gate(o, u[:, s.channels: s.channels + s.heads], s.vdim)
        return F.linear(o, self.w_out)


class LightningMixer(nn.Module):
    def __init__(self, spec: LightningSpec, width: int, eps: float, layer_idx: int, backend: HipPagedAttentionBackend,
                 dtype: torch.dtype, device) -> None:
        super().__init__()
        self.spec, self.eps, self.backend = spec, eps, backend
        inner = spec.heads * spec.vdim
        rows = spec.heads * 2 * spec.dim + 2 * inner
        self.w_in = _param(-(-rows // 8) * 8, width, dtype=dtype, device=device)  # q, k, v, output gate, padding
        self.w_out = _param(width, inner, dtype=dtype, device=device)
        self.norm = _param(inner, dtype=torch.float32, device=device)
        pad = lambda n: -(-n // 16) * 16
        self.state = backend.register_state(layer_idx, "lightning", (spec.heads, pad(spec.dim), pad(spec.vdim)), torch.float32)
        powers = torch.tensor(spec.decay, dtype=torch.float64)[:, None] ** torch.arange(DECAY_POWERS, dtype=torch.float64)
        self.register_buffer("decay_powers", powers.float().to(device).contiguous(), persistent=False)

    def load(self, get: Getter, prefix: str) -> None:
        s, at = self.spec, 0
        for name, n in (("q", s.heads * s.dim), ("k", s.heads * s.dim), ("v", s.heads * s.vdim), ("g", s.heads * s.vdim)):
            fill(self.w_in[at: at + n], get(prefix + name), prefix + name)
            at += n
        fill(self.w_out, get(prefix + "o"), prefix + "o")
        fill(self.norm, get(prefix + "norm"), prefix + "norm")

    def forward(self, h: Tensor, step: StepRows) -> Tensor:
        s, packed = self.spec, step.packed
        u = F.linear(h, self.w_in)
        inner = s.heads * s.vdim
        o = torch.empty((h.shape[0], inner), dtype=h.dtype, device=h.device)
        nd = packed.num_decodes
        if packed.decodes is not None:
            ops.lightning(u[:nd], packed.decodes, self.state, self.decay_powers, s.heads, s.dim, s.vdim, o[:nd])
        if packed.chunks is not None:
            c = packed.chunks
            need = ops.lightning_workspace_bytes(c.ctx_lens.numel(), s.heads, s.dim, s.vdim, c.max_q_len)
            ops.lightning(u, c, self.state, self.decay_powers, s.heads, s.dim, s.vdim, o,
                          workspace=self.backend._workspace_for(need) if need else None)
        g = 2 * s.heads * s.dim + inner
        o = ops.rms_gate(o, u[:, g: g + inner], self.norm, self.eps)
        return F.linear(o, self.w_out)


class GatedMLP(nn.Module):
    """``down(silu(gate h) * up h)`` with gate and up in one product."""

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
