"""Mixture-of-experts feed-forward.

Every token uses ``top`` of the experts, chosen by sigmoid scores, optionally only
among the best groups of experts; a shared expert may run for every token.  The
step stays on the device from the router to the weighted sum:

``pa_narrow_linear`` (router logits and the shared expert's gate, 32-bit) ->
``pa_moe_choose`` -> ``pa_moe_product`` with the gated
activation in its epilogue -> ``pa_moe_product``; the weighted sum over a token's
experts is part of the residual sum that follows (``pa_residual_norm``).
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import Dict, Optional

import torch
from torch import Tensor, nn

from .. import ops
from .mixers import GatedMLP, Getter, _param, fill


@dataclass(frozen=True)
class MoESpec:
    """``keep`` of ``groups`` equal groups of neighbouring experts can be chosen from; ``shared``: inner width of the expert
    that every token uses, None: there is none."""

    experts: int
    ff: int
    top: int
    groups: int = 1
    keep: int = 1
    shared: Optional[int] = None

    def __post_init__(self) -> None:
        if self.groups < 1 or self.experts % self.groups:
            raise ValueError(f"{self.experts} experts are not {self.groups} equal groups")
        if not 1 <= self.keep <= self.groups or not 1 <= self.top <= self.keep * (self.experts // self.groups):
            raise ValueError(f"top={self.top} experts cannot be chosen from keep={self.keep} of {self.groups} groups")
        if self.experts > 1024 or self.top > 64:
            raise ValueError(f"experts={self.experts} above 1024 or top={self.top} above 64")


def _pad64(n: int) -> int:
    return -(-n // 64) * 64


class MoE(nn.Module):
    def __init__(self, spec: MoESpec, width: int, dtype: torch.dtype, device) -> None:
        super().__init__()
        self.spec, self.width = spec, width
        self.inner = _pad64(spec.ff)  # (whole steps of the product kernels: the columns past ff are zeros)
        kw = dict(dtype=dtype, device=device)
        self.router = _param(spec.experts + (spec.shared is not None), width, **kw)  # the last row: the shared expert's gate
        self.w_in = _param(spec.experts, 2 * self.inner, _pad64(width), **kw)
        self.w_out = _param(spec.experts, width, self.inner, **kw)
        self.shared = GatedMLP(width, spec.shared, dtype, device) if spec.shared is not None else None

    def load(self, get: Getter, prefix: str) -> None:
        s = self.spec
        fill(self.router[: s.experts], get(prefix + "router"), prefix + "router")
        for e in range(s.experts):
            at = f"{prefix}e{e}."
            fill(self.w_in[e, : s.ff, : self.width], get(at + "gate"), at + "gate")
            fill(self.w_in[e, self.inner: self.inner + s.ff, : self.width], get(at + "up"), at + "up")
            fill(self.w_out[e, :, : s.ff], get(at + "down"), at + "down")
        if self.shared is not None:
            fill(self.router[s.experts:], get(prefix + "shared.sg"), prefix + "shared.sg")
            self.shared.load(get, prefix + "shared.")

    def branch(self, h: Tensor) -> Dict[str, Tensor]:
        s = self.spec
        choice = ops.moe_choose(ops.narrow_linear(h, self.router), s.experts, s.top, s.groups, s.keep)
        act = ops.moe_product(h, choice, self.w_in, self.inner, self.width, glu=True)
        out = {"y": ops.moe_product(act, choice, self.w_out, self.width, self.inner, glu=False), "mix": choice.weights}
        if self.shared is not None:
            out["y_extra"] = self.shared(h)
        return out
