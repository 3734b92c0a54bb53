"""Mixture-of-experts feed-forward.

Every token uses ``top`` of the experts, chosen by sigmoid or softmax scores (with a
correction that only chooses), optionally only among the best groups of experts;
some may be identity experts, which hand on their input; a shared expert may run
for every token, with or without a gate.  The step stays on the device from the router to the weighted sum:

``pa_narrow_linear`` (router logits and a shared expert's gate, 32-bit) ->
``pa_moe_choose`` -> ``pa_moe_product`` with the gated
activation in its epilogue -> ``pa_moe_product``; the weighted sum over a token's
experts is part of the residual sum that follows (``pa_residual_norm``,
``pa_hyper_norm``).
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
    that every token uses, None: there is none, ``shared_gate``: weighed by a gate of its own.  ``identity``: identity experts
    behind the ``experts``, chosen like them.  A group is as good as its ``group_top`` best choice scores together;
    ``correction``: per-expert terms of the choice scores; ``renormalize``: the chosen scores are divided by their sum."""

    experts: int
    ff: int
    top: int
    groups: int = 1
    keep: int = 1
    shared: Optional[int] = None
    shared_gate: bool = True
    identity: int = 0
    scores: str = "sigmoid"  # | "softmax"
    group_top: int = 2
    correction: bool = False
    renormalize: bool = True

    def __post_init__(self) -> None:
        if self.experts < 1 or self.identity < 0 or self.groups < 1 or self.routed % self.groups:
            raise ValueError(f"{self.routed} experts are not {self.groups} equal groups")
        if not 1 <= self.keep <= self.groups or not 1 <= self.top <= self.keep * (self.routed // self.groups):
            raise ValueError(f"top={self.top} experts cannot be chosen from keep={self.keep} of {self.groups} groups")
        if self.routed > 1024 or self.top > 64:
            raise ValueError(f"experts={self.routed} above 1024 or top={self.top} above 64")

    @property
    def routed(self) -> int:
        return self.experts + self.identity


def _pad64(n: int) -> int:
    return -(-n // 64) * 64


class MoE(nn.Module):
    def __init__(self, spec: MoESpec, width: int, dtype: torch.dtype, device) -> None:
        super().__init__()
        self.spec, self.width = spec, width
        self.inner = _pad64(spec.ff)  # (whole steps of the product kernels: the columns past ff are zeros)
        kw = dict(dtype=dtype, device=device)
        self.gated = spec.shared is not None and spec.shared_gate
        self.router = _param(spec.routed + self.gated, width, **kw)  # the last row: the shared expert's gate
        self.correction = _param(spec.routed, dtype=torch.float32, device=device) if spec.correction else None
        self.w_in = _param(spec.experts, 2 * self.inner, _pad64(width), **kw)
        self.w_out = _param(spec.experts, width, self.inner, **kw)
        self.shared = GatedMLP(width, spec.shared, dtype, device) if spec.shared is not None else None

    def load(self, get: Getter, prefix: str) -> None:
        s = self.spec
        fill(self.router[: s.routed], get(prefix + "router"), prefix + "router")
        if self.correction is not None:
            fill(self.correction, get(prefix + "correction"), prefix + "correction")
        for e in range(s.experts):
            at = f"{prefix}e{e}."
            fill(self.w_in[e, : s.ff, : self.width], get(at + "gate"), at + "gate")
            fill(self.w_in[e, self.inner: self.inner + s.ff, : self.width], get(at + "up"), at + "up")
            fill(self.w_out[e, :, : s.ff], get(at + "down"), at + "down")
        if self.gated:
            fill(self.router[s.routed:], get(prefix + "shared.sg"), prefix + "shared.sg")
        if self.shared is not None:
            self.shared.load(get, prefix + "shared.")

    def branch(self, h: Tensor) -> Dict[str, Tensor]:
        s = self.spec
        shared = None if self.shared is None else "gated" if self.gated else "plain"
        choice = ops.moe_choose(ops.narrow_linear(h, self.router), s.experts, s.top, s.groups, s.keep, shared, s.identity, s.scores,
                                s.group_top, s.renormalize, self.correction)
        act = ops.moe_product(h, choice, self.w_in, self.inner, self.width, glu=True)
        out = {"y": ops.moe_product(act, choice, self.w_out, self.width, self.inner, glu=False), "mix": choice.weights}
        if self.shared is not None:
            out["y_extra"] = self.shared(h)
        if s.identity:
            out["y_self"] = h
        return out
