"""CPU restatement of the hybrid decoder family (window attention and lightning attention).  TEST INFRASTRUCTURE.

Nothing in the product imports this file, and it imports nothing of the product.  One plain, slow function per
mechanism, whole sequences only, in the type of its inputs (the tests use float64 or float32): no cache, no state
carried between calls, no chunks.  ``decoder_forward`` strings them together for a configuration given as the plain
dictionary of a ``config.json`` and a dictionary of weights under their checkpoint names.

Shapes: ``T`` tokens of one sequence; ``x [T, width]``.

How the functions are pinned (tests/test_oracle_hybrid.py): the convolution by ``torch.nn.functional.conv1d``, the
rotation by complex multiplication, the softmax attention by ``scaled_dot_product_attention`` with an explicit mask,
lightning attention by its unrolled sum, the norms by torch's own.
"""

from __future__ import annotations

import math
from typing import Dict, List, Optional, Tuple

import torch

Tensor = torch.Tensor


def layer_norm(x: Tensor, w: Tensor, b: Tensor, eps: float) -> Tensor:
    mean = x.mean(-1, keepdim=True)
    dev = x - mean
    return dev / torch.sqrt((dev * dev).mean(-1, keepdim=True) + eps) * w + b


def unit_rms(x: Tensor, eps: float) -> Tensor:
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def silu(x: Tensor) -> Tensor:
    return x / (1 + torch.exp(-x))


def sigmoid(x: Tensor) -> Tensor:
    return 1 / (1 + torch.exp(-x))


def gelu_tanh(x: Tensor) -> Tensor:
    return 0.5 * x * (1 + torch.tanh(math.sqrt(2 / math.pi) * (x + 0.044715 * x ** 3)))


def causal_conv(u: Tensor, w: Tensor) -> Tensor:
    """``u [T, C]``, ``w [C, taps]``: y[t] = sum over j of w[:, j] u[t - taps + 1 + j]; nothing before the start."""
    taps = w.shape[1]
    y = torch.zeros_like(u)
    for t in range(u.shape[0]):
        for j in range(taps):
            src = t - taps + 1 + j
            if src >= 0:
                y[t] += w[:, j] * u[src]
    return y


def rotate_interleaved(x: Tensor, base: float, dims: int, factor: float) -> Tensor:
    """``x [T, heads, dim]``; the pair (2i, 2i+1) of the first ``dims`` dimensions turns by t base^(-2i/dims) / factor."""
    out = x.clone()
    for t in range(x.shape[0]):
        for i in range(dims // 2):
            a = t * base ** (-2 * i / dims) / factor
            c, s = math.cos(a), math.sin(a)
            u, v = x[t, :, 2 * i], x[t, :, 2 * i + 1]
            out[t, :, 2 * i] = u * c - v * s
            out[t, :, 2 * i + 1] = v * c + u * s
    return out


def window_attention(q: Tensor, k: Tensor, v: Tensor, scale: float, window: Optional[int]) -> Tensor:
    """``q [T, H, D]``, ``k [T, G, D]``, ``v [T, G, E]`` -> ``[T, H, E]``; row i sees j with 0 <= i - j < window."""
    t_len, heads, _ = q.shape
    group = heads // k.shape[1]
    out = torch.zeros(t_len, heads, v.shape[2], dtype=q.dtype)
    for i in range(t_len):
        lo = 0 if window is None else max(0, i - window + 1)
        for h in range(heads):
            g = h // group
            s = (k[lo: i + 1, g] @ q[i, h]) * scale
            p = torch.exp(s - s.max())
            out[i, h] = (p / p.sum()) @ v[lo: i + 1, g]
    return out


def mix_values(v: Tensor, v_first: Tensor, lam: Tensor) -> Tensor:
    return (1 - lam) * v + lam * v_first


def lightning_attention(q: Tensor, k: Tensor, v: Tensor, decay: List[float],
                        state: Optional[Tensor] = None) -> Tuple[Tensor, Tensor]:
    """``q, k [T, H, D]``, ``v [T, H, E]``: S <- decay S + k v^T, o = S^T q, token by token.  Returns (o, last S)."""
    t_len, heads, d = q.shape
    s = torch.zeros(heads, d, v.shape[2], dtype=q.dtype) if state is None else state.clone()
    lam = torch.tensor(decay, dtype=q.dtype)[:, None, None]
    out = torch.zeros(t_len, heads, v.shape[2], dtype=q.dtype)
    for t in range(t_len):
        s = lam * s + k[t][:, :, None] * v[t][:, None, :]
        out[t] = (s * q[t][:, :, None]).sum(1)
    return out, s


def attention_mixer(h: Tensor, w: Dict[str, Tensor], p: str, m: dict, eps: float,
                    v_first: Optional[Tensor]) -> Tuple[Tensor, Tensor]:
    """The mixer's output ``[T, width]`` and its own values (before mixing), which the first mixing layer hands on."""
    t_len = h.shape[0]
    heads, groups, dim, vdim = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (causal_conv(h @ w[p + n].T, w[p + n + ".conv"]) for n in ("q", "k", "v"))
    q, k, v = q.view(t_len, heads, dim), k.view(t_len, groups, dim), v.view(t_len, groups, vdim)
    rot = m["rot"]
    factor = rot.get("scaling", {}).get("factor", 1.0)
    q = unit_rms(rotate_interleaved(q, rot["base"], rot["dims"], factor), eps)
    k = unit_rms(rotate_interleaved(k, rot["base"], rot["dims"], factor), eps)
    own = v
    if m["v_mix"] and v_first is not None:
        v = mix_values(v, v_first, w[p + "vmix"])
    o = window_attention(q, k, v, m["scale"], m["mask"]["size"])
    o = o * sigmoid(h @ w[p + "g"].T)[:, :, None]
    return o.reshape(t_len, heads * vdim) @ w[p + "o"].T, own


def lightning_mixer(h: Tensor, w: Dict[str, Tensor], p: str, m: dict, eps: float) -> Tensor:
    t_len = h.shape[0]
    heads, dim, vdim = m["heads"], m["dim"], m["vdim"]
    q = silu(h @ w[p + "q"].T).view(t_len, heads, dim)
    k = silu(h @ w[p + "k"].T).view(t_len, heads, dim)
    v = silu(h @ w[p + "v"].T).view(t_len, heads, vdim)
    o, _ = lightning_attention(q, k, v, m["decay"])
    o = unit_rms(o.reshape(t_len, heads * vdim), eps) * w[p + "norm"]
    return (o * sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def gated_mlp(h: Tensor, w: Dict[str, Tensor], p: str) -> Tensor:
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def token_side(x: Tensor, w: Dict[str, Tensor], p: str, e: Tensor, eps: float) -> Tensor:
    """What the per-layer token input adds to ``x``; ``e [T, dim]`` is the layer's part of the second embedding."""
    y = (gelu_tanh(x @ w[p + "gate"].T) * e) @ w[p + "proj"].T
    return unit_rms(y, eps) * w[p + "norm"]


def decoder_forward(weights: Dict[str, Tensor], cfg: dict, tokens: List[int], dtype: torch.dtype = torch.float64,
                    trace: Optional[List[Tensor]] = None) -> Tensor:
    """Logits ``[T, vocab]`` of one sequence from its start; ``trace`` collects the residual after every layer."""
    w = {k: v.to(dtype) for k, v in weights.items()}
    eps = cfg["norm"]["eps"]
    ids = torch.tensor(tokens)
    x = w["embed"][ids]
    v_first = None
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        h = layer_norm(x, w[p + "norm1"], w[p + "norm1.b"], eps)
        if layer["type"] == "attention":
            y, own = attention_mixer(h, w, p + "mix.", layer["mixer"], eps, v_first)
            if layer["mixer"]["v_mix"] and v_first is None:
                v_first = own
        else:
            y = lightning_mixer(h, w, p + "mix.", layer["mixer"], eps)
        x = x + y
        if layer["mlp"] is not None:
            x = x + gated_mlp(layer_norm(x, w[p + "norm2"], w[p + "norm2.b"], eps), w, p + "mlp.")
        if cfg.get("token_side"):
            dim = cfg["token_side"]["dim"]
            x = x + token_side(x, w, p + "side.", w["side.embed"][ids][:, i * dim: (i + 1) * dim], eps)
        if trace is not None:
            trace.append(x)
    return layer_norm(x, w["final.norm"], w["final.norm.b"], eps) @ w["head"].T
