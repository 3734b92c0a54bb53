"""CPU restatement of the Loluzen design.  TEST INFRASTRUCTURE.

Nothing in the product imports this file, and it imports nothing of the product.  One plain, slow function per mechanism,
whole sequences only, in the type of its inputs (the tests use float64): no cache, no state carried between calls, no
chunks of rows.  ``decoder_forward`` strings them together for a configuration given as the plain dictionary of a
``config.json`` and a dictionary of weights under their checkpoint names.

Shapes: ``T`` tokens of one sequence; ``x [T, width]``.

How the functions are pinned (tests/test_oracle_loluzen.py): the rotation by complex multiplication, the frequencies by
their three ranges, attention by ``scaled_dot_product_attention`` with an explicit bias, mixed weights by one matrix per
row, the recurrence by its unrolled products, the convolution by ``torch.nn.functional.conv1d``.
"""

from __future__ import annotations

import math
from typing import Dict, List, Optional, Tuple

import torch

Tensor = torch.Tensor


def rms_norm(x: Tensor, eps: float) -> Tensor:
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def shifted_norm(x: Tensor, w: Tensor, eps: float) -> Tensor:
    """The weight is stored around zero."""
    return rms_norm(x, eps) * (1 + w)


def sigmoid(x: Tensor) -> Tensor:
    return 1 / (1 + torch.exp(-x))


def silu(x: Tensor) -> Tensor:
    return x * sigmoid(x)


def linear(h: Tensor, w: Dict[str, Tensor], name: str) -> Tensor:
    """With the bias where the checkpoint has one."""
    y = h @ w[name].T
    return y + w[name + ".b"] if name + ".b" in w else y


# ------------------------------------------------------------------ attention


def causal_conv(u: Tensor, w: Tensor) -> Tensor:
    """``u [T, C]``, ``w [C, taps]``: the last column weighs the current row; zeros before the start."""
    taps = w.shape[1]
    padded = torch.cat([torch.zeros(taps - 1, u.shape[1], dtype=u.dtype), u])
    return sum(w[:, j] * padded[j: j + u.shape[0]] for j in range(taps))


def pair_turns(rot: dict) -> List[float]:
    """Radians per position of every rotated pair: pairs that turn fast keep theirs, slow ones are divided by ``factor``, with
    a ramp in the number of turns over the original length between them."""
    dims, s = rot["dims"], rot.get("scaling")
    freq = [rot["base"] ** (-2.0 * i / dims) for i in range(dims // 2)]
    if not s:
        return freq
    out = []
    for f in freq:
        length = 2 * math.pi / f
        if length < s["original"] / s["high"]:
            out.append(f)
        elif length > s["original"] / s["low"]:
            out.append(f / s["factor"])
        else:
            part = (s["original"] / length - s["low"]) / (s["high"] - s["low"])
            out.append((1 - part) * f / s["factor"] + part * f)
    return out


def rotate_pairs(x: Tensor, rot: dict) -> Tensor:
    """``x [T, heads, dim]``: dimensions 2i and 2i + 1 turn together, those past the rotated ones pass."""
    freq = pair_turns(rot)
    ang = torch.arange(x.shape[0], dtype=torch.float64)[:, None] * torch.tensor(freq, dtype=torch.float64)
    c, s = (f(ang).to(x.dtype)[:, None, :] for f in (torch.cos, torch.sin))
    n = 2 * len(freq)
    u, v = x[..., 0: n: 2], x[..., 1: n: 2]
    out = x.clone()
    out[..., 0: n: 2] = u * c - v * s
    out[..., 1: n: 2] = v * c + u * s
    return out


def causal_attention(q: Tensor, k: Tensor, v: Tensor, scale: float, bias: Optional[Tensor] = None,
                     talk: Optional[Tensor] = None) -> Tensor:
    """``q [T, H, D]``, ``k [T, G, D]``, ``v [T, G, E]`` -> ``[T, H, E]``.  ``bias [H, T]`` is added to the scores by
    distance; ``talk [H, H]`` mixes the heads' weights before they meet the values."""
    t_len, heads, _ = q.shape
    group = heads // k.shape[1]
    of = torch.arange(heads) // group
    out = torch.zeros(t_len, heads, v.shape[2], dtype=q.dtype)
    keys, values = k[:, of], v[:, of]
    for i in range(t_len):
        s = (q[i] * keys[: i + 1]).sum(-1).T * scale  # [H, keys]
        if bias is not None:
            s = s + bias[:, : i + 1].flip(1)
        p = torch.exp(s - s.max(-1, keepdim=True).values)
        p = p / p.sum(-1, keepdim=True)
        if talk is not None:
            p = talk @ p
        out[i] = (p.T[:, :, None] * values[: i + 1]).sum(0)
    return out


def distance_bias(r1: Tensor, r2: Tensor, distances: int) -> Tensor:
    """``[H, distances]``: what is added to the score of a key that many positions back."""
    n = torch.arange(distances, dtype=r1.dtype)
    return -r1[:, None] * torch.log(1 + r2[:, None] * n)


def gate_heads(o: Tensor, h: Tensor, w: Tensor) -> Tensor:
    return o * sigmoid(h @ w.T)[:, :, None]


def attention_mixer(h: Tensor, w: Dict[str, Tensor], p: str, m: dict, eps: float) -> Tensor:
    t_len, heads, groups, dim, vdim = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (linear(h, w, p + n) for n in "qkv")
    if m.get("conv"):
        q, k, v = (causal_conv(u, w[f"{p}{n}.conv"]) for u, n in ((q, "q"), (k, "k"), (v, "v")))
    q = rms_norm(q.view(t_len, heads, dim), eps) * w[p + "q.norm"]
    k = rms_norm(k.view(t_len, groups, dim), eps) * w[p + "k.norm"]
    if m.get("rot"):
        q, k = rotate_pairs(q, m["rot"]), rotate_pairs(k, m["rot"])
    o = causal_attention(q, k, v.view(t_len, groups, vdim), m["scale"])
    return gate_heads(o, h, w[p + "g"]).reshape(t_len, -1) @ w[p + "o"].T


def talking_mixer(h: Tensor, w: Dict[str, Tensor], p: str, m: dict) -> Tensor:
    t_len, heads, groups, dim, vdim = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (linear(h, w, p + n) for n in "qkv")
    o = causal_attention(q.view(t_len, heads, dim), k.view(t_len, groups, dim), v.view(t_len, groups, vdim), m["scale"],
                         distance_bias(w[p + "r1"], w[p + "r2"], t_len), w[p + "talk"])
    return gate_heads(o, h, w[p + "g"]).reshape(t_len, -1) @ w[p + "o"].T


# ------------------------------------------------------------------ HGRN2


def bounded_forget(logits: Tensor, lower: Tensor) -> Tensor:
    return lower + (1 - lower) * sigmoid(logits)


def channel_recurrence(q: Tensor, f: Tensor, v: Tensor, state: Optional[Tensor] = None) -> Tuple[Tensor, Tensor]:
    """``q, f [T, H, D]``, ``v [T, H, E]``: a factor per row of the state, whose complement is written.  ``[T, H, E]`` and the
    last state ``[H, D, E]``."""
    t_len, heads, d = q.shape
    s = torch.zeros(heads, d, v.shape[2], dtype=q.dtype) if state is None else state.clone()
    out = torch.zeros(t_len, heads, v.shape[2], dtype=q.dtype)
    for t in range(t_len):
        s = f[t][:, :, None] * s + (1 - f[t])[:, :, None] * v[t][:, None, :]
        out[t] = (s * q[t][:, :, None]).sum(1)
    return out, s


def hgrn2_mixer(h: Tensor, w: Dict[str, Tensor], p: str, m: dict, eps: float) -> Tensor:
    t_len, heads, dim, vdim = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = silu(h @ w[p + "q"].T).view(t_len, heads, dim)
    f = bounded_forget(linear(h, w, p + "f"), w[p + "lower"]).view(t_len, heads, dim)
    o, _ = channel_recurrence(q, f, (h @ w[p + "v"].T).view(t_len, heads, vdim))
    return (rms_norm(o, eps) * w[p + "norm"]).reshape(t_len, -1) @ w[p + "o"].T


def parallel_mixer(h: Tensor, w: Dict[str, Tensor], p: str, m: dict, eps: float) -> Tensor:
    left = talking_mixer(h, w, p + "left.", m["left"])
    right = hgrn2_mixer(h, w, p + "right.", m["right"], eps)
    return (rms_norm(left, eps) * w[p + "left.out"] + rms_norm(right, eps) * w[p + "right.out"]) / 2


# ------------------------------------------------------------------ model


def square_relu_mlp(h: Tensor, w: Dict[str, Tensor], p: str) -> Tensor:
    return linear(torch.clamp(linear(h, w, p + "up"), min=0) ** 2, w, p + "down")


def layer_runs(cfg: dict) -> List[Tuple[int, bool]]:
    """(layer, whether the embedding is added ahead of it) of every run, in order."""
    n, loop = len(cfg["layers"]), cfg.get("loop") or {"start": 0, "stop": 0, "times": 1}
    runs = [(i, False) for i in range(loop["start"])]
    for turn in range(loop["times"]):
        runs += [(i, turn > 0 and i == loop["start"]) for i in range(loop["start"], loop["stop"])]
    return runs + [(i, False) for i in range(loop["stop"], n)]


def decoder_forward(weights: Dict[str, Tensor], cfg: dict, tokens: List[int], dtype: torch.dtype = torch.float64,
                    trace: Optional[List[Tensor]] = None) -> Tensor:
    """Logits ``[T, vocab]`` of one sequence from its start; ``trace`` collects the residual after every layer run."""
    w = {k: v.to(dtype) for k, v in weights.items()}
    eps, mult = cfg["norm"]["eps"], cfg["residual_mult"]
    x = start = w["embed"][torch.tensor(tokens)] * cfg["embedding"]["scale"]
    for i, again in layer_runs(cfg):
        layer, p = cfg["layers"][i], f"l{i}."
        if again:
            x = x + start
        mixer = {"attention": attention_mixer, "parallel": parallel_mixer}[layer["type"]]
        y = mixer(shifted_norm(x, w[p + "norm1"], eps), w, p + "mix.", layer["mixer"], eps)
        x = x + mult * shifted_norm(y, w[p + "norm1b"], eps)
        if layer.get("mlp") is not None:
            y = square_relu_mlp(shifted_norm(x, w[p + "norm2"], eps), w, p + "mlp.")
            x = x + mult * shifted_norm(y, w[p + "norm2b"], eps)
        if trace is not None:
            trace.append(x)
    return shifted_norm(x, w["final.norm"], eps) @ w["head"].T
