"""CPU restatement of the Vusalix design.  TEST INFRASTRUCTURE.

Nothing in the product imports this file, and it imports nothing of the product.  One plain, slow function per mechanism,
whole sequences only, in the type of its inputs (the tests use float64): no cache, no state carried between calls, no
chunks of rows, keys and values of latent attention written out per head.  ``decoder_forward`` strings them together for
a configuration given as the plain dictionary of a ``config.json`` and a dictionary of weights under their checkpoint
names.

Shapes: ``T`` tokens of one sequence; ``x [T, width]``.

How the functions are pinned (tests/test_oracle_vusalix.py): the rotation by complex multiplication, both kinds of
attention by a softmax over explicit masks, the buckets by their thresholds, the delta rule by its product form, the
convolution by ``torch.nn.functional.conv1d``, the router by exhaustive search, the streams by one matrix per sublayer.
"""

from __future__ import annotations

import math
from typing import Dict, List, Optional, Tuple

import torch

Tensor = torch.Tensor


def rms_norm(x: Tensor, eps: float) -> Tensor:
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def sigmoid(x: Tensor) -> Tensor:
    return 1 / (1 + torch.exp(-x))


def silu(x: Tensor) -> Tensor:
    return x * sigmoid(x)


def softplus(x: Tensor) -> Tensor:
    return torch.clamp(x, min=0) + torch.log1p(torch.exp(-x.abs()))


# ------------------------------------------------------------------ latent attention


def pair_turns(rot: dict) -> Tuple[List[float], float]:
    """Radians per position of every rotated pair, and the factor on cosine and sine."""
    dims, base, s = rot["dims"], rot["base"], rot.get("scaling")
    freq = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    if not s:
        return freq, 1.0
    where = lambda turns: dims * math.log(s["original"] / (2 * math.pi * turns)) / (2 * math.log(base))
    lo, hi = max(math.floor(where(s["fast"])), 0), min(math.ceil(where(s["slow"])), dims - 1)
    ramp = [min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0) for i in range(dims // 2)]
    return [f / s["factor"] * r + f * (1 - r) for f, r in zip(freq, ramp)], 0.1 * math.log(s["factor"]) + 1


def rotate_pairs(x: Tensor, rot: dict) -> Tensor:
    """``x [T, heads, dims]``: dimensions 2i and 2i + 1 turn together."""
    freq, amp = pair_turns(rot)
    out = torch.empty_like(x)
    for t in range(x.shape[0]):
        for i, f in enumerate(freq):
            c, s = amp * math.cos(t * f), amp * math.sin(t * f)
            u, v = x[t, :, 2 * i], x[t, :, 2 * i + 1]
            out[t, :, 2 * i] = u * c - v * s
            out[t, :, 2 * i + 1] = v * c + u * s
    return out


def visible(i: int, window: Optional[int]) -> slice:
    return slice(0 if window is None else max(0, i - window + 1), i + 1)


def softmax_attention(q: Tensor, k: Tensor, v: Tensor, scale: float, window: Optional[int]) -> Tensor:
    """``q, k [T, H, D]``, ``v [T, H, E]`` -> ``[T, H, E]``."""
    out = torch.zeros(v.shape, dtype=q.dtype)
    for i in range(q.shape[0]):
        see = visible(i, window)
        s = (q[i] * k[see]).sum(-1) * scale  # [keys, H]
        p = torch.exp(s - s.max(0).values)
        out[i] = ((p / p.sum(0))[:, :, None] * v[see]).sum(0)
    return out


def latent_mixer(h: Tensor, w: Dict[str, Tensor], p: str, m: dict, eps: float) -> Tensor:
    t_len, heads, dim, rot_dim, vdim, rank = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    rot = m["rot"]
    q = (h @ w[p + "q"].T).view(t_len, heads, dim + rot_dim)
    down = h @ w[p + "dkv"].T
    c = rms_norm(down[:, :rank], eps) * w[p + "dkv.norm"]
    k_rot = rotate_pairs(down[:, rank:].reshape(t_len, 1, rot_dim), rot)
    q = torch.cat([q[..., :dim], rotate_pairs(q[..., dim:], rot)], -1)
    k = torch.cat([(c @ w[p + "uk"].T).view(t_len, heads, dim), k_rot.expand(-1, heads, -1)], -1)
    v = (c @ w[p + "uv"].T).view(t_len, heads, vdim)
    o = softmax_attention(q, k, v, m["scale"], (m.get("mask") or {}).get("size"))
    return o.reshape(t_len, heads * vdim) @ w[p + "o"].T


# ------------------------------------------------------------------ attention with distance biases


def bucket(n: int, buckets: int, most: int) -> int:
    """Half of the buckets for single distances, the others in equal steps of the logarithm up to ``most``."""
    half = buckets // 2
    if n < half:
        return n
    steps = math.log(n / half) / math.log(most / half) * (buckets - half)
    return min(buckets - 1, half + math.floor(steps + 1e-9))  # (a whole number of steps may come out just below it)


def biased_attention(q: Tensor, k: Tensor, v: Tensor, scale: float, window: Optional[int], cap: Optional[float], rel: Tensor,
                     most: int, sink: Tensor) -> Tensor:
    """``q [T, H, D]``, ``k [T, G, D]``, ``v [T, G, E]``, ``rel [buckets, H]``, ``sink [H]`` -> ``[T, H, E]``."""
    t_len, heads, _ = q.shape
    group = heads // k.shape[1]
    which = [bucket(n, rel.shape[0], most) for n in range(t_len)]
    out = torch.zeros(t_len, heads, v.shape[2], dtype=q.dtype)
    for i in range(t_len):
        see = visible(i, window)
        for h in range(heads):
            s = (k[see, h // group] @ q[i, h]) * scale
            if cap:
                s = cap * torch.tanh(s / cap)
            s = s + rel[[which[i - j] for j in range(see.start, i + 1)], h]
            top = torch.maximum(s.max(), sink[h])
            e = torch.exp(s - top)
            out[i, h] = (e / (e.sum() + torch.exp(sink[h] - top))) @ v[see, h // group]
    return out


def attention_mixer(h: Tensor, w: Dict[str, Tensor], p: str, m: dict, eps: float) -> Tensor:
    t_len = h.shape[0]
    q = (h @ w[p + "q"].T).view(t_len, m["heads"], m["dim"])
    k = (h @ w[p + "k"].T).view(t_len, m["kv_heads"], m["dim"])
    v = (h @ w[p + "v"].T).view(t_len, m["kv_heads"], m["vdim"])
    o = biased_attention(q, k, v, m["scale"], (m.get("mask") or {}).get("size"), m.get("softcap"), w[p + "rel"], m["bias_max"],
                         w[p + "sink"])
    return o.reshape(t_len, -1) @ w[p + "o"].T


# ------------------------------------------------------------------ gated delta rule


def causal_conv(u: Tensor, w: Tensor) -> Tensor:
    """``u [T, C]``, ``w [C, taps]``: the last column weighs the current row; zeros before the start."""
    taps = w.shape[1]
    padded = torch.cat([torch.zeros(taps - 1, u.shape[1], dtype=u.dtype), u])
    return sum(w[:, j] * padded[j: j + u.shape[0]] for j in range(taps))


def unit(x: Tensor) -> Tensor:
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def delta_recurrence(q: Tensor, k: Tensor, v: Tensor, log_decay: Tensor, beta: Tensor,
                     state: Optional[Tensor] = None) -> Tuple[Tensor, Tensor]:
    """``q, k [T, H, D]`` ready to use, ``v [T, H, E]``, ``log_decay, beta [T, H]`` -> ``[T, H, E]`` and the last S
    ``[H, D, E]``."""
    t_len, heads, d = q.shape
    s = torch.zeros(heads, d, v.shape[2], dtype=q.dtype) if state is None else state.clone()
    out = torch.zeros(v.shape, dtype=q.dtype)
    for t in range(t_len):
        s = torch.exp(log_decay[t])[:, None, None] * s
        u = beta[t][:, None] * (v[t] - (s * k[t][:, :, None]).sum(1))
        s = s + k[t][:, :, None] * u[:, None, :]
        out[t] = (s * q[t][:, :, None]).sum(1)
    return out, s


def delta_mixer(h: Tensor, w: Dict[str, Tensor], p: str, m: dict, eps: float) -> Tensor:
    t_len, heads, groups, dim, vdim = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (silu(causal_conv(h @ w[p + n].T, w[f"{p}{n}.conv"])) for n in ("q", "k", "v"))
    per = heads // groups
    q = (unit(q.view(t_len, groups, dim)) * dim ** -0.5).repeat_interleave(per, 1)
    k = unit(k.view(t_len, groups, dim)).repeat_interleave(per, 1)
    beta = sigmoid(h @ w[p + "b"].T)
    log_decay = -torch.exp(w[p + "A_log"]) * softplus(h @ w[p + "a"].T + w[p + "dt_bias"])
    o, _ = delta_recurrence(q, k, v.view(t_len, heads, vdim), log_decay, beta)
    o = rms_norm(o, eps) * w[p + "norm"] * silu(h @ w[p + "g"].T).view(t_len, heads, vdim)
    return o.reshape(t_len, heads * vdim) @ w[p + "o"].T


# ------------------------------------------------------------------ feed-forward


def gated_mlp(h: Tensor, w: Dict[str, Tensor], p: str) -> Tensor:
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def route(scores: Tensor, correction: Tensor, top: int, groups: int, keep: int) -> Tuple[List[int], List[float]]:
    """One token's experts and weights from its scores."""
    s, choice = scores.tolist(), (scores + correction).tolist()
    size = len(s) // groups
    best = sorted(range(groups), key=lambda g: -max(choice[g * size: (g + 1) * size]))[:keep]
    chosen = sorted((e for e in range(len(s)) if e // size in best), key=lambda e: -choice[e])[:top]
    return chosen, [s[e] for e in chosen]


def moe(h: Tensor, w: Dict[str, Tensor], p: str, m: dict) -> Tensor:
    r = m["router"]
    groups = r.get("groups") or {"count": 1, "keep": 1}
    scores = torch.softmax(h @ w[p + "router"].T, -1)
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, weight in zip(*route(scores[t], w[p + "correction"], r["top"], groups["count"], groups["keep"])):
            out[t] += weight * (gated_mlp(h[t: t + 1], w, f"{p}e{e}.")[0] if e < r["experts"] else h[t])
    if m.get("shared"):
        out = out + gated_mlp(h, w, p + "shared.")
    return out


# ------------------------------------------------------------------ model


def hyper_sum(x: Tensor, w: Dict[str, Tensor], p: str) -> Tensor:
    """``x [streams, T, width]`` -> what a sublayer's norm reads."""
    return (w[p + "in"][:, None, None] * x).sum(0)


def hyper_update(x: Tensor, y: Tensor, w: Dict[str, Tensor], p: str) -> Tensor:
    n = x.shape[0]
    return torch.stack([sum(w[p + "mix"][s, t] * x[s] for s in range(n)) + w[p + "out"][t] * y for t in range(n)])


def decoder_forward(weights: Dict[str, Tensor], cfg: dict, tokens: List[int], dtype: torch.dtype = torch.float64,
                    trace: Optional[List[Tensor]] = None) -> Tensor:
    """Logits ``[T, vocab]`` of one sequence from its start; ``trace`` collects the sum of the streams after every layer."""
    w = {k: v.to(dtype) for k, v in weights.items()}
    eps = cfg["norm"]["eps"]
    mixers = {"latent_attention": latent_mixer, "attention": attention_mixer, "delta": delta_mixer}
    x = w["embed"][torch.tensor(tokens)].expand(cfg["streams"], -1, -1)
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        h = rms_norm(hyper_sum(x, w, p + "hc1."), eps) * w[p + "norm1"]
        x = hyper_update(x, mixers[layer["type"]](h, w, p + "mix.", layer["mixer"], eps), w, p + "hc1.")
        if layer["mlp"] is not None:
            h = rms_norm(hyper_sum(x, w, p + "hc2."), eps) * w[p + "norm2"]
            x = hyper_update(x, moe(h, w, p + "mlp.", layer["mlp"]), w, p + "hc2.")
        if trace is not None:
            trace.append(x.sum(0))
    return rms_norm(x.sum(0), eps) * w["final.norm"] @ w["head"].T
