"""CPU restatement of the Tevirax design.  TEST INFRASTRUCTURE.

Nothing in the product imports this file, and it imports nothing of the product.  One plain, slow function per mechanism,
whole sequences only, in the type of its inputs (the tests use float64): no cache, no state carried between calls, no
chunks of rows.  ``decoder_forward`` strings them together for a configuration given as the plain dictionary of a
``config.json`` and a dictionary of weights under their checkpoint names.

Shapes: ``T`` tokens of one sequence; ``x [T, width]``.

How the functions are pinned (tests/test_oracle_tevirax.py): the rotation by complex multiplication, the chunk mask by
``scaled_dot_product_attention`` with an explicit mask, both recurrences by their unrolled sums, the convolution by
``torch.nn.functional.conv1d``, the router by exhaustive search.
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


# ------------------------------------------------------------------ attention


def yarn_table(rot: Optional[dict]) -> Tuple[List[float], float]:
    """Angle per position of every rotated pair, and the factor on cosine and sine."""
    if not rot or not rot.get("dims"):
        return [], 1.0
    dims, base, s = rot["dims"], rot["base"], rot.get("scaling")
    freq = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    if not s:
        return freq, 1.0
    where = lambda turns: dims * math.log(s["original"] / (2 * math.pi * turns)) / (2 * math.log(base))
    lo = max(math.floor(where(s["fast"])), 0)
    hi = min(math.ceil(where(s["slow"])), dims - 1)
    out = []
    for i, f in enumerate(freq):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(f / s["factor"] * ramp + f * (1 - ramp))
    return out, 0.1 * math.log(s["factor"]) + 1


def rotate_halves(x: Tensor, rot: Optional[dict]) -> Tensor:
    """``x [T, heads, dim]``: dimensions i and i + dims/2 turn together."""
    freq, amp = yarn_table(rot)
    n = len(freq)
    out = x.clone()
    if n == 0:
        return out
    ang = torch.arange(x.shape[0], dtype=torch.float64)[:, None] * torch.tensor(freq, dtype=torch.float64)
    c, s = ((f(ang) * amp).to(x.dtype)[:, None, :] for f in (torch.cos, torch.sin))
    u, v = x[..., :n], x[..., n: 2 * n]
    out[..., :n] = u * c - v * s
    out[..., n: 2 * n] = v * c + u * s
    return out


def chunk_attention(q: Tensor, k: Tensor, v: Tensor, scale: float, size: Optional[int]) -> Tensor:
    """``q [T, H, D]``, ``k [T, G, D]``, ``v [T, G, E]`` -> ``[T, H, E]``; row i sees j <= i of its own chunk of ``size``
    positions, counted from the sequence's start (None: all j <= i)."""
    t_len, heads, _ = q.shape
    group = heads // k.shape[1]
    out = torch.zeros(t_len, heads, v.shape[2], dtype=q.dtype)
    for i in range(t_len):
        lo = 0 if size is None else i // size * size
        for g in range(k.shape[1]):
            hs = slice(g * group, (g + 1) * group)
            s = q[i, hs] @ k[lo: i + 1, g].T * scale
            p = torch.exp(s - s.max(-1, keepdim=True).values)
            out[i, hs] = (p / p.sum(-1, keepdim=True)) @ v[lo: i + 1, g]
    return out


def attention_heads(h: Tensor, w: Dict[str, Tensor], p: str, m: dict, eps: float) -> Tensor:
    """The attention half without its output product: ``[T, heads * vdim]``."""
    t_len = h.shape[0]
    q = (h @ w[p + "q"].T).view(t_len, m["heads"], m["dim"])
    k = (h @ w[p + "k"].T).view(t_len, m["kv_heads"], m["dim"])
    v = (h @ w[p + "v"].T).view(t_len, m["kv_heads"], m["vdim"])
    q = rotate_halves(rms_norm(q, eps) * w[p + "q.norm"], m.get("rot"))
    k = rotate_halves(rms_norm(k, eps) * w[p + "k.norm"], m.get("rot"))
    return chunk_attention(q, k, v, m["scale"], (m.get("mask") or {}).get("size")).reshape(t_len, -1)


# ------------------------------------------------------------------ mLSTM


def mlstm_recurrence(q: Tensor, k: Tensor, v: Tensor, log_i: Tensor, log_f: Tensor,
                     state: Optional[Tuple[Tensor, Tensor, Tensor]] = None) -> Tuple[Tensor, Tuple[Tensor, Tensor, Tensor]]:
    """``q, k [T, H, D]`` (q scaled already), ``v [T, H, E]``, ``log_i, log_f [T, H]`` -> ``[T, H, E]`` and (S, n, m)."""
    t_len, heads, d = q.shape
    if state is None:
        s, n = torch.zeros(heads, d, v.shape[2], dtype=q.dtype), torch.zeros(heads, d, dtype=q.dtype)
        m = torch.zeros(heads, dtype=q.dtype)
    else:
        s, n, m = (t.clone() for t in state)
    out = torch.zeros(t_len, heads, v.shape[2], dtype=q.dtype)
    for t in range(t_len):
        m_new = torch.maximum(log_f[t] + m, log_i[t])
        keep, add = torch.exp(log_f[t] + m - m_new), torch.exp(log_i[t] - m_new)
        m = m_new
        s = keep[:, None, None] * s + add[:, None, None] * k[t][:, :, None] * v[t][:, None, :]
        n = keep[:, None] * n + add[:, None] * k[t]
        num = (s * q[t][:, :, None]).sum(1)
        den = torch.maximum((n * q[t]).sum(1).abs(), torch.exp(-m)) + 1e-6
        out[t] = num / den[:, None]
    return out, (s, n, m)


def mlstm_heads(h: Tensor, w: Dict[str, Tensor], p: str, m: dict, eps: float) -> Tensor:
    t_len, heads, dim, vdim, cap = h.shape[0], m["heads"], m["dim"], m["vdim"], m["gate_cap"]
    q = (h @ w[p + "q"].T).view(t_len, heads, dim) * dim ** -0.5
    k = (h @ w[p + "k"].T).view(t_len, heads, dim)
    v = (h @ w[p + "v"].T).view(t_len, heads, vdim)
    log_i = cap * torch.tanh((h @ w[p + "i"].T + w[p + "i.b"]) / cap)
    log_f = -softplus(-cap * torch.tanh((h @ w[p + "f"].T + w[p + "f.b"]) / cap))
    o, _ = mlstm_recurrence(q, k, v, log_i, log_f)
    o = rms_norm(o, eps).reshape(t_len, heads * vdim) * w[p + "norm"]
    return o * sigmoid(h @ w[p + "g"].T)


def parallel_mixer(h: Tensor, w: Dict[str, Tensor], p: str, m: dict, eps: float) -> Tensor:
    left = attention_heads(h, w, p + "left.", m["left"], eps) @ w[p + "left.o"].T
    right = mlstm_heads(h, w, p + "right.", m["right"], eps) @ w[p + "right.o"].T
    return m["left_scale"] * left + m["right_scale"] * right


# ------------------------------------------------------------------ Mamba-2


def causal_conv(u: Tensor, w: Tensor, b: Tensor) -> Tensor:
    """``u [T, C]``, ``w [C, taps]``: the last column weighs the current row; zeros before the start."""
    taps = w.shape[1]
    padded = torch.cat([torch.zeros(taps - 1, u.shape[1], dtype=u.dtype), u])
    return b + sum(w[:, j] * padded[j: j + u.shape[0]] for j in range(taps))


def ssd_recurrence(x: Tensor, b: Tensor, c: Tensor, dt: Tensor, a: Tensor, d: Tensor,
                   state: Optional[Tensor] = None) -> Tuple[Tensor, Tensor]:
    """``x [T, H, P]``, ``b, c [T, G, N]``, ``dt [T, H]`` positive, ``a [H]`` (the state decays by exp(-a dt)), ``d [H]``
    -> ``[T, H, P]`` and the last state ``[H, N, P]``."""
    t_len, heads, p = x.shape
    per = heads // b.shape[1]
    b, c = b.repeat_interleave(per, 1), c.repeat_interleave(per, 1)
    s = torch.zeros(heads, b.shape[2], p, dtype=x.dtype) if state is None else state.clone()
    out = torch.zeros_like(x)
    for t in range(t_len):
        s = torch.exp(-a * dt[t])[:, None, None] * s + dt[t][:, None, None] * b[t][:, :, None] * x[t][:, None, :]
        out[t] = (s * c[t][:, :, None]).sum(1) + d[:, None] * x[t]
    return out, s


def gated_group_norm(y: Tensor, z: Tensor, w: Tensor, groups: int, eps: float) -> Tensor:
    """The gate first, then every part by its own root mean square."""
    y = y * silu(z)
    return rms_norm(y.view(y.shape[0], groups, -1), eps).reshape(y.shape) * w


def mamba2_mixer(h: Tensor, w: Dict[str, Tensor], p: str, m: dict, eps: float) -> Tensor:
    t_len, heads, vdim, n, g = h.shape[0], m["heads"], m["vdim"], m["state"], m["groups"]
    inner = heads * vdim
    z, xbc, dt = (h @ w[p + "in"].T).split([inner, inner + 2 * g * n, heads], 1)
    x, b, c = silu(causal_conv(xbc, w[p + "conv"], w[p + "conv.b"])).split([inner, g * n, g * n], 1)
    y, _ = ssd_recurrence(x.reshape(t_len, heads, vdim), b.reshape(t_len, g, n), c.reshape(t_len, g, n),
                          softplus(dt + w[p + "dt_bias"]), torch.exp(w[p + "A_log"]), w[p + "D"])
    return gated_group_norm(y.reshape(t_len, inner), z, w[p + "norm"], m["norm_groups"], eps) @ w[p + "o"].T


# ------------------------------------------------------------------ feed-forward


def gated_mlp(h: Tensor, w: Dict[str, Tensor], p: str) -> Tensor:
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def route(scores: Tensor, top: int, groups: int, keep: int) -> Tuple[List[int], List[float]]:
    """One token's experts and weights from its scores ``[experts]``."""
    s = scores.tolist()
    size = len(s) // groups
    value = [sum(sorted(s[g * size: (g + 1) * size], reverse=True)[:2]) for g in range(groups)]
    best = sorted(range(groups), key=lambda g: -value[g])[:keep]
    able = [e for e in range(len(s)) if e // size in best]
    chosen = sorted(able, key=lambda e: -s[e])[:top]
    total = sum(s[e] for e in chosen) + 1e-20
    return chosen, [s[e] / total for e in chosen]


def moe(h: Tensor, w: Dict[str, Tensor], p: str, m: dict) -> Tensor:
    r = m["router"]
    groups = r.get("groups") or {"count": 1, "keep": 1}
    scores = sigmoid(h @ w[p + "router"].T)
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, weight in zip(*route(scores[t], r["top"], groups["count"], groups["keep"])):
            out[t] += weight * gated_mlp(h[t: t + 1], w, f"{p}e{e}.")[0]
    if m.get("shared"):
        out = out + sigmoid(h @ w[p + "shared.sg"].T) * gated_mlp(h, w, p + "shared.")
    return out


def softcap(x: Tensor, cap: Optional[float]) -> Tensor:
    return x if not cap else cap * torch.tanh(x / cap)


# ------------------------------------------------------------------ model


def decoder_forward(weights: Dict[str, Tensor], cfg: dict, tokens: List[int], dtype: torch.dtype = torch.float64,
                    trace: Optional[List[Tensor]] = None) -> Tensor:
    """Logits ``[T, vocab]`` of one sequence from its start; ``trace`` collects the residual after every layer."""
    w = {k: v.to(dtype) for k, v in weights.items()}
    eps = cfg["norm"]["eps"]
    x = w["embed"][torch.tensor(tokens)] * cfg["embedding"]["scale"] + w["pos"][: len(tokens)]
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        mixer = {"parallel": parallel_mixer, "mamba2": mamba2_mixer}[layer["type"]]
        x = x + rms_norm(mixer(x, w, p + "mix.", layer["mixer"], eps), eps) * w[p + "norm1"]
        ff = layer["mlp"]
        if ff is not None:
            y = gated_mlp(x, w, p + "mlp.") if ff["kind"] == "dense" else moe(x, w, p + "mlp.", ff)
            x = x + rms_norm(y, eps) * w[p + "norm2"]
        if trace is not None:
            trace.append(x)
    return softcap(rms_norm(x, eps) * w["final.norm"] @ w["head"].T, cfg.get("logit_softcap"))
