"""The oracle's statement of the Loluzen mechanisms against independent routes (CPU only), and what a planted mistake does to
its logits: more than the tolerance of the tests that compare the GPU with it."""

import copy
import functools
import math

import pytest
import torch
import torch.nn.functional as F

from oracle import loluzen_oracle as lo
from tests import hybrid_helpers as hh


def _rand(*shape, seed=0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=torch.float64)


def test_norms_and_activations():
    x, w = _rand(5, 24) * 5, _rand(24, seed=1)
    assert torch.allclose(lo.rms_norm(x, 1e-3), F.rms_norm(x, (24,), None, 1e-3))
    assert torch.allclose(lo.shifted_norm(x, w, 1e-3), F.rms_norm(x, (24,), 1 + w, 1e-3))
    assert torch.allclose(lo.silu(x), F.silu(x)) and torch.allclose(lo.sigmoid(x), torch.sigmoid(x))
    weights = {"a": _rand(7, 24, seed=2), "a.b": _rand(7, seed=3), "c": _rand(7, 24, seed=4)}
    assert torch.allclose(lo.linear(x, weights, "a"), F.linear(x, weights["a"], weights["a.b"]))
    assert torch.allclose(lo.linear(x, weights, "c"), F.linear(x, weights["c"]))


@pytest.mark.parametrize("taps", [1, 2, 5])
def test_convolution_is_a_depthwise_conv1d(taps):
    u, w = _rand(11, 6), _rand(6, taps, seed=1)
    assert torch.allclose(lo.causal_conv(u, w), F.conv1d(F.pad(u.T[None], (taps - 1, 0)), w[:, None], groups=6)[0].T)


@pytest.mark.parametrize("scaling", [None, {"factor": 3.0, "original": 16, "low": 0.5, "high": 2.0}])
def test_rotation_is_complex_multiplication_of_neighbours(scaling):
    x, rot = _rand(9, 2, 14), {"base": 30.0, "dims": 10, "scaling": scaling}
    ang = torch.arange(9, dtype=torch.float64)[:, None] * torch.tensor(lo.pair_turns(rot), dtype=torch.float64)
    turned = torch.view_as_complex(x[..., :10].reshape(9, 2, 5, 2)) * torch.polar(torch.ones_like(ang), ang)[:, None]
    got = lo.rotate_pairs(x, rot)
    assert torch.allclose(got[..., :10], torch.view_as_real(turned).reshape(9, 2, 10)) and torch.equal(got[..., 10:], x[..., 10:])


def test_scaled_frequencies_by_the_number_of_waves():
    """Of the original length: at least ``high`` waves keep their frequency, at most ``low`` are slowed, a line between."""
    rot = {"base": 10000.0, "dims": 64, "scaling": {"factor": 8.0, "original": 4096, "low": 1.0, "high": 4.0}}
    plain, freq = lo.pair_turns({**rot, "scaling": None}), lo.pair_turns(rot)
    waves = [4096 * f / (2 * math.pi) for f in plain]
    assert any(w < 1 for w in waves) and any(1 < w < 4 for w in waves) and any(w > 4 for w in waves)
    for f, p, w in zip(freq, plain, waves):
        t = min(max((w - 1) / 3, 0.0), 1.0)
        assert f / p == pytest.approx(1 / 8 + t * (1 - 1 / 8))


def _heads(q, k):
    return k.repeat_interleave(q.shape[1] // k.shape[1], 1)


def test_attention_is_sdpa_under_an_explicit_bias():
    q, k, v = _rand(13, 6, 8), _rand(13, 2, 8, seed=1), _rand(13, 2, 5, seed=2)
    dist = torch.arange(13)[:, None] - torch.arange(13)[None]
    r1, r2 = torch.rand(6, dtype=torch.float64), torch.rand(6, dtype=torch.float64)
    for biased in (False, True):
        mask = torch.zeros(6, 13, 13, dtype=torch.float64)
        if biased:
            mask = -r1[:, None, None] * torch.log1p(r2[:, None, None] * dist.clamp(min=0))
        mask = mask.masked_fill(dist < 0, -math.inf)
        want = F.scaled_dot_product_attention(q.transpose(0, 1), _heads(q, k).transpose(0, 1), _heads(q, v).transpose(0, 1), attn_mask=mask, scale=0.7)
        got = lo.causal_attention(q, k, v, 0.7, lo.distance_bias(r1, r2, 13) if biased else None)
        assert torch.allclose(got, want.transpose(0, 1))


def test_mixed_heads_are_one_matrix_between_weights_and_values():
    """With the identity nothing changes; a permutation hands heads' weights to others; any matrix is a sum over the outputs that
    every head's weights would make of every kv head's values."""
    q, k, v = _rand(11, 4, 8), _rand(11, 2, 8, seed=1), _rand(11, 2, 5, seed=2)
    plain = lo.causal_attention(q, k, v, 0.6)
    assert torch.allclose(lo.causal_attention(q, k, v, 0.6, talk=torch.eye(4, dtype=torch.float64)), plain)
    talk = _rand(4, 4, seed=3)
    every = torch.stack([lo.causal_attention(q, k, v[:, g: g + 1].expand(-1, 2, -1), 0.6) for g in range(2)])  # [kv, T, H, E]
    want = torch.stack([(talk[h][None, :, None] * every[h // 2]).sum(1) for h in range(4)], 1)
    assert torch.allclose(lo.causal_attention(q, k, v, 0.6, talk=talk), want)


def test_recurrence_is_its_unrolled_product():
    q, v, z = _rand(9, 2, 4), _rand(9, 2, 3, seed=1), _rand(9, 2, 4, seed=2)
    lower = torch.rand(2, 4, dtype=torch.float64)
    f = lo.bounded_forget(z, lower)
    assert (f >= lower).all() and torch.allclose(f, lower + torch.sigmoid(z) - lower * torch.sigmoid(z))
    o, last = lo.channel_recurrence(q, f, v)
    for t in range(9):
        s = torch.zeros(2, 4, 3, dtype=torch.float64)
        for j in range(t + 1):
            s += (torch.prod(f[j + 1: t + 1], 0) * (1 - f[j]))[:, :, None] * v[j][:, None]
        assert torch.allclose(o[t], torch.matmul(q[t][:, None], s)[:, 0])
    assert torch.allclose(last, s)
    first, state = lo.channel_recurrence(q[:4], f[:4], v[:4])
    rest, end = lo.channel_recurrence(q[4:], f[4:], v[4:], state)
    assert torch.allclose(torch.cat([first, rest]), o) and torch.allclose(end, last)


def test_order_of_runs():
    cfg = {"layers": [None] * 5}
    assert lo.layer_runs(cfg) == [(i, False) for i in range(5)]
    cfg["loop"] = {"start": 1, "stop": 3, "times": 3}
    assert lo.layer_runs(cfg) == [(0, False), (1, False), (2, False), (1, True), (2, False), (1, True), (2, False), (3, False), (4, False)]


def test_model_is_causal():
    for name in ("llz-plain", "llz-odd"):
        cfg = hh.CONFIGS[name]
        w = hh.weights(cfg)
        (tokens,) = hh.prompts(cfg, [12])
        whole = hh.forward(w, cfg, tokens)
        assert torch.allclose(hh.forward(w, cfg, tokens[:7]), whole[:7]) and (hh.forward(w, cfg, tokens[1:])[-1] - whole[-1]).abs().max() > 1e-3


# ------------------------------------------------------------------ planted mistakes


def _scaled(name, factor):
    def plant(cfg, w):
        for key in w:
            if key.endswith(name):
                w[key] = w[key] * factor
    return plant


def _set(path, value):
    def plant(cfg, w):
        for layer in cfg["layers"]:
            at = layer["mixer"]
            for key in path[:-1]:
                at = at.get(key) if at else None
            if at and path[-1] in at:
                at[path[-1]] = value(at[path[-1]])
    return plant


def _changed(name, change):
    def plant(cfg, w):
        for key in w:
            if key.endswith(name):
                w[key] = change(w[key]).contiguous()
    return plant


MISTAKES = {
    "norm eps": lambda cfg, w: cfg["norm"].update(eps=0.3), "residual factor": lambda cfg, w: cfg.update(residual_mult=cfg["residual_mult"] * 1.15),
    "embedding scale": lambda cfg, w: cfg["embedding"].update(scale=cfg["embedding"]["scale"] * 1.2),
    "turns": lambda cfg, w: cfg["loop"].update(times=2), "loop end": lambda cfg, w: cfg["loop"].update(stop=3),
    "weights around one": _changed("norm1", lambda t: t - 1), "norm behind": _scaled("norm2b", 0.0), "final norm": _scaled("final.norm", 0.0),
    "rotation scaling": _set(("rot", "scaling", "factor"), lambda f: f * 2), "rotation ramp": _set(("rot", "scaling", "high"), lambda f: f * 4),
    "rotated dimensions": _set(("rot", "dims"), lambda n: n // 2), "scale": _set(("scale",), lambda s: s * 1.2),
    "scale of mixed heads": _set(("left", "scale"), lambda s: s * 1.2), "bias size": _scaled(".r1", 0.6), "bias rate": _scaled(".r2", 0.3),
    "mixing turned": _changed(".talk", lambda t: t.T), "no mixing": _changed(".talk", lambda t: torch.eye(len(t)).to(t)),
    "q bias": _scaled("left.q.b", 0.0), "v bias": _scaled("left.v.b", 0.0), "gates": _scaled("mix.left.g", 0.0), "attention gates": _scaled("l1.mix.g", 0.0),
    "q norm": _changed("q.norm", lambda t: t.flip(0)), "first tap": _changed(".conv", lambda t: torch.cat([0 * t[:, :1], t[:, 1:]], 1)),
    "forget bias": _scaled("f.b", 0.7), "lower bound": _scaled(".lower", 0.5), "head norm": _scaled("right.norm", 0.0),
    "left norm": _changed("left.out", lambda t: t.flip(0)), "right norm": _scaled("right.out", 0.8), "up bias": _scaled("up.b", 0.0), "down bias": _scaled("down.b", 0.0),
}
SMALL = ("norm eps", "rotation ramp", "bias rate", "bias size", "right norm", "lower bound", "scale", "scale of mixed heads", "rotated dimensions",
         "rotation scaling", "norm behind", "forget bias", "head norm")


@functools.lru_cache(None)
def _right():
    cfg, w = hh.CONFIGS["llz-plain"], hh.weights(hh.CONFIGS["llz-plain"])
    (tokens,) = hh.prompts(cfg, [56], seed=2)
    want = hh.forward(w, cfg, tokens)
    return cfg, w, tokens, want, hh.bf16_tolerance(hh.forward, cfg, w, tokens, want)


@pytest.mark.parametrize("mistake", sorted(MISTAKES))
def test_planted_mistakes_show(mistake):
    cfg, w, tokens, want, tol = _right()
    wrong, ww = copy.deepcopy(cfg), dict(w)
    MISTAKES[mistake](wrong, ww)
    assert wrong != cfg or any(ww[k] is not w[k] for k in w)
    err = hh.logit_error(hh.forward(ww, wrong, tokens), want)
    if mistake in SMALL:  # (a small term: what the 32-bit tests allow, many times over)
        tol = torch.full_like(tol, 4e-4)
    assert (err > tol).double().mean() > 0.1, (mistake, float((err / tol).max()), float((err > tol).double().mean()))
