"""The oracle's statement of the Tevirax mechanisms against independent routes (CPU only), and what a planted mistake does to
its logits: more than the tolerance of the tests that compare the GPU with it."""

import copy
import itertools
import math

import pytest
import torch
import torch.nn.functional as F

from oracle import tevirax_oracle as to
from tests import hybrid_helpers as hh
from tests import tevirax_helpers as tv


def _rand(*shape, seed=0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=torch.float64)


def test_norms_and_activations():
    x = _rand(5, 24) * 5
    assert torch.allclose(to.rms_norm(x, 1e-3), F.rms_norm(x, (24,), None, 1e-3))
    assert torch.allclose(to.silu(x), F.silu(x)) and torch.allclose(to.softplus(x), F.softplus(x, threshold=1e9))
    y, z, w = _rand(5, 24), _rand(5, 24, seed=1), _rand(24, seed=2)
    want = torch.cat([F.rms_norm(p, (8,), None, 1e-3) for p in (y * F.silu(z)).split(8, 1)], 1) * w
    assert torch.allclose(to.gated_group_norm(y, z, w, 3, 1e-3), want)
    assert torch.allclose(to.softcap(x, 2.0), 2 * torch.tanh(x / 2)) and to.softcap(x, None) is x


@pytest.mark.parametrize("taps", [1, 2, 4])
def test_convolution_is_a_depthwise_conv1d(taps):
    u, w, b = _rand(11, 6), _rand(6, taps, seed=1), _rand(6, seed=2)
    assert torch.allclose(to.causal_conv(u, w, b), F.conv1d(F.pad(u.T[None], (taps - 1, 0)), w[:, None], b, groups=6)[0].T)


def test_rotation_is_complex_multiplication_of_halves():
    x = _rand(9, 2, 10)
    rot = {"base": 30.0, "dims": 6, "scaling": {"factor": 3.0, "original": 16, "fast": 2.0, "slow": 0.5}}
    freq, amp = to.yarn_table(rot)
    assert amp == pytest.approx(1 + 0.1 * math.log(3.0))
    got = to.rotate_halves(x, rot)
    ang = torch.arange(9, dtype=torch.float64)[:, None] * torch.tensor(freq, dtype=torch.float64)
    turned = torch.complex(x[..., :3], x[..., 3:6]) * torch.polar(torch.full_like(ang, amp), ang)[:, None]
    assert torch.allclose(got[..., :6], torch.cat([turned.real, turned.imag], -1)) and torch.equal(got[..., 6:], x[..., 6:])
    assert torch.equal(to.rotate_halves(x, None), x)


def test_scaled_frequencies_keep_the_fast_pairs_and_divide_the_slow_ones():
    rot = {"base": 10000.0, "dims": 64, "scaling": {"factor": 8.0, "original": 4096, "fast": 32.0, "slow": 1.0}}
    plain, one = to.yarn_table({**rot, "scaling": None})
    assert one == 1.0 and plain[5] == pytest.approx(10000.0 ** (-10 / 64))
    freq, _ = to.yarn_table(rot)
    ratio = [f / p for f, p in zip(freq, plain)]
    turns = [4096 * p / (2 * math.pi) for p in plain]
    assert all(r == pytest.approx(1.0) for r, t in zip(ratio, turns) if t > 45) and all(r == pytest.approx(1 / 8) for r, t in zip(ratio, turns) if t < 0.7)
    assert all(a >= b for a, b in zip(ratio, ratio[1:])) and any(0.2 < r < 0.9 for r in ratio)


@pytest.mark.parametrize("size", [None, 1, 4, 50])
def test_chunk_attention_is_sdpa_under_the_mask(size):
    t, h, g = 13, 6, 2
    q, k, v = _rand(t, h, 8), _rand(t, g, 8, seed=1), _rand(t, g, 5, seed=2)
    i, j = torch.arange(t)[:, None], torch.arange(t)[None, :]
    mask = (i >= j) & ((i // size == j // size) if size else True)
    rep = h // g
    want = F.scaled_dot_product_attention(q.transpose(0, 1), k.repeat_interleave(rep, 1).transpose(0, 1),
                                          v.repeat_interleave(rep, 1).transpose(0, 1), attn_mask=mask, scale=0.7)
    assert torch.allclose(to.chunk_attention(q, k, v, 0.7, size), want.transpose(0, 1))


def test_matrix_memory_is_its_unrolled_sum():
    t, h, d, e = 12, 2, 5, 3
    q, k, v = _rand(t, h, d), _rand(t, h, d, seed=1), _rand(t, h, e, seed=2)
    li, lf = 2 * _rand(t, h, seed=3), -_rand(t, h, seed=4).abs()
    got, (s, n, m) = to.mlstm_recurrence(q, k, v, li, lf)
    f = lf.cumsum(0)
    for i, head in itertools.product(range(t), range(h)):
        logs = f[i, head] - f[: i + 1, head] + li[: i + 1, head]
        top = max(float(logs.max()), float(f[i, head]))  # (the maximum starts at 0 and decays as the state does)
        weight = torch.exp(logs - top)
        num = (weight * (k[: i + 1, head] @ q[i, head])) @ v[: i + 1, head]
        den = max(abs(float(weight @ (k[: i + 1, head] @ q[i, head]))), math.exp(-top)) + 1e-6
        assert torch.allclose(got[i, head], num / den)
    assert torch.allclose(m, torch.maximum(f[-1], (f[-1] - f + li).amax(0)))
    first, state = to.mlstm_recurrence(q[:5], k[:5], v[:5], li[:5], lf[:5])
    rest, last = to.mlstm_recurrence(q[5:], k[5:], v[5:], li[5:], lf[5:], state)
    assert torch.allclose(torch.cat([first, rest]), got) and torch.allclose(last[0], s) and torch.allclose(last[1], n)


def test_state_space_recurrence_is_its_unrolled_sum():
    t, h, g, p, n = 11, 4, 2, 3, 5
    x, b, c = _rand(t, h, p), _rand(t, g, n, seed=1), _rand(t, g, n, seed=2)
    dt, a, d = _rand(t, h, seed=3).abs(), _rand(h, seed=4).abs(), _rand(h, seed=5)
    got, s = to.ssd_recurrence(x, b, c, dt, a, d)
    f = (-a * dt).cumsum(0)
    for i, head in itertools.product(range(t), range(h)):
        weight = torch.exp(f[i, head] - f[: i + 1, head]) * dt[: i + 1, head]
        want = (weight * (b[: i + 1, head // 2] @ c[i, head // 2])) @ x[: i + 1, head] + d[head] * x[i, head]
        assert torch.allclose(got[i, head], want)
    first, state = to.ssd_recurrence(x[:4], b[:4], c[:4], dt[:4], a, d)
    rest, last = to.ssd_recurrence(x[4:], b[4:], c[4:], dt[4:], a, d, state)
    assert torch.allclose(torch.cat([first, rest]), got) and torch.allclose(last, s)


@pytest.mark.parametrize("experts,top,groups,keep", [(6, 2, 3, 2), (8, 3, 2, 1), (5, 4, 1, 1), (4, 2, 4, 3)])
def test_router_by_exhaustive_search(experts, top, groups, keep):
    size = experts // groups
    for seed in range(20):
        s = torch.sigmoid(_rand(experts, seed=seed))
        value = lambda g: sum(sorted(s[g * size: (g + 1) * size].tolist())[-2:])
        best = max(itertools.combinations(range(groups), keep), key=lambda gs: sum(value(g) for g in gs))
        able = [e for e in range(experts) if e // size in best]
        want = max(itertools.combinations(able, top), key=lambda es: float(sum(s[e] for e in es)))
        chosen, weights = to.route(s, top, groups, keep)
        assert sorted(chosen) == sorted(want) and sum(weights) == pytest.approx(1.0)
        assert weights == pytest.approx([float(s[e] / sum(s[list(want)])) for e in chosen])


# ------------------------------------------------------------------ planted mistakes


def _plant_chunk(cfg, w):
    for layer in cfg["layers"]:
        if layer["type"] == "parallel":
            layer["mixer"]["left"]["mask"]["size"] += 1


def _plant_eps(cfg, w):
    cfg["norm"]["eps"] = 0.3


def _scaled(name, factor):
    def plant(cfg, w):
        for key in w:
            if key.endswith(name):
                w[key] = w[key] * factor
    return plant


def _plant(path, value):
    def plant(cfg, w):
        for layer in cfg["layers"]:
            at = layer
            for key in path[:-1]:
                at = at.get(key) if at else None
            if at and path[-1] in at:
                at[path[-1]] = value(at[path[-1]])
    return plant


MISTAKES = {
    "chunk off by one": _plant_chunk, "norm eps": _plant_eps, "positions": _scaled("pos", 0.0),
    "yarn factor": _plant(("mixer", "left", "rot", "scaling", "factor"), lambda f: f * 2),
    "rotated dims": _plant(("mixer", "left", "rot", "dims"), lambda d: d - 2),
    "q norm": _scaled("left.q.norm", 0.7), "left scale": _plant(("mixer", "left_scale"), lambda s: s * 1.5),
    "gate cap": _plant(("mixer", "right", "gate_cap"), lambda c: c / 4), "input bias": _scaled("right.i.b", 0.0),
    "forget bias": _scaled("right.f.b", 0.0), "conv bias": _scaled("conv.b", 0.0), "skip": _scaled(".D", 0.0),
    "step bias": _scaled("dt_bias", 0.5), "decay": _scaled("A_log", -1.0), "shared gate": _scaled("shared.sg", 0.0),
    "experts": _plant(("mlp", "router", "top"), lambda t: t - 1), "groups": _plant(("mlp", "router", "groups", "keep"), lambda k: k - 1),
    "norm groups": _plant(("mixer", "norm_groups"), lambda n: 1), "soft cap": lambda cfg, w: cfg.update(logit_softcap=2 * cfg["logit_softcap"]),
}


@pytest.mark.parametrize("mistake", sorted(MISTAKES))
def test_planted_mistakes_show(mistake):
    name = "tvx-plain"
    cfg, w = hh.CONFIGS[name], hh.weights(hh.CONFIGS[name])
    (tokens,) = hh.prompts(cfg, [60], seed=2)
    want = hh.forward(w, cfg, tokens)
    wrong, ww = copy.deepcopy(cfg), dict(w)
    MISTAKES[mistake](wrong, ww)
    assert wrong != cfg or any(ww[k] is not w[k] for k in w)
    err = hh.logit_error(hh.forward(ww, wrong, tokens), want)
    tol = hh.bf16_tolerance(hh.forward, cfg, w, tokens, want)
    if mistake == "input bias":  # (a head's norm takes out most of it: what the 32-bit tests allow, many times over)
        tol = torch.full_like(tol, 4e-4)
    assert (err > tol).double().mean() > 0.1, (mistake, float((err / tol).max()))


def test_choices_of_experts_are_no_close_calls():
    for experts in (5, 6, 8, 12):
        s = torch.sigmoid(torch.tensor(tv.levels(experts), dtype=torch.float64))
        assert (s[:-1] / s[1:] > 1.2).all()
