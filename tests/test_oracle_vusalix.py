"""The oracle's statement of the Vusalix mechanisms against independent routes (CPU only), and what a planted mistake does to
its logits: more than the tolerance of the tests that compare the GPU with it."""

import copy
import functools
import itertools
import math

import pytest
import torch
import torch.nn.functional as F

from oracle import vusalix_oracle as vo
from tests import hybrid_helpers as hh
from tests import vusalix_helpers as vx


def _rand(*shape, seed=0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=torch.float64)


def test_norms_and_activations():
    x = _rand(5, 24) * 5
    assert torch.allclose(vo.rms_norm(x, 1e-3), F.rms_norm(x, (24,), None, 1e-3))
    assert torch.allclose(vo.silu(x), F.silu(x)) and torch.allclose(vo.softplus(x), F.softplus(x, threshold=1e9))
    assert torch.allclose(vo.unit(x).norm(dim=-1), torch.ones(5, dtype=torch.float64), atol=1e-6) and not vo.unit(0 * x).any()


@pytest.mark.parametrize("taps", [1, 2, 5])
def test_convolution_is_a_depthwise_conv1d(taps):
    u, w = _rand(11, 6), _rand(6, taps, seed=1)
    assert torch.allclose(vo.causal_conv(u, w), F.conv1d(F.pad(u.T[None], (taps - 1, 0)), w[:, None], groups=6)[0].T)


@pytest.mark.parametrize("scaling", [None, {"factor": 3.0, "original": 16, "fast": 2.0, "slow": 0.5}])
def test_rotation_is_complex_multiplication_of_neighbours(scaling):
    x, rot = _rand(9, 2, 10), {"base": 30.0, "dims": 10, "scaling": scaling}
    freq, amp = vo.pair_turns(rot)
    assert amp == pytest.approx(1 + 0.1 * math.log(3.0) if scaling else 1.0)
    ang = torch.arange(9, dtype=torch.float64)[:, None] * torch.tensor(freq, dtype=torch.float64)
    turned = torch.view_as_complex(x.view(9, 2, 5, 2)) * torch.polar(torch.full_like(ang, amp), ang)[:, None]
    assert torch.allclose(vo.rotate_pairs(x, rot), torch.view_as_real(turned).reshape(9, 2, 10))


def test_scaled_frequencies_keep_the_fast_pairs_and_divide_the_slow_ones():
    rot = {"base": 10000.0, "dims": 64, "scaling": {"factor": 8.0, "original": 4096, "fast": 32.0, "slow": 1.0}}
    plain, _ = vo.pair_turns({**rot, "scaling": None})
    freq, _ = vo.pair_turns(rot)
    ratio = [f / p for f, p in zip(freq, plain)]
    turns = [4096 * p / (2 * math.pi) for p in plain]
    assert all(r == pytest.approx(1.0) for r, t in zip(ratio, turns) if t > 45)
    assert all(r == pytest.approx(1 / 8) for r, t in zip(ratio, turns) if t < 0.7)
    assert all(a >= b for a, b in zip(ratio, ratio[1:])) and any(0.2 < r < 0.9 for r in ratio)


def _mask(t, window):
    i, j = torch.arange(t)[:, None], torch.arange(t)[None]
    return (i >= j) & ((i - j < window) if window else True)


@pytest.mark.parametrize("window", [None, 1, 4, 50])
def test_softmax_attention_is_sdpa_under_the_mask(window):
    q, k, v = _rand(13, 3, 8), _rand(13, 3, 8, seed=1), _rand(13, 3, 5, seed=2)
    want = F.scaled_dot_product_attention(q.transpose(0, 1), k.transpose(0, 1), v.transpose(0, 1), attn_mask=_mask(13, window), scale=0.7)
    assert torch.allclose(vo.softmax_attention(q, k, v, 0.7, window), want.transpose(0, 1))


def test_latent_attention_is_attention_over_the_latents():
    """The same scores with the key weights on the query's side, and the value weights behind the weighted latents."""
    m = {"heads": 3, "dim": 6, "rot_dim": 4, "vdim": 5, "kv_rank": 11, "scale": 0.4, "mask": {"size": 6}, "rot": {"base": 20.0, "dims": 4}}
    w = {"q": _rand(30, 9), "dkv": _rand(15, 9, seed=1), "dkv.norm": _rand(11, seed=2), "uk": _rand(18, 11, seed=3), "uv": _rand(15, 11, seed=4),
         "o": _rand(9, 15, seed=5)}
    h = _rand(14, 9, seed=6)
    q, down = (h @ w["q"].T).view(14, 3, 10), h @ w["dkv"].T
    c = F.rms_norm(down[:, :11], (11,), w["dkv.norm"], 1e-5)
    over = torch.matmul(q[..., :6].transpose(0, 1), w["uk"].view(3, 6, 11))
    s = torch.matmul(over, c.T) + torch.matmul(vo.rotate_pairs(q[..., 6:], m["rot"]).transpose(0, 1), vo.rotate_pairs(down[:, None, 11:], m["rot"])[:, 0].T)
    p = torch.softmax((s * 0.4).masked_fill(~_mask(14, 6), -math.inf), -1)
    o = torch.matmul(torch.matmul(p, c), w["uv"].view(3, 5, 11).transpose(1, 2)).transpose(0, 1).reshape(14, 15)
    assert torch.allclose(vo.latent_mixer(h, w, "", m, 1e-5), o @ w["o"].T)


@pytest.mark.parametrize("buckets,most", [(8, 32), (32, 256), (6, 11), (2, 2), (7, 50)])
def test_buckets_by_their_thresholds(buckets, most):
    half = buckets // 2
    rest = buckets - half
    edges = [half * (most / half) ** (k / rest) for k in range(1, rest)]  # where bucket half + k starts
    for n in range(3 * most):
        got = vo.bucket(n, buckets, most)
        if n < half:
            assert got == n
        elif not any(abs(n - e) < 1e-6 for e in edges):
            assert got == half + sum(n > e for e in edges)
    if (buckets, most) == (8, 32):  # (powers: 4, 4 * 8^(1/4), ..., exactly at 4 * 8^(2/4) there is no whole number)
        assert [vo.bucket(n, 8, 32) for n in (3, 4, 6, 7, 11, 12, 19, 20, 31, 32, 900)] == [3, 4, 4, 5, 5, 6, 6, 7, 7, 7, 7]
    if (buckets, most) == (32, 256):
        assert [vo.bucket(n, 32, 256) for n in (31, 32, 63, 64, 127, 128)] == [19, 20, 23, 24, 27, 28]


@pytest.mark.parametrize("window,cap", [(None, None), (5, 3.0), (1, 2.0)])
def test_biased_attention_is_softmax_with_one_more_column(window, cap):
    t, h, g = 12, 4, 2
    q, k, v, rel, sink = _rand(t, h, 6), _rand(t, g, 6, seed=1), _rand(t, g, 7, seed=2), _rand(6, h, seed=3), _rand(h, seed=4)
    s = torch.matmul(q.transpose(0, 1), k.repeat_interleave(2, 1).permute(1, 2, 0)) * 0.8
    s = cap * torch.tanh(s / cap) if cap else s
    dist = (torch.arange(t)[:, None] - torch.arange(t)[None]).clamp(min=0)
    s = s + rel[torch.tensor([[vo.bucket(int(d), 6, 9) for d in row] for row in dist])].permute(2, 0, 1)
    s = torch.cat([s.masked_fill(~_mask(t, window), -math.inf), sink[:, None, None].expand(-1, t, 1)], -1)
    want = torch.matmul(torch.softmax(s, -1)[..., :-1], v.repeat_interleave(2, 1).transpose(0, 1)).transpose(0, 1)
    assert torch.allclose(vo.biased_attention(q, k, v, 0.8, window, cap, rel, 9, sink), want)


def test_delta_rule_is_its_product_form():
    """S_t = g (I - beta k k^T) S_(t-1) + beta k v^T, and the state carries over a cut."""
    t, h, d, e = 12, 2, 5, 3
    q, k, v = _rand(t, h, d), vo.unit(_rand(t, h, d, seed=1)), _rand(t, h, e, seed=2)
    log_decay, beta = -_rand(t, h, seed=3).abs(), torch.sigmoid(_rand(t, h, seed=4))
    got, last = vo.delta_recurrence(q, k, v, log_decay, beta)
    for head in range(h):
        s = torch.zeros(d, e, dtype=torch.float64)
        for i in range(t):
            kk = k[i, head][:, None]
            s = math.exp(log_decay[i, head]) * (torch.eye(d, dtype=torch.float64) - beta[i, head] * kk @ kk.T) @ s + beta[i, head] * kk @ v[i, head][None]
            assert torch.allclose(got[i, head], s.T @ q[i, head])
        assert torch.allclose(last[head], s)
    first, state = vo.delta_recurrence(q[:5], k[:5], v[:5], log_decay[:5], beta[:5])
    rest, end = vo.delta_recurrence(q[5:], k[5:], v[5:], log_decay[5:], beta[5:], state)
    assert torch.allclose(torch.cat([first, rest]), got) and torch.allclose(end, last)


@pytest.mark.parametrize("experts,top,groups,keep", [(6, 2, 3, 2), (8, 3, 2, 1), (5, 4, 1, 1), (4, 2, 4, 3)])
def test_router_by_exhaustive_search(experts, top, groups, keep):
    size = experts // groups
    for seed in range(20):
        s, corr = torch.softmax(_rand(experts, seed=seed), 0), _rand(experts, seed=100 + seed) - 1.0  # (choice scores below 0, too)
        choice = (s + corr).tolist()
        best = max(itertools.combinations(range(groups), keep), key=lambda gs: sum(max(choice[g * size: (g + 1) * size]) for g in gs))
        able = [e for e in range(experts) if e // size in best]
        want = max(itertools.combinations(able, top), key=lambda es: sum(choice[e] for e in es))
        chosen, weights = vo.route(s, corr, top, groups, keep)
        assert sorted(chosen) == sorted(want) and weights == pytest.approx([float(s[e]) for e in chosen])


def test_identity_experts_hand_on_their_input():
    m = {"expert": {"ff": 4}, "router": {"experts": 2, "identity": 1, "top": 1}}
    w = {f"e{e}.{n}": _rand(*((4, 6) if n != "down" else (6, 4)), seed=e) for e in range(2) for n in ("gate", "up", "down")}
    w["router"], w["correction"] = _rand(3, 6, seed=9), torch.tensor([0.0, 0.0, 9.0], dtype=torch.float64)
    h = _rand(5, 6, seed=8)
    assert torch.allclose(vo.moe(h, w, "", m), torch.softmax(h @ w["router"].T, -1)[:, 2:] * h)


def test_streams_are_one_matrix_per_sublayer():
    n = 3
    x, y = _rand(n, 4, 5), _rand(4, 5, seed=1)
    w = {"in": _rand(n, seed=2), "mix": _rand(n, n, seed=3), "out": _rand(n, seed=4)}
    assert torch.allclose(vo.hyper_sum(x, w, ""), torch.tensordot(w["in"], x, 1))
    whole = torch.cat([w["mix"], w["out"][None]]).T  # [to, from + branch]
    assert torch.allclose(vo.hyper_update(x, y, w, ""), torch.tensordot(whole, torch.cat([x, y[None]]), 1))


# ------------------------------------------------------------------ planted mistakes


def _scaled(name, factor):
    def plant(cfg, w):
        for key in w:
            if key.endswith(name):
                w[key] = w[key] * factor
    return plant


def _plant(path, value, kind=None):
    def plant(cfg, w):
        for layer in cfg["layers"]:
            at = layer if kind in (None, layer["type"]) else None
            for key in path[:-1]:
                at = at.get(key) if at else None
            if at and path[-1] in at:
                at[path[-1]] = value(at[path[-1]])
    return plant


def _turned(name):
    def plant(cfg, w):
        for key in w:
            if key.endswith(name):
                w[key] = w[key].T.contiguous()
    return plant


def _rows_reversed(name):
    def plant(cfg, w):
        for key in w:
            if key.endswith(name):
                w[key] = w[key].flip(0)
    return plant


MISTAKES = {
    "latent window off by one": _plant(("mixer", "mask", "size"), lambda n: n + 1, "latent_attention"),
    "window off by one": _plant(("mixer", "mask", "size"), lambda n: n + 1, "attention"),
    "norm eps": lambda cfg, w: cfg["norm"].update(eps=0.3), "yarn factor": _plant(("mixer", "rot", "scaling", "factor"), lambda f: f * 2),
    "yarn length": _plant(("mixer", "rot", "scaling", "original"), lambda n: n * 8),
    "scale": _plant(("mixer", "scale"), lambda s: s * 1.2), "soft cap": _plant(("mixer", "softcap"), lambda c: c / 3),
    "sink": _scaled(".sink", 0.0), "biases": _rows_reversed(".rel"), "last distance": _plant(("mixer", "bias_max"), lambda n: n * 4),
    "latent norm": _scaled("dkv.norm", 0.7), "step bias": _scaled("dt_bias", 0.5), "decay": _scaled("A_log", -1.0), "beta": _scaled("mix.b", 0.0),
    "head norm": _scaled("mix.norm", 0.8), "streams in": _rows_reversed("hc2.in"), "streams out": _scaled("hc1.out", 0.7), "streams turned": _turned(".mix"),
    "correction": _scaled("correction", 0.0), "experts": _plant(("mlp", "router", "top"), lambda t: t - 1),
    "groups": _plant(("mlp", "router", "groups"), lambda g: {"count": 1, "keep": 1}),
}


SMALL = ("latent window off by one", "window off by one", "norm eps", "last distance", "yarn length", "sink", "head norm", "streams in", "streams turned")


@functools.lru_cache(None)
def _right():
    cfg, w = hh.CONFIGS["vsx-plain"], hh.weights(hh.CONFIGS["vsx-plain"])
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
    if mistake in SMALL:  # (one key among many, a small term: what the 32-bit tests allow, many times over)
        tol = torch.full_like(tol, 4e-4)
    assert (err > tol).double().mean() > 0.1, (mistake, float((err / tol).max()), float((err > tol).double().mean()))


def test_choices_of_experts_are_no_close_calls():
    """Of the test models: the scores that separate chosen from others differ by more than a bf16 rounding moves them."""
    for name in vx.CONFIGS:
        cfg = hh.CONFIGS[name]
        levels = torch.linspace(-1.5, 1.5, vx.router_width(cfg))
        assert levels.numel() < 2 or (levels[1:] - levels[:-1]).min() > 0.2
