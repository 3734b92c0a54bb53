"""The oracle's statement of the hybrid mechanisms against independent routes (CPU only), and what a planted mistake
does to its logits: more than the tolerance of the tests that compare the GPU with it."""

import copy
import math

import pytest
import torch
import torch.nn.functional as F

from oracle import hybrid_oracle as ho
from tests import hybrid_helpers as hh

BF16_TOL = 0.06  # what the GPU tests allow in bf16


def _rand(*shape, seed=0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=torch.float64)


def test_norms_and_activations():
    x, w, b = _rand(5, 24), _rand(24, seed=1), _rand(24, seed=2)
    assert torch.allclose(ho.layer_norm(x, w, b, 1e-3), F.layer_norm(x, (24,), w, b, 1e-3))
    assert torch.allclose(ho.unit_rms(x, 1e-3), F.rms_norm(x, (24,), None, 1e-3))
    assert torch.allclose(ho.silu(x), F.silu(x)) and torch.allclose(ho.sigmoid(x), torch.sigmoid(x))
    assert torch.allclose(ho.gelu_tanh(x), F.gelu(x, approximate="tanh"))


@pytest.mark.parametrize("taps", [1, 2, 4])
def test_convolution_is_a_depthwise_conv1d(taps):
    u, w = _rand(11, 6), _rand(6, taps, seed=1)
    want = F.conv1d(F.pad(u.T[None], (taps - 1, 0)), w[:, None], groups=6)[0].T
    assert torch.allclose(ho.causal_conv(u, w), want)


def test_rotation_is_complex_multiplication_and_depends_on_distance():
    x = _rand(9, 2, 10)
    dims, base, factor = 6, 30.0, 1.7
    got = ho.rotate_interleaved(x, base, dims, factor)
    z = torch.view_as_complex(x[..., :dims].reshape(9, 2, 3, 2).contiguous())
    ang = torch.arange(9, dtype=torch.float64)[:, None] * base ** (-torch.arange(0, dims, 2, dtype=torch.float64) / dims) / factor
    turned = z * torch.polar(torch.ones_like(ang), ang)[:, None]
    assert torch.allclose(got[..., :dims], torch.view_as_real(turned).reshape(9, 2, dims))
    assert torch.equal(got[..., dims:], x[..., dims:])
    same = x[:1].expand(9, -1, -1)
    r = ho.rotate_interleaved(same, base, dims, factor)
    assert torch.allclose((r[2] * r[5]).sum(-1), (r[4] * r[7]).sum(-1))


@pytest.mark.parametrize("window", [None, 1, 4, 50])
def test_window_attention_is_sdpa_under_the_mask(window):
    t, h, g = 13, 6, 2
    q, k, v = _rand(t, h, 8), _rand(t, g, 8, seed=1), _rand(t, g, 5, seed=2)
    i, j = torch.arange(t)[:, None], torch.arange(t)[None, :]
    mask = (i - j >= 0) & ((i - j < window) if window else True)
    rep = h // g
    want = F.scaled_dot_product_attention(q.transpose(0, 1), k.repeat_interleave(rep, 1).transpose(0, 1),
                                          v.repeat_interleave(rep, 1).transpose(0, 1), attn_mask=mask, scale=0.7)
    assert torch.allclose(ho.window_attention(q, k, v, 0.7, window), want.transpose(0, 1))


def test_lightning_attention_is_its_unrolled_sum():
    t, h = 12, 3
    q, k, v = _rand(t, h, 4), _rand(t, h, 4, seed=1), _rand(t, h, 7, seed=2)
    decay = [0.0, 0.6, 1.0]
    o, s = ho.lightning_attention(q, k, v, decay)
    for n, lam in enumerate(decay):
        for i in range(t):
            want = sum(lam ** (i - j) * (q[i, n] @ k[j, n]) * v[j, n] for j in range(i + 1))
            assert torch.allclose(o[i, n], want)
        assert torch.allclose(s[n], sum(lam ** (t - 1 - j) * torch.outer(k[j, n], v[j, n]) for j in range(t)))
    o2, s2 = ho.lightning_attention(q[5:], k[5:], v[5:], decay, ho.lightning_attention(q[:5], k[:5], v[:5], decay)[1])
    assert torch.allclose(o2, o[5:]) and torch.allclose(s2, s)


def test_mixed_values_and_head_gates():
    v, first = _rand(3, 2, 4), _rand(3, 2, 4, seed=1)
    assert torch.equal(ho.mix_values(v, first, torch.tensor(0.0)), v)
    assert torch.equal(ho.mix_values(v, first, torch.tensor(1.0)), first)
    assert math.isclose(float(ho.sigmoid(torch.tensor(0.0))), 0.5)


@pytest.mark.parametrize("name", sorted(hh.CONFIGS))
def test_forward_is_causal(name):
    cfg = hh.CONFIGS[name]
    w = hh.weights(cfg)
    (tokens,) = hh.prompts(cfg, [14])
    whole = hh.forward(w, cfg, tokens)
    assert torch.allclose(whole[:9], hh.forward(w, cfg, tokens[:9]))


PLANTED = {
    "window one longer": lambda c, w: [l["mixer"]["mask"].update(size=l["mixer"]["mask"]["size"] + 1) for l in c["layers"] if "mask" in l["mixer"]],
    "window one shorter": lambda c, w: [l["mixer"]["mask"].update(size=l["mixer"]["mask"]["size"] - 1) for l in c["layers"] if "mask" in l["mixer"]],
    "rotation not scaled": lambda c, w: [l["mixer"]["rot"].update(scaling={}) for l in c["layers"] if "rot" in l["mixer"]],
    "rotation on fewer dimensions": lambda c, w: [l["mixer"]["rot"].update(dims=l["mixer"]["rot"]["dims"] - 2) for l in c["layers"] if "rot" in l["mixer"]],
    "no value mixing": lambda c, w: [l["mixer"].update(v_mix=False) for l in c["layers"] if "rot" in l["mixer"]],
    "a decay changed": lambda c, w: [l["mixer"].update(decay=[0.97 * d for d in l["mixer"]["decay"]]) for l in c["layers"] if "decay" in l["mixer"]],
    "decays reversed": lambda c, w: [l["mixer"].update(decay=l["mixer"]["decay"][::-1]) for l in c["layers"] if "decay" in l["mixer"]],
    "a tap dropped": lambda c, w: [w[n][:, 0].zero_() for n in list(w) if n.endswith(".conv")],
    "taps reversed": lambda c, w: [w.update({n: w[n].flip(1)}) for n in list(w) if n.endswith(".conv")],
    "no norm bias": lambda c, w: [w[n].zero_() for n in list(w) if n.endswith(".b")],
    "token sides of another layer": lambda c, w: w.update({"side.embed": w["side.embed"].roll(c["token_side"]["dim"], 1)}),
}


@pytest.mark.parametrize("what", sorted(PLANTED))
def test_planted_mistakes_show(what):
    cfg = hh.CONFIGS["plain"]
    w = hh.weights(cfg)
    (tokens,) = hh.prompts(cfg, [60])
    right = hh.forward(w, cfg, tokens)
    bad_cfg, bad_w = copy.deepcopy(cfg), {k: v.clone() for k, v in w.items()}
    PLANTED[what](bad_cfg, bad_w)
    wrong = hh.forward(bad_w, bad_cfg, tokens)
    assert hh.logit_error(wrong, right).max() > 2 * BF16_TOL
