"""The host side of Vusalix without a GPU: configuration, registry, checkpoint loading into joint weights, the buckets, the
stretches of cache rows that keys and values are made from, and what the pools and states hold."""

import copy

import numpy as np
import pytest
import torch

from oracle import vusalix_oracle as vo
from research_amd.inference import HybridDecoder, registry
from research_amd.inference.attention.hip_backend import STRETCH_BLOCK, plan_stretch
from research_amd.inference.hybrid import vusalix_config
from research_amd.inference.mixers import BiasedAttentionSpec, DeltaSpec, LatentSpec, YarnScaling
from research_amd.inference.moe import MoESpec
from tests import hybrid_helpers as hh


def _config(name, change=None):
    d = copy.deepcopy(hh.CONFIGS[name])
    if change is not None:
        change(d)
    return vusalix_config(d, lambda i: 12)


def test_config_reader():
    cfg = _config("vsx-plain")
    assert (cfg.width, cfg.vocab_size, cfg.norm_eps, cfg.norm, cfg.post_norm, cfg.streams) == (96, 101, 1e-5, "rms", False, 2)
    assert cfg.layers[0].mixer == DeltaSpec(heads=4, kv_heads=2, dim=32, vdim=24, taps=4)
    assert cfg.layers[1].mixer == LatentSpec(heads=3, dim=24, rot_dim=8, vdim=40, kv_rank=56, scale=2.0 * 32 ** -0.5, window=21, rot_base=900.0,
                                             rot_yarn=YarnScaling(3.0, 60.0, 8.0, 1.0))
    assert cfg.layers[2].mixer == BiasedAttentionSpec(heads=4, kv_heads=2, dim=32, vdim=24, scale=2.0 * 32 ** -0.5, window=37, softcap=9.0,
                                                      buckets=12, bias_max=30)
    same = dict(shared_gate=False, scores="softmax", group_top=1, correction=True, renormalize=False)
    assert cfg.layers[0].ff == MoESpec(6, 24, 2, 2, 1, 40, identity=2, **same)
    assert cfg.layers[2].ff == MoESpec(7, 24, 2, 1, 1, 56, identity=1, **same)
    cc = cfg.cache_config(10, 16, 3, torch.bfloat16, "cpu")
    assert cc.layer_kv == (None, (1, 64, 0), (2, 32)) and cc.num_state_slots == 3


def test_optional_fields():
    def change(d):
        for layer in d["layers"]:
            layer["mixer"].pop("mask", None)
        d["layers"][1]["mixer"]["rot"].pop("scaling")
        d["layers"][2]["mixer"]["softcap"] = None
        del d["layers"][0]["mlp"]
        d["layers"][1]["mlp"]["router"].pop("groups")
        d["layers"][1]["mlp"]["router"].pop("identity")
        d["layers"][1]["mlp"]["shared"] = None
    cfg = _config("vsx-plain", change)
    assert cfg.layers[1].mixer.window is None and cfg.layers[1].mixer.rot_yarn is None
    assert cfg.layers[2].mixer.window is None and cfg.layers[2].mixer.softcap is None
    ff = cfg.layers[1].ff
    assert cfg.layers[0].ff is None and (ff.groups, ff.keep, ff.identity, ff.shared) == (1, 1, 0, None)


@pytest.mark.parametrize("change,message", [
    (lambda d: d["layers"][0]["mixer"].update(gate=1), "unknown fields"),
    (lambda d: d["layers"][1]["mixer"]["rot"].update(kind=1), "unknown fields"),
    (lambda d: d["layers"][1]["mixer"]["rot"]["scaling"].update(kind=1), "unknown fields"),
    (lambda d: d["layers"][2]["mixer"]["mask"].update(keep=4), "unknown fields"),
    (lambda d: d["layers"][2]["mlp"]["router"].update(bias=1), "unknown fields"),
    (lambda d: d["layers"][2]["mlp"]["shared"].update(act="gelu"), "unknown fields"),
    (lambda d: d["layers"][0].update(type="other"), "unknown mixer"),
    (lambda d: d["layers"][0]["mlp"].update(kind="dense"), "unknown feed-forward"),
    (lambda d: d["layers"][0]["mixer"].update(kv_heads=3), "multiple of kv_heads"),
    (lambda d: d["layers"][2]["mixer"].update(kv_heads=3), "multiple of kv_heads"),
    (lambda d: d["layers"][0]["mixer"].update(conv=9), "taps"),
    (lambda d: d["layers"][1]["mixer"]["rot"].update(dims=6), "rot_dim"),
    (lambda d: d["layers"][1]["mixer"]["mask"].update(size=0), "window"),
    (lambda d: d["layers"][2]["mixer"].update(bias_max=6), "bias_max"),
    (lambda d: d["layers"][2]["mixer"].update(dim=264), "above 256"),
    (lambda d: d["layers"][1]["mixer"].update(kv_rank=1040), "above 1024"),
    (lambda d: d["layers"][0]["mlp"]["router"]["groups"].update(count=3), "equal groups"),
    (lambda d: d["layers"][0]["mlp"]["router"].update(top=5), "cannot be chosen"),
    (lambda d: d.update(streams=17), "streams"),
    (lambda d: d["norm"].update(kind="layer"), "unknown fields"),
])
def test_configs_that_are_refused(change, message):
    with pytest.raises(ValueError, match=message):
        _config("vsx-plain", change)


def _load(tmp_path, name, dtype=torch.float32):
    cfg = hh.CONFIGS[name]
    w = hh.weights(cfg)
    path = hh.save(tmp_path, cfg, w)
    options = registry.LoadOptions(num_blocks=4, block_size=16, num_state_slots=2, max_positions=50, dtype=dtype, device="cpu")
    return registry.load_model(path, options), cfg, w, path


def test_checkpoint_is_loaded_into_joint_weights(tmp_path):
    assert registry.find(hh.CONFIGS["vsx-plain"]).name == "vusalix"
    model, cfg, w, path = _load(tmp_path, "vsx-plain", torch.bfloat16)
    assert isinstance(model, HybridDecoder) and registry.model_len(path, 5000) == 5000
    d = model.layers[0].mixer
    assert torch.equal(d.w_in[:224], torch.cat([w[f"l0.mix.{n}"] for n in "qkv"])) and d.w_in.shape[0] % 8 == 0
    assert torch.equal(d.conv, torch.cat([w[f"l0.mix.{n}.conv"] for n in "qkv"]).float().T)
    assert torch.allclose(d.rate, w["l0.mix.A_log"].float().exp()) and torch.equal(d.norm, w["l0.mix.norm"].float().repeat(4))
    m = model.layers[1].mixer
    assert torch.equal(m.w_in[:160], torch.cat([w["l1.mix.q"], w["l1.mix.dkv"]]))
    uk, uv = w["l1.mix.uk"].view(3, 24, 56), w["l1.mix.uv"].view(3, 40, 56)
    assert torch.equal(m.w_key[:, :, :24], uk.transpose(1, 2)) and not m.w_key[..., 24:].any()
    assert torch.equal(m.w_value[..., :56], uv) and torch.equal(m.v_made[:, :40, :56], uv)
    # a pool row times k_made: the unrotated key, then the rotated part as it is
    row = torch.randn(64).to(torch.bfloat16)
    made = m.k_made.float() @ row.float()
    assert torch.allclose(made[:, :24], uk.float() @ row[:56].float(), atol=1e-4) and torch.equal(made[:, 24:32], row[56:].float().expand(3, -1))
    b = model.layers[2].mixer
    rel = w["l2.mix.rel"].float()
    assert tuple(b.bias.shape) == (4, 31)
    assert torch.equal(b.bias, torch.stack([rel[vo.bucket(n, 12, 30)] for n in range(31)], 1))
    assert torch.equal(b.sink, w["l2.mix.sink"].float())
    e = model.layers[2].mlp
    assert torch.equal(e.router, w["l2.mlp.router"]) and e.router.shape[0] == 8 and torch.equal(e.correction, w["l2.mlp.correction"].float())
    assert e.w_in.shape[0] == 7 and torch.equal(e.w_out[6, :, :24], w["l2.mlp.e6.down"])
    s = model.layers[1].streams2
    assert torch.equal(s.between, w["l1.hc2.mix"].float()) and torch.equal(s.weights, w["l1.hc2.in"].float()) and torch.equal(s.into, w["l1.hc2.out"].float())
    with pytest.raises(KeyError, match="lacks l2.mix.sink"):
        model.load_state_dict({k: v for k, v in w.items() if k != "l2.mix.sink"})
    with pytest.raises(ValueError, match="rel"):
        model.load_state_dict({**w, "l2.mix.rel": w["l2.mix.rel"][:-1]})
    with pytest.raises(KeyError, match="does not know"):
        model.load_state_dict({**w, "l1.hc3.in": w["l1.hc2.in"]})


def test_pools_and_states(tmp_path):
    model, _, _, _ = _load(tmp_path, "vsx-odd")
    shapes = {k: tuple(v.shape) for k, v in model.backend.state.items()}
    assert shapes == {(2, "delta"): (2, 6, 32, 32), (3, "conv"): (2, 1, 2 * 44 + 84), (3, "delta"): (2, 3, 48, 32)}
    k, v = model.backend.k_cache, model.backend.v_cache
    assert [None if t is None else tuple(t.shape) for t in k] == [(64, 2, 40), (64, 1, 40), None, None, (64, 1, 48)]
    assert v[1] is None and tuple(v[0].shape) == (64, 2, 40) and not model.layers[1].mixer.remake


@pytest.mark.parametrize("buckets,most", [(2, 2), (4, 200), (6, 11), (12, 30), (32, 128), (32, 256), (64, 1000), (7, 50)])
def test_buckets_of_every_distance(buckets, most):
    spec = BiasedAttentionSpec(1, 1, 8, 8, 1.0, None, None, buckets, most)
    got = spec.bucket_of()
    assert got == [vo.bucket(n, buckets, most) for n in range(most + 1)] and got[-1] == buckets - 1
    assert all(vo.bucket(n, buckets, most) == buckets - 1 for n in range(most, 4 * most))


@pytest.mark.parametrize("window", [0, 1, 5, 40])
def test_stretches_hold_the_visible_keys(window):
    g = np.random.default_rng(0)
    bs, lens, q_lens = 8, np.array([3, 50, 17, 33]), np.array([3, 2, 16, 1])
    tables = np.full((4, 8), -1, dtype=np.int32)
    ids = g.permutation(40)
    for i, n in enumerate(-(-lens // bs)):
        tables[i, :n], ids = ids[:n], ids[n:]
    slots, new, count = plan_stretch(lens, q_lens, tables, bs, window)
    assert len(slots) % STRETCH_BLOCK == 0
    for i in range(4):
        first = max(lens[i] - q_lens[i] - window + 1, 0) if window else 0
        assert count[i] == lens[i] - first
        want = [tables[i, p // bs] * bs + p % bs for p in range(first, lens[i])]
        got = [slots[new[i, j // STRETCH_BLOCK] * STRETCH_BLOCK + j % STRETCH_BLOCK] for j in range(count[i])]
        assert got == want
    used = new[new >= 0]
    assert sorted(used.tolist()) == list(range(len(slots) // STRETCH_BLOCK))


@pytest.mark.parametrize("dim,rot,vdim,made", [(128, 64, 128, (192, 128)), (136, 24, 72, (160, 72)), (24, 8, 40, (40, 40)),
                                               (64, 16, 128, (128, 128)), (112, 32, 136, (144, 144)), (180, 32, 64, (216, 216))])
def test_sizes_of_made_keys_and_values(dim, rot, vdim, made):
    assert LatentSpec(2, dim, rot, vdim, 48, 0.1, None, 100.0).made == made
