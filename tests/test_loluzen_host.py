"""The host side of Loluzen without a GPU: configuration, registry, the order of runs, checkpoint loading into joint weights,
rotary tables, and what the pools and states hold."""

import copy
import math

import pytest
import torch

from oracle import loluzen_oracle as lo
from research_amd.inference import HybridDecoder, registry
from research_amd.inference.hybrid import HybridConfig, LayerSpec, Loop, Run, loluzen_config
from research_amd.inference.mixers import (AttentionSpec, Hgrn2Spec, LlamaScaling, MLPSpec, ParallelSpec, RotaryTables, TalkingSpec,
                                           llama_frequencies)
from tests import hybrid_helpers as hh


def _config(name, change=None):
    d = copy.deepcopy(hh.CONFIGS[name])
    if change is not None:
        change(d)
    return loluzen_config(d)


def test_config_reader():
    cfg = _config("llz-plain")
    assert (cfg.width, cfg.vocab_size, cfg.norm_eps, cfg.norm, cfg.both_norms, cfg.post_norm) == (96, 101, 1e-5, "rms", True, False)
    assert (cfg.norm_offset, cfg.residual_mult, cfg.embed_scale, cfg.loop) == (1.0, 1.2, 0.6, Loop(0, 2, 3))
    assert cfg.layers[0] == LayerSpec(ParallelSpec(TalkingSpec(4, 2, 32, 24, 2.5 * 32 ** -0.5), Hgrn2Spec(3, 16, 40), 0.5, 0.5, norms=True), MLPSpec(56, "relu2"))
    assert cfg.layers[1].mixer == AttentionSpec(heads=4, kv_heads=2, dim=24, vdim=40, scale=2.5 * 24 ** -0.5, window=None, taps=3, rot_dims=16,
                                                rot_base=500.0, qk_weights=True, rot_llama=LlamaScaling(3.0, 64.0, 1.0, 4.0))
    assert cfg.layers[2].ff is None
    assert cfg.runs() == [Run(0, 0, False), Run(1, 0, False), Run(0, 1, True), Run(1, 1, False), Run(0, 2, True), Run(1, 2, False), Run(2, 0, False)]
    cc = cfg.cache_config(10, 16, 3, torch.bfloat16, "cpu")
    assert cc.layer_kv == ((2, 32), (2, 40)) * 3 + ((2, 32),) and cc.num_state_slots == 3


@pytest.mark.parametrize("name", ["llz-plain", "llz-odd", "llz-wide", "llz-heads"])
def test_runs_are_the_oracles(name):
    assert [(r.layer, r.again) for r in _config(name).runs()] == lo.layer_runs(hh.CONFIGS[name])


def test_optional_fields():
    def change(d):
        del d["loop"], d["residual_mult"], d["embedding"]
        d["layers"][1]["mixer"].pop("conv")
        d["layers"][1]["mixer"]["rot"]["scaling"] = None
        d["layers"][0]["mlp"] = None
    cfg = _config("llz-plain", change)
    assert (cfg.loop, cfg.residual_mult, cfg.embed_scale) == (None, 1.0, 1.0) and cfg.runs() == [Run(i, 0, False) for i in range(3)]
    m = cfg.layers[1].mixer
    assert m.taps == 0 and m.rot_llama is None and m.rot_dims == 16 and cfg.layers[0].ff is None
    assert _config("llz-plain", lambda d: d["layers"][1]["mixer"].pop("rot")).layers[1].mixer.rot_dims == 0


@pytest.mark.parametrize("change,message", [
    (lambda d: d["layers"][1]["mixer"].update(window=1), "unknown fields"),
    (lambda d: d["layers"][1]["mixer"]["rot"].update(kind=1), "unknown fields"),
    (lambda d: d["layers"][1]["mixer"]["rot"]["scaling"].update(kind=1), "unknown fields"),
    (lambda d: d["layers"][0]["mixer"].update(scale=1), "unknown fields"),
    (lambda d: d["layers"][0]["mixer"]["left"].update(rot=1), "unknown fields"),
    (lambda d: d["layers"][0]["mixer"]["right"].update(conv=1), "unknown fields"),
    (lambda d: d["layers"][0]["mlp"].update(act="gelu"), "unknown fields"),
    (lambda d: d["loop"].update(every=2), "unknown fields"),
    (lambda d: d["layers"][0].update(type="other"), "unknown mixer"),
    (lambda d: d["layers"][0]["mlp"].update(kind="moe"), "unknown feed-forward"),
    (lambda d: d["layers"][0]["mixer"]["left"].update(kv_heads=3), "multiple of kv_heads"),
    (lambda d: d["layers"][0]["mixer"]["left"].update(dim=264), "above 256"),
    (lambda d: d["layers"][0]["mixer"]["left"].update(heads=130), "above 128"),
    (lambda d: d["layers"][0]["mixer"]["right"].update(dim=264), "above 256"),
    (lambda d: d["layers"][1]["mixer"]["rot"].update(dims=7), "must be even"),
    (lambda d: d["loop"].update(stop=4), "of 3 layers"),
    (lambda d: d["loop"].update(start=2), "of 3 layers"),
    (lambda d: d["loop"].update(times=0), "of 3 layers"),
])
def test_configs_that_are_refused(change, message):
    with pytest.raises(ValueError, match=message):
        _config("llz-plain", change)


def test_combinations_that_are_refused():
    layer = LayerSpec(TalkingSpec(2, 1, 8, 8, 0.5), MLPSpec(8, "relu2"))
    make = lambda **kw: HybridConfig(vocab_size=8, width=8, layers=(layer,), norm_eps=1e-5, **kw)
    for kw, message in ((dict(norm="rms", residual_mult=0.5), "residual_mult"), (dict(both_norms=True), "both sides"),
                        (dict(norm="rms", both_norms=True, post_norm=True), "both sides"), (dict(norm="rms", positions=4, loop=Loop(0, 1, 2)), "run again")):
        with pytest.raises(ValueError, match=message):
            make(**kw)


def _load(tmp_path, name, dtype=torch.float32):
    cfg = hh.CONFIGS[name]
    w = hh.weights(cfg)
    path = hh.save(tmp_path, cfg, w)
    options = registry.LoadOptions(num_blocks=4, block_size=16, num_state_slots=2, max_positions=50, dtype=dtype, device="cpu")
    return registry.load_model(path, options), cfg, w, path


def test_checkpoint_is_loaded_into_joint_weights(tmp_path):
    assert registry.find(hh.CONFIGS["llz-plain"]).name == "loluzen"
    model, cfg, w, path = _load(tmp_path, "llz-plain", torch.bfloat16)
    assert isinstance(model, HybridDecoder) and registry.model_len(path, 5000) == 5000
    p = model.layers[0].mixer
    left = [w[f"l0.mix.left.{n}"] for n in "qkvg"]
    assert torch.equal(p.left.w_in[: sum(map(len, left))], torch.cat(left)) and p.w_in.shape[0] % 8 == 0
    assert torch.equal(p.left.bias, torch.cat([w[f"l0.mix.left.{n}.b"] for n in "qkv"]).float())
    assert torch.equal(p.left.talk, w["l0.mix.left.talk"].float()) and torch.equal(p.left.bias_rate, w["l0.mix.left.r2"].float())
    right = torch.cat([w[f"l0.mix.right.{n}"] for n in "qfv"])
    assert torch.equal(p.right.w_in[: len(right)], right) and p.right.w_in.data_ptr() == p.w_in[p._in:].data_ptr()
    assert torch.equal(p.right.norm, w["l0.mix.right.norm"].float().repeat(3)) and torch.equal(p.right.lower, w["l0.mix.right.lower"].float())
    assert torch.equal(p.right_norm, 0.5 * w["l0.mix.right.out"].float()) and torch.equal(p.left.w_out, w["l0.mix.left.o"])
    layer = model.layers[0]
    assert torch.equal(layer.norm1.w, 1 + w["l0.norm1"].float()) and torch.allclose(layer.norm2b.w, 1.2 * (1 + w["l0.norm2b"].float()))
    assert torch.equal(model.norm.w, 1 + w["final.norm"].float())
    assert torch.equal(layer.mlp.in_bias, w["l0.mlp.up.b"].float()) and torch.equal(layer.mlp.w_out, w["l0.mlp.down"])
    att = model.layers[1].mixer
    assert torch.equal(att.conv, torch.cat([w[f"l1.mix.{n}.conv"] for n in "qkv"]).float().T) and torch.equal(att.q_norm, w["l1.mix.q.norm"].float())
    before = {k: v.clone() for k, v in model.state_dict().items()}
    model.load_state_dict(w)  # (again: nothing is shifted or scaled twice)
    assert all(torch.equal(v, before[k]) for k, v in model.state_dict().items())
    with pytest.raises(KeyError, match="lacks l1.norm2b"):
        model.load_state_dict({k: v for k, v in w.items() if k != "l1.norm2b"})
    with pytest.raises(ValueError, match="talk"):
        model.load_state_dict({**w, "l0.mix.left.talk": w["l0.mix.left.talk"][:-1]})
    with pytest.raises(KeyError, match="does not know"):
        model.load_state_dict({**w, "l1.mix.q.b": w["l1.mix.q.norm"]})


def test_every_turn_has_its_own_pool_and_state(tmp_path):
    model, _, _, _ = _load(tmp_path, "llz-plain")
    shapes = {k: tuple(v.shape) for k, v in model.backend.state.items()}
    channels = (4 + 2) * 24 + 2 * 40
    assert shapes == {**{(at, "hgrn2"): (2, 3, 16, 48) for at in (0, 2, 4, 6)}, **{(at, "conv"): (2, 2, channels) for at in (1, 3, 5)}}
    assert model.layers[0].mixer.site.places == (0, 2, 4) and model.layers[2].mixer.site.places == (6,)
    assert len({t.data_ptr() for t in model.backend.k_cache}) == 7
    assert [t is model.backend.state[at, "conv"] for at, t in zip((1, 3, 5), model.layers[1].mixer.conv_state)] == [True] * 3


@pytest.mark.parametrize("base,dims,scaling", [(700.0, 12, (2.0, 40, 1.0, 4.0)), (10000.0, 128, (8.0, 8192, 1.0, 4.0)), (50.0, 2, (3.0, 7, 0.5, 0.6)),
                                               (5e5, 64, (32.0, 2048, 2.0, 16.0)), (9.0, 6, (4.0, 3, 1.0, 1.0))])
def test_rotary_tables(base, dims, scaling):
    names = ("factor", "original", "low", "high")
    want = torch.tensor(lo.pair_turns({"base": base, "dims": dims, "scaling": dict(zip(names, scaling))}), dtype=torch.float64)
    spec = LlamaScaling(*scaling)
    assert torch.allclose(llama_frequencies(base, dims, spec), want, rtol=1e-12)
    tables = RotaryTables(30, "cpu")
    table = tables.get(base, dims, 1.0, spec)
    assert torch.allclose(table[29].double(), torch.stack([(29 * want).cos(), (29 * want).sin()], -1), atol=1e-6)
    assert tables.get(base, dims, 1.0, spec) is table and tables.get(base, dims, 1.0) is not table
    assert math.isfinite(float(table.sum()))
