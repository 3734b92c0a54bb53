"""The host side of Tevirax without a GPU: configuration, registry, checkpoint loading into joint and re-ordered weights, rotary
tables, chunk masks in the decode plan, and the tile arithmetic of the expert products."""

import copy
import os
import subprocess

import pytest
import torch

from oracle import tevirax_oracle as to
from research_amd.inference import HybridDecoder, registry
from research_amd.inference.hybrid import tevirax_config
from research_amd.inference.mixers import AttentionSpec, Mamba2Spec, MlstmSpec, ParallelSpec, RotaryTables, Site, YarnScaling, yarn_frequencies
from research_amd.inference.moe import MoESpec
from tests import hybrid_helpers as hh

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


def test_config_reader():
    cfg = tevirax_config(hh.CONFIGS["tvx-odd"])
    assert (cfg.width, cfg.vocab_size, cfg.norm_eps, cfg.norm, cfg.post_norm) == (76, 131, 1e-3, "rms", True)
    assert (cfg.embed_scale, cfg.positions, cfg.logit_softcap) == (3.0, 700, 7.0)
    p = cfg.layers[0].mixer
    assert isinstance(p, ParallelSpec) and (p.left_scale, p.right_scale) == (1.4, 0.5) and p.right == MlstmSpec(2, 12, 20, 3.0)
    a = p.left
    assert (a.heads, a.kv_heads, a.dim, a.vdim, a.chunk, a.rot_dims, a.rot_yarn, a.mask_window) == (6, 3, 20, 36, 7, 10, None, -7)
    assert a.rot_halves and a.qk_weights and not a.gates and a.window is None
    assert cfg.layers[1].mixer == Mamba2Spec(heads=6, vdim=20, state=18, groups=3, taps=1, norm_groups=3)
    assert [l.ff for l in cfg.layers] == [None, MoESpec(5, 22, 4), 28, None]
    assert cfg.layers[2].mixer.left.rot_yarn == YarnScaling(3.0, 24.0, 4.0, 0.5)
    cc = cfg.cache_config(10, 16, 3, torch.bfloat16, "cpu")
    assert cc.layer_kv == ((3, 40), None, (1, 48), None) and cc.num_state_slots == 3
    wide = tevirax_config(hh.CONFIGS["tvx-wide"])
    assert wide.layers[1].ff == MoESpec(12, 72, 4, 4, 3, 56)
    assert wide.layers[1].mixer.left.v_slices == 2 and wide.cache_config(1, 16, 1, torch.bfloat16, "cpu").layer_kv[1] == (4, 160)


def test_optional_fields():
    d = copy.deepcopy(hh.CONFIGS["tvx-plain"])
    d["layers"][1]["mixer"]["left"]["mask"] = None
    d["layers"][1]["mixer"]["left"]["rot"] = None
    del d["logit_softcap"], d["layers"][0]["mlp"]
    cfg = tevirax_config(d)
    assert cfg.layers[1].mixer.left.mask_window == 0 and cfg.layers[1].mixer.left.rot_dims == 0
    assert cfg.logit_softcap is None and cfg.layers[0].ff is None


@pytest.mark.parametrize("change,message", [
    (lambda d: d["layers"][0]["mixer"].update(sinks=4), "unknown fields"),
    (lambda d: d["layers"][1]["mixer"]["left"].update(bias=True), "unknown fields"),
    (lambda d: d["layers"][1]["mixer"]["left"]["mask"].update(stride=2), "unknown fields"),
    (lambda d: d["layers"][1]["mixer"]["left"]["rot"]["scaling"].update(kind=1), "unknown fields"),
    (lambda d: d["layers"][1]["mlp"]["router"].update(bias=1), "unknown fields"),
    (lambda d: d["layers"][1]["mlp"]["shared"].update(act="gelu"), "unknown fields"),
    (lambda d: d["layers"][0].update(type="other"), "unknown mixer"),
    (lambda d: d["layers"][0]["mlp"].update(kind="routed"), "unknown feed-forward"),
    (lambda d: d["layers"][1]["mixer"]["left"].update(kv_heads=3), "multiple of kv_heads"),
    (lambda d: d["layers"][1]["mixer"]["left"]["mask"].update(size=0), "chunk"),
    (lambda d: d["layers"][1]["mixer"]["right"].update(dim=260), "above 256"),
    (lambda d: d["layers"][2]["mixer"].update(groups=3), "divide"),
    (lambda d: d["layers"][2]["mixer"].update(norm_groups=7), "divide"),
    (lambda d: d["layers"][2]["mixer"].update(conv=9), "taps"),
    (lambda d: d["layers"][1]["mlp"]["router"]["groups"].update(count=4), "equal groups"),
    (lambda d: d["layers"][1]["mlp"]["router"].update(top=5), "cannot be chosen"),
    (lambda d: d["norm"].update(kind="layer"), "unknown fields"),
])
def test_configs_that_are_refused(change, message):
    d = copy.deepcopy(hh.CONFIGS["tvx-plain"])
    change(d)
    with pytest.raises(ValueError, match=message):
        tevirax_config(d)


def _load(tmp_path, name):
    cfg = hh.CONFIGS[name]
    w = hh.weights(cfg)
    path = hh.save(tmp_path, cfg, w)
    options = registry.LoadOptions(num_blocks=4, block_size=16, num_state_slots=2, max_positions=50, dtype=torch.float32, device="cpu")
    return registry.load_model(path, options), cfg, w, path


def test_registry_and_position_limits(tmp_path):
    assert registry.find(hh.CONFIGS["tvx-plain"]).name == "tevirax"
    model, cfg, w, path = _load(tmp_path, "tvx-plain")
    assert isinstance(model, HybridDecoder) and model.max_positions == 50
    assert registry.model_len(path, 5000) == 700 and registry.model_len(path, 300) == 300
    lotozen = hh.save(tmp_path / "other", hh.CONFIGS["plain"], hh.weights(hh.CONFIGS["plain"]))
    assert registry.model_len(lotozen, 5000) == 5000


def test_checkpoint_is_loaded_into_joint_weights(tmp_path):
    model, cfg, w, _ = _load(tmp_path, "tvx-plain")
    f = lambda name: w[name].float()
    m = model.layers[0].mixer
    assert torch.equal(m.w_in[: f("l0.mix.in").shape[0]], f("l0.mix.in")) and m.w_in.shape[0] % 8 == 0
    assert torch.equal(m.conv, f("l0.mix.conv").T) and torch.allclose(m.rate, f("l0.mix.A_log").exp())
    p = model.layers[1].mixer
    # the halves of a rotated head are stored as pairs, the rest of the head behind them
    order = [j for i in range(6) for j in (i, i + 6)] + list(range(12, 32))
    q = f("l1.mix.left.q").view(4, 32, -1)[:, order].reshape(128, -1)
    assert torch.equal(p.w_in[:128], q) and torch.equal(p.left.q_norm, f("l1.mix.left.q.norm")[order])
    assert torch.equal(p.w_in[192:240], f("l1.mix.left.v"))
    at = 240
    for n in ("q", "k", "v", "g", "i", "f"):
        rows = f(f"l1.mix.right.{n}")
        assert torch.equal(p.w_in[at: at + rows.shape[0]], rows)
        at += rows.shape[0]
    assert torch.equal(p.w_out, torch.cat([f("l1.mix.left.o"), f("l1.mix.right.o")], 1))
    assert torch.allclose(p.right.norm, 1.3 * f("l1.mix.right.norm")) and p.left.out_scale == 0.8
    e = model.layers[1].mlp
    assert tuple(e.w_in.shape) == (6, 128, 128) and tuple(e.w_out.shape) == (6, 88, 64)
    assert torch.equal(e.w_in[4, 64: 88, :88], f("l1.mlp.e4.up")) and not e.w_in[:, 24:64].any() and not e.w_in[..., 88:].any()
    assert torch.equal(e.router, torch.cat([f("l1.mlp.router"), f("l1.mlp.shared.sg")]))
    assert torch.equal(e.w_out[2, :, :24], f("l1.mlp.e2.down")) and not e.w_out[..., 24:].any()
    assert torch.equal(model.pos_embed, f("pos")) and model.norm.b is None
    with pytest.raises(KeyError, match="lacks l1.mlp.e3.up"):
        model.load_state_dict({k: v for k, v in w.items() if k != "l1.mlp.e3.up"})
    with pytest.raises(KeyError, match="does not know"):
        model.load_state_dict({**w, "l1.mlp.e9.up": w["embed"]})
    model.load_state_dict(w)  # (scales on stored weights are applied once)
    assert torch.allclose(p.right.norm, 1.3 * f("l1.mix.right.norm"))


def test_states_belong_to_the_backend(tmp_path):
    model, _, _, _ = _load(tmp_path, "tvx-odd")
    shapes = {k: tuple(v.shape) for k, v in model.backend.state.items()}
    assert shapes == {(0, "mlstm"): (2, 2, 16 * 32 + 32), (1, "ssd"): (2, 6, 32 * 32), (2, "mlstm"): (2, 5, 32 * 16 + 48),
                      (3, "conv"): (2, 5, 2 * 44 + 66), (3, "ssd"): (2, 2, 48 * 48)}


def test_value_heads_in_slices():
    """Copies of keys and queries per slice give the same sums as whole value heads."""
    g = torch.Generator().manual_seed(0)
    spec = AttentionSpec(heads=4, kv_heads=2, dim=6, vdim=300, scale=0.5, window=None, taps=0, rot_dims=0, rot_base=1.0, qk_weights=True,
                         gates=False)
    assert (spec.v_slices, spec.slice_dim, spec.pool_heads, spec.pool_dim) == (2, 150, 4, 152)
    from research_amd.inference.mixers import ConvAttention
    from research_amd.inference.attention import CacheConfig, HipPagedAttentionBackend

    backend = HipPagedAttentionBackend(CacheConfig(1, 4, 152, num_blocks=1, device="cpu", dtype=torch.float32))
    att = ConvAttention(spec, Site(10, 1e-5, (0,), backend, RotaryTables(4, "cpu"), torch.float32, "cpu"))
    w = {"q": torch.randn(24, 10, generator=g), "k": torch.randn(12, 10, generator=g), "v": torch.randn(600, 10, generator=g),
         "o": torch.randn(10, 1200, generator=g), "q.norm": torch.ones(6), "k.norm": torch.ones(6)}
    att.load(lambda n: w[n], "")
    h = torch.randn(5, 10, generator=g)
    u = h @ att.w_in.T
    q, k, v = u[:, :48].view(5, 8, 6), u[:, 48:72].view(5, 4, 6), u[:, 72:672].view(5, 4, 150)
    got = to.chunk_attention(q, k, v, 0.5, None).reshape(5, -1) @ att.w_out.T
    want = to.chunk_attention((h @ w["q"].T).view(5, 4, 6), (h @ w["k"].T).view(5, 2, 6), (h @ w["v"].T).view(5, 2, 300), 0.5, None)
    assert torch.allclose(got, want.reshape(5, -1) @ w["o"].T, atol=1e-3)


@pytest.mark.parametrize("base,dims,yarn", [(700.0, 12, (2.0, 40, 8.0, 1.0)), (10000.0, 128, (8.0, 4096, 32.0, 1.0)), (50.0, 2, (3.0, 7, 1.0, 1.0)),
                                            (1e6, 64, (40.0, 32768, 32.0, 1.0)), (1000.0, 48, (4.0, 3, 64.0, 60.0))])
def test_rotary_tables(base, dims, yarn):
    names = ("factor", "original", "fast", "slow")
    want, amp = to.yarn_table({"base": base, "dims": dims, "scaling": dict(zip(names, yarn))})
    freq, size = yarn_frequencies(base, dims, YarnScaling(*yarn))
    assert size == pytest.approx(amp) and torch.allclose(freq, torch.tensor(want, dtype=torch.float64))
    tables = RotaryTables(30, "cpu")
    table = tables.get(base, dims, 1.0, YarnScaling(*yarn))
    ang = torch.tensor(want, dtype=torch.float64) * 29
    assert torch.allclose(table[29].double(), amp * torch.stack([ang.cos(), ang.sin()], -1), atol=1e-6)
    assert tables.get(base, dims, 1.0) is not table and tables.get(base, 0, 1.0) is None


def test_chunk_and_tile_arithmetic(tmp_path):
    """``decode_plan.h`` and ``moe_plan.h`` in a plain C++ build: the first key of a query and the blocks it reads under a chunk
    mask, and room for every tile that lists of any lengths can make."""
    src = tmp_path / "plan.cpp"
    src.write_text('''
#include "decode_plan.h"
#include "moe_plan.h"
#include "lightning_plan.h"
#include <cstdio>
#include <cstdlib>
#include <initializer_list>
using namespace pa_decode_detail;
int main() {
    for (int size : {1, 2, 7, 16, 64, 100})
        for (int len = 1; len < 400; ++len) {
            const int first = (len - 1) / size * size;
            if (plan_first_key(len, -size) != first) return 1;
            for (int bs : {1, 16, 48})
                if (plan_blocks_of(len, bs, -size) != (len - 1) / bs - first / bs + 1) return 2;
        }
    if (plan_first_key(0, -5) != 0 || plan_blocks_of(0, 16, -5) != 0 || plan_window_span(-9) != 9 || plan_window_span(4) != 4) return 3;
    std::srand(1);
    for (int round = 0; round < 3000; ++round) {
        const int experts = 1 + std::rand() % 40, bm = 1 << (std::rand() % 9);
        int64_t items = 0, tiles = 0;
        for (int e = 0; e < experts; ++e) {
            const int c = std::rand() % 3 ? std::rand() % (1 + std::rand() % 500) : 0;
            items += c;
            tiles += (c + bm - 1) / bm;
        }
        if (tiles > moe_max_tiles(items, experts, bm)) return 4;
    }
    for (long long rows = 1; rows < 3000000; rows = rows * 3 / 2 + 1)
        for (int top : {1, 3, 8, 64}) {
            const long long part = moe_part_rows(rows, top), parts = moe_parts(rows, top);
            if (part < 1 || part * top > 8192 || part * parts < rows || part * (parts - 1) >= rows) return 7;
        }
    if (moe_shape(7, 8) != kMoeStream || moe_shape(1 << 20, 8) != kMoeTile256) return 5;
    if (gl_state_floats(true, 20, 130) != 32 * 144 + 3 * 48 || gl_workspace_bytes(2, 3, 20, 40, 4) != 2ull * 3 * 4 * (32 * 48 + 48) * 4) return 6;
    std::puts("ok");
}
''')
    exe = tmp_path / "plan"
    subprocess.run(["g++", "-std=c++17", "-I", os.path.join(ROOT, "research_amd", "csrc"), str(src), "-o", str(exe)], check=True)
    assert subprocess.run([str(exe)], stdout=subprocess.PIPE).returncode == 0
