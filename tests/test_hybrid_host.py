"""The host side of hybrid decoders without a GPU: configuration, registry, checkpoint loading, the allocator with state
slots, scheduling in portions, cache configuration, and the segment arithmetic of the linear-attention kernels."""

import copy
import os
import random
import subprocess

import pytest
import torch

from research_amd.inference import HipPagedAttentionBackend, HybridDecoder, InferenceContext
from research_amd.inference import registry
from research_amd.inference.attention import CacheConfig
from research_amd.inference.cache import PrivateKVCache
from research_amd.inference.hybrid import lotozen_config
from research_amd.inference.mixers import AttentionSpec, LightningSpec
from research_amd.inference.scheduler import schedule, step_tokens
from research_amd.inference.trace import parse_args
from research_amd.inference.types import SchedulerConfig, Sequence, SequenceStatus
from tests import hybrid_helpers as hh

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


# ------------------------------------------------------------------ configuration and registry


def test_config_reader():
    cfg = lotozen_config(hh.CONFIGS["odd"])
    assert (cfg.width, cfg.vocab_size, cfg.norm_eps, cfg.side_dim) == (76, 131, 1e-3, 5)
    assert [type(l.mixer) for l in cfg.layers] == [LightningSpec, AttentionSpec, AttentionSpec, LightningSpec, AttentionSpec]
    assert [l.ff for l in cfg.layers] == [52, None, 28, None, 30]
    assert cfg.v_roles() == [None, None, "first", None, "mix"]
    a = cfg.layers[2].mixer
    assert (a.heads, a.kv_heads, a.dim, a.vdim, a.window, a.taps, a.rot_dims, a.rot_base, a.rot_factor) == (3, 1, 44, 36, 33, 5, 44, 50.0, 3.0)
    assert a.pool_dim == 48 and a.channels == 4 * 44 + 36
    assert cfg.layers[3].mixer.decay == (0.0, 0.5, 0.9, 0.99, 1.0)
    cc = cfg.cache_config(10, 16, 3, torch.bfloat16, "cpu")
    assert cc.layer_kv == (None, (3, 40), (1, 48), None, (1, 40)) and cc.num_state_slots == 3 and cc.kv_shape(2) == (1, 48)


def test_optional_fields():
    d = copy.deepcopy(hh.CONFIGS["no-mixing"])
    del d["token_side"]
    for layer in d["layers"][:2]:
        layer["mixer"]["rot"].pop("scaling")
        layer["mixer"].pop("v_mix")
    cfg = lotozen_config(d)
    assert cfg.side_dim == 0 and cfg.v_roles() == [None, None, None]
    assert cfg.layers[0].mixer.rot_factor == 1.0


@pytest.mark.parametrize("change,message", [
    (lambda d: d["layers"][0]["mixer"].update(sinks=4), "unknown fields"),
    (lambda d: d["layers"][0]["mixer"]["mask"].update(stride=2), "unknown fields"),
    (lambda d: d["layers"][0].update(type="other"), "unknown mixer"),
    (lambda d: d["layers"][0]["mlp"].update(kind="routed"), "unknown feed-forward"),
    (lambda d: d["layers"][0]["mixer"].update(kv_heads=3), "multiple of kv_heads"),
    (lambda d: d["layers"][0]["mixer"]["rot"].update(dims=13), "rot_dims"),
    (lambda d: d["layers"][0]["mixer"]["mask"].update(size=0), "window"),
    (lambda d: d["layers"][1]["mixer"].update(decay=[0.5]), "decays"),
    (lambda d: d["layers"][2]["mixer"].update(vdim=16), "value heads"),
])
def test_configs_that_are_refused(change, message):
    d = copy.deepcopy(hh.CONFIGS["plain"])
    change(d)
    with pytest.raises(ValueError, match=message):
        lotozen_config(d)


def test_registry_picks_the_design_by_config():
    assert registry.find(hh.CONFIGS["plain"]).name == "lotozen"
    assert registry.find({"num_attention_heads": 4, "model_type": "llama"}).name == "llama"
    with pytest.raises(ValueError, match="no registered model"):
        registry.find({"architecture": "Other"})
    with pytest.raises(ValueError, match="registered already"):
        registry.register(registry.ModelEntry("llama", lambda c: False, None))


# ------------------------------------------------------------------ loading


@pytest.fixture
def loaded(tmp_path):
    cfg, w = hh.CONFIGS["plain"], hh.weights(hh.CONFIGS["plain"])
    path = hh.save(tmp_path, cfg, w)
    options = registry.LoadOptions(num_blocks=4, block_size=16, num_state_slots=2, max_positions=50, dtype=torch.float32, device="cpu")
    return registry.load_model(path, options), cfg, w


def test_checkpoint_folder_is_loaded_into_joint_projections(loaded):
    model, cfg, w = loaded
    assert isinstance(model, HybridDecoder)
    a = model.layers[0].mixer
    assert torch.equal(a.w_in[:200], torch.cat([w["l0.mix.q"], w["l0.mix.k"], w["l0.mix.v"], w["l0.mix.g"][:]])[:200].float()[:200])
    assert torch.equal(a.w_in[240:244], w["l0.mix.g"].float()) and not a.w_in[244:].any()
    assert torch.equal(a.conv[1, 128:192], w["l0.mix.k.conv"][:, 1].float())
    assert torch.equal(model.layers[2].mixer.v_lambda, w["l2.mix.vmix"].float().reshape(1))
    l = model.layers[1]
    assert torch.equal(l.mixer.w_in[48:96], w["l1.mix.k"].float()) and torch.equal(l.mlp.w_in[40:], w["l1.mlp.up"].float())
    assert torch.equal(l.mixer.decay_powers[:, 64], torch.tensor([0.7, 0.98, 0.9995], dtype=torch.float64).pow(64).float())
    assert torch.equal(l.norm2.b, w["l1.norm2.b"].float()) and torch.equal(model.side_embed, w["side.embed"].float())
    rope = a.site.rotary.get(1000.0, 12, 2.0)
    assert tuple(rope.shape) == (50, 6, 2)
    angle = torch.tensor(49 * 1000.0 ** (-4 / 12) / 2.0, dtype=torch.float64)
    assert torch.allclose(rope[49, 2].double(), torch.stack([angle.cos(), angle.sin()]), atol=1e-7)


def test_loading_refuses_wrong_checkpoints(loaded):
    model, cfg, w = loaded
    with pytest.raises(KeyError, match="lacks l1.mix.norm"):
        model.load_state_dict({k: v for k, v in w.items() if k != "l1.mix.norm"})
    with pytest.raises(ValueError, match="l0.mix.o"):
        model.load_state_dict({**w, "l0.mix.o": w["l0.mix.o"][:, :-1]})
    with pytest.raises(KeyError, match="does not know"):
        model.load_state_dict({**w, "l9.extra": w["embed"]})
    model.load_state_dict({**w, "l9.extra": w["embed"]}, strict=False)


def test_state_belongs_to_the_backend(loaded):
    model, _, _ = loaded
    state = model.backend.state
    assert sorted(state) == [(0, "conv"), (1, "lightning"), (2, "conv")]
    assert tuple(state[0, "conv"].shape) == (2, 3, 240) and tuple(state[1, "lightning"].shape) == (2, 3, 16, 32)
    state[1, "lightning"].fill_(1.0)
    model.backend.k_cache[0].fill_(1.0)
    model.backend.clear_cache()
    assert not state[1, "lightning"].any() and not model.backend.k_cache[0].any() and model.backend.k_cache[1] is None
    with pytest.raises(ValueError, match="registered already"):
        model.backend.register_state(0, "conv", (1,), torch.float32)
    plain = HipPagedAttentionBackend(CacheConfig(1, 1, 8, num_blocks=1, device="cpu"))
    with pytest.raises(ValueError, match="num_state_slots"):
        plain.register_state(0, "conv", (1,), torch.float32)


def test_cache_config_hash_only_grows_with_the_extensions():
    base = CacheConfig(2, 1, 8)
    assert hash(base) == hash(CacheConfig(2, 1, 8, layer_kv=None, num_state_slots=0))
    assert hash(base) != hash(CacheConfig(2, 1, 8, num_state_slots=2)) != hash(CacheConfig(2, 1, 8, layer_kv=((1, 8), None)))


# ------------------------------------------------------------------ packed contexts


def _ctx(**kw):
    base = dict(is_prefill=True, slot_mapping=[0, 16, 17, 18, 32], block_tables=((0,), (1,), (2,)), seq_lens=(7, 3, 1),
                q_lens=(1, 3, 1), num_decodes=1, state_slots=(1, 0, -1))
    base.update(kw)
    return InferenceContext(**base)


@pytest.fixture
def host_backend(loaded, monkeypatch):
    """The backend with its device check taken out: contexts are integers, which a CPU holds as well."""
    monkeypatch.setattr(HipPagedAttentionBackend, "_require_device", lambda self, *tensors: tensors[0].device)
    return loaded[0].backend


def test_packed_step(host_backend):
    backend = host_backend
    step = backend.packed_step(_ctx())
    assert step.num_rows == 5 and step.num_decodes == 1
    assert step.rows.ctx_lens.tolist() == [7, 3, 1] and step.rows.q_starts.tolist() == [0, 1, 4]
    assert step.rows.tiles.tolist() == [[0, 0], [1, 0], [2, 0]] and step.rows.max_q_len == 3
    assert step.decodes.ctx_lens.tolist() == [7] and step.decodes.q_lens is None and step.decodes.state_slots.tolist() == [1]
    assert step.chunks.q_lens.tolist() == [3, 1] and step.chunks.q_starts.tolist() == [1, 4] and step.chunks.state_slots.tolist() == [0, -1]
    long = backend.packed_step(_ctx(slot_mapping=[-1] * 54, seq_lens=(7, 40, 20), q_lens=(1, 33, 20)))
    assert long.rows.tiles.tolist() == [[0, 0], [1, 0], [1, 16], [1, 32], [2, 0], [2, 16]]
    single = backend.packed_step(_ctx(slot_mapping=[0, 16, 32], q_lens=None))
    assert single.num_decodes == 3 and single.chunks is None and single.rows.tiles is None


@pytest.mark.parametrize("kw,error", [
    (dict(q_lens=(1, 3)), ValueError), (dict(q_lens=(1, 4, 0)), ValueError), (dict(q_lens=(1, 3, 2)), ValueError),
    (dict(num_decodes=2), ValueError), (dict(state_slots=(1, 2, 0)), IndexError), (dict(slot_mapping=[0, 1]), IndexError),
    (dict(slot_mapping=[0, 16, 17, 18, 64]), IndexError)])
def test_packed_contexts_that_are_refused(host_backend, kw, error):
    with pytest.raises(error):
        host_backend.packed_step(_ctx(**kw))


# ------------------------------------------------------------------ allocator


def test_private_cache_hands_out_blocks_and_slots():
    c = PrivateKVCache(6, 4, num_state_slots=2)
    assert c.allocate(1, list(range(5))) == (0, 1) and c.state_slot(1) == 0 and c.num_tokens(1) == 5
    assert c.allocate(2, list(range(5))) == (2, 3) and c.state_slot(2) == 1  # equal tokens, blocks of its own
    assert not c.can_allocate(1) and c.get_cached_tokens(1) == 0
    with pytest.raises(RuntimeError, match="state slot"):
        c.allocate(3, [1])
    assert c.append_token(1, 0) is None and [c.append_token(1, 0) for _ in range(3)] == [None, None, 4]
    c.extend(2, 7)
    assert c.get_block_ids(2) == (2, 3, 5) and c.num_free_blocks() == 0
    with pytest.raises(RuntimeError, match="No free blocks"):
        c.extend(1, 10)
    assert c.num_tokens(1) == 9
    c.deallocate(1)
    c.deallocate(1)
    assert c.num_free_blocks() == 3 and c.state_slot(1) == -1 and c.can_allocate(12) and not c.can_allocate(13)
    with pytest.raises(RuntimeError, match="needs 4"):
        c.allocate(3, [0] * 13)
    assert len(c.allocate(3, [0] * 12)) == 3 and c.state_slot(3) == 0


def test_private_cache_random_operations():
    rnd = random.Random(3)
    c, live = PrivateKVCache(20, 3, num_state_slots=4), {}
    for i in range(2000):
        if rnd.random() < 0.4 and len(live) < 4:
            n = rnd.randint(1, 12)
            if c.can_allocate(n):
                c.allocate(i, [0] * n)
                live[i] = n
        elif live and rnd.random() < 0.5:
            s = rnd.choice(list(live))
            if c.num_free_blocks():
                c.append_token(s, 0)
                live[s] += 1
        elif live:
            s = rnd.choice(list(live))
            c.deallocate(s)
            del live[s]
        held = [b for s in live for b in c.get_block_ids(s)]
        slots = [c.state_slot(s) for s in live]
        assert len(held) == len(set(held)) == sum(-(-n // 3) for n in live.values()) == 20 - c.num_free_blocks()
        assert len(set(slots)) == len(live) and all(0 <= s < 4 for s in slots)


# ------------------------------------------------------------------ scheduling in portions


def _seq(i, n, computed=0, running=False):
    return Sequence(i, [0] * n, [], n, SequenceStatus.RUNNING if running else SequenceStatus.WAITING, 0.0, 5, frozenset(), [],
                    num_computed=computed)


def test_schedule_counts_portions():
    cfg = SchedulerConfig(max_batch_size=4, max_tokens_per_batch=20, block_size=4, prefill_portion=8)
    running = [_seq(0, 30, 29, True), _seq(1, 30, 16, True)]  # a decode, and the next portion of a prompt
    waiting = [_seq(2, 50), _seq(3, 3), _seq(4, 2)]
    assert [step_tokens(s, cfg) for s in running + waiting] == [1, 8, 8, 3, 2]
    out = schedule(waiting, running, 100, cfg)
    assert out.decode_seqs == (0, 1) and out.prefill_seqs == (2, 3)  # 1 + 8 + 8 + 3 tokens
    assert schedule(waiting, running, 12, cfg).prefill_seqs == ()    # blocks for the whole prompt are reserved
    whole = SchedulerConfig(max_batch_size=4, max_tokens_per_batch=20, block_size=4)
    assert schedule(waiting, running, 100, whole).prefill_seqs == ()  # 50 tokens do not fit at once
    assert schedule(waiting[1:], running, 100, whole).prefill_seqs == (3, 4)


def test_trace_arguments():
    a = parse_args(["--model", "m", "--dtype", "float32", "--out", "o", "--max-tokens", "128"])
    assert (a.model, a.dtype, a.out, a.max_tokens, a.max_sequences) == ("m", "float32", "o", 128, 4)


# ------------------------------------------------------------------ segments


def test_segment_arithmetic(tmp_path):
    """``lightning_plan.h`` in a plain C++ build: segments cover every portion once, never crowd the compute units and are
    never shorter than their fixed cost is worth."""
    src = tmp_path / "plan.cpp"
    src.write_text('''
#include "lightning_plan.h"
#include <cstdio>
#include <initializer_list>
int main() {
    for (int cus : {64, 256})
        for (long long wgs : {1LL, 3LL, 32LL, 100LL, 256LL, 4000LL})
            for (int len = 1; len < 40000; len = len * 3 / 2 + 1) {
                const int s = la_segments(wgs, cus, len), rows = la_segment_rows(len, s);
                const long long chunks = (len + kLaChunk - 1) / kLaChunk;
                if (s < 1 || s > kLaMaxSegments || rows % kLaChunk || (long long)s * rows < len) return 1;
                if (s > 1 && (wgs * s > cus || chunks / s < kLaMinSegChunks)) return 2;
                if (la_workspace_bytes(2, 3, 20, 40, s) != (s > 1 ? 2ull * 3 * s * 32 * 48 * 4 : 0)) return 3;
            }
    if (la_segments(1, 256, 100000) != 64 || la_segments(32, 256, 16384) != 8 || la_segments(256, 256, 16384) != 1) return 4;
    std::puts("ok");
}
''')
    exe = tmp_path / "plan"
    subprocess.run(["g++", "-std=c++17", "-I", os.path.join(ROOT, "research_amd", "csrc"), str(src), "-o", str(exe)], check=True)
    assert subprocess.run([str(exe)], stdout=subprocess.PIPE).returncode == 0
