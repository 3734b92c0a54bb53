"""Hybrid decoders on the GPU, loaded from a checkpoint folder and run by the engine, against the oracle's forward:
whole prompts, portions, single tokens, mixed batches with blocks and slots used again, and generation."""

import io
import json
import os

import numpy as np
import pytest
import torch

from research_amd.inference import EngineConfig, InferenceEngine, SamplingParams
from tests import hybrid_helpers as hh
from tests.gpu_helpers import announce

pytestmark = pytest.mark.gpu

F32_TOL = 2e-5


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    made = {}

    def get(name):
        if name not in made:
            cfg = hh.CONFIGS[name]
            w = hh.weights(cfg)
            made[name] = (hh.save(tmp_path_factory.mktemp(name), cfg, w), cfg, w)
        return made[name]
    return get


def _engine(path, dtype, blocks=40, slots=4, max_len=640, **kw):
    return InferenceEngine(EngineConfig(model_path=path, cache_type="private", block_size=16, max_batch_size=slots,
                                        max_model_len=max_len, num_kv_blocks=blocks, dtype=dtype, **kw))


class Wanted:
    """The oracle's logits of one sequence, and how far from them each position may be."""

    def __init__(self, cfg, w, tokens, dtype):
        with torch.no_grad():
            self.logits = hh.forward(w, cfg, tokens)
            self.tol = torch.full((len(tokens),), F32_TOL, dtype=torch.float64)
            if dtype == "bfloat16":
                self.tol = hh.bf16_tolerance(hh.forward, cfg, w, tokens, self.logits)
        self.scale = self.logits.pow(2).mean().sqrt()

    def check(self, got, places, what):
        want = self.logits[places]
        err = (got.double() - want) - (got.double() - want).mean(-1, keepdim=True)
        err = err.pow(2).mean(-1).sqrt() / self.scale
        assert torch.isfinite(got).all()
        assert (err < self.tol[places]).all(), (what, int((err / self.tol[places]).argmax()), float(err.max()))


def _wanted(cfg, w, prompts, dtype):
    return [Wanted(cfg, w, p, dtype) for p in prompts]


def _rows(engine, hidden, lo, n):
    with torch.no_grad():
        return engine.model.logits(hidden[lo: lo + n]).float().cpu()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(hh.CONFIGS))
def test_whole_prompts_of_unequal_length_in_one_batch(folders, name, dtype):
    announce(f"hybrid whole {name} {dtype}")
    path, cfg, w = folders(name)
    prompts = hh.prompts(cfg, [1, 2, 3, 90])
    engine = _engine(path, dtype)
    seqs = [engine.open_sequence() for _ in prompts]
    hidden, first = engine.feed(list(zip(seqs, prompts)))
    for p, at, want in zip(prompts, first, _wanted(cfg, w, prompts, dtype)):
        want.check(_rows(engine, hidden, at, len(p)), slice(None), len(p))
    for s in seqs:
        engine.close_sequence(s)
    assert engine.cache.num_free_blocks() == 40 and len(engine.cache.free_state_slots) == 4


@pytest.mark.parametrize("name", ["odd", "tvx-odd", "tvx-wide", "vsx-plain", "vsx-odd", "vsx-wide", "llz-plain", "llz-odd", "llz-wide",
                                  "llz-heads"])
def test_residual_after_every_layer(folders, name):
    announce(f"hybrid layers {name}")
    path, cfg, w = folders(name)
    (prompt,) = hh.prompts(cfg, [37])
    want = []
    hh.forward(w, cfg, prompt, trace=want)
    engine = _engine(path, "float32")
    forward, got = engine.model.forward, []
    engine.model.forward = lambda ids, pos, ctx: forward(ids, pos, ctx, got)
    engine.feed([(engine.open_sequence(), prompt)])
    for i, (g, x) in enumerate(zip(got, want)):
        assert (g.cpu().double() - x).abs().max() < 1e-4, i
    assert len(got) == len(want) == len(engine.model.runs) >= len(cfg["layers"])


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(hh.CONFIGS))
def test_portions_and_token_by_token(folders, name, dtype):
    """The same sequence whole, one token at a time and in portions of changing size: every position's logits."""
    announce(f"hybrid portions {name} {dtype}")
    path, cfg, w = folders(name)
    (prompt,) = hh.prompts(cfg, [110], seed=4)
    (want,) = _wanted(cfg, w, [prompt], dtype)
    engine = _engine(path, dtype)
    for cut in ([1] * 110, [2] * 55, [2, 3, 2, 15, 16, 17, 2, 1, 1, 31, 20], [64, 1, 45], [63, 2, 1, 1, 43]):
        assert sum(cut) == 110
        seq, at = engine.open_sequence(), 0
        for n in cut:
            hidden, _ = engine.feed([(seq, prompt[at: at + n])])
            want.check(_rows(engine, hidden, 0, n), slice(at, at + n), (cut[:3], at))
            at += n
        engine.close_sequence(seq)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["plain", "odd", "tvx-plain", "tvx-odd", "vsx-plain", "vsx-odd", "vsx-wide",
                                  "llz-plain", "llz-odd", "llz-heads"])
def test_mixed_batches_use_blocks_and_slots_again(folders, name, dtype):
    """Up to three live sequences in a pool that barely holds them: portions of some beside single tokens of others,
    sequences that pause, and successors in the blocks and state slots of the ones that ended."""
    announce(f"hybrid mixed {name} {dtype}")
    path, cfg, w = folders(name)
    g = np.random.default_rng(8)
    prompts = hh.prompts(cfg, [70, 33, 90, 5, 64, 41, 17, 80], seed=6)
    want = _wanted(cfg, w, prompts, dtype)
    engine = _engine(path, dtype, blocks=16, slots=3, max_len=96)
    waiting, live, at, used = list(range(len(prompts))), {}, {}, set()
    while waiting or live:
        while waiting and len(live) < 3:
            held = sum(-(-len(prompts[i]) // 16) for i in live)
            if held + -(-len(prompts[waiting[0]]) // 16) > 16:
                break
            i = waiting.pop(0)
            live[i], at[i] = engine.open_sequence(), 0
        order = [i for i in live if g.random() < 0.8] or list(live)[:1]
        g.shuffle(order)
        counts = [min(len(prompts[i]) - at[i], int(g.choice([1, 1, 2, 3, 16, 25]))) for i in order]
        hidden, first = engine.feed([(live[i], prompts[i][at[i]: at[i] + n]) for i, n in zip(order, counts)])
        for i, n, row in zip(order, counts, first):
            want[i].check(_rows(engine, hidden, row, n), slice(at[i], at[i] + n), (i, at[i], n))
            at[i] += n
            used.add((i, engine.cache.state_slot(live[i].seq_id)))
            if at[i] == len(prompts[i]):
                engine.close_sequence(live.pop(i))
    assert len({s for _, s in used}) == 3 and len(used) == len(prompts)
    assert engine.cache.num_free_blocks() == 16


def _by_prompt(samples):
    return {s.prompt_tokens: s for s in samples}


@pytest.mark.parametrize("name,kw", [("plain", {}), ("plain", {"use_graphs": True}), ("odd", {"prefill_portion": 7}),
                                     ("no-mixing", {"use_graphs": True, "prefill_portion": 20}),
                                     ("tvx-plain", {"use_graphs": True}), ("tvx-odd", {"prefill_portion": 7}),
                                     ("tvx-wide", {"use_graphs": True, "prefill_portion": 20}),
                                     ("vsx-plain", {"use_graphs": True}), ("vsx-odd", {"prefill_portion": 7}),
                                     ("vsx-wide", {"use_graphs": True, "prefill_portion": 20}),
                                     ("llz-plain", {"use_graphs": True}), ("llz-odd", {"prefill_portion": 7}),
                                     ("llz-heads", {"use_graphs": True, "prefill_portion": 20})])
def test_greedy_generation_through_the_scheduler(folders, name, kw):
    """Long greedy decoding of ragged prompts by ``generate``: the tokens are the oracle's argmax at every position,
    the log probabilities its own; graphs are replayed between eager prefills."""
    announce(f"hybrid generate {name} {kw}")
    path, cfg, w = folders(name)
    engine = _engine(path, "float32", blocks=80, slots=6, max_len=300, **kw)
    prompts = hh.prompts(cfg, [1, 2, 30, 17, 64, 50, 45, 3], seed=3)
    for round_ in range(2 if "use_graphs" in kw else 1):
        samples = _by_prompt(engine.generate(prompts, SamplingParams(temperature=0.0, max_tokens=40 + 60 * round_)))
        for p in prompts:
            s = samples[tuple(p)]
            tokens = list(p) + list(s.completion_tokens)
            with torch.no_grad():
                lp = torch.log_softmax(hh.forward(w, cfg, tokens[:-1])[len(p) - 1:], -1)
            assert len(s.completion_tokens) == 40 + 60 * round_
            assert lp.argmax(-1).tolist() == list(s.completion_tokens)
            assert s.logprobs == pytest.approx(lp.max(-1).values.tolist(), abs=2e-4)
    assert engine.cache.num_free_blocks() == 80


@pytest.mark.parametrize("name", ["plain", "tvx-plain", "vsx-plain", "llz-plain"])
def test_preemption_starts_the_state_over(folders, name):
    announce(f"hybrid preemption {name}")
    path, cfg, w = folders(name)
    engine = _engine(path, "float32", blocks=9, slots=4, max_len=120, prefill_portion=10)
    prompts = hh.prompts(cfg, [30, 25, 28], seed=5)
    samples = _by_prompt(engine.generate(prompts, SamplingParams(temperature=0.0, max_tokens=40)))
    assert engine.num_preemptions > 0
    for p in prompts:
        tokens = list(p) + list(samples[tuple(p)].completion_tokens)
        with torch.no_grad():
            assert hh.forward(w, cfg, tokens[:-1])[len(p) - 1:].argmax(-1).tolist() == tokens[len(p):]


@pytest.mark.parametrize("name,tensor", [("plain", "l0.mix.o"), ("tvx-plain", "l1.mix.left.o"), ("vsx-plain", "l1.mix.uk"), ("llz-plain", "l0.mix.left.talk")])
def test_weight_updates_keep_graphs_and_restart_sequences(folders, name, tensor):
    announce(f"hybrid update {name}")
    path, cfg, _ = folders(name)
    engine = _engine(path, "float32", use_graphs=True)
    prompts = hh.prompts(cfg, [9, 20])
    engine.generate(prompts, SamplingParams(temperature=0.0, max_tokens=5))
    w = hh.weights(cfg, seed=77)
    engine.update_weights(w)
    engine.flush_cache()
    samples = _by_prompt(engine.generate(prompts, SamplingParams(temperature=0.0, max_tokens=12)))
    for p in prompts:
        tokens = list(p) + list(samples[tuple(p)].completion_tokens)
        with torch.no_grad():
            assert hh.forward(w, cfg, tokens[:-1])[len(p) - 1:].argmax(-1).tolist() == tokens[len(p):]
    with pytest.raises(KeyError, match="checkpoint lacks"):
        engine.update_weights({k: v for k, v in w.items() if k != tensor})


@pytest.mark.parametrize("name", ["plain", "tvx-plain", "vsx-plain", "llz-plain"])
def test_trace_replay(folders, tmp_path, name):
    announce(f"hybrid trace {name}")
    from research_amd.inference.trace import replay

    path, cfg, w = folders(name)
    a, b, c = hh.prompts(cfg, [40, 21, 30], seed=9)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:38], "want": [0, 37]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[38:39], "want": []}, {"id": "b", "tokens": b, "want": [20, 5]}], "end": ["b"]},
             {"step": 2, "entries": [{"id": "c", "tokens": c[:2], "want": [1]}, {"id": "a", "tokens": a[39:], "want": [0]}], "end": ["a"]},
             {"step": 3, "entries": [{"id": "c", "tokens": c[2:], "want": [27]}], "end": ["c"]}]
    engine = _engine(path, "float32", blocks=5, slots=2, max_len=80)
    said = io.StringIO()
    replay(engine, [json.dumps(s) + "\n" for s in steps], str(tmp_path), said)
    assert said.getvalue().split("\n") == ["done 0", "done 1", "done 2", "done 3", ""]
    wa, wb, wc = _wanted(cfg, w, [a, b, c], "float32")
    for step, wanted in ((0, [(wa, 0), (wa, 37)]), (1, [(wb, 20), (wb, 5)]), (2, [(wc, 1), (wa, 39)]), (3, [(wc, 29)])):
        got = torch.from_numpy(np.fromfile(os.path.join(tmp_path, f"{step}.f32"), "<f4").reshape(len(wanted), -1))
        for row, (want, place) in zip(got, wanted):
            want.check(row[None], slice(place, place + 1), (step, place))


def test_llama_runs_packed_batches_too(tmp_path):
    """The trace path on the other registered design: portions and single tokens equal its own whole-prompt logits."""
    announce("llama packed")
    from research_amd.inference import CacheConfig, HipPagedAttentionBackend, ModelConfig, PagedLlama

    cfg = ModelConfig(vocab_size=89, hidden_size=64, intermediate_size=96, num_layers=2, num_heads=4, num_kv_heads=2, head_dim=32,
                      max_position_embeddings=256)
    backend = HipPagedAttentionBackend(CacheConfig(num_layers=2, num_kv_heads=2, head_dim=32, num_blocks=20, block_size=16,
                                                   dtype=torch.float32))
    torch.manual_seed(1)
    model = PagedLlama(cfg, backend).float().cuda().eval()
    engine = InferenceEngine(EngineConfig(model_path="", cache_type="private", block_size=16, max_batch_size=4, max_model_len=200,
                                          num_kv_blocks=20), model=model)
    g = np.random.default_rng(0)
    p, q = g.integers(0, 89, 70).tolist(), g.integers(0, 89, 25).tolist()
    s1, s2 = engine.open_sequence(), engine.open_sequence()
    hidden, first = engine.feed([(s1, p), (s2, q)])
    want = [_rows(engine, hidden, first[0], 70), _rows(engine, hidden, first[1], 25)]
    engine.close_sequence(s1)
    engine.close_sequence(s2)
    s1, s2 = engine.open_sequence(), engine.open_sequence()
    for (a, b), (c, d) in (((0, 30), (0, 1)), ((30, 31), (1, 20)), ((31, 69), (20, 24)), ((69, 70), (24, 25))):
        hidden, first = engine.feed([(s1, p[a:b]), (s2, q[c:d])])
        for want_rows, lo, hi, row in ((want[0], a, b, first[0]), (want[1], c, d, first[1])):
            assert (_rows(engine, hidden, row, hi - lo) - want_rows[lo:hi]).abs().max() < 1e-4
