"""The kernels of the Vusalix mechanisms, each against the oracle's function or a plain float64 statement: residual streams,
latent rows and attention over them, capped and biased scores with sinks at the edges of windows, buckets and blocks, the
delta rule (outputs and carried states), the softmax router with identity experts."""

import numpy as np
import pytest
import torch

from oracle import vusalix_oracle as vo
from research_amd import ops
from research_amd.inference import CacheConfig, HipPagedAttentionBackend, InferenceContext
from research_amd.inference.mixers import BiasedAttentionSpec
from tests.gpu_helpers import DEV, announce, assert_close
from tests.test_gpu_tevirax_ops import _i32, _portions, _rand

pytestmark = pytest.mark.gpu

BF, F32 = torch.bfloat16, torch.float32
TOL = {F32: 3e-6, BF: 8e-3}


# ------------------------------------------------------------------ residual streams


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("streams,width", [(1, 64), (2, 37), (3, 260), (4, 1000), (5, 2048), (9, 516), (16, 40), (4, 5000)])
def test_streams_are_mixed_summed_and_normed(streams, width, dtype):
    announce(f"streams {streams} {width} {dtype}")
    rows, m = 6, 3
    table, ids = _rand(9, width, dtype=dtype), torch.tensor([3, 8, 0, 9, -1, 3])
    x = torch.full((rows, streams, width), float("nan"), device=DEV)
    w, h_in = _rand(width, seed=1), _rand(streams, seed=2)
    got = ops.hyper_norm(x, dtype, ids=ids.to(DEV), table=table.to(DEV), sum_weight=h_in.to(DEV), weight=w.to(DEV), eps=1e-3)
    emb = torch.stack([table[i].double() if 0 <= i < 9 else torch.zeros(width, dtype=torch.float64) for i in ids.tolist()])
    want = emb.expand(streams, -1, -1)
    hc = {"in": h_in.double(), "mix": _rand(streams, streams, seed=3).double() * streams ** -0.5, "out": _rand(streams, seed=4).double()}
    assert_close(x.transpose(0, 1), want, 2e-6, "embedding")
    assert_close(got, vo.rms_norm(vo.hyper_sum(want, hc, ""), 1e-3) * w.double(), TOL[dtype], "normed embedding")
    kw = dict(between=hc["mix"].float().to(DEV), into=hc["out"].float().to(DEV))
    y = _rand(rows, width, dtype=dtype, seed=5)
    want = vo.hyper_update(want, y.double(), hc, "")
    assert_close(ops.hyper_norm(x, dtype, y=y.to(DEV), **kw, want="sum"), want.sum(0), 4e-6, "sum")
    assert_close(x.transpose(0, 1), emb.expand(streams, -1, -1), 2e-6, "a sum leaves the streams")
    got = ops.hyper_norm(x, dtype, y=y.to(DEV), **kw, sum_weight=h_in.to(DEV), weight=w.to(DEV), eps=1e-3)
    assert_close(x.transpose(0, 1), want, 4e-6, "update")
    assert_close(got, vo.rms_norm(vo.hyper_sum(want, hc, ""), 1e-3) * w.double(), TOL[dtype], "normed sum")
    # a weighted branch: items of weight 0 have no row, the row's own input and an extra row come along
    items, extra, own, mix = _rand(rows * m, width, dtype=dtype, seed=6), _rand(rows, width, dtype=dtype, seed=7), _rand(rows, width, dtype=dtype, seed=8), _rand(rows, m + 2, seed=9)
    branch = (mix[:, :m, None].double() * items.double().view(rows, m, width)).sum(1) + mix[:, m, None].double() * extra.double() + mix[:, m + 1, None].double() * own.double()
    mix0, items0 = mix.clone(), items.clone().view(rows, m, width)
    mix0[2, 1] = 0
    items0[2, 1] = float("nan")
    branch[2] -= mix[2, 1].double() * items[2 * m + 1].double()
    want = vo.hyper_update(want, branch, hc, "")
    ops.hyper_norm(x, dtype, y=items0.view(-1, width).to(DEV), mix=mix0.to(DEV), y_extra=extra.to(DEV), y_self=own.to(DEV), **kw, weight=w.to(DEV))
    assert_close(x.transpose(0, 1), want, 1e-5, "weighted branch")


# ------------------------------------------------------------------ router


@pytest.mark.parametrize("rows,experts,identity,top,groups,keep,shared", [
    (1, 6, 0, 2, 3, 2, None), (37, 7, 1, 3, 2, 1, "plain"), (130, 5, 3, 4, 1, 1, "plain"), (64, 200, 56, 8, 8, 4, None), (9, 90, 10, 20, 100, 40, "gated"),
    (2000, 13, 3, 4, 4, 2, "plain"), (3, 1, 0, 1, 1, 1, None), (50, 960, 40, 10, 20, 5, "plain"), (70, 2, 6, 3, 2, 1, "plain")])
@pytest.mark.parametrize("renormalize", [False, True])
def test_softmax_choice_with_corrections_and_identity_experts(rows, experts, identity, top, groups, keep, shared, renormalize):
    announce(f"softmax choose {rows} {experts} {identity} {top} {groups} {keep}")
    every = experts + identity
    logits, corr = 2 * _rand(rows, every + (shared == "gated"), seed=rows), 0.4 * _rand(every, seed=1) - 0.3
    c = ops.moe_choose(logits.to(DEV), experts, top, groups, keep, shared, identity, "softmax", 1, renormalize, corr.to(DEV))
    ids, weights, counts, lists = (t.cpu() for t in c)
    scores = torch.softmax(logits[:, :every].double(), -1)
    for r in range(min(rows, 60)):
        want, ww = vo.route(scores[r], corr.double(), top, groups, keep)
        if renormalize:
            ww = [x / (sum(ww) + 1e-20) for x in ww]
        assert ids[r].tolist() == [e if e < experts else -1 for e in want]
        assert weights[r, :top].tolist() == pytest.approx([x if e < experts else 0.0 for e, x in zip(want, ww)], rel=2e-5, abs=1e-30)
        if identity:
            assert float(weights[r, top + 1]) == pytest.approx(sum(x for e, x in zip(want, ww) if e >= experts), rel=2e-5, abs=1e-30)
    assert weights.shape[1] == top + (2 if identity else 1)
    wanted = {None: torch.zeros(rows), "plain": torch.ones(rows), "gated": torch.sigmoid(logits[:, -1])}[shared]
    assert torch.allclose(weights[:, top], wanted, atol=1e-6)
    assert counts.numel() == experts
    for e in range(experts):
        want = torch.nonzero(ids.reshape(-1) == e).reshape(-1)
        assert counts[e] == want.numel() and torch.equal(lists[e, : counts[e]].long(), want)


# ------------------------------------------------------------------ delta rule


class DeltaCase:
    """Random rows of some sequences, the oracle's outputs and states."""

    def __init__(self, lens, heads, groups, dim, vdim, dtype, seed=0, keep=2.0):
        self.heads, self.groups, self.dim, self.vdim, self.dtype, self.lens = heads, groups, dim, vdim, dtype, lens
        self.bias, self.rate = _rand(heads, seed=seed + 1), torch.exp(_rand(heads, seed=seed + 2) - keep)
        self.rows, self.want, self.states = [], [], []
        for i, n in enumerate(lens):
            parts = [_rand(n, w, dtype=dtype, seed=seed + 10 * i + j) for j, w in enumerate((groups * dim, groups * dim, heads * vdim, heads, heads))]
            # neighbouring keys that resemble each other, so that a chunk's system is far from the identity
            parts[1][1::2] = (parts[1][1::2].float() * 0.3 + parts[1][: 2 * (n // 2): 2].float()).to(dtype)
            self.rows.append(torch.cat(parts, 1))
            q, k, v, a, b = (t.double() for t in parts)
            per = heads // groups
            q = (vo.unit(q.view(n, groups, dim)) * dim ** -0.5).repeat_interleave(per, 1)
            k = vo.unit(k.view(n, groups, dim)).repeat_interleave(per, 1)
            o, s = vo.delta_recurrence(q, k, v.view(n, heads, vdim), -self.rate.double() * vo.softplus(a + self.bias.double()), vo.sigmoid(b))
            self.want.append(o.reshape(n, -1))
            self.states.append(s)
        pad = lambda x: -(-x // 16) * 16
        self.state = torch.full((len(lens) + 1, heads, pad(dim), pad(vdim)), float("nan"), device=DEV)

    def run(self, picks, slots, decode=False, chunks=True):
        u = torch.cat([self.rows[b][lo: lo + n] for b, lo, n in picks]).to(DEV)
        sizes = [self.groups * self.dim, self.groups * self.dim, self.heads * self.vdim, self.heads, self.heads]
        q, k, v, a, b = u.split(sizes, 1)
        p = _portions(picks, slots, tiles=False)
        if decode:
            p = ops.Portions(p.ctx_lens, p.state_slots)
        out = torch.full((u.shape[0], self.heads * self.vdim), float("nan"), dtype=self.dtype, device=DEV)
        need = ops.delta_workspace_bytes(len(picks), self.heads, self.dim, self.vdim, p.max_q_len)
        ws = torch.empty(need, dtype=torch.uint8, device=DEV) if chunks and not decode else None
        ops.delta_rule(q, k, v, a, b, self.bias.to(DEV), self.rate.to(DEV), p, self.state, self.heads, self.dim, self.vdim, self.dim ** -0.5, out,
                       heads_per_group=self.heads // self.groups, workspace=ws)
        at = 0
        for i, lo, n in picks:
            assert_close(out[at: at + n], self.want[i][lo: lo + n], 1e-5 if self.dtype == F32 else 8e-3, (i, lo, n))
            at += n

    def check_states(self, slots):
        for i, s in enumerate(self.states):
            got = self.state[slots[i]].cpu().double()
            assert_close(got[:, : self.dim, : self.vdim], s, 2e-5, ("state", i))
            assert not got[:, self.dim:].any() and not got[:, :, self.vdim:].any()


DELTA = [(2, 2, 64, 64, BF), (3, 1, 128, 128, BF), (4, 2, 48, 40, BF), (2, 1, 72, 144, BF), (2, 2, 256, 96, BF), (6, 3, 20, 200, BF), (1, 1, 130, 24, BF),
         (3, 3, 7, 5, BF), (2, 1, 64, 80, F32), (4, 2, 33, 17, F32), (1, 1, 256, 64, F32)]


@pytest.mark.parametrize("heads,groups,dim,vdim,dtype", DELTA)
def test_delta_rule_of_whole_sequences(heads, groups, dim, vdim, dtype):
    announce(f"delta whole {heads} {groups} {dim} {vdim} {dtype}")
    case = DeltaCase([1, 2, 64, 65, 150, 63, 257], heads, groups, dim, vdim, dtype)
    slots = [3, 0, 6, 1, 5, 2, 7]
    case.run([(i, 0, n) for i, n in enumerate(case.lens)], slots)
    case.check_states(slots)


@pytest.mark.parametrize("heads,groups,dim,vdim,dtype", DELTA)
def test_delta_rule_in_portions_and_single_tokens(heads, groups, dim, vdim, dtype):
    announce(f"delta portions {heads} {groups} {dim} {vdim} {dtype}")
    case = DeltaCase([140, 97], heads, groups, dim, vdim, dtype, seed=3)
    for b, cuts in ((0, [2, 1, 64, 1, 66, 2, 4]), (1, [63, 2, 1, 31])):
        at = 0
        for n in cuts:
            case.run([(b, at, n)], [1, 0], decode=n == 1)
            at += n
    case.check_states([1, 0])
    case.run([(1, 0, 97)], [1, 2])  # a slot that held a state, and a portion that starts at position 0
    case.run([(0, 0, 30), (1, 0, 2)], [2, 0])
    case.run([(1, 2, 95), (0, 30, 110)], [2, 0])
    case.check_states([2, 0])


def test_delta_rule_many_heads_take_wide_slices():
    announce("delta wide slices")
    for heads, batch, vdim in ((160, 2, 128), (160, 2, 64), (300, 1, 72)):
        case = DeltaCase([70, 64][:batch], heads, heads // 4, 64, vdim, BF, seed=5)
        case.run([(i, 0, n) for i, n in enumerate(case.lens)], [0, 1])
        case.check_states([0, 1])


@pytest.mark.parametrize("dtype", [F32, BF])
def test_delta_rule_remembers_a_far_token(dtype):
    """Slow decay, one large value at the start, everything else written elsewhere: it is read out long after."""
    announce(f"delta far {dtype}")
    n, dim = 400, 64
    case = DeltaCase([n], 1, 1, dim, 32, dtype, keep=9.0)
    eye = torch.eye(dim)
    k = eye[1 + torch.arange(n) % 40]
    k[0] = eye[0]
    q = k.clone()
    q[-1] = eye[0]
    v = 0.1 * _rand(n, 32)
    v[0] = 10 + torch.arange(32)
    u = torch.cat([q, k, v, torch.full((n, 1), -2.0), torch.full((n, 1), 4.0)], 1).to(dtype)
    case.rows = [u]
    q, k, v, a, b = (t.double() for t in u.split([dim, dim, 32, 1, 1], 1))
    o, s = vo.delta_recurrence(vo.unit(q)[:, None] * dim ** -0.5, vo.unit(k)[:, None], v[:, None], -case.rate.double() * vo.softplus(a + case.bias.double()), vo.sigmoid(b))
    case.want, case.states = [o.reshape(n, -1)], [s]
    assert o[-1].abs().min() > 1
    for cuts in ([n], [399, 1], [2] * 200):
        at = 0
        for c in cuts:
            case.run([(0, at, c)], [0], decode=c == 1)
            at += c
        case.check_states([0])


# ------------------------------------------------------------------ attention with score terms


class Paged:
    """Keys and values of sequences in a pool of 16-token blocks in mixed order, blocks of other contents in between."""

    def __init__(self, lens, kv, kd, vd, dtype, one=False, seed=0):
        g = np.random.default_rng(seed)
        self.bs, self.lens = 16, lens
        need = [-(-n // 16) for n in lens]
        ids = g.permutation(sum(need) + 5)
        self.k = _rand((sum(need) + 5) * 16, kv, kd, seed=seed + 1).to(dtype)
        self.v = self.k if one else _rand((sum(need) + 5) * 16, kv, vd, seed=seed + 2).to(dtype)
        self.tables = np.full((len(lens), max(need) + 2), -1, dtype=np.int32)
        at = 0
        for i, n in enumerate(need):
            self.tables[i, :n] = ids[at: at + n]
            at += n

    def rows(self, pool, i, lo=0):
        p = np.arange(lo, self.lens[i])
        return pool[torch.from_numpy(self.tables[i, p // 16].astype(np.int64) * 16 + p % 16)]


def _scored(paged, picks, q, vdim, dtype, scale, window, decode=False, splits=True, **terms):
    p = _portions(picks, [0] * len(paged.lens), tiles=False)
    if decode:
        p = ops.Portions(p.ctx_lens, p.state_slots)
    k = paged.k.to(DEV)
    v = k if paged.v is paged.k else paged.v.to(DEV)
    rows, heads = q[0].shape[:2]
    tables = torch.from_numpy(paged.tables[[b for b, _, _ in picks]]).to(DEV)
    out = torch.full((rows, heads, vdim), float("nan"), dtype=dtype, device=DEV)
    need = ops.scored_workspace_bytes(len(picks), heads, k.shape[1], sum(t.shape[2] for t in q), vdim, v is k, tables.shape[1] * 16, window) if decode else 0
    ws = torch.empty(need, dtype=torch.uint8, device=DEV) if need and splits else None
    return ops.scored_attention(tuple(t.to(DEV) for t in q), k, v, vdim, p, tables, 16, scale, window, out, workspace=ws,
                                **{n: (t.to(DEV) if torch.is_tensor(t) else t) for n, t in terms.items()})


def _whole(paged, i, q, vdim, scale, window, cap, rel, most, sink):
    """The oracle over a whole sequence: queries only of the asked rows (others are zeros)."""
    k, v = paged.rows(paged.k, i).double(), paged.rows(paged.v, i).double()[..., :vdim]
    return vo.biased_attention(q.double(), k[..., : q.shape[2]], v, scale, window, cap, rel.double(), most, sink.double())


SCORED = [  # heads, kv heads, dim, vdim, window, cap, buckets, bias_max
    (6, 2, 40, 56, 70, 18.0, 16, 90), (4, 1, 64, 32, 33, 5.0, 8, 20), (4, 2, 184, 120, 80, 12.0, 14, 50), (3, 3, 160, 72, 45, None, 10, 60),
    (8, 2, 128, 96, 100, 30.0, 32, 128), (3, 3, 20, 36, 17, None, 4, 9),
    (20, 1, 40, 40, None, 8.0, 12, 300), (2, 1, 136, 200, 64, 15.0, 6, 64), (5, 5, 24, 16, 1, 4.0, 2, 3), (9, 3, 33, 21, 50, 12.0, 10, 40)]


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("heads,kv,dim,vdim,window,cap,buckets,most", SCORED)
def test_biased_attention_in_portions_and_single_rows(heads, kv, dim, vdim, window, cap, buckets, most, dtype):
    announce(f"scored {heads} {kv} {dim} {vdim} {window} {cap} {buckets} {most} {dtype}")
    pad = lambda n: -(-n // 8) * 8
    lens = [1, 2, 150, 97, 330]
    d = pad(max(dim, vdim))
    paged = Paged(lens, kv, d, d, dtype)
    paged.k[..., dim:] = 0
    rel, sink = 1.5 * _rand(buckets, heads, seed=5), 2 * _rand(heads, seed=6)
    spec = BiasedAttentionSpec(heads, kv, dim, vdim, 1.0, window, cap, buckets, most)
    bias = rel[torch.tensor(spec.bucket_of())].t().contiguous()
    scale = 2.0 * dim ** -0.5
    qs = [torch.nn.functional.pad(_rand(n, heads, dim, seed=20 + i), (0, pad(dim) - dim)).to(dtype) for i, n in enumerate(lens)]
    want = [_whole(paged, i, q[..., :dim], vdim, scale, window, cap, rel, most, sink) for i, q in enumerate(qs)]
    kw = dict(softcap=cap or 0.0, bias=bias, sink=sink)
    tol = 6e-6 if dtype == F32 else 1e-2

    def run(picks, lens_now, decode=False):
        old = paged.lens
        got = _scored(paged, picks, (torch.cat([qs[b][lo: lo + n] for b, lo, n in picks]),), vdim, dtype, scale, window or 0, decode, **kw).cpu()
        at = 0
        for b, lo, n in picks:
            assert_close(got[at: at + n], want[b][lo: lo + n], tol, (b, lo, n))
            at += n
        paged.lens = old
    run([(i, 0, n) for i, n in enumerate(lens)], lens)
    run([(2, 148, 2), (4, 15, 40), (3, 90, 7), (4, 300, 30)], lens)
    for places in ([0, 1, 149, 96, 329], [0, 0, 16, 15, 64], [0, 1, 70, 33, 128]):
        run([(i, p, 1) for i, p in enumerate(places)], lens, decode=True)


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("window,most", [(40, 30), (16, 200), (64, 64)])
def test_one_key_at_the_edges_of_the_window(window, most, dtype):
    """One key scores far above all others and carries its own value: it is seen up to window - 1 tokens later, in prompts and
    in decoding, wherever blocks of 16 and tiles of 32 and 64 keys begin."""
    announce(f"scored edge {window} {most} {dtype}")
    n, heads, dim = 260, 4, 32
    rel, sink = _rand(8, heads, seed=2), torch.zeros(heads)
    bias = rel[torch.tensor(BiasedAttentionSpec(heads, 2, dim, dim, 1.0, window, 60.0, 8, most).bucket_of())].t().contiguous()
    for far in (0, 15, 16, 31, 63, 64, 100):
        paged = Paged([n], 2, dim, dim, dtype, seed=far)
        at = int(paged.tables[0, far // 16]) * 16 + far % 16
        paged.k *= 0.1
        paged.v *= 0.1
        paged.k[at], paged.v[at] = 8.0, 50.0
        q = torch.ones(n, heads, dim).to(dtype)
        got = _scored(paged, [(0, 0, n)], (q,), dim, dtype, dim ** -0.5, window, softcap=60.0, bias=bias, sink=sink).cpu().float()
        seen = (got[:, :, 0] > 25).all(1)
        assert seen.tolist() == [far <= i < far + window for i in range(n)]
        rows = [i for i in (far, far + 1, far + window - 1, far + window, far + window + 1) if i < n]
        for i in rows:
            one = _scored(paged, [(0, i, 1)], (q[:1],), dim, dtype, dim ** -0.5, window, decode=True, softcap=60.0, bias=bias, sink=sink).cpu()
            assert bool((one[0, :, 0] > 25).all()) == (i < far + window)


@pytest.mark.parametrize("dtype", [F32, BF])
def test_sinks_and_biases_carry_weight(dtype):
    """Equal scores: the weights are the biases' and the sink's alone."""
    announce(f"scored sink {dtype}")
    n, heads, dim = 90, 3, 16
    paged = Paged([n], 1, dim, dim, dtype)
    paged.k *= 0
    paged.v[:] = 1
    rel = _rand(6, heads, seed=1)
    sink = torch.tensor([-3.0, 0.0, 4.0])
    which = BiasedAttentionSpec(heads, 1, dim, dim, 1.0, 30, 10.0, 6, 25).bucket_of()
    bias = rel[torch.tensor(which)].t().contiguous()
    got = _scored(paged, [(0, 0, n)], (torch.zeros(n, heads, dim).to(dtype),), dim, dtype, 1.0, 30, softcap=10.0, bias=bias, sink=sink).cpu()
    for i in (0, 1, 29, 30, 89):
        total = torch.stack([torch.exp(rel[vo.bucket(x, 6, 25)].double()) for x in range(min(i + 1, 30))]).sum(0)
        assert_close(got[i, :, 0], total / (total + torch.exp(sink.double())), 3e-6 if dtype == F32 else 4e-3, i)


@pytest.mark.parametrize("splits", [False, True])
@pytest.mark.parametrize("heads,rank,rot,window", [(4, 64, 16, None), (16, 128, 32, 700), (20, 200, 64, None), (40, 512, 64, 1500), (3, 24, 8, 5)])
def test_decode_over_latents_with_long_contexts(heads, rank, rot, window, splits):
    announce(f"latent decode {heads} {rank} {rot} {window} {splits}")
    lens = [2000, 1, 17, 900, 64]
    paged = Paged(lens, 1, rank + rot, 0, BF, one=True)
    q = [_rand(len(lens), heads, n, dtype=BF, seed=s) * n ** -0.5 * 3 for s, n in ((1, rank), (2, rot))]
    got = _scored(paged, [(i, n - 1, 1) for i, n in enumerate(lens)], q, rank, BF, 0.9, window or 0, decode=True, splits=splits).cpu()
    for i, n in enumerate(lens):
        rows = paged.rows(paged.k, i)[:, 0].double()[vo.visible(n - 1, window)]
        p = torch.softmax(torch.cat(q, -1)[i].double() @ rows.T * 0.9, -1)
        assert_close(got[i], p @ rows[:, :rank], 1e-2, i)


def test_decode_pieces_with_sinks_and_padding_rows():
    announce("scored pieces")
    heads, dim, lens = 2, 64, [3000, 5]
    paged = Paged(lens, 1, dim, dim, BF)
    rel, sink = _rand(32, heads, seed=3), torch.tensor([6.0, -1.0])
    bias = rel[torch.tensor(BiasedAttentionSpec(heads, 1, dim, dim, 1.0, None, None, 32, 500).bucket_of())].t().contiguous()
    q = _rand(2, heads, dim, dtype=BF, seed=9)
    want = []
    for i, n in enumerate(lens):
        k, v = (paged.rows(t, i)[:, 0].double() for t in (paged.k, paged.v))
        s = q[i].double() @ k.T * 0.2 + rel[[vo.bucket(n - 1 - j, 32, 500) for j in range(n)]].double().T
        e = torch.exp(s)
        want.append(e @ v / (e.sum(-1, keepdim=True) + torch.exp(sink.double())[:, None]))
    for splits in (False, True):
        got = _scored(paged, [(i, n - 1, 1) for i, n in enumerate(lens)], (q,), dim, BF, 0.2, 0, decode=True, splits=splits, bias=bias, sink=sink).cpu()
        assert_close(got, torch.stack(want), 1e-2, splits)


# ------------------------------------------------------------------ latent rows


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("heads,dim,rot,rank", [(3, 24, 8, 40), (2, 72, 16, 120), (5, 20, 10, 30), (1, 0, 6, 17), (16, 128, 64, 512)])
def test_latent_rows_are_normed_turned_and_appended(heads, dim, rot, rank, dtype):
    announce(f"latent append {heads} {dim} {rot} {rank} {dtype}")
    pad = lambda n: -(-n // 8) * 8
    picks = [(0, 5, 1), (1, 0, 40), (2, 30, 2)]
    rows, size = sum(n for _, _, n in picks), dim + rot
    u = _rand(rows, heads * size + rank + rot + 3, dtype=dtype)
    norm, slots = _rand(rank, seed=2), torch.from_numpy(np.random.default_rng(0).permutation(64)[:rows].copy())
    slots[3] = -1
    ang = torch.rand(64, rot // 2, generator=torch.Generator().manual_seed(3)) * 6
    rope = torch.stack([ang.cos(), ang.sin()], -1).contiguous()
    pool = torch.full((64, 1, pad(rank + rot)), 7.0, dtype=dtype, device=DEV)
    q = ops.latent_append(u.to(DEV), _portions(picks, [0, 0, 0]), slots.to(DEV), pool, norm.to(DEV), 1e-4, rope.to(DEV), heads, dim, rot, rank,
                          pad(size) + 8, 0.37).cpu().double()
    pos = torch.cat([torch.arange(lo, lo + n) for _, lo, n in picks])
    c, s = rope[pos].double()[:, None].unbind(-1)

    def turn(x):
        y = torch.empty_like(x)
        y[..., 0::2], y[..., 1::2] = x[..., 0::2] * c - x[..., 1::2] * s, x[..., 1::2] * c + x[..., 0::2] * s
        return y
    x = u.double()
    heads_in = x[:, : heads * size].view(rows, heads, size)
    assert_close(q[..., :size], 0.37 * torch.cat([heads_in[..., :dim], turn(heads_in[..., dim:])], -1), TOL[dtype], "q")
    assert not q[..., size:].any()
    down = x[:, heads * size: heads * size + rank + rot]
    want = torch.cat([vo.rms_norm(down[:, :rank], 1e-4) * norm.double(), turn(down[:, None, rank:])[:, 0]], -1)
    live = slots >= 0
    got = pool.cpu().double()[slots[live], 0]
    assert_close(got[:, : rank + rot], want[live], TOL[dtype], "pool")
    assert not got[:, rank + rot:].any()
    untouched = torch.ones(64, dtype=torch.bool)
    untouched[slots[live]] = False
    assert (pool.cpu()[untouched] == 7).all()
    took = ops.latent_gather(pool, torch.tensor([5, -1, 63, 64, 0], device=DEV)).cpu()
    assert torch.equal(took[[0, 2, 4]], pool.cpu()[[5, 63, 0], 0]) and not took[[1, 3]].any()
