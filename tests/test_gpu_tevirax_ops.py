"""The kernels of the Tevirax mechanisms, each against the oracle's function or a plain float64 statement: embeddings with
positions, weighted branch sums, grouped gated norms, weighted q/k norms, chunk masks at their edges, the short convolution,
both gated recurrences (outputs and carried states) and the expert products."""

import math

import numpy as np
import pytest
import torch

from oracle import tevirax_oracle as to
from research_amd import ops
from research_amd.inference import CacheConfig, HipPagedAttentionBackend, InferenceContext
from tests.gpu_helpers import DEV, announce, assert_close
from tests.test_gpu_hybrid_ops import _one_key_stands_out

pytestmark = pytest.mark.gpu

BF, F32 = torch.bfloat16, torch.float32
TOL = {F32: 2e-6, BF: 8e-3}


def _rand(*shape, dtype=F32, seed=0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed)).to(dtype)


def _i32(values):
    return torch.tensor(list(values), dtype=torch.int32, device=DEV)


def _portions(picks, slots, tiles=True):
    """``picks``: (sequence, first row, rows) in the order of the packed rows."""
    q_lens = [n for _, _, n in picks]
    cut = [(i, r) for i, n in enumerate(q_lens) for r in range(0, n, ops.QKV_TILE_ROWS)]
    return ops.Portions(_i32(lo + n for _, lo, n in picks), _i32(slots[b] for b, _, _ in picks), _i32(q_lens),
                        _i32(np.cumsum([0] + q_lens[:-1])), torch.tensor(cut, dtype=torch.int32, device=DEV) if tiles else None, max(q_lens))


# ------------------------------------------------------------------ rows


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("width", [37, 88, 260, 2048, 5000])
def test_embeddings_and_weighted_branches(width, dtype):
    announce(f"embedding and mix {width} {dtype}")
    rows, m = 7, 3
    table, pos = _rand(11, width, dtype=dtype), _rand(20, width, dtype=dtype, seed=1)
    ids, at = torch.tensor([3, 0, 10, 3, -1, 11, 2]), torch.tensor([0, 19, 4, 20, 5, 6, -1])
    x = torch.full((rows, width), float("nan"), device=DEV)
    w = _rand(width, seed=2)
    got = ops.residual_norm(x, dtype, ids=ids.to(DEV), table=table.to(DEV), table_scale=3.7, positions=at.to(DEV), pos_table=pos.to(DEV),
                            norm="rms", weight=w.to(DEV), eps=1e-3)
    zero = torch.zeros(width, dtype=torch.float64)
    want = torch.stack([(3.7 * table[i].double() if 0 <= i < 11 else zero) + (pos[p].double() if 0 <= p < 20 else zero)
                        for i, p in zip(ids.tolist(), at.tolist())])
    assert_close(x, want, 2e-6, "embedding")
    assert_close(got, to.rms_norm(want, 1e-3) * w.double(), TOL[dtype], "normed embedding")
    x0 = _rand(rows, width, seed=3)
    y, extra, mix = _rand(rows * m, width, dtype=dtype, seed=4), _rand(rows, width, dtype=dtype, seed=5), _rand(rows, m + 1, seed=6)
    for with_extra in (False, True):
        x = x0.to(DEV)
        branch = (y.double().view(rows, m, width) * mix[:, :m, None].double()).sum(1)
        if with_extra:
            branch = branch + mix[:, m:].double() * extra.double()
        got = ops.residual_norm(x, dtype, y=y.to(DEV), mix=mix.to(DEV), y_extra=extra.to(DEV) if with_extra else None, y_weight=w.to(DEV), y_eps=1e-2)
        want = x0.double() + to.rms_norm(branch, 1e-2) * w.double()
        assert_close(x, want, 4e-6, "mixed branch")
        assert_close(got, want, TOL[dtype], "mixed branch, cast")
    with pytest.raises(ValueError):
        ops.residual_norm(x, dtype, y=y[: rows].to(DEV), mix=mix.to(DEV))


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("groups,per", [(1, 48), (3, 24), (5, 14), (4, 72), (2, 200), (8, 128), (2, 2048), (3, 33)])
def test_gated_norms_of_groups(groups, per, dtype):
    announce(f"gated norm {groups} x {per} {dtype}")
    rows, width = 9, groups * per
    o, w = _rand(rows, width, dtype=dtype), _rand(width, seed=1)
    wide = _rand(rows, width + 16, dtype=dtype, seed=2).to(DEV)
    for lo in (0, 8, 3):
        g = wide[:, lo: lo + width]
        gc, oc = g.cpu().double(), o.double()
        out = torch.zeros(rows, width + 24, dtype=dtype, device=DEV)
        got = ops.rms_gate(o.to(DEV), g, w.to(DEV), 1e-2, groups=groups, out=out[:, lo: lo + width])
        want = to.rms_norm(oc.view(rows, groups, per), 1e-2).reshape(rows, width) * w.double() * to.sigmoid(gc)
        assert_close(got, want, TOL[dtype], "sigmoid last")
        assert not out[:, :lo].any() and not out[:, lo + width:].any()
        got = ops.rms_gate(o.to(DEV), g, w.to(DEV), 1e-2, groups=groups, order="silu_first")
        assert_close(got, to.gated_group_norm(oc, gc, w.double(), groups, 1e-2), 2 * TOL[dtype], "silu first")


@pytest.mark.parametrize("dtype", [F32, BF])
def test_head_packing_with_a_scale_and_capped_logits(dtype):
    announce(f"head scale, softcap {dtype}")
    o = _rand(6, 3, 40, dtype=dtype)
    for lo, vdim in ((0, 24), (8, 40), (5, 17)):
        out = torch.zeros(6, 160, dtype=dtype, device=DEV)
        ops.head_gate(o.to(DEV), None, vdim, 1.3, out[:, lo: lo + 3 * vdim])
        assert_close(out[:, lo: lo + 3 * vdim], 1.3 * o[:, :, :vdim].double().reshape(6, -1), TOL[dtype], "scaled")
        assert not out[:, :lo].any() and not out[:, lo + 3 * vdim:].any()
    for shape in ((5, 101), (3, 64)):
        x = (_rand(*shape, seed=1) * 40).to(dtype)
        got = ops.softcap(x.to(DEV), 15.0)
        assert got.dtype == F32
        assert_close(got, 15 * torch.tanh(x.double() / 15), 4e-6, "softcap")


# ------------------------------------------------------------------ q, k, v


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("hq,hkv,dim,vdim,rot", [(4, 2, 32, 24, 12), (6, 3, 20, 36, 10), (3, 1, 96, 192, 96), (2, 2, 44, 28, 0), (8, 2, 256, 64, 128)])
def test_weighted_norms_ahead_of_the_rotation(hq, hkv, dim, vdim, rot, dtype):
    announce(f"qk norm {hq} {hkv} {dim} {vdim} {rot} {dtype}")
    n, eps, d = 37, 1e-2, -(-max(dim, vdim) // 8) * 8
    cfg = {"base": 60.0, "dims": rot, "scaling": {"factor": 2.0, "original": 20, "fast": 3.0, "slow": 0.5}} if rot else None
    order = torch.arange(dim)
    order[:rot] = order[:rot].view(2, -1).t().reshape(-1)
    u = _rand(n, (hq + hkv) * dim + hkv * vdim, dtype=dtype)
    qw, kw = 1 + 0.3 * _rand(dim, seed=1), 1 + 0.3 * _rand(dim, seed=2)
    q, k, v = u.double().split([hq * dim, hkv * dim, hkv * vdim], 1)
    want_q = to.rotate_halves(to.rms_norm(q.view(n, hq, dim), eps) * qw.double(), cfg)
    want_k = to.rotate_halves(to.rms_norm(k.view(n, hkv, dim), eps) * kw.double(), cfg)
    rope = None
    if rot:
        freq, amp = to.yarn_table(cfg)
        ang = torch.arange(64, dtype=torch.float64)[:, None] * torch.tensor(freq, dtype=torch.float64)
        rope = (amp * torch.stack([ang.cos(), ang.sin()], -1)).float().contiguous().to(DEV)
    stored = torch.cat([u[:, : (hq + hkv) * dim].view(n, -1, dim)[..., order].reshape(n, -1), u[:, (hq + hkv) * dim:]], 1)
    kc = torch.zeros(64, hkv, d, dtype=dtype, device=DEV)
    vc = torch.zeros_like(kc)
    slots = torch.randperm(64, generator=torch.Generator().manual_seed(3))[:n]
    got, at = [], 0
    for size in (2, 20, 15):
        rows = stored[at: at + size].to(DEV)
        got.append(ops.qkv_conv_append(rows, _portions([(0, at, size)], [-1]), slots[at: at + size].to(DEV), kc, vc, hq, dim, vdim, 0.4, eps, False,
                                       rope, rot, None, None, q_norm=qw[order].to(DEV), k_norm=kw[order].to(DEV)).cpu())
        at += size
    tol = 4 * TOL[dtype]
    assert_close(torch.cat(got)[..., :dim], 0.4 * want_q[..., order], tol, "q")
    assert_close(kc.cpu()[slots][..., :dim], want_k[..., order], tol, "k")
    assert_close(vc.cpu()[slots][..., :vdim], v.view(n, hkv, vdim), TOL[dtype], "v")


# ------------------------------------------------------------------ chunk masks


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("size", [1, 2, 15, 16, 17, 40, 64, 100])
def test_chunk_edges_in_decode(size, dtype):
    announce(f"chunk edge decode {size} {dtype}")
    for total in (1, size, size + 1, 2 * size, 2 * size + 1, 65, 113, 128):
        first = (total - 1) // size * size
        for target in {first, first - 1, total - 1, 0}:
            if not 0 <= target < total:
                continue
            o = _one_key_stands_out(dtype, 32, -size, 16, 1, total, target)
            assert (o > 0.99).all() if target >= first else not o.any(), (total, target)


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("d", [32, 64, 128, 192, 256])
@pytest.mark.parametrize("size", [1, 16, 33, 50, 120])
def test_chunk_edges_in_portions(size, d, dtype):
    announce(f"chunk edge prefill {size} {d} {dtype}")
    for total, rows in ((130, 130), (130, 2), (131, 37), (420, 300)):
        edge = (total - 1) // size * size
        for target in {0, 15, 16, total - rows, edge, edge - 1, total - rows - (total - rows) % size, (total - rows) // size * size - 1}:
            if not 0 <= target < total:
                continue
            o = _one_key_stands_out(dtype, d, -size, 16, rows, total, target)
            p = torch.arange(total - rows, total)
            inside = (p >= target) & (p // size == target // size)
            assert (o[inside] > 0.99).all() and not o[~inside].any(), (total, rows, target)


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("heads,kv,d,size", [(6, 2, 40, 20), (5, 1, 96, 64), (4, 4, 16, 200), (12, 4, 192, 70), (14, 2, 160, 33)])
def test_packed_batches_under_a_chunk_mask(heads, kv, d, size, dtype):
    announce(f"packed chunks {heads} {kv} {d} {size} {dtype}")
    bs, lens, rows = 16, [77, 1, 33, 150, 64, 2], [1, 1, 1, 90, 64, 2]
    per = [-(-n // bs) for n in lens]
    backend = HipPagedAttentionBackend(CacheConfig(num_layers=1, num_kv_heads=kv, head_dim=d, num_blocks=sum(per), block_size=bs, dtype=dtype,
                                                   layer_kv=((kv, d),)))
    perm = np.random.default_rng(1).permutation(sum(per)).astype(np.int32)
    tables, at = np.full((6, max(per)), -1, dtype=np.int32), 0
    backend.k_cache[0].copy_(_rand(sum(per) * bs, kv, d, seed=1))
    backend.v_cache[0].copy_(_rand(sum(per) * bs, kv, d, seed=2))
    for b, n in enumerate(per):
        tables[b, :n] = perm[at: at + n]
        at += n
    q = _rand(sum(rows), heads, d, dtype=dtype, seed=3)
    ctx = InferenceContext(is_prefill=True, block_tables=tables, seq_lens=np.asarray(lens), q_lens=np.asarray(rows), num_decodes=3)
    got = backend.attend_packed(q.to(DEV), 0, backend.packed_step(ctx), d ** -0.5, -size).cpu()
    kc, vc, r = backend.k_cache[0].cpu().double(), backend.v_cache[0].cpu().double(), 0
    for b, n in enumerate(lens):
        idx = torch.tensor([tables[b, p // bs] * bs + p % bs for p in range(n)])
        full = torch.zeros(n, heads, d, dtype=torch.float64)
        full[n - rows[b]:] = q[r: r + rows[b]].double()
        want = to.chunk_attention(full, kc[idx], vc[idx], d ** -0.5, size)[n - rows[b]:]
        assert_close(got[r: r + rows[b]], want, 2e-2 if dtype == BF else 1e-5, f"sequence {b}")
        r += rows[b]


# ------------------------------------------------------------------ short convolution


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("channels,taps,act", [(40, 4, "silu"), (33, 3, "silu"), (2056, 2, "silu"), (24, 8, None), (16, 1, "silu"), (66, 6, None)])
def test_short_convolution_in_portions(channels, taps, act, dtype):
    """Two sequences in portions down to one and two tokens, single tokens beside a padding row, slots used before."""
    announce(f"short conv {channels} {taps} {act} {dtype}")
    lens = [45, 38]
    us = [_rand(n, channels + 16, dtype=dtype, seed=i) for i, n in enumerate(lens)]
    w, bias = _rand(channels, taps, seed=5), _rand(channels, seed=6)
    want = [to.causal_conv(u[:, 8: 8 + channels].double(), w.double(), bias.double()) for u in us]
    if act:
        want = [to.silu(y) for y in want]
    state = _rand(4, taps - 1, channels, dtype=dtype, seed=9).to(DEV) if taps > 1 else None
    before = None if state is None else state.clone()
    slots, at = [2, 0], [0, 0]
    for n0, n1 in [(2, 17), (1, 2), (19, 1), (1, 1), (2, 3), (16, 14), (4, 0)]:
        picks = [(b, at[b], n) for b, n in ((0, n0), (1, n1)) if n]
        rows = torch.cat([us[b][lo: lo + n] for b, lo, n in picks])
        if [n for _, _, n in picks] == [1, 1]:
            rows = torch.cat([rows, rows[:1]])
            por = ops.Portions(_i32([at[0] + 1, at[1] + 1, 0]), _i32([2, 0, -1]))
        else:
            por = _portions(picks, slots)
        got = ops.short_conv(rows.to(DEV)[:, 8: 8 + channels], por, w.t().contiguous().to(DEV), bias.to(DEV), state, act).cpu()
        r = 0
        for b, lo, n in picks:
            assert_close(got[r: r + n], want[b][lo: lo + n], 2 * TOL[dtype], f"{b} {lo}")
            r += n
            at[b] += n
    assert at == lens
    if state is not None:
        for b in (0, 1):
            assert torch.equal(state[slots[b]].cpu(), us[b][lens[b] - taps + 1:, 8: 8 + channels])
        assert torch.equal(state[1], before[1]) and torch.equal(state[3], before[3])


# ------------------------------------------------------------------ gated recurrences


class Case:
    """Random rows of some sequences with the oracle's outputs and states, for either kind of recurrence."""

    def __init__(self, kind, lens, heads, dim, vdim, dtype, groups=None, seed=0, remember=3.0):
        g = torch.Generator().manual_seed(seed)
        rnd = lambda *s: torch.randn(*s, generator=g)
        self.kind, self.heads, self.dim, self.vdim, self.dtype = kind, heads, dim, vdim, dtype
        self.groups = groups or heads
        self.cap, self.q_scale = 5.0, dim ** -0.5
        n_qk = self.groups * dim
        self.sizes = [n_qk, n_qk, heads * vdim, heads, heads]
        self.rows = [rnd(n, sum(self.sizes) + 8).to(dtype) for n in lens]
        if kind == "ssd":
            self.constants = (torch.linspace(-4, 1, heads), torch.exp(0.7 * rnd(heads)), 1 + 0.5 * rnd(heads))
        else:
            self.constants = (rnd(heads), remember + rnd(heads), None)
        self.want, self.final = [], []
        for r in self.rows:
            o, final = self.oracle(r)
            self.want.append(o.reshape(-1, heads * vdim))
            self.final.append(final)
        floats = ops.gated_linear_state_floats(kind, dim, vdim)
        self.state = torch.full((len(lens) + 2, heads, floats), 7.0, device=DEV)  # whatever a slot holds, a sequence starts empty

    def oracle(self, rows):
        q, k, v, a, b = rows.double()[:, : sum(self.sizes)].split(self.sizes, 1)
        q, k, v = q.reshape(-1, self.groups, self.dim), k.reshape(-1, self.groups, self.dim), v.reshape(-1, self.heads, self.vdim)
        c0, c1, c2 = (c.double() if c is not None else None for c in self.constants)
        if self.kind == "ssd":
            return to.ssd_recurrence(v, k, q, to.softplus(a + c0), c1, c2)
        li = self.cap * torch.tanh((a + c0) / self.cap)
        lf = -to.softplus(-self.cap * torch.tanh((b + c1) / self.cap))
        return to.mlstm_recurrence(q * self.q_scale, k, v, li, lf)

    def call(self, rows, por, out, workspace=None):
        u = rows.to(DEV)[:, : sum(self.sizes)]
        q, k, v, a, b = u.split(self.sizes, 1)
        ops.gated_linear(self.kind, q, k, v, (a, b if self.kind == "mlstm" else None), tuple(c.to(DEV) if c is not None else None for c in self.constants), por,
                         self.state, self.heads, self.dim, self.vdim, out, heads_per_group=self.heads // self.groups, cap=self.cap,
                         q_scale=self.q_scale, den_eps=1e-6, workspace=workspace)

    def run(self, picks, slots, use_ws=True):
        rows = torch.cat([self.rows[b][lo: lo + n] for b, lo, n in picks])
        out = torch.full((rows.shape[0], self.heads * self.vdim), float("nan"), dtype=self.dtype, device=DEV)
        por = _portions(picks, slots, tiles=False)
        need = ops.gated_linear_workspace_bytes(len(picks), self.heads, self.dim, self.vdim, por.max_q_len)
        ws = torch.full((need,), 0x7f, dtype=torch.uint8, device=DEV) if need and use_ws else None
        self.call(rows, por, out, ws)
        return out.cpu().split([n for _, _, n in picks])

    def check(self, b, lo, got):
        want = self.want[b][lo: lo + got.shape[0]]
        scale = want.abs().mean(-1, keepdim=True) + want.abs().mean() * 0.2
        err = (got.double() - want).abs() / (scale + want.abs())
        assert torch.isfinite(got.double()).all()
        assert err.max() < (1e-4 if self.dtype == F32 else 1e-2), (b, lo, int(err.max(1).values.argmax()), float(err.max()))

    def check_state(self, b, slot):
        pad = lambda n: -(-n // 16) * 16
        dp, vp = pad(self.dim), pad(self.vdim)
        got = self.state[slot].cpu().double()
        s = got[:, : dp * vp].view(self.heads, dp, vp)[:, : self.dim, : self.vdim]
        want = self.final[b] if self.kind == "ssd" else self.final[b][0]
        assert (s - want).abs().max() / want.abs().max() < 2e-4
        if self.kind == "mlstm":
            for rep in range(-(-self.vdim // 64)):  # a copy of n and m per 64 value columns
                at = dp * vp + rep * (dp + 16)
                assert (got[:, at: at + self.dim] - self.final[b][1]).abs().max() / self.final[b][1].abs().max() < 2e-4
                assert (got[:, at + dp] / math.log2(math.e) - self.final[b][2]).abs().max() < 2e-3


SHAPES = [("mlstm", 3, 16, 16, None), ("mlstm", 2, 48, 80, None), ("mlstm", 1, 136, 200, None), ("mlstm", 2, 128, 128, None), ("mlstm", 1, 256, 300, None),
          ("mlstm", 2, 36, 20, None), ("mlstm", 2, 30, 14, None), ("mlstm", 1, 64, 64, None),
          ("ssd", 4, 24, 16, 2), ("ssd", 3, 48, 32, 1), ("ssd", 2, 128, 64, 2), ("ssd", 2, 160, 144, 1), ("ssd", 6, 18, 20, 3), ("ssd", 2, 33, 44, 1), ("ssd", 1, 256, 72, 1)]


@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("kind,heads,dim,vdim,groups", SHAPES)
def test_whole_sequences_of_unequal_length(kind, heads, dim, vdim, groups, dtype):
    announce(f"gated {kind} {heads}x{dim}x{vdim} {dtype}")
    lens = [1, 2, 63, 64, 65, 150]
    case = Case(kind, lens, heads, dim, vdim, dtype, groups)
    slots = [3, 0, 5, 1, 6, 2]
    got = case.run([(b, 0, n) for b, n in enumerate(lens)], slots)
    for b in range(len(lens)):
        case.check(b, 0, got[b])
        case.check_state(b, slots[b])


@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("kind,heads,dim,vdim,groups", [("mlstm", 3, 80, 144, None), ("ssd", 4, 48, 40, 2)])
def test_portions_and_single_tokens_continue_the_state(kind, heads, dim, vdim, groups, dtype):
    announce(f"gated portions {kind} {dtype}")
    case = Case(kind, [200, 131], heads, dim, vdim, dtype, groups, seed=2)
    slots, at = [1, 3], [0, 0]
    sizes = [[2, 3, 64, 61, 2, 5, 63], [70, 2, 2, 33, 2, 7, 15]]
    for i in range(7):
        picks = [(b, at[b], sizes[b][i]) for b in (0, 1)]
        for (b, lo, n), got in zip(picks, case.run(picks, slots)):
            case.check(b, lo, got)
            at[b] += n
    assert at == [200, 131]
    for b in (0, 1):
        case.check_state(b, slots[b])


@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("kind,heads,dim,vdim,groups", [("mlstm", 2, 64, 96, None), ("ssd", 4, 40, 72, 1)])
def test_decode_rows_equal_the_recurrence_and_padding_rows_are_skipped(kind, heads, dim, vdim, groups, dtype):
    announce(f"gated decode {kind} {dtype}")
    case = Case(kind, [40, 40, 40], heads, dim, vdim, dtype, groups, seed=3)
    before = case.state.clone()
    for t in range(40):
        rows = torch.stack([r[t] for r in case.rows] + [case.rows[0][t]])
        out = torch.zeros(4, heads * vdim, dtype=dtype, device=DEV)
        case.call(rows, ops.Portions(_i32([t + 1, t + 1, t + 1, 0]), _i32([2, 4, 0, -1])), out)
        for b in range(3):
            case.check(b, t, out[b: b + 1].cpu())
        assert not out[3].any()
    for b, slot in enumerate((2, 4, 0)):
        case.check_state(b, slot)
    assert torch.equal(case.state[1], before[1]) and torch.equal(case.state[3], before[3])


@pytest.mark.parametrize("kind,heads,dim,vdim,groups", [("mlstm", 2, 128, 200, None), ("mlstm", 1, 64, 48, None), ("ssd", 4, 128, 64, 1), ("ssd", 2, 256, 80, 2)])
def test_long_portions_in_segments(kind, heads, dim, vdim, groups):
    """Few sequences of many chunks: with a workspace the portion runs in segments; the same without one."""
    lens = [1125, 700]
    announce(f"gated segments {kind} {heads}x{dim}x{vdim}")
    assert ops.gated_linear_workspace_bytes(2, heads, dim, vdim, 1125) > 0
    case = Case(kind, lens, heads, dim, vdim, BF, groups, seed=4, remember=4.5)
    for use_ws in (True, False):
        for first in (0, 37):
            if first:
                case.run([(0, 0, first), (1, 0, first)], [1, 2])
            got = case.run([(b, first, lens[b] - first) for b in (0, 1)], [1, 2], use_ws)
            for b in (0, 1):
                case.check(b, first, got[b])
                case.check_state(b, 1 + b)


@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("kind", ["mlstm", "ssd"])
def test_a_far_token_is_remembered(kind, dtype):
    """Hundreds of tokens write next to nothing but one, whose key the last queries ask for."""
    announce(f"gated far {kind} {dtype}")
    n, target = 400, 21
    case = Case(kind, [n], 2, 32, 48, dtype, 1 if kind == "ssd" else None, seed=5)
    q, k, v, a, b = case.rows[0][:, : sum(case.sizes)].split(case.sizes, 1)
    a.fill_(-4.0), b.fill_(40.0)  # weak writes, nothing forgotten
    case.constants = (torch.full((2,), -6.0 if kind == "ssd" else 0.0), torch.full((2,), 0.01), torch.zeros(2) if kind == "ssd" else None)
    k.mul_(0.05)
    a[target], k[target] = (6.0 if kind == "ssd" else 40.0), 1.0
    q[-20:] = 1.0
    o, final = case.oracle(case.rows[0])
    case.want, case.final = [o.reshape(n, -1)], [final]
    target_v = v[target].double().view(2, 48)
    for t in (-1, -20):
        cos = torch.nn.functional.cosine_similarity(o[t], target_v, dim=-1)
        assert (cos > 0.9).all()
    for cut in ([n], [target + 1, 2, n - target - 3], [64, 200, n - 264]):
        at, got = 0, []
        for size in cut:
            got.append(case.run([(0, at, size)], [1])[0])
            at += size
        got = torch.cat(got)
        for lo in (target, 63, n - 20):
            err = (got[lo: lo + 20].double() - case.want[0][lo: lo + 20]).abs().max() / case.want[0][lo: lo + 20].abs().max()
            assert err < (1e-4 if dtype == F32 else 1e-2), (cut, lo, float(err))


# ------------------------------------------------------------------ experts


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("rows,n,k", [(1, 3, 40), (5, 65, 256), (70, 130, 76), (33, 9, 33), (2100, 64, 200), (130, 257, 1024)])
def test_narrow_products_are_32_bit(rows, n, k, dtype):
    announce(f"narrow {rows} {n} {k} {dtype}")
    x, w = _rand(rows, k + 8, dtype=dtype), _rand(n, k, dtype=dtype, seed=1)
    for lo in (0, 8, 1):
        if lo + k > k + 8:
            continue
        got = ops.narrow_linear(x.to(DEV)[:, lo: lo + k], w.to(DEV))
        want = x[:, lo: lo + k].double() @ w.double().T
        assert got.dtype == F32 and tuple(got.shape) == (rows, n)
        assert ((got.cpu().double() - want).abs() / (want.abs() + k ** 0.5)).max() < 2e-6


@pytest.mark.parametrize("rows,experts,top,groups,keep,shared", [(1, 6, 2, 3, 2, True), (37, 8, 3, 2, 1, False), (130, 5, 4, 1, 1, True), (64, 256, 8, 8, 4, True),
                                                                (9, 100, 20, 100, 40, False), (2000, 16, 4, 4, 2, True), (3, 1, 1, 1, 1, False),
                                                                (50, 1000, 10, 20, 5, True), (5000, 120, 6, 12, 12, True)])
def test_choice_of_experts(rows, experts, top, groups, keep, shared):
    announce(f"choose {rows} {experts} {top} {groups} {keep}")
    logits = _rand(rows, experts + shared, seed=rows)
    c = ops.moe_choose(logits.to(DEV), experts, top, groups, keep, "gated" if shared else None)
    ids, weights, counts, lists = (t.cpu() for t in c)
    for r in range(min(rows, 60)):
        want, ww = to.route(torch.sigmoid(logits[r, :experts].double()), top, groups, keep)
        assert ids[r].tolist() == want
        assert weights[r, :top].tolist() == pytest.approx(ww, rel=1e-5)
    gate = torch.sigmoid(logits[:, experts]) if shared else torch.zeros(rows)
    assert torch.allclose(weights[:, top], gate, atol=1e-6)
    for e in range(experts):
        want = torch.nonzero(ids.reshape(-1) == e).reshape(-1)
        assert counts[e] == want.numel() and torch.equal(lists[e, : counts[e]].long(), want)


def test_rows_of_nan_have_no_experts():
    announce("choose nan")
    logits = _rand(70, 8)
    logits[3] = float("nan")
    ids, _, counts, _ = (t.cpu() for t in ops.moe_choose(logits.to(DEV), 8, 2, 2, 1))
    assert (ids[3] == -1).all() and counts.sum() == 2 * 69 and (ids[4] >= 0).all()


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("rows,experts,top,width,ff", [(1, 4, 2, 64, 40), (9, 6, 2, 88, 24), (40, 8, 3, 128, 96), (130, 7, 2, 256, 200), (300, 5, 4, 72, 48),
                                                       (60, 3, 1, 76, 22), (1200, 6, 3, 320, 136), (33, 40, 4, 192, 64)])
def test_expert_products(rows, experts, top, width, ff, dtype):
    """From one item per expert to hundreds, so that every kernel runs; lists of very unequal length."""
    announce(f"experts {rows} {experts} {top} {width} {ff} {dtype}")
    pad = lambda n: -(-n // 64) * 64
    logits = _rand(rows, experts, seed=1) + torch.linspace(2, -2, experts)
    c = ops.moe_choose(logits.to(DEV), experts, top, 1, 1)
    h = _rand(rows, width, dtype=dtype, seed=2)
    g, u, d = (_rand(experts, *s, dtype=dtype, seed=i) * s[1] ** -0.5 for i, s in ((3, (ff, width)), (4, (ff, width)), (5, (width, ff))))
    w_in = torch.zeros(experts, 2 * pad(ff), pad(width), dtype=dtype)
    w_in[:, :ff, :width], w_in[:, pad(ff): pad(ff) + ff, :width] = g, u
    w_out = torch.zeros(experts, width, pad(ff), dtype=dtype)
    w_out[..., :ff] = d
    act = ops.moe_product(h.to(DEV), c, w_in.to(DEV), pad(ff), width, glu=True)
    y = ops.moe_product(act, c, w_out.to(DEV), width, pad(ff), glu=False)
    e = c.ids.cpu().long().reshape(-1)
    x = h.double().repeat_interleave(top, 0)
    want_act = torch.zeros(rows * top, ff, dtype=torch.float64)
    want = torch.zeros(rows * top, width, dtype=torch.float64)
    for k in range(experts):
        m = e == k
        want_act[m] = to.silu(x[m] @ g[k].double().T) * (x[m] @ u[k].double().T)
        seen = act.cpu().double()[m][:, :ff]
        want[m] = seen @ d[k].double().T
    assert_close(act[:, :ff], want_act, 2e-5 if dtype == F32 else 8e-3, "activations")
    assert not act[:, ff:].any()
    assert_close(y, want, 2e-5 if dtype == F32 else 8e-3, "outputs")
