"""The kernels of the Loluzen mechanisms, each against the oracle's function or a plain float64 statement: residual sums with
embeddings and pairs of normed branches, biases and activations, attention with mixed heads, HGRN2 (outputs and carried
states)."""

import numpy as np
import pytest
import torch
import torch.nn.functional as F

from oracle import loluzen_oracle as lo
from research_amd import ops
from tests.gpu_helpers import DEV, announce, assert_close
from tests.test_gpu_tevirax_ops import _i32, _portions, _rand
from tests.test_gpu_vusalix_ops import Paged

pytestmark = pytest.mark.gpu

BF, F32 = torch.bfloat16, torch.float32
TOL = {F32: 3e-6, BF: 8e-3}


# ------------------------------------------------------------------ rows


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("width", [37, 88, 260, 2048, 5000])
def test_two_normed_branches_biases_and_the_embedding_again(width, dtype):
    announce(f"branches {width} {dtype}")
    rows = 6
    x0, y, z = _rand(rows, width, seed=1), 3 * _rand(rows, width, dtype=dtype, seed=2), 0.2 * _rand(rows, width, dtype=dtype, seed=3)
    wy, wz, w1, w2, b = (_rand(width, seed=s) for s in range(4, 9))
    table, ids = _rand(9, width, dtype=dtype, seed=9), torch.tensor([3, 8, 0, 9, -1, 3])
    emb = torch.stack([table[i].double() if 0 <= i < 9 else torch.zeros(width, dtype=torch.float64) for i in ids.tolist()])
    kw = dict(norm="rms", weight=w2.to(DEV), eps=1e-3)
    x = x0.to(DEV)
    got = ops.residual_norm(x, dtype, y=y.to(DEV), y2=(z.to(DEV), wy.to(DEV), wz.to(DEV)), y_weight=w1.to(DEV), y_eps=1e-2, **kw)
    both = lo.rms_norm(y.double(), 1e-2) * wy.double() + lo.rms_norm(z.double(), 1e-2) * wz.double()
    want = x0.double() + lo.rms_norm(both, 1e-2) * w1.double()
    assert_close(x, want, 4e-6, "pair")
    assert_close(got, lo.rms_norm(want, 1e-3) * w2.double(), TOL[dtype], "normed pair")
    ops.residual_norm(x, dtype, y=y.to(DEV), y2=(z.to(DEV), wy.to(DEV), wz.to(DEV)), y_eps=1e-2, want_out=False)
    want = want + both
    assert_close(x, want, 6e-6, "pair as it is")
    got = ops.residual_norm(x, dtype, y=y.to(DEV), y_bias=b.to(DEV), y_weight=w1.to(DEV), y_eps=1e-2, ids=ids.to(DEV), table=table.to(DEV),
                            table_scale=2.5, ids_add=True, **kw)
    want = want + lo.rms_norm(y.double() + b.double(), 1e-2) * w1.double() + 2.5 * emb
    assert_close(x, want, 8e-6, "bias and embedding")
    assert_close(got, lo.rms_norm(want, 1e-3) * w2.double(), TOL[dtype], "normed")
    ops.residual_norm(x, dtype, ids=ids.to(DEV), table=table.to(DEV), ids_add=True, want_out=False)
    assert_close(x, want + emb, 8e-6, "embedding alone")


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("width", [5, 48, 1000, 4100])
def test_bias_and_activation(width, dtype):
    announce(f"bias act {width} {dtype}")
    wide, b = 3 * _rand(7, width + 16, dtype=dtype), _rand(width, seed=1)
    for x in (wide[:, :width], wide[:, 8: 8 + width], wide[:, 3: 3 + width]):
        for bias in (None, b):
            z = x.double() + (0 if bias is None else bias.double())
            for act, f in (("relu2", lambda t: torch.clamp(t, min=0) ** 2), ("silu", F.silu), ("gelu_tanh", lambda t: F.gelu(t, approximate="tanh")),
                           (None, lambda t: t)):
                dev = wide.to(DEV)[:, x.storage_offset(): x.storage_offset() + width]
                assert_close(ops.bias_act(dev, None if bias is None else bias.to(DEV), act), f(z), 1e-5 if dtype == F32 else 8e-3, (act, bias is None))


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("width,groups", [(64, 1), (84, 3), (2048, 16), (30, 5)])
def test_norm_of_groups_without_a_gate(width, groups, dtype):
    announce(f"group norm {width} {groups} {dtype}")
    x, w = _rand(9, width, dtype=dtype), _rand(width, seed=1)
    out = torch.zeros(9, width + 8, dtype=dtype, device=DEV)
    ops.rms_gate(x.to(DEV), None, w.to(DEV), 1e-3, groups=groups, order=None, out=out[:, :width])
    want = lo.rms_norm(x.double().view(9, groups, -1), 1e-3).reshape(9, width) * w.double()
    assert_close(out[:, :width], want, TOL[dtype])
    assert not out[:, width:].any()


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("heads,kv,dim,vdim", [(4, 2, 32, 24), (6, 3, 20, 28), (3, 3, 13, 44), (2, 1, 136, 200)])
def test_projections_with_biases_are_appended(heads, kv, dim, vdim, dtype):
    announce(f"append with bias {heads} {kv} {dim} {vdim} {dtype}")
    pad = lambda n: -(-n // 8) * 8
    d, n = pad(max(dim, vdim)), 21
    channels = (heads + kv) * dim + kv * vdim
    u, bias = _rand(n, pad(channels + 3), dtype=dtype), _rand(channels, seed=1)
    kc = torch.full((48, kv, d), float("nan"), dtype=dtype, device=DEV)
    vc = kc.clone()
    slots = torch.randperm(48, generator=torch.Generator().manual_seed(0))[:n]
    q = ops.qkv_conv_append(u.to(DEV), _portions([(0, 30, n)], [0]), slots.to(DEV), kc, vc, heads, dim, vdim, 1.0, 0.0, False, None, 0, None, None,
                            bias=bias.to(DEV))
    want = u[:, :channels].double() + bias.double()
    parts = want.split([heads * dim, kv * dim, kv * vdim], 1)
    for got, part, h, size in ((q, parts[0], heads, dim), (kc[slots.to(DEV)], parts[1], kv, dim), (vc[slots.to(DEV)], parts[2], kv, vdim)):
        assert_close(got[..., :size], part.view(n, h, size), 1e-6 if dtype == F32 else 4e-3)
        assert not got[..., size:].any()


# ------------------------------------------------------------------ attention with mixed heads


class Talking:
    def __init__(self, lens, heads, kv, dim, vdim, dtype, seed=0, biased=True, odd_talk=False):
        pad = lambda n: -(-n // 8) * 8
        self.heads, self.kv, self.dim, self.vdim, self.dtype, self.pad = heads, kv, dim, vdim, dtype, pad(dim)
        d = pad(max(dim, vdim))
        self.paged = Paged(lens, kv, d, d, dtype, seed=seed)
        self.paged.k[..., dim:] = 0
        self.scale = 2.0 * dim ** -0.5
        self.talk = torch.eye(heads) + 0.9 * heads ** -0.5 * _rand(heads, heads, seed=seed + 3)
        if not odd_talk:
            self.talk = self.talk.to(BF).float()
        g = torch.Generator().manual_seed(seed + 4)
        self.size = 0.05 + 1.5 * torch.rand(heads, generator=g) if biased else None
        self.rate = 0.05 + 0.6 * torch.rand(heads, generator=g) if biased else None
        self.q = [F.pad(_rand(n, heads, dim, seed=seed + 20 + i), (0, self.pad - dim)).to(dtype) for i, n in enumerate(lens)]

    def solve(self):
        self.want = []
        for i, q in enumerate(self.q):
            k, v = self.paged.rows(self.paged.k, i).double(), self.paged.rows(self.paged.v, i).double()[..., : self.vdim]
            bias = None if self.size is None else lo.distance_bias(self.size.double(), self.rate.double(), len(q))
            self.want.append(lo.causal_attention(q.double()[..., : self.dim], k[..., : self.dim], v, self.scale, bias, self.talk.double()))
        return self

    def run(self, picks, decode=False, workspace=True):
        p = _portions(picks, [0] * len(self.q), tiles=False)
        if decode:
            p = ops.Portions(p.ctx_lens, p.state_slots)
        q = torch.cat([self.q[b][at: at + n] for b, at, n in picks]).to(DEV)
        tables = torch.from_numpy(self.paged.tables[[b for b, _, _ in picks]]).to(DEV)
        out = torch.full((q.shape[0], self.heads, self.vdim), float("nan"), dtype=self.dtype, device=DEV)
        need = ops.talking_workspace_bytes(q.shape[0], p, self.heads, self.kv, self.vdim, tables.shape[1] * 16)
        if not workspace:  # (enough for the sums only)
            need = -(-q.shape[0] * self.heads * 4 // 256) * 256
        ws = torch.full((need,), 0x7f, dtype=torch.uint8, device=DEV)
        dev = lambda t: None if t is None else t.to(DEV)
        ops.talking_attention(q, self.paged.k.to(DEV), self.paged.v.to(DEV), self.vdim, p, tables, 16, self.scale, dev(self.talk), out,
                              dev(self.size), dev(self.rate), workspace=ws)
        return out.cpu().split([n for _, _, n in picks])

    def check(self, picks, **kw):
        # (errors against the size of the rows: mixed weights have both signs and their sums may nearly cancel)
        for (b, at, n), got in zip(picks, self.run(picks, **kw)):
            want = self.want[b][at: at + n]
            err = (got.double() - want).abs() / (1.0 + want.abs())
            assert torch.isfinite(got.double()).all()
            worst = float(err.max())
            assert worst < (1e-5 if self.dtype == F32 else 1.5e-2), (b, at, n, worst, int(err.flatten(1).max(1).values.argmax()))


TALKING = [  # heads, kv heads, dim, vdim
    (6, 2, 40, 56), (4, 1, 64, 32), (3, 3, 20, 36), (16, 4, 128, 96), (8, 2, 128, 128), (20, 4, 72, 64), (24, 8, 64, 128), (32, 8, 128, 128),
    (32, 32, 16, 8), (1, 1, 8, 8), (40, 8, 48, 40), (20, 1, 64, 64), (5, 5, 136, 200), (34, 2, 24, 72), (66, 3, 16, 24), (9, 3, 33, 21)]


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("heads,kv,dim,vdim", TALKING)
def test_mixed_heads_in_portions_and_single_rows(heads, kv, dim, vdim, dtype):
    announce(f"talking {heads} {kv} {dim} {vdim} {dtype}")
    lens = [1, 2, 110, 63, 200]
    case = Talking(lens, heads, kv, dim, vdim, dtype).solve()
    case.check([(i, 0, n) for i, n in enumerate(lens)])
    case.check([(4, 130, 2), (2, 37, 30), (3, 15, 17), (1, 0, 2)])
    case.check([(4, 64, 136), (2, 108, 2)])
    for at in (0, 1, 15, 16, 17, 31, 32, 62):
        case.check([(3, at, 1), (2, at + 40, 1), (4, at + 130, 1)], decode=True)
    case.check([(i, n - 1, 1) for i, n in enumerate(lens)], decode=True)
    case.check([(i, n - 1, 1) for i, n in enumerate(lens)], decode=True, workspace=False)


@pytest.mark.parametrize("heads,kv,dim,vdim", [(8, 2, 64, 64), (20, 4, 48, 72)])
def test_long_decode_steps_run_in_pieces(heads, kv, dim, vdim):
    """One or two sequences of a few thousand tokens: their keys are spread over the device in up to sixteen pieces."""
    announce(f"talking pieces {heads} {kv} {dim} {vdim}")
    for lens in ([4097], [1500, 257], [3000, 1, 255]):
        case = Talking(lens, heads, kv, dim, vdim, BF, seed=len(lens))
        picks = [(i, n - 1, 1) for i, n in enumerate(lens)]
        case.want = []
        for i, n in enumerate(lens):  # the last row only
            k, v = case.paged.rows(case.paged.k, i).double(), case.paged.rows(case.paged.v, i).double()[..., :vdim]
            of = torch.arange(heads) // (heads // kv)
            s = (case.q[i][-1].double()[:, None, :dim] * k[:, of, :dim].transpose(0, 1)).sum(-1) * case.scale
            s = s + lo.distance_bias(case.size.double(), case.rate.double(), n).flip(1)
            p = case.talk.double() @ torch.softmax(s, -1)
            row = (p[:, :, None] * v[:, of].transpose(0, 1)).sum(1)
            case.want.append(torch.cat([torch.zeros(n - 1, heads, vdim, dtype=torch.float64), row[None]]))
        case.check(picks, decode=True)
        case.check(picks + [(0, lens[0] - 1, 1)] * 40, decode=True)


@pytest.mark.parametrize("dtype", [F32, BF])
def test_without_biases_and_with_a_matrix_of_more_than_16_bits(dtype):
    announce(f"talking plain {dtype}")
    for heads, kv, dim, vdim in ((6, 3, 32, 40), (20, 5, 64, 64)):
        for biased, odd in ((False, False), (True, True)):
            case = Talking([70, 45], heads, kv, dim, vdim, dtype, seed=5, biased=biased, odd_talk=odd).solve()
            case.check([(0, 0, 70), (1, 0, 45)])
            case.check([(0, 69, 1), (1, 30, 1)], decode=True)


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("far", [0, 15, 16, 31, 32, 63, 64, 199])
def test_one_far_key_of_one_head_shows_in_every_head(far, dtype):
    """One score of one head stands out: its value reaches every head by the mixing matrix alone, wherever the key lies."""
    announce(f"talking far {far} {dtype}")
    for heads, kv, dim, vdim in ((6, 2, 40, 24), (24, 8, 64, 32)):
        n, head = 300, heads // 2
        case = Talking([n], heads, kv, dim, vdim, dtype, seed=7)
        slot = int(case.paged.tables[0, far // 16]) * 16 + far % 16
        case.paged.k[..., : dim // 2] = 0  # these dimensions belong to the one key
        case.paged.k[slot, head // (heads // kv), 0] = 8.0
        case.paged.v[slot] = (20 + torch.arange(case.paged.v.shape[-1])).to(dtype) / 8
        case.q[0][:, :, : dim // 2] = 0
        case.q[0][:, head, 0] = 2.0 * dim ** 0.5
        case.solve()
        late = case.want[0][far + 1:]
        assert ((late - case.talk[:, head, None].double() * case.paged.v[slot, 0, :vdim].double()).abs().mean() < 1.5)
        case.check([(0, 0, n)])
        case.check([(0, 250, 50)])
        for at in {far, far + 1, 290}:
            case.check([(0, at, 1)], decode=True)


def test_decode_rows_of_length_zero_are_padding():
    announce("talking padding")
    case = Talking([40, 20], 6, 2, 32, 24, BF).solve()
    p = ops.Portions(_i32([40, 0, 20]), _i32([0, 0, 0]))
    q = torch.stack([case.q[0][39], case.q[0][0], case.q[1][19]]).to(DEV)
    tables = torch.from_numpy(case.paged.tables[[0, 0, 1]]).to(DEV)
    out = torch.full((3, 6, 24), 5.0, dtype=BF, device=DEV)
    need = ops.talking_workspace_bytes(3, p, 6, 2, 24, tables.shape[1] * 16)
    ops.talking_attention(q, case.paged.k.to(DEV), case.paged.v.to(DEV), 24, p, tables, 16, case.scale, case.talk.to(DEV), out, case.size.to(DEV),
                          case.rate.to(DEV), workspace=torch.zeros(need, dtype=torch.uint8, device=DEV))
    assert_close(out[0], case.want[0][39], 1.5e-2)
    assert_close(out[2], case.want[1][19], 1.5e-2)
    assert (out[1] == 5.0).all()


# ------------------------------------------------------------------ HGRN2


class Channels:
    """Random rows of some sequences, the oracle's outputs and states.  ``logit``: size of the forget logits; ``shift``: their
    bias is spread around it."""

    def __init__(self, lens, heads, dim, vdim, dtype, seed=0, logit=1.0, shift=3.0, low=0.95):
        self.heads, self.dim, self.vdim, self.dtype, self.lens = heads, dim, vdim, dtype, lens
        n = heads * dim
        self.bias = shift + 4 * (torch.rand(n, generator=torch.Generator().manual_seed(seed)) * 2 - 1)
        self.lower = low * torch.rand(n, generator=torch.Generator().manual_seed(seed + 1)) * torch.linspace(0, 1, n)
        self.rows, self.want, self.states = [], [], []
        for i, t in enumerate(lens):
            parts = [_rand(t, w, dtype=dtype, seed=seed + 10 * i + j) for j, w in enumerate((n, n, heads * vdim))]
            parts[1] = (logit * parts[1].float()).to(dtype)
            self.add(parts)
        pad = lambda x: -(-x // 16) * 16
        self.state = torch.full((len(lens) + 1, heads, pad(dim), pad(vdim)), float("nan"), device=DEV)

    def add(self, parts):
        self.rows.append(torch.cat(parts, 1))
        q, z, v = (p.double() for p in parts)
        t = len(q)
        f = lo.bounded_forget(z + self.bias.double(), self.lower.double()).view(t, self.heads, self.dim)
        o, s = lo.channel_recurrence(lo.silu(q).view(t, self.heads, self.dim), f, v.view(t, self.heads, self.vdim))
        self.want.append(o.reshape(t, -1))
        self.states.append(s)

    def run(self, picks, slots, decode=False, use_ws=True):
        u = torch.cat([self.rows[b][at: at + n] for b, at, n in picks]).to(DEV)
        q, z, v = u.split([self.heads * self.dim, self.heads * self.dim, self.heads * self.vdim], 1)
        p = _portions(picks, slots, tiles=False)
        if decode:
            p = ops.Portions(p.ctx_lens, p.state_slots)
        out = torch.full((u.shape[0], self.heads * self.vdim), float("nan"), dtype=self.dtype, device=DEV)
        need = ops.channel_linear_workspace_bytes(len(picks), self.heads, self.dim, self.vdim, p.max_q_len)
        ws = torch.full((need,), 0x7f, dtype=torch.uint8, device=DEV) if need and use_ws and not decode else None
        ops.channel_linear(q, z, v, self.bias.to(DEV), self.lower.to(DEV), p, self.state, self.heads, self.dim, self.vdim, out, q_act="silu", workspace=ws)
        at = 0
        for i, first, n in picks:
            want = self.want[i][first: first + n]
            got = out[at: at + n].cpu().double()
            assert torch.isfinite(got).all()
            err = (got - want).abs() / (want.abs() + 0.3 * want.abs().mean() + 1e-3)
            worst = float(err.max())
            assert worst < (5e-5 if self.dtype == F32 else 1e-2), (i, first, n, worst, int(err.max(1).values.argmax()))
            at += n
        return need

    def check_states(self, slots):
        for i, s in enumerate(self.states):
            got = self.state[slots[i]].cpu().double()
            assert_close(got[:, : self.dim, : self.vdim], s, 3e-5, ("state", i))
            assert not got[:, self.dim:].any() and not got[:, :, self.vdim:].any()


CHANNELS = [(2, 64, 64, BF), (3, 128, 128, BF), (4, 48, 40, BF), (2, 72, 144, BF), (2, 256, 96, BF), (1, 200, 32, BF), (6, 20, 200, BF), (1, 130, 24, BF),
            (3, 7, 5, BF), (2, 8, 4, BF), (2, 128, 64, BF), (2, 64, 80, F32), (4, 33, 17, F32), (1, 256, 64, F32)]


@pytest.mark.parametrize("heads,dim,vdim,dtype", CHANNELS)
def test_channel_gates_of_whole_sequences(heads, dim, vdim, dtype):
    announce(f"channels whole {heads} {dim} {vdim} {dtype}")
    case = Channels([1, 2, 64, 65, 150, 63, 257, 16, 17], heads, dim, vdim, dtype)
    slots = [3, 0, 6, 1, 5, 2, 7, 8, 4]
    case.run([(i, 0, n) for i, n in enumerate(case.lens)], slots)
    case.check_states(slots)


@pytest.mark.parametrize("heads,dim,vdim,dtype", CHANNELS)
def test_channel_gates_in_portions_and_single_tokens(heads, dim, vdim, dtype):
    announce(f"channels portions {heads} {dim} {vdim} {dtype}")
    case = Channels([140, 97], heads, dim, vdim, dtype, seed=3)
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


@pytest.mark.parametrize("shift,logit", [(-30.0, 1.0), (-8.0, 6.0), (0.0, 25.0), (60.0, 1.0), (12.0, 1.0)])
def test_channel_gates_that_forget_everything_or_nothing(shift, logit):
    """Factors so small that their products over a block have no reciprocal (some channels of some blocks, or all), and so close
    to one that what is written is a rounding of them."""
    announce(f"channels extreme {shift} {logit}")
    for heads, dim, vdim in ((2, 64, 48), (2, 128, 128), (1, 256, 32), (3, 40, 72)):
        for low in (0.0, 0.9):
            case = Channels([130, 65, 18], heads, dim, vdim, BF, seed=8, logit=logit, shift=shift, low=low)
            slots = [0, 2, 1]
            case.run([(i, 0, n) for i, n in enumerate(case.lens)], slots)
            case.check_states(slots)
            case.run([(0, 0, 33), (1, 0, 2)], slots)
            case.run([(0, 33, 97), (1, 2, 63)], slots)
            case.check_states(slots[:2] + [1])


@pytest.mark.parametrize("heads,dim,vdim", [(2, 64, 64), (1, 128, 128), (1, 256, 80), (2, 96, 200)])
def test_long_portions_run_in_segments(heads, dim, vdim):
    announce(f"channels segments {heads} {dim} {vdim}")
    case = Channels([2050, 530], heads, dim, vdim, BF, seed=4)
    assert case.run([(0, 0, 2050), (1, 0, 530)], [1, 0]) > 0
    case.check_states([1, 0])
    case.run([(0, 0, 1025), (1, 0, 3)], [0, 2])
    case.run([(0, 1025, 1025), (1, 3, 527)], [0, 2])
    case.check_states([0, 2])
    case.run([(0, 0, 2050), (1, 0, 530)], [0, 1], use_ws=False)
    case.check_states([0, 1])


@pytest.mark.parametrize("dtype", [F32, BF])
def test_channel_gates_remember_a_far_token(dtype):
    """Slow channels hold one large value of the first token; it is read out long after, beside fast channels that lost it."""
    announce(f"channels far {dtype}")
    n, dim, vdim = 400, 32, 32
    case = Channels([], 1, dim, vdim, dtype)
    case.lens = [n]
    case.bias, case.lower = torch.zeros(dim), torch.zeros(dim)
    z = torch.full((n, dim), 2.0)
    z[:, : dim // 2] = 12.0   # slow: nothing is forgotten, nothing is written
    z[0, : dim // 2] = -4.0   # except at the start
    v = 0.1 * _rand(n, vdim)
    v[0] = 10 + torch.arange(vdim)
    q = torch.full((n, dim), -30.0)  # (silu: nothing)
    q[-1, : dim // 2] = 1.0
    case.add([t.to(dtype) for t in (q, z, v)])
    assert case.want[0][-1].abs().min() > 10
    case.state = torch.full((1, 1, 32, 32), float("nan"), device=DEV)
    for cuts in ([n], [399, 1], [2] * 200, [17] * 23 + [9]):
        at = 0
        for c in cuts:
            case.run([(0, at, c)], [0], decode=c == 1)
            at += c
        case.check_states([0])


def test_padding_rows_and_other_slots_are_left_alone():
    announce("channels padding")
    case = Channels([40, 40], 2, 48, 72, BF, seed=3)
    case.state.fill_(7.0)
    u = lambda t: torch.stack([case.rows[0][t], case.rows[1][t], case.rows[0][t]]).to(DEV)
    for t in range(40):
        q, z, v = u(t).split([96, 96, 144], 1)
        out = torch.zeros(3, 144, dtype=BF, device=DEV)
        ops.channel_linear(q, z, v, case.bias.to(DEV), case.lower.to(DEV), ops.Portions(_i32([t + 1, t + 1, 0]), _i32([2, 0, -1])), case.state, 2, 48, 72,
                           out, q_act="silu")
        for b in (0, 1):
            assert_close(out[b], case.want[b][t], 1e-2)
        assert not out[2].any()
    case.check_states([2, 0])
    assert (case.state[1] == 7.0).all()
