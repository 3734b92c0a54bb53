"""Lightning attention on the GPU against the oracle's token-by-token recurrence: outputs and carried states, whole
sequences, portions of any length, unequal batches, slots used again, and long portions cut into segments."""

import numpy as np
import pytest
import torch

from oracle import hybrid_oracle as ho
from research_amd import ops
from tests.gpu_helpers import DEV, announce

pytestmark = pytest.mark.gpu

BF, F32 = torch.bfloat16, torch.float32


def _i32(values):
    return torch.tensor(list(values), dtype=torch.int32, device=DEV)


def _powers(decay):
    p = torch.tensor(decay, dtype=torch.float64)[:, None] ** torch.arange(65, dtype=torch.float64)
    return p.float().to(DEV).contiguous()


class Case:
    """Random projection rows ``[q | k | v | gate]`` of some sequences and the oracle's outputs and states."""

    def __init__(self, lens, heads, dim, vdim, decay, dtype, seed=0):
        g = torch.Generator().manual_seed(seed)
        self.heads, self.dim, self.vdim, self.dtype, self.decay = heads, dim, vdim, dtype, decay
        self.width = heads * (2 * dim + 2 * vdim)
        self.rows = [torch.randn(n, self.width, generator=g).to(dtype) for n in lens]
        self.want, self.final = [], []
        for r in self.rows:
            act = ho.silu(r.double())
            if dtype == BF:  # (activations are rounded to the type of the products)
                act = act.to(BF).double()
            q, k, v = act.split([heads * dim, heads * dim, 2 * heads * vdim], 1)
            o, s = ho.lightning_attention(q.view(-1, heads, dim), k.view(-1, heads, dim),
                                          v[:, : heads * vdim].reshape(-1, heads, vdim), decay)
            self.want.append(o.reshape(-1, heads * vdim))
            self.final.append(s)
        self.state = ops.lightning_state(len(lens) + 2, heads, dim, vdim, DEV)
        self.state.fill_(7.0)  # whatever a slot holds, a sequence starts empty

    def run(self, picks, slots, use_ws=True):
        """``picks``: (sequence, first row, rows) of one batch; returns the outputs row by row."""
        u = torch.cat([self.rows[b][lo: lo + n] for b, lo, n in picks]).to(DEV)
        out = torch.full((u.shape[0], self.heads * self.vdim), float("nan"), dtype=self.dtype, device=DEV)
        q_lens = [n for _, _, n in picks]
        por = ops.Portions(_i32(lo + n for _, lo, n in picks), _i32(slots[b] for b, _, _ in picks), _i32(q_lens),
                           _i32(np.cumsum([0] + q_lens[:-1])), None, max(q_lens))
        ws = None
        need = ops.lightning_workspace_bytes(len(picks), self.heads, self.dim, self.vdim, max(q_lens))
        if need and use_ws:
            ws = torch.full((need,), 0x7f, dtype=torch.uint8, device=DEV)
        ops.lightning(u, por, self.state, _powers(self.decay), self.heads, self.dim, self.vdim, out, workspace=ws)
        return out.cpu().split(q_lens)

    def check(self, b, lo, got):
        want = self.want[b][lo: lo + got.shape[0]]
        scale = want.abs().mean(-1, keepdim=True) + 1e-6
        tol = 1e-4 if self.dtype == F32 else 1.2e-2  # (the output is rounded to bf16)
        err = (got.double() - want).abs() / (scale + want.abs())
        assert torch.isfinite(got.double()).all()
        assert err.max() < tol, (b, lo, int(err.max(1).values.argmax()), float(err.max()))

    def check_state(self, b, slot):
        got = self.state[slot].cpu().double()[:, : self.dim, : self.vdim]
        err = (got - self.final[b]).abs().max() / self.final[b].abs().max()
        # (bf16: an activation at a rounding tie may fall to either side)
        assert err < (2e-5 if self.dtype == F32 else 1e-3), (b, float(err))


SHAPES = [(3, 16, 16), (2, 48, 80), (5, 64, 32), (2, 128, 128), (1, 96, 200), (2, 136, 72), (1, 256, 144), (2, 36, 20)]


@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("heads,dim,vdim", SHAPES)
def test_whole_sequences_of_unequal_length(heads, dim, vdim, dtype):
    announce(f"lightning {heads}x{dim}x{vdim} {dtype}")
    decay = [0.3, 0.97, 0.9995, 1.0, 0.0][:heads]
    lens = [1, 2, 63, 64, 65, 150]
    case = Case(lens, heads, dim, vdim, decay, dtype)
    slots = [3, 0, 5, 1, 6, 2]
    got = case.run([(b, 0, n) for b, n in enumerate(lens)], slots)
    for b in range(len(lens)):
        case.check(b, 0, got[b])
        case.check_state(b, slots[b])


@pytest.mark.parametrize("dtype", [BF, F32])
def test_portions_and_single_tokens_continue_the_state(dtype):
    announce(f"lightning portions {dtype}")
    heads, dim, vdim = 3, 80, 48
    case = Case([200, 131], heads, dim, vdim, [0.5, 0.99, 0.9999], dtype, seed=2)
    slots = [1, 3]
    at = [0, 0]
    sizes = [[2, 3, 64, 61, 2, 5, 63], [70, 2, 2, 33, 2, 7, 15]]
    for i in range(7):
        picks = [(b, at[b], sizes[b][i]) for b in (0, 1)]
        for (b, lo, n), got in zip(picks, case.run(picks, slots)):
            case.check(b, lo, got)
            at[b] += n
    assert at == [200, 131]
    for b in (0, 1):
        case.check_state(b, slots[b])


def test_decode_rows_equal_the_recurrence_and_padding_rows_are_skipped():
    announce("lightning decode")
    for dtype in (BF, F32):
        heads, dim, vdim = 2, 64, 96
        case = Case([40, 40, 40], heads, dim, vdim, [0.8, 0.999], dtype, seed=3)
        powers = _powers(case.decay)
        before = case.state.clone()
        for t in range(40):
            u = torch.stack([r[t] for r in case.rows] + [case.rows[0][t]]).to(DEV)
            out = torch.zeros(4, heads * vdim, dtype=dtype, device=DEV)
            por = ops.Portions(_i32([t + 1, t + 1, t + 1, 0]), _i32([2, 4, 0, -1]))
            ops.lightning(u, por, case.state, powers, heads, dim, vdim, out)
            for b in range(3):
                case.check(b, t, out[b: b + 1].cpu())
            assert not out[3].any()
        for b, slot in enumerate((2, 4, 0)):
            case.check_state(b, slot)
        assert torch.equal(case.state[1], before[1]) and torch.equal(case.state[3], before[3])


@pytest.mark.parametrize("heads,dim,vdim", [(2, 128, 128), (4, 64, 48), (1, 256, 80)])
def test_long_portions_in_segments(heads, dim, vdim):
    """Few sequences of many chunks: with a workspace the portion runs in segments; the same without one."""
    lens = [1125, 700]
    announce(f"lightning segments {heads}x{dim}x{vdim}")
    assert ops.lightning_workspace_bytes(2, heads, dim, vdim, 1125) > 0
    case = Case(lens, heads, dim, vdim, [0.999, 0.9, 0.99, 0.5][:heads], BF, seed=4)
    for use_ws in (True, False):
        for first in (0, 37):
            if first:
                case.run([(0, 0, first), (1, 0, first)], [1, 2])
            got = case.run([(b, first, lens[b] - first) for b in (0, 1)], [1, 2], use_ws)
            for b in (0, 1):
                case.check(b, first, got[b])
                case.check_state(b, 1 + b)
