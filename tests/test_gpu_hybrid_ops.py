"""The kernels around attention in hybrid blocks, each against a plain float32 statement or the oracle: residual sums
and norms, gates, the joint q/k/v step with its carried rows, and packed attention at the edges of windows and pages."""

import numpy as np
import pytest
import torch
import torch.nn.functional as F

from oracle import hybrid_oracle as ho
from research_amd import _lib, ops
from research_amd.inference import CacheConfig, HipPagedAttentionBackend, InferenceContext
from tests.gpu_helpers import DEV, announce, assert_close

pytestmark = pytest.mark.gpu

BF, F32 = torch.bfloat16, torch.float32
TOL = {F32: 2e-6, BF: 8e-3}


def _rand(*shape, dtype=F32, seed=0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed)).to(dtype)


def _i32(values):
    return torch.tensor(list(values), dtype=torch.int32, device=DEV)


# ------------------------------------------------------------------ rows


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("width", [4, 37, 76, 256, 260, 1000, 1030, 2048, 3000, 8192, 9000, 16384])
def test_residual_sums_and_norms(width, dtype):
    announce(f"residual {width} {dtype}")
    rows = 7
    x0, y = _rand(rows, width) * 3 + 1, _rand(rows, width, dtype=dtype, seed=1)
    w, b, yw = _rand(width, seed=2), _rand(width, seed=3), _rand(width, seed=4)
    dev = lambda t: t.to(DEV)
    for norm in ("layer", "rms", None):
        for branch in ("none", "plain", "normed"):
            x = dev(x0.clone())
            args = {} if branch == "none" else {"y": dev(y)}
            want = x0.double()
            if branch == "plain":
                want = want + y.double()
            if branch == "normed":
                args.update(y_weight=dev(yw), y_eps=1e-2)
                want = want + ho.unit_rms(y.double(), 1e-2) * yw.double()
            if norm is not None:
                args.update(weight=dev(w), bias=dev(b))
            got = ops.residual_norm(x, dtype, norm=norm, eps=1e-3, **args)
            assert_close(x, want, 2e-6, f"{norm} {branch} x")
            out = want
            if norm == "layer":
                out = ho.layer_norm(want, w.double(), b.double(), 1e-3)
            if norm == "rms":
                out = ho.unit_rms(want, 1e-3) * w.double() + b.double()
            assert_close(got, out, TOL[dtype], f"{norm} {branch}")
    table, ids = _rand(11, width, dtype=dtype, seed=5), torch.tensor([3, 0, 10, 3, -1, 11, 2])
    x = torch.full((rows, width), float("nan"), device=DEV)
    got = ops.residual_norm(x, dtype, ids=dev(ids), table=dev(table), norm="layer", weight=dev(w), bias=dev(b), eps=1e-3)
    want = torch.stack([table[i].double() if 0 <= i < 11 else torch.zeros(width, dtype=torch.float64) for i in ids.tolist()])
    assert torch.equal(x.cpu().double(), want)
    assert_close(got, ho.layer_norm(want, w.double(), b.double(), 1e-3), TOL[dtype], "embedding")
    pick = torch.tensor([6, 0, 0])
    got = ops.residual_norm(x, dtype, row_index=dev(pick), norm="rms", weight=dev(w), eps=1e-3)
    assert_close(got, ho.unit_rms(want[pick], 1e-3) * w.double(), TOL[dtype], "picked rows")


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("width", [8, 20, 33, 640, 4096, 9008])
def test_gates_and_activations(width, dtype):
    announce(f"gates {width} {dtype}")
    rows = 5
    wide = _rand(rows, 3 * width + 3, dtype=dtype).to(DEV)
    for lo in (0, 3):  # a slice that is aligned, and one that is not
        a, g = wide[:, lo: lo + width], wide[:, lo + width: lo + 2 * width]
        ac, gc = a.cpu().double(), g.cpu().double()
        assert_close(ops.glu(a, g, "silu"), ho.silu(ac) * gc, TOL[dtype], "silu")
        assert_close(ops.glu(a, g, "gelu_tanh"), ho.gelu_tanh(ac) * gc, TOL[dtype], "gelu")
        o, w = _rand(rows, width, dtype=dtype, seed=1), _rand(width, seed=2)
        got = ops.rms_gate(o.to(DEV), g, w.to(DEV), 1e-2)
        assert_close(got, ho.unit_rms(o.double(), 1e-2) * w.double() * ho.sigmoid(gc), TOL[dtype], "rms gate")
    table, ids = _rand(9, 4 * width, dtype=dtype, seed=3), torch.tensor([8, 0, 9, 4, -2])
    col = table[:, width: 2 * width]
    got = ops.glu(wide[:, :width], table.to(DEV)[:, width: 2 * width], "gelu_tanh", ids=ids.to(DEV))
    want = torch.stack([col[i].double() if 0 <= i < 9 else torch.zeros(width, dtype=torch.float64) for i in ids.tolist()])
    assert_close(got, ho.gelu_tanh(wide[:, :width].cpu().double()) * want, TOL[dtype], "token rows")


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("heads,d,vdim", [(3, 40, 24), (2, 16, 16), (5, 24, 17), (1, 256, 200)])
def test_head_gates_pack_the_value_part(heads, d, vdim, dtype):
    announce(f"head gate {heads} {d} {vdim} {dtype}")
    o, g = _rand(6, heads, d, dtype=dtype), _rand(6, heads + 2, dtype=dtype, seed=1)
    got = ops.head_gate(o.to(DEV), g.to(DEV)[:, 1: 1 + heads], vdim)
    want = o.double()[:, :, :vdim] * ho.sigmoid(g.double()[:, 1: 1 + heads])[:, :, None]
    assert_close(got, want.reshape(6, -1), TOL[dtype], "gated")
    assert torch.equal(ops.head_gate(o.to(DEV), None, vdim).cpu(), o[:, :, :vdim].reshape(6, -1))


# ------------------------------------------------------------------ joint q/k/v step


def _qkv_want(u, hq, hkv, dim, vdim, conv, rot, base, factor, eps, norm):
    t = u.shape[0]
    y = u[:, : (hq + hkv) * dim + hkv * vdim]
    if conv is not None:
        y = ho.causal_conv(y, conv.T)
    q, k, v = y.split([hq * dim, hkv * dim, hkv * vdim], 1)
    q = ho.rotate_interleaved(q.reshape(t, hq, dim), base, rot, factor)
    k = ho.rotate_interleaved(k.reshape(t, hkv, dim), base, rot, factor)
    if norm:
        q, k = ho.unit_rms(q, eps), ho.unit_rms(k, eps)
    return q, k, v.reshape(t, hkv, vdim)


QKV = [  # hq, hkv, dim, vdim, taps, rotated dims
    (4, 2, 32, 24, 4, 12), (3, 1, 64, 64, 3, 64), (2, 2, 20, 36, 2, 10), (6, 3, 96, 136, 5, 32), (1, 1, 256, 8, 8, 2),
    (5, 5, 8, 16, 0, 8), (2, 1, 28, 28, 1, 0), (4, 4, 136, 200, 6, 40),
]


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("hq,hkv,dim,vdim,taps,rot", QKV)
def test_qkv_step_in_portions(hq, hkv, dim, vdim, taps, rot, dtype):
    """Two sequences in portions down to one and two tokens, beside a padding row in the decode form; slots in shuffled
    blocks; the carried rows of a slot that another sequence used before."""
    announce(f"qkv {hq} {hkv} {dim} {vdim} {taps} {rot} {dtype}")
    lens, base, factor, eps = [45, 38], 60.0, 1.5, 1e-2
    chans, d, bs = (hq + hkv) * dim + hkv * vdim, -(-max(dim, vdim) // 8) * 8, 8
    us = [_rand(n, chans + 3, dtype=dtype, seed=i) for i, n in enumerate(lens)]
    conv = _rand(taps, chans, seed=7) if taps else None
    firsts = [_rand(n, hkv * vdim, dtype=dtype, seed=20 + i) for i, n in enumerate(lens)]
    lam = torch.tensor([0.3], device=DEV)
    want = [_qkv_want(u.double(), hq, hkv, dim, vdim, None if conv is None else conv.double(), rot, base, factor, eps, True)
            for u in us]
    freq = base ** (-torch.arange(0, rot, 2, dtype=torch.float64) / max(rot, 1)) / factor
    ang = torch.arange(64, dtype=torch.float64)[:, None] * freq
    rope = torch.stack([ang.cos(), ang.sin()], -1).float().contiguous().to(DEV) if rot else None
    perm = torch.randperm(16, generator=torch.Generator().manual_seed(5)).tolist()
    blocks = [perm[:6], perm[6:12]]
    kc = torch.zeros(16 * bs, hkv, d, dtype=dtype, device=DEV)
    vc = torch.zeros_like(kc)
    state = _rand(4, max(taps - 1, 1), chans, dtype=dtype, seed=9).to(DEV) if taps > 1 else None
    before = None if state is None else state.clone()
    sslot = [2, 0]
    got_q = [torch.zeros(n, hq, d) for n in lens]
    mode = {0: None, 1: "first", 2: "mix"}[(hq + taps) % 3]
    seen_first = [torch.zeros(n, hkv * vdim) for n in lens]
    at = [0, 0]
    sizes = [(2, 17), (1, 2), (19, 1), (1, 1), (2, 3), (16, 14), (4, 0)]
    for n0, n1 in sizes:
        picks = [(b, at[b], n) for b, n in ((0, n0), (1, n1)) if n]
        decode = all(n == 1 for _, _, n in picks) and len(picks) == 2
        rows = torch.cat([us[b][lo: lo + n] for b, lo, n in picks])
        vf = torch.cat([firsts[b][lo: lo + n] for b, lo, n in picks]).to(DEV) if mode == "mix" else \
            torch.zeros(rows.shape[0], hkv * vdim, dtype=dtype, device=DEV)
        slots = [blocks[b][p // bs] * bs + p % bs for b, lo, n in picks for p in range(lo, lo + n)]
        ctx, q_lens, st = [lo + n for _, lo, n in picks], [n for _, _, n in picks], [sslot[b] for b, _, _ in picks]
        if decode:  # with a padding row
            rows, vf = torch.cat([rows, rows[:1]]), torch.cat([vf, vf[:1]])
            por = ops.Portions(_i32(ctx + [0]), _i32(st + [-1]))
            slots = slots + [-1]
        else:
            starts = np.cumsum([0] + q_lens[:-1]).tolist()
            tiles = [(i, r) for i, n in enumerate(q_lens) for r in range(0, n, ops.QKV_TILE_ROWS)]
            por = ops.Portions(_i32(ctx), _i32(st), _i32(q_lens), _i32(starts),
                               torch.tensor(tiles, dtype=torch.int32, device=DEV), max(q_lens))
        q = ops.qkv_conv_append(rows.to(DEV), por, torch.tensor(slots, device=DEV), kc, vc, hq, dim, vdim, 0.4, eps, True, rope,
                                rot, None if conv is None else conv.to(DEV), state, mode, vf, lam if mode == "mix" else None)
        r = 0
        for b, lo, n in picks:
            got_q[b][lo: lo + n] = q[r: r + n].float().cpu()
            seen_first[b][lo: lo + n] = vf[r: r + n].float().cpu()
            r += n
            at[b] += n
    assert at == lens
    for b in (0, 1):
        idx = torch.tensor([blocks[b][p // bs] * bs + p % bs for p in range(lens[b])])
        k, v = kc.cpu()[idx], vc.cpu()[idx]
        wq, wk, wv = want[b]
        assert_close(got_q[b][..., :dim], 0.4 * wq, 4 * TOL[dtype], "q")
        assert_close(k[..., :dim], wk, 4 * TOL[dtype], "k")
        if mode == "mix":
            wv = 0.7 * wv + 0.3 * firsts[b].double().view(wv.shape)
        assert_close(v[..., :vdim], wv, 4 * TOL[dtype], "v")
        if mode == "first":
            assert_close(seen_first[b], wv.reshape(lens[b], -1), 4 * TOL[dtype], "first values")
        assert not got_q[b][..., dim:].any() and not k[..., dim:].any() and not v[..., vdim:].any()
        if state is not None:
            assert torch.equal(state[sslot[b]].cpu(), us[b][lens[b] - taps + 1:, :chans])  # the last projected rows
    if state is not None:  # slots of other sequences are untouched
        assert torch.equal(state[1], before[1]) and torch.equal(state[3], before[3])


# ------------------------------------------------------------------ packed attention


def _one_key_stands_out(dtype, d, window, bs, q_rows, total, target):
    """Scores are zero except that key ``target`` of every sequence scores 40; its value is all ones, all others zero.
    Returns the backend's packed output for the last ``q_rows`` positions of a ``total``-token sequence."""
    backend = HipPagedAttentionBackend(CacheConfig(num_layers=1, num_kv_heads=1, head_dim=d, num_blocks=-(-total // bs) + 3,
                                                   block_size=bs, dtype=dtype, layer_kv=((1, d),)))
    blocks = torch.randperm(-(-total // bs) + 3, generator=torch.Generator().manual_seed(total)).tolist()
    slot = lambda p: blocks[p // bs] * bs + p % bs
    kc, vc = backend.k_cache[0], backend.v_cache[0]
    kc[slot(target), 0, 0] = 8.0
    vc[slot(target)] = 1.0
    q = torch.zeros(q_rows, 2, d, dtype=dtype, device=DEV)
    q[:, :, 0] = 5.0
    ctx = InferenceContext(is_prefill=True, block_tables=np.asarray([blocks[: -(-total // bs)]], dtype=np.int32),
                           seq_lens=np.asarray([total]), q_lens=np.asarray([q_rows]), num_decodes=1 if q_rows == 1 else 0)
    return backend.attend_packed(q, 0, backend.packed_step(ctx), 1.0, window).float().cpu()


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("window", [1, 2, 15, 16, 17, 33, 64, 95])
def test_window_edges_in_decode(window, dtype):
    announce(f"window edge decode {window} {dtype}")
    for total in (window, window + 1, 64, 65, 113, 128, 129):
        for target in {max(0, total - window), total - window - 1, total - 1, 0}:
            if not 0 <= target < total:
                continue
            o = _one_key_stands_out(dtype, 32, window, 16, 1, total, target)
            inside = total - 1 - target < window
            assert (o > 0.99).all() if inside else not o.any(), (total, target)


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("window", [1, 16, 31, 50, 64])
def test_window_edges_in_portions(window, dtype):
    announce(f"window edge prefill {window} {dtype}")
    for total, rows in ((130, 130), (130, 2), (131, 37), (200, 64)):
        for target in (0, 15, 16, total - rows, total - rows - window, total - window, total - 1):
            if not 0 <= target < total:
                continue
            o = _one_key_stands_out(dtype, 32, window, 16, rows, total, target)
            dist = torch.arange(total - rows, total) - target
            inside = (dist >= 0) & (dist < window)
            assert (o[inside] > 0.99).all() and not o[~inside].any(), (total, rows, target)


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("heads,kv,d,window", [(6, 2, 40, 20), (5, 1, 96, 0), (4, 4, 16, 200), (12, 1, 160, 70)])
def test_packed_batches_of_decodes_and_portions(heads, kv, d, window, dtype):
    announce(f"packed attention {heads} {kv} {d} {window} {dtype}")
    bs = 16
    lens, rows = [77, 1, 33, 150, 64, 2], [1, 1, 1, 90, 64, 2]
    per = [-(-n // bs) for n in lens]
    backend = HipPagedAttentionBackend(CacheConfig(num_layers=2, num_kv_heads=kv, head_dim=d, num_blocks=sum(per), block_size=bs,
                                                   dtype=dtype, layer_kv=(None, (kv, d))))
    perm = np.random.default_rng(1).permutation(sum(per)).astype(np.int32)
    tables, at = np.full((6, max(per)), -1, dtype=np.int32), 0
    backend.k_cache[1].copy_(_rand(sum(per) * bs, kv, d, seed=1))
    backend.v_cache[1].copy_(_rand(sum(per) * bs, kv, d, seed=2))
    for b, n in enumerate(per):
        tables[b, :n] = perm[at: at + n]
        at += n
    q = _rand(sum(rows), heads, d, dtype=dtype, seed=3)
    ctx = InferenceContext(is_prefill=True, block_tables=tables, seq_lens=np.asarray(lens), q_lens=np.asarray(rows), num_decodes=3)
    got = backend.attend_packed(q.to(DEV), 1, backend.packed_step(ctx), d ** -0.5, window).cpu()
    kc, vc, r = backend.k_cache[1].cpu().double(), backend.v_cache[1].cpu().double(), 0
    for b, n in enumerate(lens):
        idx = torch.tensor([tables[b, p // bs] * bs + p % bs for p in range(n)])
        full_q = torch.zeros(n, heads, d, dtype=torch.float64)
        full_q[n - rows[b]:] = q[r: r + rows[b]].double()
        want = ho.window_attention(full_q, kc[idx], vc[idx], d ** -0.5, window or None)[n - rows[b]:]
        assert_close(got[r: r + rows[b]], want, 2e-2 if dtype == BF else 1e-5, f"sequence {b}")
        r += rows[b]


def test_bad_arguments_are_refused():
    x = torch.zeros(2, 8, device=DEV)
    with pytest.raises(ValueError):
        ops.residual_norm(x, F32, y=torch.zeros(3, 8, device=DEV))
    with pytest.raises(ValueError):
        ops.glu(x, torch.zeros(2, 9, device=DEV), "silu")
    with pytest.raises(_lib.PagedAttnError):
        ops.residual_norm(torch.zeros(1, 16388, device=DEV), F32, norm="rms", weight=torch.ones(16388, device=DEV))
