"""The C ABI without a GPU: the library loads, exports every symbol the header
declares, and rejects bad arguments with a status code and a message before it
touches any device (so none of these calls computes anything)."""

import ctypes
import os
import re

import pytest

from research_amd import _lib

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
HEADER = os.path.join(ROOT, "include", "paged_attn.h")


def _declared_functions():
    text = re.sub(r"/\*.*?\*/", "", open(HEADER).read(), flags=re.S)
    return sorted(set(re.findall(r"\b(pa_[a-z0-9_]+)\s*\(", text)))


def test_library_exports_every_declared_symbol():
    lib = ctypes.CDLL(_lib.LIB_PATH)
    names = _declared_functions()
    assert len(names) >= 10
    for name in names:
        assert hasattr(lib, name), f"{name} declared in paged_attn.h but not exported"


def test_binding_table_matches_header():
    assert sorted(_lib.SIGNATURES) == _declared_functions()


def test_version_and_dtype_sizes():
    lib = _lib.load()
    assert lib.pa_version() == 10
    assert [lib.pa_dtype_bytes(c) for c in (0, 1, 2, 3, 4, -1)] == [4, 2, 2, 1, 0, 0]


def test_missing_library_fails_loudly(tmp_path):
    with pytest.raises(FileNotFoundError, match="no other implementation"):
        _lib.load(str(tmp_path / "libpaged_attn.so"))


FAKE = ctypes.c_void_p(0x1000)  # never dereferenced: every call below is rejected first


def _status(name, *args):
    lib = _lib.load()
    rc = getattr(lib, name)(*args)
    return rc, _lib.last_error()


def test_scatter_argument_errors():
    rc, msg = _status("pa_kv_scatter", FAKE, FAKE, FAKE, FAKE, FAKE, 4, 64, 8, 128, 3, None)
    assert rc == _lib.PA_ERR_INVALID_ARG and "elem_bytes" in msg
    rc, msg = _status("pa_kv_scatter", FAKE, FAKE, FAKE, FAKE, FAKE, -1, 64, 8, 128, 2, None)
    assert rc == _lib.PA_ERR_INVALID_ARG and "n_tokens" in msg
    rc, msg = _status("pa_kv_scatter", None, FAKE, FAKE, FAKE, FAKE, 4, 64, 8, 128, 2, None)
    assert rc == _lib.PA_ERR_INVALID_ARG and "NULL" in msg
    rc, msg = _status("pa_kv_scatter", FAKE, FAKE, FAKE, FAKE, FAKE, 4, 64, 1, 3, 1, None)
    assert rc == _lib.PA_ERR_INVALID_ARG and "multiple of 4" in msg
    # nothing to do is fine and needs no pointers
    assert _status("pa_kv_scatter", None, None, None, None, None, 0, 64, 8, 128, 2, None)[0] == _lib.PA_OK


def test_gather_argument_errors():
    rc, msg = _status("pa_kv_gather", FAKE, FAKE, FAKE, FAKE, FAKE, 4, FAKE, 2, 16, 8, 0, 8, 128, 2, None)
    assert rc == _lib.PA_ERR_INVALID_ARG and "block_size" in msg
    rc, msg = _status("pa_kv_gather", FAKE, FAKE, None, FAKE, FAKE, 4, FAKE, 2, 16, 8, 16, 8, 128, 2, None)
    assert rc == _lib.PA_ERR_INVALID_ARG and "NULL" in msg
    assert _status("pa_kv_gather", None, None, None, None, None, 0, None, 0, 0, 8, 16, 8, 128, 2, None)[0] == 0


def _decode_args(**kw):
    a = dict(q=FAKE, k=FAKE, v=FAKE, out=FAKE, bt=FAKE, bt_stride=4, lens=FAKE, ez=None, ks=None, vs=None,
             batch=2, hq=32, hkv=8, d=128, bs=16, nb=64, scale=0.088, window=0, qd=_lib.PA_BF16, kvd=_lib.PA_BF16,
             ws=FAKE, ws_bytes=1 << 30, stream=None)
    a.update(kw)
    return [a[k] for k in ("q", "k", "v", "out", "bt", "bt_stride", "lens", "ez", "ks", "vs", "batch", "hq", "hkv",
                           "d", "bs", "nb", "scale", "window", "qd", "kvd", "ws", "ws_bytes", "stream")]


def test_decode_argument_errors():
    rc, msg = _status("pa_decode", *_decode_args(hq=30))
    assert rc == _lib.PA_ERR_INVALID_ARG and "multiple of num_kv_heads" in msg
    rc, msg = _status("pa_decode", *_decode_args(bs=0))
    assert rc == _lib.PA_ERR_INVALID_ARG and "block_size" in msg
    for entry in ("pa_decode_split", "pa_decode_reduce"):
        rc, msg = _status(entry, *_decode_args(hq=30))
        assert rc == _lib.PA_ERR_INVALID_ARG
    rc, msg = _status("pa_decode", *_decode_args(d=100))  # (any multiple of 8 up to 256 has a kernel)
    assert rc == _lib.PA_ERR_UNSUPPORTED and "head_dim=100" in msg
    rc, msg = _status("pa_decode", *_decode_args(d=264))
    assert rc == _lib.PA_ERR_UNSUPPORTED
    rc, msg = _status("pa_decode", *_decode_args(qd=_lib.PA_F32))
    assert rc == _lib.PA_ERR_UNSUPPORTED  # q and pool types must match unless the pool is fp8
    rc, msg = _status("pa_decode", *_decode_args(kvd=_lib.PA_FP8_E4M3))
    assert rc == _lib.PA_ERR_INVALID_ARG and "k_scale" in msg
    rc, msg = _status("pa_decode", *_decode_args(ws_bytes=1024))
    assert rc == _lib.PA_ERR_WORKSPACE and "need" in msg
    rc, msg = _status("pa_decode", *_decode_args(ws=None))
    assert rc == _lib.PA_ERR_WORKSPACE
    # more than 8192 sequences are taken 8192 at a time through a workspace sized for 8192
    lib = _lib.load()
    assert (lib.pa_decode_workspace_bytes(10000, 32, 8, 128, _lib.PA_BF16)
            == lib.pa_decode_workspace_bytes(8192, 32, 8, 128, _lib.PA_BF16))
    rc, msg = _status("pa_decode", *_decode_args(batch=10000, ws_bytes=1024))
    assert rc == _lib.PA_ERR_WORKSPACE
    rc, msg = _status("pa_decode", *_decode_args(q=None))
    assert rc == _lib.PA_ERR_INVALID_ARG and "NULL" in msg
    assert _status("pa_decode", *_decode_args(batch=0, q=None, ws=None, ws_bytes=0))[0] == _lib.PA_OK


def test_decode_static_argument_errors():
    """The entry point without a workspace rejects bad arguments, and shapes whose partials exceed the library's
    fixed scratch array, before it touches a device."""
    static = lambda **kw: _decode_args(**kw)[:-3] + [None]
    rc, msg = _status("pa_decode_static", *static(hq=30))
    assert rc == _lib.PA_ERR_INVALID_ARG and "multiple of num_kv_heads" in msg
    rc, msg = _status("pa_decode_static", *static(d=100))
    assert rc == _lib.PA_ERR_UNSUPPORTED
    rc, msg = _status("pa_decode_static", *static(batch=8192))
    assert rc == _lib.PA_ERR_WORKSPACE and "scratch" in msg and "pa_decode_workspace_bytes" in msg
    assert _status("pa_decode_static", *static(batch=0, q=None))[0] == _lib.PA_OK


def test_decode_workspace_arithmetic():
    lib = _lib.load()
    small = lib.pa_decode_workspace_bytes(1, 1, 1, 32, _lib.PA_F32)
    c4 = lib.pa_decode_workspace_bytes(256, 32, 8, 128, _lib.PA_BF16)
    # (4096 + planes*batch) slots of hpw*NREP heads x (D+2) floats: shapes only, no lengths
    assert 0 < small < c4 and c4 >= (4096 + 2 * 256) * 16 * 130 * 4
    assert c4 % 256 == 0
    assert lib.pa_decode_workspace_bytes(256, 32, 8, 128, _lib.PA_FP8_E4M3) > 0
    assert lib.pa_decode_workspace_bytes(-1, 32, 8, 128, _lib.PA_BF16) == 0
    assert "pa_decode_workspace_bytes" in _lib.last_error()
    # head sizes between the compiled ones take the next larger kernel (and its workspace); odd ones have none
    assert (lib.pa_decode_workspace_bytes(4, 32, 8, 96, _lib.PA_BF16)
            == lib.pa_decode_workspace_bytes(4, 32, 8, 128, _lib.PA_BF16))
    assert lib.pa_decode_workspace_bytes(4, 32, 8, 100, _lib.PA_BF16) == 0
    assert lib.pa_decode_workspace_bytes(4, 30, 8, 128, _lib.PA_BF16) == 0


def test_prefill_and_quantize_argument_errors():
    args = [FAKE, FAKE, FAKE, FAKE, FAKE, 4, FAKE, FAKE, FAKE, None, 2, 16, 32, 8, 128, 16, 64, 0.088, 0,
            _lib.PA_FP8_E4M3, None]
    rc, msg = _status("pa_prefill_paged", *args)
    assert rc == _lib.PA_ERR_INVALID_ARG and "dtype" in msg
    args[-2] = _lib.PA_BF16
    args[14] = 84  # (not a multiple of 8: no kernel)
    rc, msg = _status("pa_prefill_paged", *args)
    assert rc == _lib.PA_ERR_UNSUPPORTED
    rc, msg = _status("pa_quantize_kv_e4m3", FAKE, FAKE, FAKE, 4, 16, 8, 128, _lib.PA_FP8_E4M3, None)
    assert rc == _lib.PA_ERR_INVALID_ARG and "src_dtype" in msg
    rc, msg = _status("pa_quantize_kv_e4m3", None, FAKE, FAKE, 4, 16, 8, 128, _lib.PA_F32, None)
    assert rc == _lib.PA_ERR_INVALID_ARG and "NULL" in msg
    append = [FAKE, FAKE, FAKE, FAKE, FAKE, FAKE, FAKE, 5, FAKE, 2, None, None, 64, 16, 8, 128, _lib.PA_BF16, None]
    bad = list(append); bad[16] = _lib.PA_FP8_E4M3
    rc, msg = _status("pa_kv_append_e4m3", *bad)
    assert rc == _lib.PA_ERR_INVALID_ARG and "src_dtype" in msg
    bad = list(append); bad[13] = 1024
    rc, msg = _status("pa_kv_append_e4m3", *bad)
    assert rc == _lib.PA_ERR_INVALID_ARG and "block_size" in msg
    bad = list(append); bad[8] = None
    rc, msg = _status("pa_kv_append_e4m3", *bad)
    assert rc == _lib.PA_ERR_INVALID_ARG and "NULL" in msg
    bad = list(append); bad[10] = FAKE  # a row order without the block starts
    rc, msg = _status("pa_kv_append_e4m3", *bad)
    assert rc == _lib.PA_ERR_INVALID_ARG and "row_order" in msg
    bad = list(append); bad[7] = 0  # nothing to append: fine even with no device
    rc, msg = _status("pa_kv_append_e4m3", *bad)
    assert rc == _lib.PA_OK


def test_rope_argument_errors():
    rope = [FAKE, FAKE, FAKE, FAKE, None, FAKE, FAKE, FAKE, FAKE, None, 8, FAKE, 4, 64, 32, 8, 128, _lib.PA_BF16, None]
    bad = list(rope); bad[17] = _lib.PA_FP8_E4M3
    rc, msg = _status("pa_rope_kv_append", *bad)
    assert rc == _lib.PA_ERR_INVALID_ARG and "dtype" in msg
    bad = list(rope); bad[16] = 24  # half a head = 12 bf16 = 24 bytes
    rc, msg = _status("pa_rope_kv_append", *bad)
    assert rc == _lib.PA_ERR_UNSUPPORTED and "16 bytes" in msg
    bad = list(rope); bad[10] = 3  # 3 table rows for 4 tokens and no positions
    rc, msg = _status("pa_rope_kv_append", *bad)
    assert rc == _lib.PA_ERR_INVALID_ARG and "positions" in msg
    bad = list(rope); bad[11] = None  # no slots and no k_out
    rc, msg = _status("pa_rope_kv_append", *bad)
    assert rc == _lib.PA_ERR_INVALID_ARG and "nowhere" in msg
    bad = list(rope); bad[0] = None
    rc, msg = _status("pa_rope_kv_append", *bad)
    assert rc == _lib.PA_ERR_INVALID_ARG and "NULL" in msg
    bad = list(rope); bad[12] = 0
    assert _status("pa_rope_kv_append", *bad)[0] == _lib.PA_OK
    fp8 = [FAKE, FAKE, FAKE, FAKE, FAKE, FAKE, FAKE, FAKE, FAKE, FAKE, None, 8, FAKE, 4, FAKE, 1, None, None, 64, 16, 32,
           8, 128, _lib.PA_BF16, None]
    bad = list(fp8); bad[19] = 1024
    rc, msg = _status("pa_rope_kv_append_e4m3", *bad)
    assert rc == _lib.PA_ERR_INVALID_ARG and "block_size" in msg
    bad = list(fp8); bad[11] = 2
    rc, msg = _status("pa_rope_kv_append_e4m3", *bad)
    assert rc == _lib.PA_ERR_INVALID_ARG and "positions" in msg
    bad = list(fp8); bad[13] = 0
    assert _status("pa_rope_kv_append_e4m3", *bad)[0] == _lib.PA_OK


def test_error_text_is_cleared_by_a_good_call():
    _status("pa_kv_scatter", FAKE, FAKE, FAKE, FAKE, FAKE, -1, 64, 8, 128, 2, None)
    assert _lib.last_error() != ""
    assert _status("pa_kv_scatter", None, None, None, None, None, 0, 64, 8, 128, 2, None)[0] == 0
    assert _lib.last_error() == ""


@pytest.mark.parametrize("script,generated", [("gen_prefill_loop.py", "prefill_mfma_loop.inc"),
                                              ("gen_prefill_loop_d256.py", "prefill_d256_loop.inc")])
def test_generated_prefill_loop_is_current(tmp_path, script, generated):
    """The committed assembly loops (head_dim 128: prefill_mfma_loop.inc; head_dim 256: prefill_d256_loop.inc) are
    what their generators write (the generators also check the instruction distances the hardware does not
    interlock, so a schedule that violates one cannot be committed)."""
    import os
    import subprocess
    import sys
    csrc = os.path.join(os.path.dirname(os.path.dirname(os.path.abspath(__file__))), "research_amd", "csrc")
    out = tmp_path / "loop.inc"
    subprocess.run([sys.executable, os.path.join(csrc, script), str(out)], check=True, stdout=subprocess.DEVNULL)
    assert out.read_text() == open(os.path.join(csrc, generated)).read()


def test_block_entry_points_check_their_arguments():
    """The kernels around attention in hybrid blocks: rejected before any device call."""
    f32, bf16 = _lib.PA_F32, _lib.PA_BF16
    residual = lambda **kw: [{**dict(x=FAKE, y=FAKE, mw=None, mix=0, yx=None, yb=None, y2=None, yp=None, y2p=None, yw=None, ye=0.0, ids=None, ia=0, table=None, tr=0,
                                     ts=1.0, pos=None, pt=None, pr=0, ri=None, xr=4, w=FAKE, b=FAKE, eps=1e-6,
                                     norm=_lib.PA_NORM_LAYER, out=FAKE, rows=4, width=64, dt=bf16, s=None), **kw}[k]
                             for k in ("x", "y", "mw", "mix", "yx", "yb", "y2", "yp", "y2p", "yw", "ye", "ids", "ia", "table", "tr", "ts", "pos", "pt", "pr", "ri",
                                       "xr", "w", "b", "eps", "norm", "out", "rows", "width", "dt", "s")]
    for kw, status, text in ((dict(x=None), -1, "neither"), (dict(norm=7), -1, "norm=7"), (dict(width=20000), -2, "above"),
                             (dict(dt=_lib.PA_F16), -2, "dtype"), (dict(ids=FAKE), -1, "table"), (dict(ri=FAKE), -1, "row_index"),
                             (dict(y=None, out=None), -1, "nothing"), (dict(y=None, yw=FAKE), -1, "y_weight"),
                             (dict(norm=_lib.PA_NORM_NONE), -1, "without a norm"), (dict(pos=FAKE, pt=FAKE), -1, "positions"),
                             (dict(mw=FAKE), -1, "mix_weight"), (dict(yx=FAKE), -1, "y_extra"), (dict(ia=1), -1, "ids_add"),
                             (dict(y=None, yb=FAKE), -1, "y_bias"), (dict(mw=FAKE, mix=2, y2=FAKE, yp=FAKE, y2p=FAKE), -1, "y2"),
                             (dict(y2=FAKE, yp=FAKE), -1, "together"), (dict(yp=FAKE), -1, "together")):
        rc, msg = _status("pa_residual_norm", *residual(**kw))
        assert rc == status and text in msg, (kw, msg)
    assert _status("pa_residual_norm", *residual(rows=0, x=None))[0] == 0
    rc, msg = _status("pa_rms_gate", FAKE, FAKE, 60, FAKE, 1e-6, FAKE, 64, 4, 64, 1, 0, f32, None)
    assert rc == -1 and "gate_stride" in msg
    rc, msg = _status("pa_rms_gate", FAKE, FAKE, 64, FAKE, 1e-6, FAKE, 60, 4, 64, 1, 0, f32, None)
    assert rc == -1 and "out_stride" in msg
    rc, msg = _status("pa_rms_gate", FAKE, FAKE, 64, FAKE, 1e-6, FAKE, 64, 4, 64, 3, 0, f32, None)
    assert rc == -1 and "equal groups" in msg
    rc, msg = _status("pa_softcap", FAKE, FAKE, 4, 0.0, f32, None)
    assert rc == -1 and "cap" in msg
    rc, msg = _status("pa_glu", FAKE, 64, FAKE, 64, None, 0, FAKE, 4, 64, 9, f32, None)
    assert rc == -1 and "act" in msg
    rc, msg = _status("pa_head_gate", FAKE, FAKE, 4, 1.0, FAKE, 96, 4, 4, 16, 24, f32, None)
    assert rc == -1 and "sizes" in msg

    qkv = lambda **kw: [{**dict(u=FAKE, ld=200, n=4, ub=None, cw=FAKE, taps=3, cs=FAKE, sr=2, rope=FAKE, rr=9, rot=8, cl=FAKE, ql=None,
                                qs=None, ss=FAKE, tiles=None, nt=4, batch=4, slots=FAKE, ts=64, q=FAKE, k=FAKE, v=FAKE, vf=None,
                                lam=None, vm=0, qn=None, kn=None, hq=4, hkv=2, dim=16, vdim=24, d=24, un=1, eps=1e-6, qsc=1.0, dt=bf16, s=None),
                           **kw}[k] for k in ("u", "ld", "n", "ub", "cw", "taps", "cs", "sr", "rope", "rr", "rot", "cl", "ql", "qs", "ss",
                                              "tiles", "nt", "batch", "slots", "ts", "q", "k", "v", "vf", "lam", "vm", "qn", "kn", "hq", "hkv",
                                              "dim", "vdim", "d", "un", "eps", "qsc", "dt", "s")]
    for kw, status, text in ((dict(hkv=3), -1, "multiple"), (dict(d=20), -1, "pool_dim"), (dict(rot=9), -1, "rot_dims"),
                             (dict(taps=9), -2, "taps"), (dict(cw=None), -1, "convolution"), (dict(cs=None), -1, "carried"),
                             (dict(rope=None), -1, "table"), (dict(vm=2, vf=FAKE), -1, "v_lambda"), (dict(vm=1), -1, "v_first"),
                             (dict(nt=3), -1, "one row"), (dict(ld=100), -1, "u_stride"), (dict(tiles=FAKE), -1, "tiles"),
                             (dict(dt=_lib.PA_F16), -2, "dtype"), (dict(d=264), -2, "above 256"), (dict(qn=FAKE), -1, "together"),
                             (dict(ub=FAKE), -1, "bias")):
        rc, msg = _status("pa_qkv_conv_append", *qkv(**kw))
        assert rc == status and text in msg, (kw, msg)
    assert _status("pa_qkv_conv_append", *qkv(n=0, u=None, batch=0, nt=0))[0] == 0

    lib = _lib.load()
    assert lib.pa_lightning_state_floats(20, 40) == 32 * 48
    chunked = lambda **kw: [{**dict(u=FAKE, ld=200, n=4, st=FAKE, sr=2, dp=FAKE, cl=FAKE, ql=FAKE, qs=FAKE, ss=FAKE, batch=2, mq=4,
                                    out=FAKE, h=2, dim=16, vdim=24, dt=bf16, ws=None, wb=0, s=None), **kw}[k]
                            for k in ("u", "ld", "n", "st", "sr", "dp", "cl", "ql", "qs", "ss", "batch", "mq", "out", "h", "dim",
                                      "vdim", "dt", "ws", "wb", "s")]
    for kw, status, text in ((dict(dt=f32), -2, "BF16"), (dict(dim=300, ld=2000), -2, "above 256"), (dict(ld=100), -1, "u_stride"),
                             (dict(qs=None), -1, "together"), (dict(st=None), -1, "NULL"), (dict(mq=-1), -1, "max_q_len")):
        rc, msg = _status("pa_lightning_chunked", *chunked(**kw))
        assert rc == status and text in msg, (kw, msg)
    rc, msg = _status("pa_lightning_recurrent", FAKE, 200, 1, FAKE, 2, FAKE, FAKE, None, None, FAKE, 2, FAKE, 2, 16, 24, f32, None)
    assert rc == -1 and "below batch" in msg
    assert lib.pa_lightning_workspace_bytes(-1, 2, 16, 24, 8) == 0 and "pa_lightning_workspace_bytes" in _lib.last_error()


def test_recurrence_and_expert_entry_points_check_their_arguments():
    f32, bf16 = _lib.PA_F32, _lib.PA_BF16
    conv = lambda **kw: [{**dict(u=FAKE, ld=64, n=4, w=FAKE, b=None, taps=3, act=_lib.PA_ACT_SILU, cs=FAKE, sr=2, cl=FAKE, ql=None,
                                 qs=None, ss=FAKE, tiles=None, nt=4, batch=4, out=FAKE, ch=48, dt=bf16, s=None), **kw}[k]
                         for k in ("u", "ld", "n", "w", "b", "taps", "act", "cs", "sr", "cl", "ql", "qs", "ss", "tiles", "nt", "batch",
                                   "out", "ch", "dt", "s")]
    for kw, status, text in ((dict(ld=40), -1, "u_stride"), (dict(taps=9), -2, "taps"), (dict(act=1), -1, "act"), (dict(cs=None), -1, "carried"),
                             (dict(nt=3), -1, "one row"), (dict(tiles=FAKE), -1, "tiles"), (dict(dt=_lib.PA_F16), -2, "dtype")):
        rc, msg = _status("pa_short_conv", *conv(**kw))
        assert rc == status and text in msg, (kw, msg)

    lib = _lib.load()
    assert lib.pa_gated_linear_state_floats(_lib.PA_GL_SSD, 20, 130) == 32 * 144
    assert lib.pa_gated_linear_state_floats(_lib.PA_GL_MLSTM, 20, 130) == 32 * 144 + 3 * (32 + 16)
    assert lib.pa_gated_linear_state_floats(5, 20, 130) == 0
    names = ("kind", "q", "lq", "k", "lk", "v", "lv", "hpg", "ga", "gb", "lg", "ha", "hb", "hc", "cap", "qsc", "eps", "n", "st", "sr", "cl",
             "ql", "qs", "ss", "batch", "mq", "out", "h", "dim", "vdim", "dt", "ws", "wb", "s")
    gated = lambda **kw: [{**dict(kind=_lib.PA_GL_MLSTM, q=FAKE, lq=64, k=FAKE, lk=64, v=FAKE, lv=96, hpg=1, ga=FAKE, gb=FAKE, lg=4, ha=FAKE,
                                  hb=FAKE, hc=None, cap=2.0, qsc=1.0, eps=1e-6, n=4, st=FAKE, sr=2, cl=FAKE, ql=FAKE, qs=FAKE, ss=FAKE, batch=2,
                                  mq=2, out=FAKE, h=4, dim=16, vdim=24, dt=bf16, ws=None, wb=0, s=None), **kw}[k] for k in names]
    for kw, status, text in ((dict(kind=3), -1, "kind"), (dict(hpg=3), -1, "heads_per_group"), (dict(dim=264, lq=2000, lk=2000), -2, "above 256"),
                             (dict(lv=90), -1, "stride"), (dict(lg=3), -1, "stride"), (dict(cap=0.0), -1, "cap"), (dict(gb=None), -1, "NULL"),
                             (dict(kind=_lib.PA_GL_SSD), -1, "NULL"), (dict(ql=None), -1, "together"),
                             (dict(ql=None, qs=None, batch=5), -1, "below batch"), (dict(dt=_lib.PA_F16), -2, "dtype")):
        rc, msg = _status("pa_gated_linear", *gated(**kw))
        assert rc == status and text in msg, (kw, msg)
    assert lib.pa_gated_linear_workspace_bytes(2, 0, 16, 24, 8) == 0 and "workspace_bytes" in _lib.last_error()

    rc, msg = _status("pa_narrow_linear", FAKE, 30, FAKE, FAKE, 4, 8, 32, f32, None)
    assert rc == -1 and "x_stride" in msg
    names = ("logits", "ld", "rows", "e", "ident", "top", "groups", "keep", "shared", "scores", "gtop", "renorm", "corr", "ids", "w", "c", "l", "ws",
             "wb", "s")
    choose = lambda **kw: [{**dict(logits=FAKE, ld=4096, rows=4, e=8, ident=0, top=2, groups=1, keep=1, shared=0, scores=0, gtop=2, renorm=1,
                                   corr=None, ids=FAKE, w=FAKE, c=FAKE, l=FAKE, ws=FAKE, wb=1 << 20, s=None), **kw}[k] for k in names]
    for kw, status, text in ((dict(e=9, groups=2), -1, "equal groups"), (dict(e=8, ident=1, groups=2), -1, "equal groups"),
                             (dict(top=5, groups=2), -1, "cannot be chosen"), (dict(groups=2, keep=3), -1, "cannot be chosen"),
                             (dict(e=2048), -2, "above"), (dict(e=1024, ident=2), -2, "above"), (dict(scores=2), -1, "scores"),
                             (dict(gtop=3), -1, "group_top"), (dict(shared=3), -1, "shared"), (dict(ld=8, shared=1), -1, "logits_stride"),
                             (dict(ld=9, ident=2), -1, "logits_stride"), (dict(c=None), -1, "NULL"), (dict(wb=8), -3, "needed")):
        rc, msg = _status("pa_moe_choose", *choose(**kw))
        assert rc == status and text in msg, (kw, msg)
    assert lib.pa_moe_workspace_bytes(16384, 64, 8) == 256 * 64 * 4
    product = lambda **kw: [{**dict(x=FAKE, lx=64, ipr=2, w=FAKE, wr=96, lw=64, k=64, c=FAKE, l=FAKE, rows=4, top=2, e=8, glu=1, out=FAKE, n=48,
                                    dt=bf16, s=None), **kw}[k] for k in ("x", "lx", "ipr", "w", "wr", "lw", "k", "c", "l", "rows", "top", "e",
                                                                         "glu", "out", "n", "dt", "s")]
    for kw, status, text in ((dict(wr=90), -1, "w_rows"), (dict(lx=60), -1, "stride"), (dict(c=None), -1, "NULL"), (dict(dt=_lib.PA_F16), -2, "dtype"),
                             (dict(ipr=0), -1, "out of range")):
        rc, msg = _status("pa_moe_product", *product(**kw))
        assert rc == status and text in msg, (kw, msg)


def test_argument_checks_of_the_latent_scored_delta_and_stream_kernels():
    lib = _lib.load()
    def cases(name, names, good, bad):
        for kw, status, text in bad:
            rc, msg = _status(name, *[{**good, **kw}[k] for k in names])
            assert rc == status and text in msg, (name, kw, msg)

    bf16 = _lib.PA_BF16
    cases("pa_hyper_norm", ("x", "y", "mw", "mix", "ml", "ye", "ys", "bt", "into", "ids", "tab", "tr", "sw", "nw", "eps", "out", "sum", "rows",
                            "n", "width", "dt", "s"),
          dict(x=FAKE, y=FAKE, mw=None, mix=0, ml=0, ye=None, ys=None, bt=FAKE, into=FAKE, ids=None, tab=None, tr=0, sw=None, nw=FAKE, eps=1e-5,
               out=FAKE, sum=None, rows=2, n=3, width=64, dt=bf16, s=None),
          [(dict(n=17), -2, "streams"), (dict(width=20000), -2, "width"), (dict(n=0), -1, "out of range"), (dict(x=None), -1, "NULL"),
           (dict(bt=None), -1, "without its weights"), (dict(ids=FAKE), -1, "ids"), (dict(mw=FAKE, mix=2, ml=2, ye=FAKE), -1, "does not fit"),
           (dict(ye=FAKE), -1, "without mix_weight"), (dict(nw=None), -1, "norm_weight"), (dict(y=None, out=None), -1, "nothing"),
           (dict(dt=_lib.PA_F16), -2, "dtype")])
    cases("pa_latent_append", ("u", "lu", "n", "nw", "eps", "rope", "rr", "cl", "ql", "qs", "t", "nt", "batch", "slots", "ts", "q", "pool", "h",
                               "dim", "rot", "rank", "qd", "row", "sc", "dt", "s"),
          dict(u=FAKE, lu=200, n=2, nw=FAKE, eps=1e-5, rope=FAKE, rr=8, cl=FAKE, ql=None, qs=None, t=None, nt=2, batch=2, slots=FAKE, ts=32,
               q=FAKE, pool=FAKE, h=4, dim=24, rot=8, rank=40, qd=32, row=48, sc=1.0, dt=bf16, s=None),
          [(dict(rot=7), -1, "out of range"), (dict(qd=24), -1, "multiples of 8"), (dict(row=50), -1, "multiples of 8"), (dict(lu=100), -1, "u_stride"),
           (dict(nt=3), -1, "one row"), (dict(t=FAKE), -1, "tiles"), (dict(rope=None), -1, "table"), (dict(dt=_lib.PA_F16), -2, "dtype"),
           (dict(pool=None), -1, "NULL")])
    cases("pa_scored_attention", ("q1", "r1", "h1", "n1", "q2", "r2", "h2", "n2", "k", "kd", "v", "vd", "vdim", "bt", "bs_", "bs", "nb", "cl", "ql",
                                  "qs", "n", "batch", "mq", "hq", "hkv", "sc", "win", "cap", "bias", "bn", "sink", "out", "dt", "ws", "wb", "s"),
          dict(q1=FAKE, r1=128, h1=32, n1=32, q2=None, r2=0, h2=0, n2=0, k=FAKE, kd=32, v=FAKE, vd=32, vdim=24, bt=FAKE, bs_=4, bs=16, nb=8,
               cl=FAKE, ql=None, qs=None, n=2, batch=2, mq=1, hq=4, hkv=2, sc=1.0, win=0, cap=0.0, bias=None, bn=0, sink=None, out=FAKE, dt=bf16,
               ws=None, wb=0, s=None),
          [(dict(n1=40), -1, "fit the pool"), (dict(vdim=40), -1, "fit the pool"), (dict(hq=3), -1, "multiple"), (dict(win=-1), -1, "window"),
           (dict(bias=FAKE), -1, "bias_n"), (dict(ql=FAKE), -1, "together"), (dict(n2=8, kd=48), -1, "NULL"), (dict(batch=3), -1, "below batch"),
           (dict(vdim=1032, vd=1032), -2, "above 1024"), (dict(dt=_lib.PA_F16), -2, "dtype")])
    cases("pa_delta", ("q", "lq", "k", "lk", "v", "lv", "hpg", "ga", "gb", "lg", "bias", "rate", "sc", "n", "st", "sr", "cl", "ql", "qs", "ss", "batch",
                       "mq", "out", "h", "dim", "vdim", "dt", "ws", "wb", "s"),
          dict(q=FAKE, lq=64, k=FAKE, lk=64, v=FAKE, lv=96, hpg=1, ga=FAKE, gb=FAKE, lg=4, bias=FAKE, rate=FAKE, sc=0.25, n=4, st=FAKE, sr=2,
               cl=FAKE, ql=FAKE, qs=FAKE, ss=FAKE, batch=2, mq=2, out=FAKE, h=4, dim=16, vdim=24, dt=bf16, ws=None, wb=0, s=None),
          [(dict(hpg=3), -1, "heads_per_group"), (dict(dim=264, lq=2000, lk=2000), -2, "above 256"), (dict(lv=90), -1, "stride"),
           (dict(lg=3), -1, "stride"), (dict(gb=None), -1, "NULL"), (dict(ql=None), -1, "together"), (dict(ql=None, qs=None, batch=5), -1, "below batch"),
           (dict(dt=_lib.PA_F16), -2, "dtype")])
    assert lib.pa_scored_workspace_bytes(0, 4, 2, 32, 32, 0, 100, 0) == 0
    assert lib.pa_delta_workspace_bytes(2, 3, 64, 64, 65) == 2 * 3 * 2 * (4 * 64 * 64 * 2 + 1024)


def test_entry_points_of_mixed_heads_and_channel_gates_check_their_arguments():
    f32, bf16 = _lib.PA_F32, _lib.PA_BF16
    rc, msg = _status("pa_bias_act", FAKE, 60, None, FAKE, 4, 64, _lib.PA_ACT_RELU2, f32, None)
    assert rc == -1 and "x_stride" in msg
    rc, msg = _status("pa_bias_act", FAKE, 64, None, FAKE, 4, 64, 4, f32, None)
    assert rc == -1 and "act" in msg
    assert _status("pa_bias_act", None, 64, None, None, 0, 64, _lib.PA_ACT_NONE, bf16, None)[0] == 0
    rc, msg = _status("pa_glu", FAKE, 64, FAKE, 64, None, 0, FAKE, 4, 64, _lib.PA_ACT_RELU2, f32, None)
    assert rc == -1 and "act" in msg
    rc, msg = _status("pa_rms_gate", FAKE, None, 0, FAKE, 1e-6, FAKE, 64, 4, 64, 1, 0, f32, None)
    assert rc == -1 and "NULL" in msg

    lib = _lib.load()
    names = ("q", "qr", "qh", "dim", "k", "kd", "v", "vd", "vdim", "bt", "bts", "bs", "nb", "cl", "ql", "qs", "n", "batch", "mq", "h", "hkv", "scale", "size",
             "rate", "talk", "out", "dt", "ws", "wb", "s")
    talk = lambda **kw: [{**dict(q=FAKE, qr=128, qh=32, dim=32, k=FAKE, kd=32, v=FAKE, vd=32, vdim=24, bt=FAKE, bts=4, bs=16, nb=8, cl=FAKE, ql=FAKE,
                                 qs=FAKE, n=4, batch=2, mq=2, h=4, hkv=2, scale=0.1, size=FAKE, rate=FAKE, talk=FAKE, out=FAKE, dt=bf16, ws=FAKE,
                                 wb=1 << 20, s=None), **kw}[k] for k in names]
    for kw, status, text in ((dict(hkv=3), -1, "multiple"), (dict(dim=33), -1, "fit the pool"), (dict(vdim=33), -1, "fit the pool"), (dict(ql=None), -1, "together"),
                             (dict(rate=None), -1, "together"), (dict(bs=0), -1, "block_size"), (dict(dt=_lib.PA_F16), -2, "dtype"),
                             (dict(dim=264, kd=264), -2, "above 256"), (dict(h=130, hkv=1), -2, "above 128"), (dict(talk=None), -1, "NULL"),
                             (dict(ws=None), -3, "workspace"), (dict(wb=16), -3, "workspace"), (dict(ql=None, qs=None, batch=5), -1, "below batch")):
        rc, msg = _status("pa_talking_attention", *talk(**kw))
        assert rc == status and text in msg, (kw, msg)
    assert _status("pa_talking_attention", *talk(n=0, q=None))[0] == 0
    assert lib.pa_talking_workspace_bytes(5, 2, 4, 2, 24, 1000, 0) == 256 and lib.pa_talking_workspace_bytes(5, 2, 0, 2, 24, 1000, 0) == 0

    names = ("q", "lq", "act", "f", "lf", "fb", "lo", "v", "lv", "n", "st", "sr", "cl", "ql", "qs", "ss", "batch", "mq", "out", "h", "dim", "vdim", "dt", "ws",
             "wb", "s")
    chan = lambda **kw: [{**dict(q=FAKE, lq=64, act=_lib.PA_ACT_SILU, f=FAKE, lf=64, fb=None, lo=FAKE, v=FAKE, lv=96, n=4, st=FAKE, sr=2, cl=FAKE, ql=FAKE,
                                 qs=FAKE, ss=FAKE, batch=2, mq=2, out=FAKE, h=4, dim=16, vdim=24, dt=bf16, ws=None, wb=0, s=None), **kw}[k] for k in names]
    for kw, status, text in ((dict(act=_lib.PA_ACT_GELU_TANH), -1, "q_act"), (dict(lq=63), -1, "stride"), (dict(lf=63), -1, "stride"), (dict(lv=95), -1, "stride"),
                             (dict(dim=264, lq=2000, lf=2000), -2, "above 256"), (dict(lo=None), -1, "NULL"), (dict(qs=None), -1, "together"),
                             (dict(ql=None, qs=None, batch=5), -1, "below batch"), (dict(dt=_lib.PA_F16), -2, "dtype"), (dict(vdim=0), -1, "positive")):
        rc, msg = _status("pa_channel_linear", *chan(**kw))
        assert rc == status and text in msg, (kw, msg)
    assert _status("pa_channel_linear", *chan(n=0, q=None))[0] == 0
    assert lib.pa_channel_linear_workspace_bytes(2, 0, 16, 24, 8) == 0 and "workspace_bytes" in _lib.last_error()
