"""Tensor-level wrappers of the C ABI (one function per ``pa_*`` entry point).

Each wrapper takes torch tensors that already live on the HIP device, passes
their raw pointers, sizes and the current stream to ``libpaged_attn.so`` and
raises ``PagedAttnError`` on a negative status.  No computation happens in
Python and nothing is routed to torch kernels.
"""

from __future__ import annotations

from typing import NamedTuple, Optional, Tuple

import torch
from torch import Tensor

from . import _lib

PA_DTYPE = {torch.float32: _lib.PA_F32, torch.bfloat16: _lib.PA_BF16, torch.float16: _lib.PA_F16,
            torch.float8_e4m3fn: _lib.PA_FP8_E4M3, torch.uint8: _lib.PA_FP8_E4M3}

QKV_TILE_ROWS = _lib.PA_QKV_TILE_ROWS


def _ptr(t: Optional[Tensor]) -> Optional[int]:
    return None if t is None else t.data_ptr()


def _stream(t: Tensor) -> Optional[int]:
    if t.device.type != "cuda":
        raise RuntimeError(f"libpaged_attn computes only on a HIP device; got a tensor on {t.device}")
    return torch.cuda.current_stream(t.device).cuda_stream or None


def _run(name: str, *args) -> None:
    _lib.check(name, getattr(_lib.load(), name)(*args))


def kv_scatter(k_cache: Tensor, v_cache: Tensor, k_src: Tensor, v_src: Tensor, slots: Tensor) -> None:
    """``cache[slots[i]] = src[i]``; caches ``[total_slots, Hkv, D]``, src ``[N, Hkv, D]``, slots int64 ``[N]``."""
    total_slots, hkv, d = k_cache.shape
    _run("pa_kv_scatter", _ptr(k_cache), _ptr(v_cache), _ptr(k_src), _ptr(v_src), _ptr(slots), slots.numel(),
         total_slots, hkv, d, k_cache.element_size(), _stream(k_cache))


def kv_gather(k_cache: Tensor, v_cache: Tensor, block_tables: Tensor, seq_lens: Tensor, max_len: int,
              block_size: int, out: Optional[Tuple[Tensor, Tensor]] = None) -> Tuple[Tensor, Tensor]:
    """Zero-padded ``[B, max_len, Hkv, D]`` copies; block_tables int32 ``[B, W]`` (-1 padded), seq_lens int32.
    ``out``: a pair of contiguous tensors of that shape and the pool's type to write into."""
    total_slots, hkv, d = k_cache.shape
    batch = block_tables.shape[0]
    if out is None:
        k_out = torch.empty((batch, max_len, hkv, d), dtype=k_cache.dtype, device=k_cache.device)
        v_out = torch.empty_like(k_out)
    else:
        k_out, v_out = out
        for t in (k_out, v_out):
            if tuple(t.shape) != (batch, max_len, hkv, d) or t.dtype != k_cache.dtype or not t.is_contiguous():
                raise ValueError("kv_gather: out tensors must be contiguous [B, max_len, Hkv, D] of the pool's type")
    _run("pa_kv_gather", _ptr(k_cache), _ptr(v_cache), _ptr(k_out), _ptr(v_out), _ptr(block_tables),
         block_tables.shape[1], _ptr(seq_lens), batch, max_len, total_slots // block_size, block_size, hkv, d,
         k_cache.element_size(), _stream(k_cache))
    return k_out, v_out


def decode_workspace_bytes(batch: int, num_q_heads: int, num_kv_heads: int, head_dim: int,
                           kv_dtype: torch.dtype) -> int:
    """Bytes of workspace ``decode`` needs for these shapes (independent of the sequence lengths)."""
    n = int(_lib.load().pa_decode_workspace_bytes(batch, num_q_heads, num_kv_heads, head_dim, PA_DTYPE[kv_dtype]))
    if n == 0:
        raise _lib.PagedAttnError("pa_decode_workspace_bytes", 0, _lib.last_error())
    return n


def decode_workspace(q: Tensor, k_cache: Tensor) -> Tensor:
    """A fresh workspace tensor sized for ``decode(q, k_cache, ...)``, zero-filled: the library's arrival
    counters at its start must read zero before the first call that uses them."""
    batch, hq, d = q.shape
    n = decode_workspace_bytes(batch, hq, k_cache.shape[1], d, k_cache.dtype)
    return torch.zeros(n, dtype=torch.uint8, device=q.device)


def decode(q: Tensor, k_cache: Tensor, v_cache: Tensor, block_tables: Tensor, seq_lens: Tensor, block_size: int,
           scale: float, workspace: Tensor, extra_zero_keys: Optional[Tensor] = None,
           k_scale: Optional[Tensor] = None, v_scale: Optional[Tensor] = None, out: Optional[Tensor] = None,
           entry: str = "pa_decode", window: int = 0) -> Tensor:
    """Paged decode attention; q ``[B, Hq, D]`` -> out ``[B, Hq, D]`` (same dtype).

    ``entry`` may name ``pa_decode_split`` or ``pa_decode_reduce`` to run one pass only; ``window`` > 0
    restricts every sequence to its last ``window`` keys, < 0 to its last chunk of ``-window`` positions.
    """
    batch, hq, d = q.shape
    total_slots, hkv, _ = k_cache.shape
    if out is None:
        out = torch.empty_like(q)
    _run(entry, _ptr(q), _ptr(k_cache), _ptr(v_cache), _ptr(out), _ptr(block_tables), block_tables.shape[1],
         _ptr(seq_lens), _ptr(extra_zero_keys), _ptr(k_scale), _ptr(v_scale), batch, hq, hkv, d, block_size,
         total_slots // block_size, float(scale), int(window), PA_DTYPE[q.dtype], PA_DTYPE[k_cache.dtype],
         _ptr(workspace),
         workspace.numel() * workspace.element_size(), _stream(q))
    return out


def decode_static(q: Tensor, k_cache: Tensor, v_cache: Tensor, block_tables: Tensor, seq_lens: Tensor,
                  block_size: int, scale: float, extra_zero_keys: Optional[Tensor] = None,
                  k_scale: Optional[Tensor] = None, v_scale: Optional[Tensor] = None, out: Optional[Tensor] = None,
                  window: int = 0) -> Tensor:
    """``decode`` through ``pa_decode_static``: the partials go to the library's own fixed scratch array, the
    call allocates nothing (pass ``out``); shapes beyond the scratch raise ``PagedAttnError``."""
    batch, hq, d = q.shape
    total_slots, hkv, _ = k_cache.shape
    if out is None:
        out = torch.empty_like(q)
    _run("pa_decode_static", _ptr(q), _ptr(k_cache), _ptr(v_cache), _ptr(out), _ptr(block_tables),
         block_tables.shape[1], _ptr(seq_lens), _ptr(extra_zero_keys), _ptr(k_scale), _ptr(v_scale), batch, hq, hkv,
         d, block_size, total_slots // block_size, float(scale), int(window), PA_DTYPE[q.dtype],
         PA_DTYPE[k_cache.dtype], _stream(q))
    return out


def prefill_workspace_bytes(q: Tensor, block_tables: Tensor, max_q_len: int, block_size: int, num_kv_heads: int,
                            window: int = 0) -> int:
    """Bytes of workspace with which ``prefill_paged`` spreads a launch of few rows over the device (0: the launch
    fills it anyway, or its shapes have no split kernel)."""
    total_q, hq, d = q.shape
    if q.dtype not in PA_DTYPE:
        return 0
    return int(_lib.load().pa_prefill_workspace_bytes(block_tables.shape[0], int(max_q_len), total_q,
                                                      block_tables.shape[1], block_size, int(window), hq,
                                                      num_kv_heads, d, PA_DTYPE[q.dtype]))


def prefill_paged(q: Tensor, k_cache: Tensor, v_cache: Tensor, block_tables: Tensor, ctx_lens: Tensor,
                  q_lens: Tensor, q_starts: Tensor, max_q_len: int, block_size: int, scale: float,
                  out: Optional[Tensor] = None, window: int = 0, row_first_key: Optional[Tensor] = None,
                  rowwise: bool = False, workspace: Optional[Tensor] = None) -> Tensor:
    """Causal prefill over a paged context; q ``[total_q, Hq, D]`` packed rows; ``window`` > 0 adds the
    sliding window (a row at position p sees keys p - window < j <= p), < 0 chunks of ``-window`` positions (it sees
    keys of its own chunk); ``row_first_key`` (int32 per q row,
    non-decreasing along a sequence) adds a per-row first key, e.g. the start of the row's document;
    ``rowwise`` selects the vector kernel (``pa_prefill_paged_rowwise``) also where a matrix-core kernel exists;
    ``workspace`` (uint8, ``prefill_workspace_bytes`` or more) lets a launch of few rows split its keys over
    several workgroups (``pa_prefill_paged_ws``)."""
    total_q, hq, d = q.shape
    if row_first_key is not None and (row_first_key.dtype != torch.int32 or row_first_key.numel() != total_q):
        raise ValueError("row_first_key must hold one int32 per q row")
    total_slots, hkv, _ = k_cache.shape
    if out is None:
        out = torch.empty_like(q)
    args = (_ptr(q), _ptr(k_cache), _ptr(v_cache), _ptr(out), _ptr(block_tables), block_tables.shape[1],
            _ptr(ctx_lens), _ptr(q_lens), _ptr(q_starts), _ptr(row_first_key) if row_first_key is not None else None,
            block_tables.shape[0], max_q_len, hq, hkv, d, block_size, total_slots // block_size, float(scale),
            int(window), PA_DTYPE[q.dtype], _stream(q))
    if workspace is not None and not rowwise:
        # (``pa_prefill_paged_ws``: the launch is cut into pieces over the keys when it has too few rows for the device)
        _run("pa_prefill_paged_ws", *args, total_q, _ptr(workspace), workspace.numel() * workspace.element_size())
    else:
        _run("pa_prefill_paged_rowwise" if rowwise else "pa_prefill_paged", *args)
    return out


def pack_mask(keep: Tensor) -> Tensor:
    """Bits of a boolean mask ``[rows, heads (or 1), keys]`` as int32 words ``[rows, heads, ceil(keys / 32)]``
    (bit j of word j // 32 = keep[..., j]), the layout ``attend_masked`` takes.  Packed with byte arithmetic, a
    bounded number of rows at a time: the temporaries stay near the size of the boolean input."""
    rows, heads, keys = keep.shape
    words = max(1, -(-keys // 32))
    out = torch.empty((rows, heads, words), dtype=torch.int32, device=keep.device)
    per_row = max(1, heads * words * 32)
    chunk = max(1, (1 << 27) // per_row)  # about 128 MiB of bytes per round
    for at in range(0, rows, chunk):
        part = keep[at: at + chunk]
        n = part.shape[0]
        if keys == words * 32:
            bits = part.contiguous().view(torch.uint8) if part.dtype == torch.bool else part.to(torch.uint8)
        else:
            bits = torch.zeros((n, heads, words * 32), dtype=torch.uint8, device=keep.device)
            bits[..., :keys] = part
        bits = bits.reshape(n, heads, words * 4, 8)
        byte = bits[..., 0].clone()
        for k in range(1, 8):
            byte |= bits[..., k] << k
        out[at: at + n] = byte.contiguous().view(torch.int32).view(n, heads, words)  # little-endian: byte 0 = bits 0..7
    return out


def attend_masked(q: Tensor, k_cache: Tensor, v_cache: Tensor, block_tables: Tensor, ctx_lens: Tensor, q_lens: Tensor,
                  q_starts: Tensor, max_q_len: int, block_size: int, scale: float, mask_words: Tensor, n_keys: int,
                  out: Optional[Tensor] = None, k_scale: Optional[Tensor] = None,
                  v_scale: Optional[Tensor] = None) -> Tensor:
    """Attention of packed q rows ``[total_q, Hq, D]`` over a paged context under an arbitrary mask
    (``pa_attend_masked``): ``mask_words`` int32 ``[total_q, 1 or Hq, words]`` from ``pack_mask``; row r attends
    key j < n_keys iff its bit is set; keys at or past ``ctx_lens[b]`` are zero rows.  An fp8-e4m3 pool comes with
    its ``k_scale`` / ``v_scale``."""
    total_q, hq, d = q.shape
    total_slots, hkv, _ = k_cache.shape
    if mask_words.dtype != torch.int32 or mask_words.dim() != 3 or mask_words.shape[0] != total_q:
        raise ValueError("mask_words must be int32 [total_q, heads, words]")
    if out is None:
        out = torch.empty_like(q)
    _run("pa_attend_masked", _ptr(q), _ptr(k_cache), _ptr(v_cache), _ptr(out), _ptr(block_tables),
         block_tables.shape[1], _ptr(ctx_lens), _ptr(q_lens), _ptr(q_starts), _ptr(mask_words), mask_words.shape[1],
         mask_words.shape[2], int(n_keys), block_tables.shape[0], max_q_len, hq, hkv, d, block_size,
         total_slots // block_size, float(scale), PA_DTYPE[q.dtype], PA_DTYPE[k_cache.dtype], _ptr(k_scale),
         _ptr(v_scale), _stream(q))
    return out


def quantize_kv_e4m3(pool: Tensor, block_size: int) -> Tuple[Tensor, Tensor]:
    """e4m3fn bytes (as ``torch.float8_e4m3fn``) and ``float32 [num_blocks, Hkv]`` scales of a pool."""
    total_slots, hkv, d = pool.shape
    num_blocks = total_slots // block_size
    dst = torch.empty(pool.shape, dtype=torch.float8_e4m3fn, device=pool.device)
    scale = torch.empty((num_blocks, hkv), dtype=torch.float32, device=pool.device)
    _run("pa_quantize_kv_e4m3", _ptr(pool), _ptr(dst), _ptr(scale), num_blocks, block_size, hkv, d,
         PA_DTYPE[pool.dtype], _stream(pool))
    return dst, scale


class TouchedBlocks(NamedTuple):
    """The distinct blocks a slot list writes to and the index of its rows by block that ``pa_kv_append_e4m3``
    takes: rows ``row_order[block_start[i]:block_start[i + 1]]`` are the tokens whose slots fall in ``blocks[i]``."""

    blocks: Tensor       # int32 [n_touched]
    row_order: Tensor    # int32 [n_rows], token indices grouped by block
    block_start: Tensor  # int32 [n_touched + 1]


def touched_blocks(slots: Tensor, block_size: int, num_blocks: int) -> TouchedBlocks:
    """Distinct blocks (int32, on the device) that the non-negative, in-pool slots fall in, with the rows of
    each: an append workgroup then reads the slots of its own block instead of the whole list."""
    blocks = torch.div(slots, block_size, rounding_mode="floor")
    rows = torch.nonzero((slots >= 0) & (blocks < num_blocks)).reshape(-1)
    uniq, inverse, counts = torch.unique(blocks[rows], return_inverse=True, return_counts=True)
    order = rows[torch.argsort(inverse, stable=True)]
    start = torch.zeros(uniq.numel() + 1, dtype=torch.int32, device=slots.device)
    start[1:] = torch.cumsum(counts, 0)
    return TouchedBlocks(uniq.to(torch.int32), order.to(torch.int32).contiguous(), start)


def _touched_args(touched, slots: Tensor, block_size: int, num_blocks: int):
    """(blocks, row_order, block_start) for the append calls: ``touched`` is a TouchedBlocks, a bare int32 tensor
    of blocks (no index: every workgroup scans the slot list) or None (computed here)."""
    if touched is None:
        touched = touched_blocks(slots, block_size, num_blocks)
    if isinstance(touched, TouchedBlocks):
        return touched.blocks, touched.row_order, touched.block_start
    return touched, None, None


def kv_append_e4m3(k_cache: Tensor, v_cache: Tensor, k_scale: Tensor, v_scale: Tensor, k_src: Tensor, v_src: Tensor,
                   slots: Tensor, block_size: int, touched=None) -> None:
    """Append rows to an fp8-e4m3 pool with the "re-round on growth" policy of ``pa_kv_append_e4m3``.

    k_cache/v_cache ``[total_slots, Hkv, D]`` float8_e4m3fn, scales ``float32 [num_blocks, Hkv]`` (updated in
    place), k_src/v_src ``[N, Hkv, D]`` fp32/bf16/fp16, slots ``int64 [N]``.  ``touched`` (a ``TouchedBlocks``
    from ``touched_blocks``, or a bare int32 tensor of the distinct target blocks without the row index) is
    computed with torch when not given.
    """
    total_slots, hkv, d = k_cache.shape
    num_blocks = total_slots // block_size
    blocks, order, start = _touched_args(touched, slots, block_size, num_blocks)
    _run("pa_kv_append_e4m3", _ptr(k_cache), _ptr(v_cache), _ptr(k_scale), _ptr(v_scale), _ptr(k_src), _ptr(v_src),
         _ptr(slots), slots.numel(), _ptr(blocks), blocks.numel(), _ptr(order), _ptr(start), num_blocks, block_size,
         hkv, d, PA_DTYPE[k_src.dtype], _stream(k_cache))


def rope_kv_append(q: Tensor, k_src: Tensor, v_src: Tensor, cos: Tensor, sin: Tensor, k_cache: Optional[Tensor],
                   v_cache: Optional[Tensor], slots: Optional[Tensor], positions: Optional[Tensor] = None,
                   q_out: Optional[Tensor] = None, k_out: Optional[Tensor] = None) -> Tensor:
    """Rotary embedding of q and k fused with the KV append (``pa_rope_kv_append``).

    q ``[N, Hq, D]``, k_src/v_src ``[N, Hkv, D]``, cos/sin ``[R, D]`` of the same dtype; ``positions`` int32 ``[N]``
    picks the table row per token (None: row i for token i).  The rotated k and v go to the caches at ``slots``
    (int64 ``[N]``; None: no cache write) and the rotated k also to ``k_out`` when given.  Returns rotated q
    (``q_out``, or q itself rotated in place when ``q_out`` is None).
    """
    n, hq, d = q.shape
    hkv = k_src.shape[1]
    if q_out is None:
        q_out = q
    for t in (k_src, v_src, cos, sin):
        if t.dtype != q.dtype:
            raise RuntimeError("q, k, v, cos and sin must have the same dtype")
    if positions is not None and positions.dtype != torch.int32:
        raise ValueError("positions must be int32")
    if cos.shape != sin.shape or cos.dim() != 2 or cos.shape[1] != d:
        raise ValueError("cos / sin must be [rows, head_dim]")
    total_slots = k_cache.shape[0] if k_cache is not None else 0
    _run("pa_rope_kv_append", _ptr(q), _ptr(q_out), _ptr(k_src), _ptr(v_src), _ptr(k_out), _ptr(k_cache),
         _ptr(v_cache), _ptr(cos), _ptr(sin), _ptr(positions), cos.shape[0], _ptr(slots), n, total_slots, hq, hkv, d,
         PA_DTYPE[q.dtype], _stream(q))
    return q_out


def rope_kv_append_e4m3(q: Tensor, k_src: Tensor, v_src: Tensor, cos: Tensor, sin: Tensor, k_cache: Tensor,
                        v_cache: Tensor, k_scale: Tensor, v_scale: Tensor, slots: Tensor, block_size: int,
                        positions: Optional[Tensor] = None, q_out: Optional[Tensor] = None,
                        touched=None) -> Tensor:
    """``rope_kv_append`` into an fp8-e4m3 pool (``pa_rope_kv_append_e4m3``): k is rotated while the fp8 append
    reads it; arguments as in ``rope_kv_append`` and ``kv_append_e4m3``."""
    n, hq, d = q.shape
    total_slots, hkv, _ = k_cache.shape
    num_blocks = total_slots // block_size
    if q_out is None:
        q_out = q
    for t in (k_src, v_src, cos, sin):
        if t.dtype != q.dtype:
            raise RuntimeError("q, k, v, cos and sin must have the same dtype")
    if positions is not None and positions.dtype != torch.int32:
        raise ValueError("positions must be int32")
    blocks, order, start = _touched_args(touched, slots, block_size, num_blocks)
    _run("pa_rope_kv_append_e4m3", _ptr(q), _ptr(q_out), _ptr(k_src), _ptr(v_src), _ptr(k_cache), _ptr(v_cache),
         _ptr(k_scale), _ptr(v_scale), _ptr(cos), _ptr(sin), _ptr(positions), cos.shape[0], _ptr(slots), n,
         _ptr(blocks), blocks.numel(), _ptr(order), _ptr(start), num_blocks, block_size, hq, hkv, d,
         PA_DTYPE[q.dtype], _stream(q))
    return q_out


def dequantize_blocks_e4m3(cache: Tensor, scale: Tensor, block_ids: Tensor, block_size: int,
                           dtype: torch.dtype = torch.bfloat16) -> Tensor:
    """Compact 16-bit pool ``[len(block_ids) * block_size, Hkv, D]`` holding the listed blocks of an fp8-e4m3
    pool dequantised (``pa_dequantize_blocks_e4m3``); ``block_ids`` int32 on the device."""
    total_slots, hkv, d = cache.shape
    if block_ids.dtype != torch.int32:
        raise ValueError("block_ids must be int32")
    dst = torch.empty((block_ids.numel() * block_size, hkv, d), dtype=dtype, device=cache.device)
    _run("pa_dequantize_blocks_e4m3", _ptr(cache), _ptr(scale), _ptr(block_ids), block_ids.numel(), _ptr(dst),
         total_slots // block_size, block_size, hkv, d, PA_DTYPE[dtype], _stream(cache))
    return dst


# ------------------------------------------------------------------ decoder blocks around attention


def _row_stride(t: Tensor) -> int:
    """Elements between the rows of a 2-D tensor whose rows are contiguous (a column slice of a wider one)."""
    if t.dim() != 2 or (t.shape[1] > 1 and t.stride(1) != 1):
        raise ValueError("expected a 2-D tensor with contiguous rows")
    return t.stride(0) if t.shape[0] > 1 else max(t.stride(0), t.shape[1])


def _dense(*tensors: Optional[Tensor]) -> None:
    for t in tensors:
        if t is not None and not t.is_contiguous():
            raise ValueError("expected contiguous tensors")


def _typed(dtype: torch.dtype, *tensors: Optional[Tensor]) -> None:
    for t in tensors:
        if t is not None and t.dtype != dtype:
            raise ValueError(f"expected {dtype}, got {t.dtype}")


_NORMS = {None: _lib.PA_NORM_NONE, "layer": _lib.PA_NORM_LAYER, "rms": _lib.PA_NORM_RMS}
_ACTS = {"silu": _lib.PA_ACT_SILU, "gelu_tanh": _lib.PA_ACT_GELU_TANH, None: _lib.PA_ACT_NONE, "relu2": _lib.PA_ACT_RELU2}
_GATES = {"sigmoid_last": _lib.PA_GATE_SIGMOID_LAST, "silu_first": _lib.PA_GATE_SILU_FIRST,
          "silu_last": _lib.PA_GATE_SILU_LAST, None: _lib.PA_GATE_NONE}
_SCORES = {"sigmoid": _lib.PA_MOE_SIGMOID, "softmax": _lib.PA_MOE_SOFTMAX}
_SHARED = {None: _lib.PA_MOE_NO_SHARED, "gated": _lib.PA_MOE_SHARED_GATED, "plain": _lib.PA_MOE_SHARED}
_GATED = {"ssd": _lib.PA_GL_SSD, "mlstm": _lib.PA_GL_MLSTM}
_V_MODES = {None: _lib.PA_V_PLAIN, "first": _lib.PA_V_FIRST, "mix": _lib.PA_V_MIX}


def residual_norm(x: Tensor, dtype: torch.dtype, y: Optional[Tensor] = None, y_weight: Optional[Tensor] = None,
                  y_eps: float = 0.0, ids: Optional[Tensor] = None, table: Optional[Tensor] = None,
                  row_index: Optional[Tensor] = None, norm: Optional[str] = None, weight: Optional[Tensor] = None,
                  bias: Optional[Tensor] = None, eps: float = 0.0, want_out: bool = True, table_scale: float = 1.0,
                  positions: Optional[Tensor] = None, pos_table: Optional[Tensor] = None, mix: Optional[Tensor] = None,
                  y_extra: Optional[Tensor] = None, y_bias: Optional[Tensor] = None,
                  y2: Optional[Tuple[Tensor, Tensor, Tensor]] = None, ids_add: bool = False) -> Optional[Tensor]:
    """Residual sum and norm in one pass over the rows (``pa_residual_norm``): ``x`` float32 ``[rows, width]`` is
    updated in place (``table[ids] * table_scale``, with ``positions`` also their rows of ``pos_table``, or itself,
    plus ``y`` or its RMS norm times ``y_weight``), and ``norm(x) * weight + bias`` (``"layer"``, ``"rms"`` or None: a
    cast) comes back in ``dtype``.  With ``mix`` float32 ``[rows, m + 1]`` the branch is a weighted sum: of ``y``
    ``[rows * m, width]``, m rows each, and of ``y_extra``.  ``y_bias`` is added to ``y``; ``y2`` ``(branch, weight of y's
    own norm, weight of the branch's)``: y is the sum of two normed branches.  ``ids_add``: the table's rows are added to
    ``x``.  ``row_index`` picks rows of ``x`` instead of updating it."""
    rows, width = x.shape
    other, own_part, other_part = y2 if y2 is not None else (None, None, None)
    _dense(x, y, y_weight, ids, table, row_index, weight, bias, positions, pos_table, mix, y_extra, y_bias, other, own_part, other_part)
    _typed(torch.float32, x, y_weight, weight, bias, mix, y_bias, own_part, other_part)
    _typed(torch.int64, ids, row_index, positions)
    _typed(dtype, y, table, pos_table, y_extra, other)
    n = rows if row_index is None else row_index.numel()
    m = mix.shape[1] - 1 if mix is not None else 0
    if (y is not None and tuple(y.shape) != (rows * (m or 1), width)) or (ids is not None and ids.numel() != rows):
        raise ValueError("y / ids do not fit the residual")
    if (mix is not None and mix.shape[0] != rows) or (y_extra is not None and tuple(y_extra.shape) != (rows, width)):
        raise ValueError("mix / y_extra do not fit the residual")
    if positions is not None and positions.numel() != rows:
        raise ValueError("positions do not fit the residual")
    for t in (table, pos_table):
        if t is not None and t.shape[1] != width:
            raise ValueError("table rows are not as wide as the residual")
    if other is not None and tuple(other.shape) != (rows, width):
        raise ValueError("y2 does not fit the residual")
    for w in (y_weight, weight, bias, y_bias, own_part, other_part):
        if w is not None and w.numel() != width:
            raise ValueError("norm weights are not as wide as the residual")
    out = torch.empty((n, width), dtype=dtype, device=x.device) if want_out else None
    _run("pa_residual_norm", _ptr(x), _ptr(y), _ptr(mix), m, _ptr(y_extra), _ptr(y_bias), _ptr(other), _ptr(own_part),
         _ptr(other_part), _ptr(y_weight), float(y_eps), _ptr(ids), int(ids_add), _ptr(table),
         table.shape[0] if table is not None else 0, float(table_scale), _ptr(positions), _ptr(pos_table),
         pos_table.shape[0] if pos_table is not None else 0, _ptr(row_index), rows, _ptr(weight), _ptr(bias), float(eps),
         _NORMS[norm], _ptr(out), n, width, PA_DTYPE[dtype], _stream(x))
    return out


def rms_gate(o: Tensor, gate: Optional[Tensor], weight: Tensor, eps: float, groups: int = 1, order: Optional[str] = "sigmoid_last",
             out: Optional[Tensor] = None) -> Tensor:
    """The gated RMS norm of every one of ``groups`` equal parts of a row (``pa_rms_gate``): ``"sigmoid_last"``:
    ``o / rms(o) * weight * sigmoid(gate)``; ``"silu_last"`` likewise with the silu; ``"silu_first"``: ``z / rms(z) * weight`` of ``z = o * silu(gate)``; None: the norm alone.
    ``gate`` and ``out`` may be column slices."""
    rows, width = o.shape
    _dense(o, weight)
    _typed(o.dtype, gate)
    _typed(torch.float32, weight)
    if (gate is None) != (order is None) or (gate is not None and tuple(gate.shape) != (rows, width)) or weight.numel() != width:
        raise ValueError("gate / weight do not fit o")
    if out is None:
        out = torch.empty_like(o)
    _typed(o.dtype, out)
    if tuple(out.shape) != (rows, width):
        raise ValueError("out does not fit o")
    _run("pa_rms_gate", _ptr(o), _ptr(gate), _row_stride(gate) if gate is not None else 0, _ptr(weight), float(eps), _ptr(out), _row_stride(out), rows,
         width, groups, _GATES[order], PA_DTYPE[o.dtype], _stream(o))
    return out


def glu(gate: Tensor, up: Tensor, act: str, ids: Optional[Tensor] = None) -> Tensor:
    """``act(gate) * up`` (``pa_glu``); both may be column slices.  With ``ids`` the factor of row r is row
    ``ids[r]`` of ``up``."""
    rows, width = gate.shape
    _typed(gate.dtype, up)
    _typed(torch.int64, ids)
    if up.shape[1] != width or (up.shape[0] if ids is None else ids.numel()) != rows:
        raise ValueError("up / ids do not fit gate")
    out = torch.empty((rows, width), dtype=gate.dtype, device=gate.device)
    _run("pa_glu", _ptr(gate), _row_stride(gate), _ptr(up), _row_stride(up), _ptr(ids), up.shape[0], _ptr(out), rows,
         width, _ACTS[act], PA_DTYPE[gate.dtype], _stream(gate))
    return out


def bias_act(x: Tensor, bias: Optional[Tensor], act: Optional[str]) -> Tensor:
    """``act(x + bias)`` (``pa_bias_act``), ``"relu2"`` the square of the positive part; ``x`` may be a column slice."""
    rows, width = x.shape
    _dense(bias)
    _typed(torch.float32, bias)
    if bias is not None and bias.numel() != width:
        raise ValueError("bias does not fit x")
    out = torch.empty((rows, width), dtype=x.dtype, device=x.device)
    _run("pa_bias_act", _ptr(x), _row_stride(x), _ptr(bias), _ptr(out), rows, width, _ACTS[act], PA_DTYPE[x.dtype], _stream(x))
    return out


def head_gate(o: Tensor, gate: Optional[Tensor], vdim: int, scale: float = 1.0, out: Optional[Tensor] = None) -> Tensor:
    """``[rows, heads, d]`` -> ``[rows, heads * vdim]``: the leading ``vdim`` of every head times ``scale`` and the
    sigmoid of its gate logit (``pa_head_gate``); ``out`` may be a column slice."""
    rows, heads, d = o.shape
    _dense(o)
    if gate is not None:
        _typed(o.dtype, gate)
        if tuple(gate.shape) != (rows, heads):
            raise ValueError("gate must hold one logit per row and head")
    if out is None:
        out = torch.empty((rows, heads * vdim), dtype=o.dtype, device=o.device)
    _typed(o.dtype, out)
    if tuple(out.shape) != (rows, heads * vdim):
        raise ValueError("out does not fit o")
    _run("pa_head_gate", _ptr(o), _ptr(gate), _row_stride(gate) if gate is not None else 0, float(scale), _ptr(out),
         _row_stride(out), rows, heads, d, vdim, PA_DTYPE[o.dtype], _stream(o))
    return out


class Portions(NamedTuple):
    """Runs of new rows, one per sequence, as the kernels take them (int32 on the device).  ``q_lens`` /
    ``q_starts`` None: one row per sequence, in order."""

    ctx_lens: Tensor
    state_slots: Optional[Tensor]
    q_lens: Optional[Tensor] = None
    q_starts: Optional[Tensor] = None
    tiles: Optional[Tensor] = None  # [n, 2]: (sequence, first row) of every PA_QKV_TILE_ROWS rows
    max_q_len: int = 1


def qkv_conv_append(u: Tensor, portions: Portions, slots: Tensor, k_cache: Tensor, v_cache: Tensor, num_q_heads: int,
                    dim: int, vdim: int, q_scale: float, eps: float, unit_norm: bool, rope: Optional[Tensor], rot_dims: int,
                    conv_weight: Optional[Tensor], conv_state: Optional[Tensor], v_mode: Optional[str] = None,
                    v_first: Optional[Tensor] = None, v_lambda: Optional[Tensor] = None,
                    q_out: Optional[Tensor] = None, q_norm: Optional[Tensor] = None,
                    k_norm: Optional[Tensor] = None, bias: Optional[Tensor] = None) -> Tensor:
    """Projection rows to rotated, normalised q and appended k / v (``pa_qkv_conv_append``).  Returns q
    ``[rows, Hq, D]`` with D the pool's head size; k and v go to ``k_cache`` / ``v_cache`` ``[slots, Hkv, D]``.
    ``q_norm`` / ``k_norm`` float32 ``[dim]``: weights of RMS norms ahead of the rotation; ``bias`` float32 ``[channels]``."""
    rows = u.shape[0]
    total_slots, hkv, d = k_cache.shape
    taps = conv_weight.shape[0] if conv_weight is not None else 1
    channels = (num_q_heads + hkv) * dim + hkv * vdim
    _dense(slots, k_cache, v_cache, rope, conv_weight, conv_state, v_first, q_norm, k_norm, bias, *portions[:5])
    _typed(u.dtype, k_cache, v_cache, conv_state, v_first)
    _typed(torch.int32, *portions[:5])
    _typed(torch.float32, rope, conv_weight, v_lambda, q_norm, k_norm, bias)
    if bias is not None and bias.numel() != channels:
        raise ValueError("bias must hold one number per channel")
    for t in (q_norm, k_norm):
        if t is not None and t.numel() != dim:
            raise ValueError("q_norm / k_norm must hold one weight per dimension")
    _typed(torch.int64, slots)
    batch = portions.ctx_lens.numel()
    if slots.numel() != rows or v_cache.shape != k_cache.shape or u.shape[1] < channels:
        raise ValueError("slots / v_cache / u do not fit")
    if conv_weight is not None and (conv_weight.shape[1] != channels or (taps > 1 and tuple(conv_state.shape[1:]) != (taps - 1, channels))):
        raise ValueError("convolution weights or state of another size")
    if rope is not None and tuple(rope.shape[1:]) != (rot_dims // 2, 2):
        raise ValueError("rope must be [positions, rot_dims / 2, 2]")
    if v_first is not None and tuple(v_first.shape) != (rows, hkv * vdim):
        raise ValueError("v_first must be [rows, Hkv * vdim]")
    if q_out is None:
        q_out = torch.empty((rows, num_q_heads, d), dtype=u.dtype, device=u.device)
    n_tiles = batch if portions.tiles is None else portions.tiles.shape[0]
    _run("pa_qkv_conv_append", _ptr(u), _row_stride(u), rows, _ptr(bias), _ptr(conv_weight), taps, _ptr(conv_state),
         conv_state.shape[0] if conv_state is not None else 0, _ptr(rope), rope.shape[0] if rope is not None else 0,
         rot_dims if rope is not None else 0, _ptr(portions.ctx_lens), _ptr(portions.q_lens), _ptr(portions.q_starts),
         _ptr(portions.state_slots), _ptr(portions.tiles), n_tiles, batch, _ptr(slots), total_slots, _ptr(q_out),
         _ptr(k_cache), _ptr(v_cache), _ptr(v_first), _ptr(v_lambda), _V_MODES[v_mode], _ptr(q_norm), _ptr(k_norm),
         num_q_heads, hkv, dim, vdim, d, int(unit_norm), float(eps), float(q_scale), PA_DTYPE[u.dtype], _stream(u))
    return q_out


def lightning_state(num_slots: int, heads: int, dim: int, vdim: int, device) -> Tensor:
    """The zero-filled state pool of one lightning layer, float32 ``[slots, heads, pad16(dim), pad16(vdim)]``."""
    pad = lambda n: -(-n // 16) * 16
    return torch.zeros((num_slots, heads, pad(dim), pad(vdim)), dtype=torch.float32, device=device)


def lightning_workspace_bytes(batch: int, heads: int, dim: int, vdim: int, max_q_len: int) -> int:
    return int(_lib.load().pa_lightning_workspace_bytes(batch, heads, dim, vdim, max_q_len))


def lightning(u: Tensor, portions: Portions, state: Tensor, decay_powers: Tensor, heads: int, dim: int, vdim: int,
              out: Tensor, workspace: Optional[Tensor] = None) -> Tensor:
    """Lightning attention over projection rows ``[q | k | v | ...]`` with the state carried in ``state`` (see
    ``lightning_state``): portions of bf16 rows in chunks on the matrix cores (``pa_lightning_chunked``), single rows
    and float32 rows token by token (``pa_lightning_recurrent``).  ``out`` ``[rows, heads * vdim]``."""
    _dense(state, decay_powers, out, *portions[:4])
    _typed(torch.int32, *portions[:4])
    _typed(torch.float32, state, decay_powers)
    _typed(u.dtype, out)
    rows, batch = u.shape[0], portions.ctx_lens.numel()
    pad = lambda n: -(-n // 16) * 16
    if tuple(state.shape[1:]) != (heads, pad(dim), pad(vdim)) or tuple(decay_powers.shape) != (heads, 65):
        raise ValueError("state or decay table of another size")
    if tuple(out.shape) != (rows, heads * vdim):
        raise ValueError("out must be [rows, heads * vdim]")
    head = (_ptr(u), _row_stride(u), rows, _ptr(state), state.shape[0], _ptr(decay_powers), _ptr(portions.ctx_lens),
            _ptr(portions.q_lens), _ptr(portions.q_starts), _ptr(portions.state_slots), batch)
    tail = (_ptr(out), heads, dim, vdim, PA_DTYPE[u.dtype])
    if portions.q_lens is None or u.dtype == torch.float32:
        _run("pa_lightning_recurrent", *head, *tail, _stream(u))
    else:
        _run("pa_lightning_chunked", *head, portions.max_q_len, *tail, _ptr(workspace),
             workspace.numel() * workspace.element_size() if workspace is not None else 0, _stream(u))
    return out


def softcap(x: Tensor, cap: float) -> Tensor:
    """``cap * tanh(x / cap)`` as float32 (``pa_softcap``)."""
    _dense(x)
    out = torch.empty(x.shape, dtype=torch.float32, device=x.device)
    _run("pa_softcap", _ptr(x), _ptr(out), x.numel(), float(cap), PA_DTYPE[x.dtype], _stream(x))
    return out


def short_conv(u: Tensor, portions: Portions, weight: Tensor, bias: Optional[Tensor], conv_state: Optional[Tensor],
               act: Optional[str]) -> Tensor:
    """Causal convolution over time with its carried rows (``pa_short_conv``): ``u`` ``[rows, channels]`` (may be a column
    slice), ``weight`` float32 ``[taps, channels]``, ``conv_state`` ``[slots, taps - 1, channels]``."""
    rows, channels = u.shape
    taps = weight.shape[0]
    _dense(weight, bias, conv_state, *portions[:5])
    _typed(torch.float32, weight, bias)
    _typed(torch.int32, *portions[:5])
    _typed(u.dtype, conv_state)
    if weight.shape[1] != channels or (bias is not None and bias.numel() != channels):
        raise ValueError("weight / bias do not fit u")
    if taps > 1 and (conv_state is None or tuple(conv_state.shape[1:]) != (taps - 1, channels)):
        raise ValueError("carried rows of another size")
    batch = portions.ctx_lens.numel()
    out = torch.empty((rows, channels), dtype=u.dtype, device=u.device)
    _run("pa_short_conv", _ptr(u), _row_stride(u), rows, _ptr(weight), _ptr(bias), taps, _ACTS[act], _ptr(conv_state),
         conv_state.shape[0] if conv_state is not None else 0, _ptr(portions.ctx_lens), _ptr(portions.q_lens),
         _ptr(portions.q_starts), _ptr(portions.state_slots), _ptr(portions.tiles),
         batch if portions.tiles is None else portions.tiles.shape[0], batch, _ptr(out), channels, PA_DTYPE[u.dtype], _stream(u))
    return out


def gated_linear_state_floats(kind: str, dim: int, vdim: int) -> int:
    """Floats per head of a gated recurrence's state."""
    return int(_lib.load().pa_gated_linear_state_floats(_GATED[kind], dim, vdim))


def gated_linear_workspace_bytes(batch: int, heads: int, dim: int, vdim: int, max_q_len: int) -> int:
    return int(_lib.load().pa_gated_linear_workspace_bytes(batch, heads, dim, vdim, max_q_len))


def gated_linear(kind: str, q: Tensor, k: Tensor, v: Tensor, gates: Tuple[Tensor, Optional[Tensor]],
                 constants: Tuple[Tensor, Tensor, Optional[Tensor]], portions: Portions, state: Tensor, heads: int, dim: int,
                 vdim: int, out: Tensor, heads_per_group: int = 1, cap: float = 1.0, q_scale: float = 1.0, den_eps: float = 0.0,
                 workspace: Optional[Tensor] = None) -> Tensor:
    """A linear recurrence with gates per token and head (``pa_gated_linear``), ``kind`` ``"ssd"`` or ``"mlstm"``.  q, k, v
    and the gates ``[rows, heads]`` may be column slices; ``constants`` float32 ``[heads]`` each: dt bias, decay rate and
    skip, or the biases of the two gates; ``state`` float32 ``[slots, heads, gated_linear_state_floats]``."""
    rows, batch = v.shape[0], portions.ctx_lens.numel()
    ga, gb = gates
    _dense(state, out, *constants, *portions[:4])
    _typed(torch.int32, *portions[:4])
    _typed(torch.float32, state, *constants)
    _typed(v.dtype, q, k, ga, gb, out)
    qk = (rows, heads // heads_per_group * dim)
    if tuple(q.shape) != qk or tuple(k.shape) != qk or tuple(v.shape) != (rows, heads * vdim) or out.shape != v.shape:
        raise ValueError("q / k / v / out do not fit each other")
    if any(c is not None and c.numel() != heads for c in constants) or tuple(ga.shape) != (rows, heads):
        raise ValueError("gates / constants do not fit the heads")
    if gb is not None and (tuple(gb.shape) != (rows, heads) or _row_stride(gb) != _row_stride(ga)):
        raise ValueError("the two gates differ in their rows")
    if tuple(state.shape[1:]) != (heads, gated_linear_state_floats(kind, dim, vdim)):
        raise ValueError("state of another size")
    _run("pa_gated_linear", _GATED[kind], _ptr(q), _row_stride(q), _ptr(k), _row_stride(k), _ptr(v), _row_stride(v),
         heads_per_group, _ptr(ga), _ptr(gb), _row_stride(ga), *(_ptr(c) for c in constants), float(cap), float(q_scale),
         float(den_eps), rows, _ptr(state), state.shape[0], _ptr(portions.ctx_lens), _ptr(portions.q_lens),
         _ptr(portions.q_starts), _ptr(portions.state_slots), batch, portions.max_q_len, _ptr(out), heads, dim, vdim,
         PA_DTYPE[v.dtype], _ptr(workspace), workspace.numel() * workspace.element_size() if workspace is not None else 0,
         _stream(v))
    return out


def narrow_linear(x: Tensor, w: Tensor) -> Tensor:
    """``x w^T`` summed and returned in float32 (``pa_narrow_linear``), for a few outputs."""
    _dense(w)
    _typed(x.dtype, w)
    if w.shape[1] != x.shape[1]:
        raise ValueError("w does not fit x")
    out = torch.empty((x.shape[0], w.shape[0]), dtype=torch.float32, device=x.device)
    _run("pa_narrow_linear", _ptr(x), _row_stride(x), _ptr(w), _ptr(out), x.shape[0], w.shape[0], w.shape[1],
         PA_DTYPE[x.dtype], _stream(x))
    return out


class ExpertChoice(NamedTuple):
    """Which experts every row uses: ``ids`` int32 ``[rows, top]``, ``weights`` float32 ``[rows, top + 1]`` (the last one the
    shared expert's; with identity experts one more, the sum of theirs) and, per expert, how many and which items (row * top
    + place)."""

    ids: Tensor
    weights: Tensor
    counts: Tensor
    lists: Tensor


def moe_choose(logits: Tensor, experts: int, top: int, groups: int, keep: int, shared: Optional[str] = None, identity: int = 0,
               scores: str = "sigmoid", group_top: int = 2, renormalize: bool = True,
               correction: Optional[Tensor] = None) -> ExpertChoice:
    """``pa_moe_choose`` over float32 ``logits`` ``[rows, experts + identity]``; ``shared`` ``"gated"`` (one column more, its
    gate), ``"plain"`` or None."""
    rows, every = logits.shape[0], experts + identity
    _dense(logits, correction)
    _typed(torch.float32, logits, correction)
    if logits.shape[1] != every + (shared == "gated") or (correction is not None and correction.numel() != every):
        raise ValueError("logits must hold one column per expert, and one for a gated shared expert; correction likewise")
    dev = logits.device
    ids = torch.empty((rows, top), dtype=torch.int32, device=dev)
    weights = torch.empty((rows, top + (2 if identity else 1)), dtype=torch.float32, device=dev)
    counts = torch.empty(every, dtype=torch.int32, device=dev)
    lists = torch.empty((every, rows), dtype=torch.int32, device=dev)
    workspace = torch.empty(int(_lib.load().pa_moe_workspace_bytes(rows, every, top)), dtype=torch.uint8, device=dev)
    _run("pa_moe_choose", _ptr(logits), logits.shape[1], rows, experts, identity, top, groups, keep, _SHARED[shared], _SCORES[scores],
         group_top, int(renormalize), _ptr(correction), _ptr(ids), _ptr(weights), _ptr(counts), _ptr(lists), _ptr(workspace),
         workspace.numel(), _stream(logits))
    return ExpertChoice(ids, weights, counts[:experts], lists[:experts])


def moe_product(x: Tensor, choice: ExpertChoice, w: Tensor, n: int, k: int, glu: bool) -> Tensor:
    """Every item's product with its expert's weights (``pa_moe_product``): ``x`` ``[rows, k]`` or one row per item,
    ``w`` ``[experts, n (glu: 2n), stride]`` zero past k -> ``[rows * top, n]``."""
    rows, top = choice.ids.shape
    _dense(w, *choice)
    _typed(x.dtype, w)
    if x.shape[0] not in (rows, rows * top) or x.shape[1] != k:
        raise ValueError("x does not fit the choice")
    if w.shape[0] != choice.counts.numel() or w.shape[1] < n * (2 if glu else 1) or w.shape[2] < k:
        raise ValueError("w does not fit the choice")
    out = torch.empty((rows * top, n), dtype=x.dtype, device=x.device)
    _run("pa_moe_product", _ptr(x), _row_stride(x), rows * top // x.shape[0] if x.shape[0] else 1, _ptr(w), w.shape[1], w.shape[2], k,
         _ptr(choice.counts), _ptr(choice.lists), rows, top, w.shape[0], int(glu), _ptr(out), n, PA_DTYPE[x.dtype], _stream(x))
    return out


def delta_workspace_bytes(batch: int, heads: int, dim: int, vdim: int, max_q_len: int) -> int:
    return int(_lib.load().pa_delta_workspace_bytes(batch, heads, dim, vdim, max_q_len))


def delta_rule(q: Tensor, k: Tensor, v: Tensor, decay_logits: Tensor, beta_logits: Tensor, decay_bias: Tensor, decay_rate: Tensor,
               portions: Portions, state: Tensor, heads: int, dim: int, vdim: int, q_scale: float, out: Tensor,
               heads_per_group: int = 1, workspace: Optional[Tensor] = None) -> Tensor:
    """The gated delta rule (``pa_delta``).  q, k, v and the logits ``[rows, heads]`` may be column slices; ``state`` float32
    ``[slots, heads, pad16(dim), pad16(vdim)]``."""
    rows, batch = v.shape[0], portions.ctx_lens.numel()
    pad = lambda n: -(-n // 16) * 16
    _dense(state, out, decay_bias, decay_rate, *portions[:4])
    _typed(torch.int32, *portions[:4])
    _typed(torch.float32, state, decay_bias, decay_rate)
    _typed(v.dtype, q, k, decay_logits, beta_logits, out)
    qk = (rows, heads // heads_per_group * dim)
    if tuple(q.shape) != qk or tuple(k.shape) != qk or tuple(v.shape) != (rows, heads * vdim) or out.shape != v.shape:
        raise ValueError("q / k / v / out do not fit each other")
    if any(tuple(g.shape) != (rows, heads) for g in (decay_logits, beta_logits)) or _row_stride(decay_logits) != _row_stride(beta_logits):
        raise ValueError("the two logits do not fit the heads, or differ in their rows")
    if decay_bias.numel() != heads or decay_rate.numel() != heads or tuple(state.shape[1:]) != (heads, pad(dim), pad(vdim)):
        raise ValueError("constants or state of another size")
    _run("pa_delta", _ptr(q), _row_stride(q), _ptr(k), _row_stride(k), _ptr(v), _row_stride(v), heads_per_group, _ptr(decay_logits),
         _ptr(beta_logits), _row_stride(decay_logits), _ptr(decay_bias), _ptr(decay_rate), float(q_scale), rows, _ptr(state),
         state.shape[0], _ptr(portions.ctx_lens), _ptr(portions.q_lens), _ptr(portions.q_starts), _ptr(portions.state_slots), batch,
         portions.max_q_len, _ptr(out), heads, dim, vdim, PA_DTYPE[v.dtype], _ptr(workspace),
         workspace.numel() * workspace.element_size() if workspace is not None else 0, _stream(v))
    return out


def hyper_norm(x: Tensor, dtype: torch.dtype, y: Optional[Tensor] = None, between: Optional[Tensor] = None,
               into: Optional[Tensor] = None, mix: Optional[Tensor] = None, y_extra: Optional[Tensor] = None,
               y_self: Optional[Tensor] = None, ids: Optional[Tensor] = None, table: Optional[Tensor] = None,
               sum_weight: Optional[Tensor] = None, weight: Optional[Tensor] = None, eps: float = 0.0, want: str = "out") -> Tensor:
    """One step of residual streams ``x`` float32 ``[rows, streams, width]`` (``pa_hyper_norm``): they start as
    ``table[ids]``, or are mixed by ``between`` and take ``y`` by ``into``.  ``want`` ``"out"``: updates x and returns the
    RMS norm of their weighted sum in ``dtype``; ``"sum"``: returns the float32 sum and leaves x.  ``mix`` float32
    ``[rows, m + 1]`` or, with ``y_self``, ``[rows, m + 2]``: y is a weighted sum of ``y`` ``[rows * m, width]``, ``y_extra``
    and ``y_self``."""
    rows, streams, width = x.shape
    _dense(x, y, between, into, mix, y_extra, y_self, ids, table, sum_weight, weight)
    _typed(torch.float32, x, between, into, mix, sum_weight, weight)
    _typed(torch.int64, ids)
    _typed(dtype, y, y_extra, y_self, table)
    m = mix.shape[1] - (1 if y_self is None else 2) if mix is not None else 0
    if y is not None and tuple(y.shape) != (rows * (m or 1), width):
        raise ValueError("y does not fit the streams")
    if (mix is not None and mix.shape[0] != rows) or any(t is not None and tuple(t.shape) != (rows, width) for t in (y_extra, y_self)):
        raise ValueError("mix / y_extra / y_self do not fit the streams")
    if ids is not None and (ids.numel() != rows or table.shape[1] != width):
        raise ValueError("ids / table do not fit the streams")
    if (between is not None and tuple(between.shape) != (streams, streams)) or \
            any(t is not None and t.numel() != streams for t in (into, sum_weight)) or (weight is not None and weight.numel() != width):
        raise ValueError("weights do not fit the streams")
    if want == "out":
        out, sum_ = torch.empty((rows, width), dtype=dtype, device=x.device), None
    else:
        out, sum_ = None, torch.empty((rows, width), dtype=torch.float32, device=x.device)
    _run("pa_hyper_norm", _ptr(x), _ptr(y), _ptr(mix), m, mix.shape[1] if mix is not None else 0, _ptr(y_extra), _ptr(y_self),
         _ptr(between), _ptr(into), _ptr(ids), _ptr(table), table.shape[0] if table is not None else 0, _ptr(sum_weight), _ptr(weight),
         float(eps), _ptr(out), _ptr(sum_), rows, streams, width, PA_DTYPE[dtype], _stream(x))
    return out if sum_ is None else sum_


def latent_append(u: Tensor, portions: Portions, slots: Tensor, pool: Tensor, norm: Tensor, eps: float, rope: Optional[Tensor],
                  heads: int, dim: int, rot_dim: int, rank: int, q_dim: int, q_scale: float) -> Tensor:
    """Projection rows to rotated queries ``[rows, heads, q_dim]`` and the appended pool rows ``[slots, 1, row]``
    (``pa_latent_append``)."""
    rows, batch = u.shape[0], portions.ctx_lens.numel()
    total_slots, one, pool_row = pool.shape
    _dense(slots, pool, norm, rope, *portions[:5])
    _typed(torch.int32, *portions[:5])
    _typed(torch.float32, norm, rope)
    _typed(u.dtype, pool)
    _typed(torch.int64, slots)
    if one != 1 or slots.numel() != rows or norm.numel() != rank or u.shape[1] < heads * (dim + rot_dim) + rank + rot_dim:
        raise ValueError("slots / pool / norm / u do not fit")
    if rot_dim and tuple(rope.shape[1:]) != (rot_dim // 2, 2):
        raise ValueError("rope must be [positions, rot_dim / 2, 2]")
    q = torch.empty((rows, heads, q_dim), dtype=u.dtype, device=u.device)
    n_tiles = batch if portions.tiles is None else portions.tiles.shape[0]
    _run("pa_latent_append", _ptr(u), _row_stride(u), rows, _ptr(norm), float(eps), _ptr(rope), rope.shape[0] if rope is not None else 0,
         _ptr(portions.ctx_lens), _ptr(portions.q_lens), _ptr(portions.q_starts), _ptr(portions.tiles), n_tiles, batch, _ptr(slots),
         total_slots, _ptr(q), _ptr(pool), heads, dim, rot_dim, rank, q_dim, pool_row, float(q_scale), PA_DTYPE[u.dtype], _stream(u))
    return q


def latent_gather(pool: Tensor, slots: Tensor) -> Tensor:
    """Rows ``[n, row]`` of a latent pool, zeros for slots out of range (``pa_latent_gather``)."""
    _dense(pool, slots)
    _typed(torch.int64, slots)
    total_slots, _, row = pool.shape
    out = torch.empty((slots.numel(), row), dtype=pool.dtype, device=pool.device)
    _run("pa_latent_gather", _ptr(pool), _ptr(slots), total_slots, _ptr(out), slots.numel(), row, PA_DTYPE[pool.dtype], _stream(pool))
    return out


def scored_workspace_bytes(batch: int, heads: int, kv_heads: int, key_size: int, vdim: int, one_tensor: bool, max_keys: int,
                           window: int) -> int:
    """Bytes with which a decode step spreads its sequences' keys over the device; ``one_tensor``: values are part of the keys."""
    return int(_lib.load().pa_scored_workspace_bytes(batch, heads, kv_heads, key_size, vdim, int(one_tensor), max_keys, window))


def scored_attention(q: Tuple[Tensor, ...], k_cache: Tensor, v_cache: Tensor, vdim: int, portions: Portions, block_tables: Tensor,
                     block_size: int, scale: float, window: int, out: Tensor, softcap: float = 0.0, bias: Optional[Tensor] = None,
                     sink: Optional[Tensor] = None, workspace: Optional[Tensor] = None) -> Tensor:
    """Paged attention with score terms (``pa_scored_attention``): ``q`` one or two pieces ``[rows, heads, n]`` whose last
    dimension is contiguous, ``bias`` float32 ``[heads, distances]``, ``sink`` float32 ``[heads]``; ``out`` ``[rows, heads,
    vdim]``.  ``v_cache`` may be ``k_cache``: the values are its first ``vdim`` elements."""
    rows, heads = q[0].shape[:2]
    total_slots, kv_heads, k_dim = k_cache.shape
    _dense(k_cache, v_cache, block_tables, bias, sink, out, *portions[:4])
    _typed(torch.int32, block_tables, *portions[:4])
    _typed(torch.float32, bias, sink)
    _typed(out.dtype, k_cache, v_cache, *q)
    if any(tuple(t.shape[:2]) != (rows, heads) or t.stride(2) != 1 for t in q) or not 1 <= len(q) <= 2:
        raise ValueError("q pieces do not fit each other")
    if tuple(v_cache.shape[:2]) != (total_slots, kv_heads) or tuple(out.shape) != (rows, heads, vdim):
        raise ValueError("v_cache / out do not fit")
    if (bias is not None and bias.shape[0] != heads) or (sink is not None and sink.numel() != heads):
        raise ValueError("bias / sink must have a row per head")
    piece = lambda t: (_ptr(t), t.stride(0), t.stride(1), t.shape[2])
    second = piece(q[1]) if len(q) == 2 else (None, 0, 0, 0)
    batch = portions.ctx_lens.numel()
    _run("pa_scored_attention", *piece(q[0]), *second, _ptr(k_cache), k_dim, _ptr(v_cache), v_cache.shape[2], vdim, _ptr(block_tables),
         block_tables.shape[1], block_size, total_slots // block_size, _ptr(portions.ctx_lens), _ptr(portions.q_lens),
         _ptr(portions.q_starts), rows, batch, portions.max_q_len, heads, kv_heads, float(scale), int(window), float(softcap), _ptr(bias),
         bias.shape[1] if bias is not None else 0, _ptr(sink), _ptr(out), PA_DTYPE[out.dtype], _ptr(workspace),
         workspace.numel() * workspace.element_size() if workspace is not None else 0, _stream(out))
    return out


def talking_workspace_bytes(rows: int, portions: Portions, heads: int, kv_heads: int, vdim: int, max_keys: int) -> int:
    return int(_lib.load().pa_talking_workspace_bytes(rows, portions.ctx_lens.numel(), heads, kv_heads, vdim, max_keys, int(portions.q_lens is None)))


def talking_attention(q: Tensor, k_cache: Tensor, v_cache: Tensor, vdim: int, portions: Portions, block_tables: Tensor, block_size: int,
                      scale: float, talk: Tensor, out: Tensor, bias_size: Optional[Tensor] = None, bias_rate: Optional[Tensor] = None,
                      workspace: Optional[Tensor] = None) -> Tensor:
    """Paged attention whose heads' weights are mixed by ``talk`` float32 ``[heads, heads]`` (``pa_talking_attention``): ``q``
    ``[rows, heads, dim]`` whose last dimension is contiguous, ``bias_size`` and ``bias_rate`` float32 ``[heads]``; ``out``
    ``[rows, heads, vdim]``.  The workspace (``talking_workspace_bytes``) is needed."""
    rows, heads, dim = q.shape
    total_slots, kv_heads, k_dim = k_cache.shape
    _dense(k_cache, v_cache, block_tables, talk, bias_size, bias_rate, out, *portions[:4])
    _typed(torch.int32, block_tables, *portions[:4])
    _typed(torch.float32, talk, bias_size, bias_rate)
    _typed(out.dtype, k_cache, v_cache, q)
    if q.stride(2) != 1 or tuple(v_cache.shape[:2]) != (total_slots, kv_heads) or tuple(out.shape) != (rows, heads, vdim):
        raise ValueError("q / v_cache / out do not fit")
    if tuple(talk.shape) != (heads, heads) or any(t is not None and t.numel() != heads for t in (bias_size, bias_rate)):
        raise ValueError("talk / bias_size / bias_rate do not fit the heads")
    _run("pa_talking_attention", _ptr(q), q.stride(0), q.stride(1), dim, _ptr(k_cache), k_dim, _ptr(v_cache), v_cache.shape[2], vdim,
         _ptr(block_tables), block_tables.shape[1], block_size, total_slots // block_size, _ptr(portions.ctx_lens), _ptr(portions.q_lens),
         _ptr(portions.q_starts), rows, portions.ctx_lens.numel(), portions.max_q_len, heads, kv_heads, float(scale), _ptr(bias_size),
         _ptr(bias_rate), _ptr(talk), _ptr(out), PA_DTYPE[out.dtype], _ptr(workspace),
         workspace.numel() * workspace.element_size() if workspace is not None else 0, _stream(out))
    return out


def channel_linear_workspace_bytes(batch: int, heads: int, dim: int, vdim: int, max_q_len: int) -> int:
    return int(_lib.load().pa_channel_linear_workspace_bytes(batch, heads, dim, vdim, max_q_len))


def channel_linear(q: Tensor, forget: Tensor, v: Tensor, f_bias: Optional[Tensor], lower: Tensor, portions: Portions, state: Tensor,
                   heads: int, dim: int, vdim: int, out: Tensor, q_act: Optional[str] = None, workspace: Optional[Tensor] = None) -> Tensor:
    """Linear attention with a forget gate per channel (``pa_channel_linear``).  q, the gate's logits and v may be column slices;
    ``f_bias`` and ``lower`` float32 ``[heads * dim]``, ``state`` float32 ``[slots, heads, pad16(dim), pad16(vdim)]``."""
    rows, batch = v.shape[0], portions.ctx_lens.numel()
    pad = lambda n: -(-n // 16) * 16
    _dense(state, out, f_bias, lower, *portions[:4])
    _typed(torch.int32, *portions[:4])
    _typed(torch.float32, state, f_bias, lower)
    _typed(v.dtype, q, forget, out)
    if any(tuple(t.shape) != (rows, heads * dim) for t in (q, forget)) or tuple(v.shape) != (rows, heads * vdim) or out.shape != v.shape:
        raise ValueError("q / forget / v / out do not fit each other")
    if any(t is not None and t.numel() != heads * dim for t in (f_bias, lower)) or tuple(state.shape[1:]) != (heads, pad(dim), pad(vdim)):
        raise ValueError("constants or state of another size")
    _run("pa_channel_linear", _ptr(q), _row_stride(q), _ACTS[q_act], _ptr(forget), _row_stride(forget), _ptr(f_bias), _ptr(lower), _ptr(v),
         _row_stride(v), rows, _ptr(state), state.shape[0], _ptr(portions.ctx_lens), _ptr(portions.q_lens), _ptr(portions.q_starts),
         _ptr(portions.state_slots), batch, portions.max_q_len, _ptr(out), heads, dim, vdim, PA_DTYPE[v.dtype], _ptr(workspace),
         workspace.numel() * workspace.element_size() if workspace is not None else 0, _stream(v))
    return out
