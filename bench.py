#!/usr/bin/env python3
"""Benchmark of the paged decode-attention hot path on one MI355X.

One step = one ``pa_decode`` call over one batch of the synthetic workload,
inputs resident in HBM.  The headline workload is workload c4 (Llama-3-8B
shape, B=256, bf16 pool, lognormal context lengths, seed 1004).  Prints one
JSON line; with the default workload the line also carries short runs of the
other configurations (c2, c5 decode; c3 append + chunked prefill; the c3 shape at
head_dim 256 and 64; dense prefill of 64 x 512 and 4 x 8192 tokens; one chunk
behind 200 000 cached keys at head_dim 128 and 256) under ``secondary``.

    python bench.py [--gpus 1] [--steps K] [--warmup W] [--no-secondary]
                    [--workload c4|c2|c5|c1|c3|c3-d256|c3-d64|c3-d96|long-d128|long-d256|dense-64x512|dense-4x8192|engine|lotozen|tevirax|vusalix|loluzen]
    python bench.py --traffic-from-pmc NAME KERNEL FETCH.csv WRITE.csv   # refresh profiles/traffic.json
"""

from __future__ import annotations

import argparse
import json
import os
import sys
import time

import numpy as np
import torch

ROOT = os.path.dirname(os.path.abspath(__file__))
if ROOT not in sys.path:
    sys.path.insert(0, ROOT)

HBM_PEAK_GBPS = 8000.0  # MI355X HBM3E, vendor figure
MFMA_BF16_PEAK_TFLOPS = 2500.0  # MI355X dense bf16 matrix peak, vendor figure

# HBM traffic of one launch of each workload's dominant kernel, from rocprofv3 --pmc FETCH_SIZE / WRITE_SIZE runs
# scaled by a device copy of known size in the same run: written by `--traffic-from-pmc` from the counter files,
# never typed in; a workload without an entry reports null.
TRAFFIC_FILE = os.path.join(ROOT, "profiles", "traffic.json")


def calibration_copy(dev) -> None:
    """One device copy of 1 GiB (reads 1 GiB, writes 1 GiB): what `--traffic-from-pmc` scales the counters by."""
    src = torch.empty(1 << 30, dtype=torch.uint8, device=dev)
    dst = torch.empty_like(src)
    dst.copy_(src)
    torch.cuda.synchronize()
    del src, dst


def measured_traffic(name):
    try:
        with open(TRAFFIC_FILE) as f:
            entry = json.load(f).get(name)
    except (OSError, ValueError):
        return None
    return None if entry is None else entry["bytes"]


def traffic_from_pmc(name, kernel, fetch_csv, write_csv) -> int:
    """Average FETCH_SIZE / WRITE_SIZE (KiB per dispatch) of `kernel` in two rocprofv3 counter_collection CSVs,
    each scaled by what the same counter reads for the 1 GiB device copy of `--copy-calibration` in the same file;
    stores the sum as workload `name` in profiles/traffic.json."""
    import csv

    def one(path, counter, copied_kib):
        mine, copy = [], []
        with open(path) as f:
            for r in csv.DictReader(f):
                if r["Counter_Name"] != counter:
                    continue
                if kernel in r["Kernel_Name"]:
                    mine.append(float(r["Counter_Value"]))
                elif "copyBuffer" in r["Kernel_Name"]:
                    copy.append(float(r["Counter_Value"]))
        if not mine or not copy:
            raise SystemExit(f"{path}: no {counter} rows for {kernel!r} or for the calibration copy")
        # the calibration copy (1 GiB, in one dispatch or split in two) is the largest device copy of the run
        big = [c for c in copy if c >= 0.9 * max(copy)]
        factor = copied_kib / sum(big)
        return sum(mine) / len(mine) * factor * 1024.0, factor

    fetch, f_scale = one(fetch_csv, "FETCH_SIZE", 1024 * 1024)
    write, w_scale = one(write_csv, "WRITE_SIZE", 1024 * 1024)
    try:
        with open(TRAFFIC_FILE) as f:
            table = json.load(f)
    except (OSError, ValueError):
        table = {}
    table[name] = {"bytes": int(round(fetch + write)), "kernel": kernel, "fetch_bytes": int(round(fetch)),
                   "write_bytes": int(round(write)), "fetch_scale": round(f_scale, 4), "write_scale": round(w_scale, 4)}
    with open(TRAFFIC_FILE, "w") as f:
        json.dump(table, f, indent=1, sort_keys=True)
        f.write("\n")
    print(json.dumps({name: table[name]}))
    return 0


def parse_args():
    ap = argparse.ArgumentParser()
    ap.add_argument("--gpus", type=int, default=1)
    ap.add_argument("--steps", type=int, default=50)
    ap.add_argument("--warmup", type=int, default=10)
    ap.add_argument("--workload", default="c4", choices=["c1", "c2", "c3", "c3-d256", "c3-d64", "c3-d96", "long-d128", "long-d256", "dense-64x512",
                                                         "dense-4x8192", "c4", "c5", "engine", "lotozen",
                                                         "tevirax", "vusalix", "loluzen"])
    ap.add_argument("--preheat-s", type=float, default=0.5,
                    help="seconds of untimed steps before the warmup steps: an idle GPU sits at its lowest clocks "
                         "and takes a few hundred milliseconds of work to leave them")
    ap.add_argument("--no-cpu-baseline", action="store_true")
    ap.add_argument("--cpu-seconds", type=float, default=15.0, help="rough budget of the CPU baseline sample")
    ap.add_argument("--copy-calibration", action="store_true",
                    help="also run one plain 1 GiB device copy, as the known-size kernel HBM counters are scaled by")
    ap.add_argument("--no-secondary", action="store_true",
                    help="with the default workload: leave out the short runs of c2, c5 and c3")
    ap.add_argument("--traffic-from-pmc", nargs=4, metavar=("NAME", "KERNEL", "FETCH_CSV", "WRITE_CSV"),
                    help="no benchmark: compute a workload's HBM traffic from two rocprofv3 counter files")
    return ap.parse_args()


def cpu_baseline(w, budget_s: float):
    """Time the vectorised CPU restatement (index gather + SDPA per sequence) on a bounded sample."""
    from oracle import paged_oracle as po

    threads = torch.get_num_threads()
    order = np.argsort(w.seq_lens)  # shortest first so the sample can be cut to the budget
    tables = [w.block_tables[i].tolist() for i in order]
    lens = w.seq_lens[order]
    q = w.q[torch.from_numpy(order)][:, None]
    k_pool, v_pool = w.k_pool, w.v_pool
    if w.kv_format == "fp8_e4m3":  # the CPU path of the fp8 workload is dequantise-then-attend
        kb, ks = po.quantize_kv_e4m3(k_pool, w.block_size)
        vb, vs = po.quantize_kv_e4m3(v_pool, w.block_size)
        k_pool = po.dequantize_kv_e4m3(kb, ks, w.block_size).to(w.dtype)
        v_pool = po.dequantize_kv_e4m3(vb, vs, w.block_size).to(w.dtype)
    po.decode_per_sequence(q[:2], k_pool, v_pool, tables[:2], lens[:2], w.block_size, w.scale)  # warm up
    done_tokens, done_seqs, at, t0 = 0, 0, 0, time.perf_counter()
    # walk the batch (again from the start once it is exhausted) until the budget is used
    while time.perf_counter() - t0 < budget_s:
        n = min(4, len(lens) - at)
        sl = slice(at, at + n)
        po.decode_per_sequence(q[sl], k_pool, v_pool, tables[sl], lens[sl], w.block_size, w.scale)
        done_seqs += n
        done_tokens += int(lens[sl].sum())
        at = (at + n) % len(lens)
    dt = time.perf_counter() - t0
    # the same bytes per key as the GPU figure counts: one per element of an fp8 pool (the CPU path itself reads
    # the dequantised 16-bit copy)
    kv_size = 1 if w.kv_format == "fp8_e4m3" else w.q.element_size()
    sample_bytes = done_tokens * w.num_kv_heads * w.head_dim * 2 * kv_size
    return {
        "value": sample_bytes / dt / 1e9,
        "unit": "GB/s",
        "cores": threads,
        "kind": "port",
        "tokens_per_s": done_seqs / dt,
        "sample": f"{done_seqs} sequence passes over the {len(lens)} sequences of {w.name}, shortest first, "
                  f"cycling ({done_tokens} keys), per-sequence index gather + torch SDPA on {threads} threads, "
                  f"{dt:.1f} s",
    }


def cpu_literal(w):
    """One pass of the literal restatement of the reference's decode (token-by-token gather loop into a
    zero-padded batch, repeat_interleave, unmasked SDPA) over the whole workload; only for the workloads small
    enough to run it as written (c1, c2)."""
    from oracle import paged_oracle as po

    tables = [t.tolist() for t in w.block_tables]
    t0 = time.perf_counter()
    po.decode_literal(w.q[:, None], w.k_pool, w.v_pool, tables, w.seq_lens, w.block_size, w.scale)
    dt = time.perf_counter() - t0
    padded = 2 * w.batch * int(w.seq_lens.max()) * w.num_q_heads * w.head_dim * w.q.element_size()
    return {"value": w.algorithmic_bytes() / dt / 1e9, "unit": "GB/s", "cores": torch.get_num_threads(),
            "kind": "port", "seconds": dt, "tokens_per_s": w.batch / dt,
            "sample": f"the whole of {w.name} once: {2 * int(w.seq_lens.sum())} row copies issued from Python, "
                      f"{padded / 1e9:.2f} GB of padded and head-expanded K/V, one SDPA call"}


def preheat(fn, seconds):
    """Untimed calls of `fn` for about `seconds`, so that the timed region does not start on idle clocks."""
    t0 = time.perf_counter()
    while time.perf_counter() - t0 < seconds:
        for _ in range(20):
            fn()
        torch.cuda.synchronize()


def timed_ms(fn, steps):
    """Average milliseconds per call: HIP events on the launch stream around `steps` calls."""
    start, stop = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
    torch.cuda.synchronize()
    start.record()
    for _ in range(steps):
        fn()
    stop.record()
    torch.cuda.synchronize()
    return start.elapsed_time(stop) / steps


def timed_steps(fn, steps):
    """(mean, median) milliseconds per call over exactly `steps` calls: one HIP event on the launch stream before
    the first call and one behind every call; the mean is the whole bracket, the median is over the steps."""
    marks = [torch.cuda.Event(enable_timing=True) for _ in range(steps + 1)]
    torch.cuda.synchronize()
    marks[0].record()
    for i in range(steps):
        fn()
        marks[i + 1].record()
    torch.cuda.synchronize()
    each = sorted(marks[i].elapsed_time(marks[i + 1]) for i in range(steps))
    return marks[0].elapsed_time(marks[steps]) / steps, each[steps // 2]


KERNEL_LAUNCHES = 50  # launches the dominant kernel's average duration is taken over


def bench_prefill_c3(args, dev) -> dict:
    """Workload c3: append 32 x 256 new K/V rows, then chunked causal prefill over 2048 shared prefix keys.

    One step = pa_kv_scatter + pa_prefill_paged.  The value is the step's attention FLOP rate; the roofline
    entry is the matrix-core prefill kernel alone; the append is reported beside it in GB/s.
    """
    from oracle import paged_oracle as po
    from research_amd import ops
    from research_amd.workloads import make_prefill_c3

    w = make_prefill_c3()
    S, C, P = w.num_seqs, w.chunk_len, w.prefix_len
    shape = (w.num_blocks * w.block_size, w.num_kv_heads, w.head_dim)
    kc = torch.zeros(shape, dtype=w.dtype, device=dev)
    vc = torch.zeros_like(kc)
    ops.kv_scatter(kc, vc, w.k_prefix.to(dev), w.v_prefix.to(dev), torch.from_numpy(w.prefix_slots()).to(dev))
    k_new = w.k_chunk.reshape(S * C, *shape[1:]).to(dev)
    v_new = w.v_chunk.reshape(S * C, *shape[1:]).to(dev)
    slots = torch.from_numpy(w.chunk_slots()).to(dev)
    q = w.q.reshape(S * C, w.num_q_heads, w.head_dim).to(dev)
    tables = torch.from_numpy(np.stack(w.block_tables).astype(np.int32)).to(dev)
    ctx = torch.full((S,), P + C, dtype=torch.int32, device=dev)
    ql = torch.full((S,), C, dtype=torch.int32, device=dev)
    qs = torch.arange(S, dtype=torch.int32, device=dev) * C
    out = torch.empty_like(q)

    def append():
        ops.kv_scatter(kc, vc, k_new, v_new, slots)

    def prefill():
        ops.prefill_paged(q, kc, vc, tables, ctx, ql, qs, C, w.block_size, w.scale, out=out)

    def step():
        append()
        prefill()

    if args.copy_calibration:
        calibration_copy(dev)
    preheat(step, args.preheat_s)
    for _ in range(args.warmup):
        step()
    ms_step_mean, ms_step = timed_steps(step, args.steps)
    ms_prefill = timed_ms(prefill, max(args.steps, KERNEL_LAUNCHES))
    ms_append = timed_ms(append, max(args.steps, KERNEL_LAUNCHES))
    # The same append with the rotary embedding of q and k fused in (the step a model runs right before this
    # path), beside the two-pass form: rotation into dense buffers, then the scatter.
    pos = (torch.arange(C, dtype=torch.int32, device=dev) + P).repeat(S)
    inv_freq = 1.0 / (10000.0 ** (torch.arange(0, w.head_dim, 2, device=dev).float() / w.head_dim))
    angles = torch.arange(P + C, device=dev).float()[:, None] * inv_freq[None, :]
    cos_t = torch.cat((angles, angles), dim=-1).cos().to(w.dtype)
    sin_t = torch.cat((angles, angles), dim=-1).sin().to(w.dtype)
    q_rot, k_rot = torch.empty_like(q), torch.empty_like(k_new)
    kc2, vc2 = torch.zeros_like(kc), torch.zeros_like(vc)  # scratch pool: the timed pool keeps its unrotated rows

    def rope_fused():
        ops.rope_kv_append(q, k_new, v_new, cos_t, sin_t, kc2, vc2, slots, positions=pos, q_out=q_rot)

    def rope_two_pass():
        ops.rope_kv_append(q, k_new, v_new, cos_t, sin_t, None, None, None, positions=pos, q_out=q_rot, k_out=k_rot)
        ops.kv_scatter(kc2, vc2, k_rot, v_new, slots)

    preheat(rope_fused, 0.1)
    ms_rope = timed_ms(rope_fused, args.steps)
    ms_rope2 = timed_ms(rope_two_pass, args.steps)
    eb = q.element_size()
    rope_bytes = (2 * q.numel() + 4 * k_new.numel()) * eb + 2 * S * C * w.head_dim * eb + S * C * 12
    flops = w.attention_flops()
    achieved = flops / (ms_prefill * 1e-3) / 1e12
    result = {
        "metric": "prefill-attn TFLOP/s", "value": flops / (ms_step * 1e-3) / 1e12, "unit": "TFLOP/s",
        "tokens_per_s": S * C / (ms_step * 1e-3), "n_gpus": 1, "steps": args.steps, "warmup": args.warmup,
        "preheat_s": args.preheat_s, "ms_per_step": ms_step, "ms_per_step_mean": ms_step_mean, "step_statistic": "median of the timed steps",
        "higher_is_better": True, "scaling": "weak", "vs_baseline": None, "dtype": "bf16",
        "data": "synthetic",
        "config": {"workload": "c3 shared-prefix chunked prefill + KV append, 32 x (2048 + 256), bf16",
                   "num_seqs": S, "prefix_len": P, "chunk_len": C, "num_q_heads": w.num_q_heads,
                   "num_kv_heads": w.num_kv_heads, "head_dim": w.head_dim, "block_size": w.block_size,
                   "attention_flops": flops, "append_bytes": w.append_bytes(), "seed": 1003},
        "roofline": {"bound": "mfma", "kernel": "prefill_asm_kernel", "achieved": achieved,
                     "peak": MFMA_BF16_PEAK_TFLOPS, "unit": "TFLOP/s", "frac": achieved / MFMA_BF16_PEAK_TFLOPS,
                     "traffic": measured_traffic("c3"), "kernel_ms": ms_prefill,
                     "kernel_launches": max(args.steps, KERNEL_LAUNCHES)},
        "append": {"kernel": "kv_scatter_kernel", "kernel_ms": ms_append,
                   "achieved_gbps": w.append_bytes() / (ms_append * 1e-3) / 1e9, "peak_gbps": HBM_PEAK_GBPS},
        "rope_append": {"kernel": "rope_kv_append_kernel", "kernel_ms": ms_rope, "bytes": rope_bytes,
                        "achieved_gbps": rope_bytes / (ms_rope * 1e-3) / 1e9, "peak_gbps": HBM_PEAK_GBPS,
                        "two_pass_ms": ms_rope2},
    }
    if not args.no_cpu_baseline:
        threads = torch.get_num_threads()
        kcc, vcc = kc.cpu(), vc.cpu()
        n = 0  # sequence passes of the sample (cycling over the batch)
        t0 = time.perf_counter()
        while time.perf_counter() - t0 < args.cpu_seconds:
            s = n % S
            blocks = np.asarray(w.block_tables[s])
            pos = np.arange(P + C)
            idx = torch.from_numpy(blocks[pos // w.block_size] * w.block_size + pos % w.block_size)
            k_full, v_full = kcc[idx][None], vcc[idx][None]
            q_full = torch.cat([torch.zeros(P, w.num_q_heads, w.head_dim, dtype=w.dtype), w.q[s]])[None]
            po.prefill_literal(q_full, k_full, v_full, w.scale)
            n += 1
        dt = time.perf_counter() - t0
        result["cpu_baseline"] = {
            "value": flops / S * n / dt / 1e12, "unit": "TFLOP/s", "cores": threads, "kind": "port",
            "sample": f"{n} sequence passes over the {S} sequences (cycling): index gather of prefix+chunk, then the reference's full-sequence causal "
                      f"SDPA over {P + C} tokens (rows {P}..{P + C - 1} are the chunk), {threads} threads, {dt:.1f} s; "
                      "FLOPs counted for the chunk rows only",
        }
    return result


# the c3 shape at other head sizes: workload -> (query heads, kv heads, head_dim, seed, kernel)
PREFILL_HEAD_SHAPES = {"c3-d256": (16, 8, 256, 1006, "prefill_d256_kernel"),
                       "c3-d64": (32, 8, 64, 1007, "prefill_asm_kernel"),
                       # a head size between the compiled ones: the head_dim-128 kernel, rows of 96 in memory
                       "c3-d96": (32, 8, 96, 1011, "prefill_asm_kernel")}


def bench_prefill_head(args, dev, name) -> dict:
    """The c3 shape (32 x (2048 shared + 256 own) tokens, 16-token blocks, bf16) with 16 query / 8 kv heads of 256,
    or 32 query / 8 kv heads of 64 or 96: the chunked-prefill kernel for that head size alone, against the bf16
    matrix-core peak (head_dim 96 runs the head_dim-128 kernel; its FLOP count is that of 96)."""
    from research_amd import ops
    from research_amd.workloads import make_prefill_c3

    hq, hkv, head_dim, seed, kernel = PREFILL_HEAD_SHAPES[name]
    w = make_prefill_c3(num_q_heads=hq, num_kv_heads=hkv, head_dim=head_dim, seed=seed)
    S, C, P = w.num_seqs, w.chunk_len, w.prefix_len
    shape = (w.num_blocks * w.block_size, w.num_kv_heads, w.head_dim)
    kc = torch.zeros(shape, dtype=w.dtype, device=dev)
    vc = torch.zeros_like(kc)
    ops.kv_scatter(kc, vc, w.k_prefix.to(dev), w.v_prefix.to(dev), torch.from_numpy(w.prefix_slots()).to(dev))
    ops.kv_scatter(kc, vc, w.k_chunk.reshape(S * C, *shape[1:]).to(dev), w.v_chunk.reshape(S * C, *shape[1:]).to(dev),
                   torch.from_numpy(w.chunk_slots()).to(dev))
    q = w.q.reshape(S * C, w.num_q_heads, w.head_dim).to(dev)
    tables = torch.from_numpy(np.stack(w.block_tables).astype(np.int32)).to(dev)
    ctx = torch.full((S,), P + C, dtype=torch.int32, device=dev)
    ql = torch.full((S,), C, dtype=torch.int32, device=dev)
    qs = torch.arange(S, dtype=torch.int32, device=dev) * C
    out = torch.empty_like(q)

    def prefill():
        ops.prefill_paged(q, kc, vc, tables, ctx, ql, qs, C, w.block_size, w.scale, out=out)

    if args.copy_calibration:
        calibration_copy(dev)
    preheat(prefill, args.preheat_s)
    for _ in range(args.warmup):
        prefill()
    ms_step_mean, ms_step = timed_steps(prefill, args.steps)
    ms_kernel = timed_ms(prefill, max(args.steps, KERNEL_LAUNCHES))
    flops = w.attention_flops()
    achieved = flops / (ms_kernel * 1e-3) / 1e12
    return {
        "metric": "prefill-attn TFLOP/s", "value": flops / (ms_step * 1e-3) / 1e12, "unit": "TFLOP/s",
        "tokens_per_s": S * C / (ms_step * 1e-3), "n_gpus": 1, "steps": args.steps, "warmup": args.warmup,
        "preheat_s": args.preheat_s, "ms_per_step": ms_step, "ms_per_step_mean": ms_step_mean, "step_statistic": "median of the timed steps",
        "higher_is_better": True, "scaling": "weak", "vs_baseline": None, "dtype": "bf16", "data": "synthetic",
        "config": {"workload": f"c3 shape at head_dim {head_dim}: chunked prefill, 32 x (2048 + 256), {hq} q / {hkv} kv heads, bf16",
                   "num_seqs": S, "prefix_len": P, "chunk_len": C, "num_q_heads": w.num_q_heads,
                   "num_kv_heads": w.num_kv_heads, "head_dim": w.head_dim, "block_size": w.block_size,
                   "attention_flops": flops, "seed": seed},
        "roofline": {"bound": "mfma", "kernel": kernel, "achieved": achieved,
                     "peak": MFMA_BF16_PEAK_TFLOPS, "unit": "TFLOP/s", "frac": achieved / MFMA_BF16_PEAK_TFLOPS,
                     "traffic": measured_traffic(name), "kernel_ms": ms_kernel,
                     "kernel_launches": max(args.steps, KERNEL_LAUNCHES)},
    }


# one long sequence: workload -> (query heads, kv heads, head_dim, seed, kernel)
PREFILL_LONG_SHAPES = {"long-d128": (8, 2, 128, 1008, "prefill_asm_kernel"),
                       "long-d256": (8, 2, 256, 1009, "prefill_d256_kernel")}


def bench_prefill_long(args, dev, name) -> dict:
    """A 2048-token chunk of ONE sequence behind 200 000 cached keys (16-token blocks in random pool order, bf16,
    8 query / 2 kv heads): more keys than the prefill kernels' LDS slot tables hold, so the instances that fill them
    again on the way run; few rows: 64 (head_dim 128) or 128 (256) workgroups for 256 CUs, so the call hands over a
    workspace and the head_dim 128 launch runs every workgroup's keys in pieces (kernel_ms then covers the piece
    kernel and the merge of the pieces)."""
    from research_amd import ops

    hq, hkv, head_dim, seed, kernel = PREFILL_LONG_SHAPES[name]
    P, C, bs = 200_000, 2048, 16
    nblk = -(-(P + C) // bs)
    gen = torch.Generator(device=dev).manual_seed(seed)
    kc = torch.randn(nblk * bs, hkv, head_dim, device=dev, dtype=torch.bfloat16, generator=gen)
    vc = torch.randn(nblk * bs, hkv, head_dim, device=dev, dtype=torch.bfloat16, generator=gen)
    q = torch.randn(C, hq, head_dim, device=dev, dtype=torch.bfloat16, generator=gen)
    tables = torch.randperm(nblk, device=dev, generator=gen).to(torch.int32).reshape(1, -1).contiguous()
    ctx = torch.tensor([P + C], dtype=torch.int32, device=dev)
    ql = torch.tensor([C], dtype=torch.int32, device=dev)
    qs = torch.zeros(1, dtype=torch.int32, device=dev)
    out = torch.empty_like(q)
    scale = head_dim ** -0.5

    # few rows: with a workspace the library cuts every workgroup's keys into pieces run side by side
    ws_bytes = ops.prefill_workspace_bytes(q, tables, C, bs, hkv)
    ws = torch.empty(ws_bytes, dtype=torch.uint8, device=dev) if ws_bytes else None
    pieces = ws_bytes // (C * hq * (head_dim + 2) * 4)

    def prefill():
        ops.prefill_paged(q, kc, vc, tables, ctx, ql, qs, C, bs, scale, out=out, workspace=ws)

    if args.copy_calibration:
        calibration_copy(dev)
    preheat(prefill, args.preheat_s)
    for _ in range(args.warmup):
        prefill()
    ms_step_mean, ms_step = timed_steps(prefill, args.steps)
    ms_kernel = timed_ms(prefill, max(args.steps, KERNEL_LAUNCHES))
    flops = 4 * head_dim * hq * (C * P + C * (C + 1) // 2)  # two products, every visible (row, key) pair
    achieved = flops / (ms_kernel * 1e-3) / 1e12
    return {
        "metric": "prefill-attn TFLOP/s", "value": flops / (ms_step * 1e-3) / 1e12, "unit": "TFLOP/s",
        "tokens_per_s": C / (ms_step * 1e-3), "n_gpus": 1, "steps": args.steps, "warmup": args.warmup,
        "preheat_s": args.preheat_s, "ms_per_step": ms_step, "ms_per_step_mean": ms_step_mean, "step_statistic": "median of the timed steps",
        "higher_is_better": True, "scaling": "weak", "vs_baseline": None, "dtype": "bf16", "data": "synthetic",
        "config": {"workload": f"one sequence, chunked prefill, 200000 + 2048, {hq} q / {hkv} kv heads of {head_dim}, bf16",
                   "num_seqs": 1, "prefix_len": P, "chunk_len": C, "num_q_heads": hq, "num_kv_heads": hkv,
                   "head_dim": head_dim, "block_size": bs, "attention_flops": flops, "seed": seed,
                   "key_pieces_per_workgroup": max(1, pieces), "workspace_bytes": ws_bytes},
        "roofline": {"bound": "mfma", "kernel": kernel, "achieved": achieved,
                     "peak": MFMA_BF16_PEAK_TFLOPS, "unit": "TFLOP/s", "frac": achieved / MFMA_BF16_PEAK_TFLOPS,
                     "traffic": measured_traffic(name), "kernel_ms": ms_kernel,
                     "kernel_launches": max(args.steps, KERNEL_LAUNCHES)},
    }


# dense causal prefill (no cached prefix): workload -> (sequences, tokens each, query heads, kv heads, head_dim, seed)
PREFILL_DENSE_SHAPES = {"dense-64x512": (64, 512, 32, 8, 128, 1010), "dense-4x8192": (4, 8192, 32, 8, 128, 1011)}


def bench_prefill_dense(args, dev, name) -> dict:
    """Dense causal prefill as ``_prefill_attention`` issues it: the step's own [B, T, Hkv, D] K/V handed to the
    paged kernel as a pool of B blocks of T tokens with the identity table.  64 prompts of 512 tokens are what an
    engine step of fresh prompts looks like: eight tiles of keys at most per workgroup, so the kernel's set-up and
    write-out weigh as much as its loop."""
    from research_amd import ops

    B, T, hq, hkv, head_dim, seed = PREFILL_DENSE_SHAPES[name]
    gen = torch.Generator(device=dev).manual_seed(seed)
    q = torch.randn(B * T, hq, head_dim, device=dev, dtype=torch.bfloat16, generator=gen)
    k = torch.randn(B * T, hkv, head_dim, device=dev, dtype=torch.bfloat16, generator=gen)
    v = torch.randn(B * T, hkv, head_dim, device=dev, dtype=torch.bfloat16, generator=gen)
    tables = torch.arange(B, dtype=torch.int32, device=dev).reshape(B, 1).contiguous()
    lens = torch.full((B,), T, dtype=torch.int32, device=dev)
    starts = torch.arange(B, dtype=torch.int32, device=dev) * T
    out = torch.empty_like(q)
    scale = head_dim ** -0.5

    def prefill():
        ops.prefill_paged(q, k, v, tables, lens, lens, starts, T, T, scale, out=out)

    if args.copy_calibration:
        calibration_copy(dev)
    preheat(prefill, args.preheat_s)
    for _ in range(args.warmup):
        prefill()
    ms_step_mean, ms_step = timed_steps(prefill, args.steps)
    ms_kernel = timed_ms(prefill, max(args.steps, KERNEL_LAUNCHES))
    flops = 4 * head_dim * hq * B * (T * (T + 1) // 2)  # two products, every visible (row, key) pair
    achieved = flops / (ms_kernel * 1e-3) / 1e12
    return {
        "metric": "prefill-attn TFLOP/s", "value": flops / (ms_step * 1e-3) / 1e12, "unit": "TFLOP/s",
        "tokens_per_s": B * T / (ms_step * 1e-3), "n_gpus": 1, "steps": args.steps, "warmup": args.warmup,
        "preheat_s": args.preheat_s, "ms_per_step": ms_step, "ms_per_step_mean": ms_step_mean,
        "step_statistic": "median of the timed steps", "higher_is_better": True, "scaling": "weak",
        "vs_baseline": None, "dtype": "bf16", "data": "synthetic",
        "config": {"workload": f"dense causal prefill, {B} x {T} tokens, {hq} q / {hkv} kv heads of {head_dim}, bf16",
                   "num_seqs": B, "prefix_len": 0, "chunk_len": T, "num_q_heads": hq, "num_kv_heads": hkv,
                   "head_dim": head_dim, "attention_flops": flops, "seed": seed},
        "roofline": {"bound": "mfma", "kernel": "prefill_asm_kernel", "achieved": achieved,
                     "peak": MFMA_BF16_PEAK_TFLOPS, "unit": "TFLOP/s", "frac": achieved / MFMA_BF16_PEAK_TFLOPS,
                     "traffic": measured_traffic(name), "kernel_ms": ms_kernel,
                     "kernel_launches": max(args.steps, KERNEL_LAUNCHES)},
    }


def bench_engine(args, dev) -> int:
    """The engine loop on a Qwen2.5-0.5B-shaped model with random weights (24 layers, 14 query / 2 kv heads of
    64, vocabulary 151 936, bf16): 8 prompts of 512 tokens, 16 rollouts each, 64 new tokens per rollout at
    temperature 1.  One step = one whole ``generate`` call.  Timed for the paged path (radix allocator: the
    rollouts of a prompt share its prefix blocks) and, beside it, for the reference engine's own design, the
    cache-less loop that recomputes every sequence each step (engine.py:218-250), through the same model."""
    from research_amd.inference import (CacheConfig, EngineConfig, HipPagedAttentionBackend, InferenceEngine,
                                        ModelConfig, PagedLlama, SamplingParams)

    cfg = ModelConfig(vocab_size=151936, hidden_size=896, intermediate_size=4864, num_layers=24, num_heads=14,
                      num_kv_heads=2, head_dim=64, rope_theta=1e6, rms_norm_eps=1e-6, max_position_embeddings=2048,
                      tie_word_embeddings=True, attention_bias=True)
    n_prompts, n_rollouts, prompt_len, new_tokens = 8, 16, 512, 64
    g = torch.Generator().manual_seed(7)
    prompts = [torch.randint(0, cfg.vocab_size, (prompt_len,), generator=g).tolist() for _ in range(n_prompts)]
    batch = [p for p in prompts for _ in range(n_rollouts)]
    params = SamplingParams(temperature=1.0, max_tokens=new_tokens)
    backend = HipPagedAttentionBackend(CacheConfig(
        num_layers=cfg.num_layers, num_kv_heads=cfg.num_kv_heads, head_dim=cfg.head_dim, num_blocks=8192,
        block_size=16, device="cuda", dtype=torch.bfloat16))
    torch.manual_seed(0)
    model = PagedLlama(cfg, backend).to(torch.bfloat16).to(dev).eval()

    def run(cache_type, reps, use_graphs=False):
        engine = InferenceEngine(EngineConfig(model_path="", cache_type=cache_type, block_size=16,
                                              max_batch_size=len(batch), max_model_len=2048, num_kv_blocks=8192,
                                              use_graphs=use_graphs),
                                 model=model)
        times = []
        for _ in range(reps):
            engine.flush_cache()
            torch.manual_seed(1)
            torch.cuda.synchronize()
            t0 = time.perf_counter()
            samples = engine.generate(batch, params)
            torch.cuda.synchronize()
            times.append(time.perf_counter() - t0)
            assert len(samples) == len(batch) and all(len(s.completion_tokens) == new_tokens for s in samples)
        return times

    run("radix", max(1, args.warmup // 5))  # untimed
    eager = run("radix", max(1, args.steps // 10))
    paged = run("radix", max(1, args.steps // 10) + 1, use_graphs=True)[1:]  # the first call captures the graph
    recompute = run("none", 1)
    n_new = len(batch) * new_tokens
    best = min(paged)
    result = {
        "metric": "engine generated tokens/s", "value": n_new / best, "unit": "tokens/s", "n_gpus": 1,
        "steps": len(paged), "warmup": max(1, args.warmup // 5), "ms_per_step": 1e3 * best,
        "higher_is_better": True, "scaling": "weak", "vs_baseline": None, "dtype": "bf16", "data": "synthetic",
        "config": {"workload": "engine: Qwen2.5-0.5B-shaped model, 8 prompts x 16 rollouts, 512 + 64 tokens",
                   "cache_type": "radix", "use_graphs": True, "block_size": 16, "sequences": len(batch),
                   "prompt_len": prompt_len, "new_tokens": new_tokens, "all_ms": [round(1e3 * t, 1) for t in paged]},
        "without_graphs": {"tokens_per_s": n_new / min(eager), "ms": 1e3 * min(eager)},
        "recompute_loop": {"tokens_per_s": n_new / recompute[0], "ms": 1e3 * recompute[0],
                           "note": "cache_type none: the reference engine's cache-less loop through the same model"},
        "speedup_over_recompute": recompute[0] / best,
    }
    print(json.dumps(result))
    return 0


def bench_decode(name, args, dev) -> dict:
    """One decode workload: the pa_decode step, its dominant kernel alone, the CPU restatement beside it."""
    from research_amd import _lib, ops
    from research_amd.workloads import make_decode

    t_gen = time.perf_counter()
    w = make_decode(name)
    t_gen = time.perf_counter() - t_gen

    q = w.q.to(dev)
    if w.kv_format == "fp8_e4m3":
        k_pool, k_scale = ops.quantize_kv_e4m3(w.k_pool.to(dev), w.block_size)
        v_pool, v_scale = ops.quantize_kv_e4m3(w.v_pool.to(dev), w.block_size)
    else:
        k_pool, v_pool, k_scale, v_scale = w.k_pool.to(dev), w.v_pool.to(dev), None, None
    tables = torch.from_numpy(w.padded_tables()).to(dev)
    lens = torch.from_numpy(w.seq_lens.astype(np.int32)).to(dev)
    ws = ops.decode_workspace(q, k_pool)
    out = torch.empty_like(q)
    # A workload whose K/V fit several times into HBM but not far beyond the 256 MB last-level cache is rotated
    # over 4 copies of its pools, so that no launch finds the previous launch's lines on chip.
    kv_bytes = 2 * k_pool.numel() * k_pool.element_size()
    n_pools = 4 if kv_bytes < (1 << 30) else 1
    pools = [(k_pool, v_pool)] + [(k_pool.clone(), v_pool.clone()) for _ in range(n_pools - 1)]
    turn = [0]
    # one launch (the split pass merges the pieces itself) or two (split pass, reduction pass)
    passes = int(_lib.load().pa_decode_passes(w.batch, w.num_q_heads, w.num_kv_heads, w.head_dim,
                                              ops.PA_DTYPE[k_pool.dtype]))

    def step(entry="pa_decode"):
        kp, vp = pools[turn[0] % n_pools]
        turn[0] += 1
        ops.decode(q, kp, vp, tables, lens, w.block_size, w.scale, ws, k_scale=k_scale, v_scale=v_scale,
                   out=out, entry=entry)

    if args.copy_calibration:
        calibration_copy(dev)
    preheat(step, args.preheat_s)
    for _ in range(args.warmup):
        step()
    torch.cuda.synchronize()
    wall = time.perf_counter()
    ms_step_mean, ms_step = timed_steps(step, args.steps)
    wall = time.perf_counter() - wall
    n_kernel = max(args.steps, KERNEL_LAUNCHES)
    # the dominant kernel alone: the split pass (with one launch per step it IS the step)
    ms_split = timed_ms(lambda: step("pa_decode" if passes == 1 else "pa_decode_split"), n_kernel)
    ms_reduce = None if passes == 1 else timed_ms(lambda: step("pa_decode_reduce"), n_kernel)

    host_path = None
    if w.kv_format != "fp8_e4m3" and not getattr(args, "secondary_run", False):
        # What a decode call costs through the backend class, host side included, by the form the context's
        # integer fields arrive in: the reference's tuples of tuples (converted block id by block id in Python),
        # padded int32 arrays, or device tensors (used in place).  A new context object per call, as a new step
        # brings; wall time of one call including the wait for the GPU, best of three.
        from research_amd.inference import CacheConfig, HipPagedAttentionBackend, InferenceContext

        be = HipPagedAttentionBackend(CacheConfig(num_layers=1, num_kv_heads=w.num_kv_heads, head_dim=w.head_dim,
                                                  num_blocks=1, block_size=w.block_size, dtype=k_pool.dtype,
                                                  device=str(dev)))
        be.set_num_heads(w.num_q_heads)
        be.config = CacheConfig(num_layers=1, num_kv_heads=w.num_kv_heads, head_dim=w.head_dim,
                                num_blocks=k_pool.shape[0] // w.block_size, block_size=w.block_size,
                                dtype=k_pool.dtype, device=str(dev))
        be.k_cache, be.v_cache = k_pool.unsqueeze(0), v_pool.unsqueeze(0)  # the workload's pools, not a copy
        q4 = q.unsqueeze(1)
        forms = {
            "tuples": lambda: (tuple(tuple(int(x) for x in t) for t in w.block_tables), tuple(int(n) for n in w.seq_lens)),
            "int32_arrays": lambda: (w.padded_tables(), w.seq_lens.astype(np.int32)),
            "device_tensors": lambda: (tables, lens),
        }
        host_path = {"unit": "ms per backend decode call, host and GPU", "kernel_ms": ms_step}
        for form, make in forms.items():
            best = None
            for _ in range(3):
                bt, sl = make()  # the caller's own bookkeeping, outside the timed call
                torch.cuda.synchronize()
                t0 = time.perf_counter()
                be._decode_attention(q4, 0, InferenceContext(is_prefill=False, block_tables=bt, seq_lens=sl,
                                                             max_seq_len=int(w.seq_lens.max())))
                torch.cuda.synchronize()
                dt = (time.perf_counter() - t0) * 1e3
                best = dt if best is None else min(best, dt)
            host_path[form] = best
        del be

    gather = None
    if name in ("c1", "c2") and not getattr(args, "secondary_run", False):
        # the reference's own decode materialises this copy first (_gather_kv_from_cache): the block-table
        # gather into zero-padded [B, max_len, Hkv, D] tensors, bit-exact, bound by HBM
        max_len = int(w.seq_lens.max())
        gk = torch.empty((w.batch, max_len, w.num_kv_heads, w.head_dim), dtype=k_pool.dtype, device=dev)
        gv = torch.empty_like(gk)
        run_gather = lambda: ops.kv_gather(k_pool, v_pool, tables, lens, max_len, w.block_size, out=(gk, gv))
        for _ in range(3):
            run_gather()
        ms_gather = timed_ms(run_gather, args.steps)
        row = w.num_kv_heads * w.head_dim * k_pool.element_size()
        g_bytes = 2 * w.batch * max_len * row + 2 * w.total_tokens * row + 4 * int(sum(len(t) for t in w.block_tables)) + 4 * w.batch
        gather = {"kernel": "kv_gather_kernel", "kernel_ms": ms_gather, "bytes": g_bytes,
                  "achieved": g_bytes / (ms_gather * 1e-3) / 1e9, "unit": "GB/s",
                  "frac": g_bytes / (ms_gather * 1e-3) / 1e9 / HBM_PEAK_GBPS,
                  "note": "written 2*B*max_len rows + read 2*sum(L) rows + tables"}
        del gk, gv

    alg_bytes = w.algorithmic_bytes()
    achieved = alg_bytes / (ms_split * 1e-3) / 1e9
    result = {
        "metric": "decode-attn HBM GB/s",
        "value": alg_bytes / (ms_step * 1e-3) / 1e9,
        "unit": "GB/s",
        "pct_of_hbm_peak": 100.0 * alg_bytes / (ms_step * 1e-3) / 1e9 / HBM_PEAK_GBPS,
        "tokens_per_s": w.batch / (ms_step * 1e-3),
        "n_gpus": 1,
        "steps": args.steps,
        "warmup": args.warmup,
        "preheat_s": args.preheat_s,
        "ms_per_step": ms_step,
        "ms_per_step_mean": ms_step_mean,
        "step_statistic": "median of the timed steps",
        "value_at_mean": alg_bytes / (ms_step_mean * 1e-3) / 1e9,
        "wall_ms_per_step": wall * 1e3 / args.steps,
        "higher_is_better": True,
        "scaling": "weak",
        "vs_baseline": None,
        "dtype": ("fp8-e4m3 KV, bf16 q" if w.kv_format == "fp8_e4m3" else
                  "bf16" if w.dtype == torch.bfloat16 else str(w.dtype).replace("torch.", "")),
        "data": "synthetic",
        "config": {
            "workload": {"c1": "c1 fp32 decode B=4", "c2": "c2 Qwen3-0.6B-shaped decode B=64 bf16",
                         "c4": "c4 Llama-3-8B-shaped decode B=256 bf16 paged KV",
                         "c5": "c5 long-context fp8-e4m3 KV decode B=8"}[name],
            "batch": w.batch, "num_q_heads": w.num_q_heads, "num_kv_heads": w.num_kv_heads,
            "head_dim": w.head_dim, "block_size": w.block_size, "total_keys": w.total_tokens,
            "max_len": int(w.seq_lens.max()), "kv_format": w.kv_format or str(w.dtype).replace("torch.", ""),
            "algorithmic_bytes": alg_bytes, "pool_copies_rotated": n_pools, "launches_per_step": passes,
            "seed": 1000 + int(name[1]), "generate_s": round(t_gen, 1),
        },
        "roofline": {
            "bound": "hbm", "kernel": "decode_split_kernel", "achieved": achieved, "peak": HBM_PEAK_GBPS,
            "unit": "GB/s", "frac": achieved / HBM_PEAK_GBPS, "traffic": measured_traffic(name),
            "kernel_ms": ms_split, "kernel_launches": n_kernel, "reduce_kernel_ms": ms_reduce,
        },
    }
    if gather is not None:
        result["gather"] = gather
    if host_path is not None:
        result["host_path"] = host_path
    if not args.no_cpu_baseline:
        result["cpu_baseline"] = cpu_baseline(w, args.cpu_seconds)
        if name in ("c1", "c2") and args.cpu_seconds > 0 and not getattr(args, "secondary_run", False):
            result["cpu_baseline_literal"] = cpu_literal(w)
    return result


HYBRID_SHAPES = {
    # width, query heads, kv heads, dim, vdim, lightning heads (of 128 x 128), feed-forward, token-side columns
    "w2048": (2048, 16, 4, 128, 128, 16, 5632, 128),
    "w2048-v64": (2048, 16, 4, 128, 64, 16, 5632, 128),
    "w4096": (4096, 32, 8, 128, 128, 32, 14336, 256),
}
HYBRID_LAYERS, HYBRID_WINDOW, HYBRID_VOCAB = 8, 1024, 32000
HYBRID_PREFILL, HYBRID_DECODE = (8, 2048), (128, 2048)  # (sequences, tokens), (sequences, cached tokens)


def hybrid_model(shape, dev, num_blocks, slots, max_positions):
    """A Lotozen-shaped model (window attention and lightning layers in turn) with random weights."""
    from research_amd.inference import HipPagedAttentionBackend, HybridConfig, HybridDecoder
    from research_amd.inference.hybrid import LayerSpec
    from research_amd.inference.mixers import AttentionSpec, LightningSpec

    width, heads, kv, dim, vdim, lheads, ff, side = shape
    att = AttentionSpec(heads=heads, kv_heads=kv, dim=dim, vdim=vdim, scale=dim ** -0.5, window=HYBRID_WINDOW, taps=4,
                        rot_dims=dim // 2, rot_base=10000.0, rot_factor=2.0, v_mix=True)
    lin = LightningSpec(heads=lheads, dim=128, vdim=128, decay=tuple(1.0 - 2.0 ** -(2 + 6 * h / lheads) for h in range(lheads)))
    cfg = HybridConfig(vocab_size=HYBRID_VOCAB, width=width, norm_eps=1e-6, side_dim=side,
                       layers=tuple(LayerSpec(att if i % 2 == 0 else lin, ff) for i in range(HYBRID_LAYERS)))
    backend = HipPagedAttentionBackend(cfg.cache_config(num_blocks, 16, slots, torch.bfloat16, "cuda"))
    model = HybridDecoder(cfg, backend, max_positions)
    with torch.no_grad():
        for p in model.parameters():
            p.normal_(0.0, p.shape[-1] ** -0.5)
    return model.eval()


def llama_model(shape, dev, num_blocks, max_positions):
    """The closest other model at equal size: the same width, heads, feed-forward and layer count."""
    from research_amd.inference import CacheConfig, HipPagedAttentionBackend, ModelConfig, PagedLlama

    width, heads, kv, dim, _, _, ff, _ = shape
    cfg = ModelConfig(vocab_size=HYBRID_VOCAB, hidden_size=width, intermediate_size=ff, num_layers=HYBRID_LAYERS,
                      num_heads=heads, num_kv_heads=kv, head_dim=dim, max_position_embeddings=max_positions)
    backend = HipPagedAttentionBackend(CacheConfig(num_layers=HYBRID_LAYERS, num_kv_heads=kv, head_dim=dim,
                                                   num_blocks=num_blocks, block_size=16, device="cuda",
                                                   dtype=torch.bfloat16))
    with torch.device(dev):
        model = PagedLlama(cfg, backend).to(torch.bfloat16)
    return model.eval()


def hybrid_throughput(model, dev, packed, steps, warmup, preheat_s):
    """Milliseconds of one prefill pass and of one decode step (replayed from a captured graph)."""
    from research_amd.inference import InferenceContext
    from research_amd.inference.engine import _DecodeGraph

    g = np.random.default_rng(3)
    n_seq, n_tok = HYBRID_PREFILL
    per = n_tok // 16
    tables = g.permutation(n_seq * per).reshape(n_seq, per).astype(np.int32)
    pos = np.tile(np.arange(n_tok), (n_seq, 1))
    slots = np.take_along_axis(tables, pos // 16, 1).astype(np.int64) * 16 + pos % 16
    ids = torch.from_numpy(g.integers(0, HYBRID_VOCAB, (n_seq, n_tok))).to(dev)
    lens = np.full(n_seq, n_tok)
    extra = dict(q_lens=lens, state_slots=np.arange(n_seq)) if packed else dict(prefix_lens=np.zeros(n_seq, dtype=np.int64))
    ctx = InferenceContext(is_prefill=True, slot_mapping=slots.reshape(-1), block_tables=tables, seq_lens=lens,
                           max_seq_len=n_tok, **extra)
    tpos = torch.from_numpy(pos).to(dev)
    fn = lambda: model(ids, tpos, ctx)
    out = {}
    with torch.no_grad():
        preheat(fn, preheat_s)
        for _ in range(warmup):
            fn()
        out["prefill_ms"] = timed_steps(fn, steps)[1]
        batch, ctx_len = HYBRID_DECODE
        width = ctx_len // 16 + 1
        graph = _DecodeGraph(model, batch, width, dev)
        tables = g.permutation(batch * width).reshape(batch, width).astype(np.int32)
        args = (g.integers(0, HYBRID_VOCAB, (batch, 1)), np.full(batch, ctx_len),
                tables[:, ctx_len // 16].astype(np.int64) * 16 + ctx_len % 16, tables, np.full(batch, ctx_len + 1))
        graph.run(*args, np.arange(batch, dtype=np.int32) if packed else None)
        fn = graph.graph.replay
        preheat(fn, preheat_s)
        for _ in range(warmup):
            fn()
        out["decode_ms"] = timed_steps(fn, steps)[1]
    out["prefill_tokens_per_s"] = n_seq * n_tok / out["prefill_ms"] * 1e3
    out["decode_tokens_per_s"] = batch / out["decode_ms"] * 1e3
    return out


def kernel_table(steps):
    """A list of kernels with their times and rooflines, and the function that adds one."""
    rows_out = []

    def add(phase, name, fn, like, n_bytes=0.0, flops=0.0):
        # (a graph of several launches: what the host takes to launch a short kernel is not the kernel's time)
        fn()
        torch.cuda.synchronize()
        graph = torch.cuda.CUDAGraph()
        with torch.cuda.graph(graph):
            for _ in range(8):
                fn()
        preheat(graph.replay, 0.05)
        ms = timed_ms(graph.replay, max(1, steps // 4)) / 8
        bound = max(n_bytes / HBM_PEAK_GBPS / 1e6, flops / MFMA_BF16_PEAK_TFLOPS / 1e9)
        rows_out.append({"phase": phase, "kernel": name, "like": like, "us": round(1e3 * ms, 2),
                         "pct_of_roofline": round(100.0 * bound / ms, 1),
                         "bound": "mfma" if flops / MFMA_BF16_PEAK_TFLOPS / 1e9 > n_bytes / HBM_PEAK_GBPS / 1e6 else "hbm"})

    return rows_out, add


def hybrid_kernels(shape, dev, steps):
    """Every kernel of the new blocks alone at the layer's shapes, against its roofline, with the like kernel of the
    Llama block.  Bytes and FLOPs are the algorithmic ones (heads unpadded)."""
    from research_amd import ops

    width, heads, kv, dim, vdim, lheads, ff, side = shape
    bf, f32 = torch.bfloat16, torch.float32
    rnd = lambda *s, dtype=bf: torch.randn(*s, device=dev, dtype=torch.float32).to(dtype)
    i32 = lambda a: torch.as_tensor(np.ascontiguousarray(a), dtype=torch.int32).to(dev)
    rows_out, add = kernel_table(steps)
    d = -(-max(dim, vdim) // 8) * 8
    chans = (heads + kv) * dim + kv * vdim
    for phase, (batch, length) in (("prefill", HYBRID_PREFILL), ("decode", HYBRID_DECODE)):
        dec = phase == "decode"
        n = batch if dec else batch * length
        per = length // 16 + (1 if dec else 0)
        tables = np.random.default_rng(5).permutation(batch * per).reshape(batch, per).astype(np.int32)
        ctx = np.full(batch, length + 1 if dec else length)
        pos = np.full((batch, 1), length) if dec else np.tile(np.arange(length), (batch, 1))
        slots = torch.from_numpy((np.take_along_axis(tables, pos // 16, 1).astype(np.int64) * 16 + pos % 16).reshape(-1)).to(dev)
        bt, lens, sslots = i32(tables), i32(ctx), i32(np.arange(batch))
        if dec:
            por = ops.Portions(lens, sslots)
        else:
            first = np.arange(0, length, ops.QKV_TILE_ROWS)
            tiles = np.stack([np.repeat(np.arange(batch), len(first)), np.tile(first, batch)], 1)
            por = ops.Portions(lens, sslots, i32(ctx), i32(np.arange(batch) * length), i32(tiles), length)
        x, y = rnd(n, width, dtype=f32), rnd(n, width)
        w = rnd(width, dtype=f32)
        add(phase, "residual + layer norm", lambda: ops.residual_norm(x, bf, y=y, norm="layer", weight=w, bias=w, eps=1e-6),
            "rope_kv_append", n * width * 12.0)
        add(phase, "residual + RMS-normed branch + layer norm",
            lambda: ops.residual_norm(x, bf, y=y, y_weight=w, y_eps=1e-6, norm="layer", weight=w, bias=w, eps=1e-6),
            "rope_kv_append", n * width * 12.0)
        u2 = rnd(n, 2 * ff)
        add(phase, "silu(gate) * up", lambda: ops.glu(u2[:, :ff], u2[:, ff:], "silu"), "rope_kv_append", n * ff * 6.0)
        del u2
        sg, st, ids = rnd(n, side), rnd(HYBRID_VOCAB, side * HYBRID_LAYERS), torch.randint(0, HYBRID_VOCAB, (n,), device=dev)
        add(phase, "gelu(gate) * token row", lambda: ops.glu(sg, st[:, side: 2 * side], "gelu_tanh", ids=ids), "rope_kv_append",
            n * (side * 6.0 + 8))
        del x, y, st
        # attention layer
        u = rnd(n, chans + heads)
        total = batch * per * 16
        kc, vc = rnd(total, kv, d), rnd(total, kv, d)
        conv = rnd(4, chans, dtype=f32)
        cstate = torch.zeros(batch, 3, chans, dtype=bf, device=dev)
        rope = rnd(length + 1, dim // 4, 2, dtype=f32)
        vf, lam = rnd(n, kv * vdim), rnd(1, dtype=f32)
        q = torch.empty(n, heads, d, dtype=bf, device=dev)
        conv_bytes = n * 2.0 * (2 * chans + kv * vdim) + (batch * 2.0 * 2 * 3 * chans if dec else 0.0) + chans * 16.0
        add(phase, "conv + rotation + unit norm + append",
            lambda: ops.qkv_conv_append(u, por, slots, kc, vc, heads, dim, vdim, 1.0, 1e-6, True, rope, dim // 2, conv, cstate,
                                        "mix", vf, lam, q_out=q), "rope_kv_append", conv_bytes)
        cos = rnd(length + 1, d)
        k0, v0 = rnd(n, kv, d), rnd(n, kv, d)
        tpos = i32(pos.reshape(-1))
        add(phase, "like: rope_kv_append", lambda: ops.rope_kv_append(q, k0, v0, cos, cos, kc, vc, slots, positions=tpos, q_out=q),
            "", n * 2.0 * d * (2 * heads + 4 * kv))
        o = torch.empty_like(q)
        seen = np.minimum(ctx, HYBRID_WINDOW)
        if dec:
            ws = ops.decode_workspace(q, kc)
            att = lambda win: ops.decode(q, kc, vc, bt, lens, 16, 0.1, ws, out=o, window=win)
            add(phase, "decode attention, window", lambda: att(HYBRID_WINDOW), "decode attention",
                2.0 * kv * (dim + vdim) * float(seen.sum()))
            add(phase, "like: decode attention", lambda: att(0), "", 4.0 * kv * d * float(ctx.sum()))
        else:
            att = lambda win: ops.prefill_paged(q, kc, vc, bt, lens, por.q_lens, por.q_starts, length, 16, 0.1, out=o, window=win)
            vis = np.minimum(np.arange(1, length + 1), HYBRID_WINDOW).sum() * batch
            add(phase, "prefill attention, window", lambda: att(HYBRID_WINDOW), "prefill attention",
                flops=2.0 * (dim + vdim) * heads * float(vis))
            add(phase, "like: prefill attention", lambda: att(0), "",
                flops=4.0 * d * heads * batch * length * (length + 1) / 2.0)
        add(phase, "head gate", lambda: ops.head_gate(o, u[:, chans: chans + heads], vdim), "rope_kv_append",
            n * heads * 2.0 * (2 * vdim + 1))
        del u, kc, vc, q, o, k0, v0, vf
        # lightning layer
        inner = lheads * 128
        u = rnd(n, 4 * inner)
        state = ops.lightning_state(batch, lheads, 128, 128, dev)
        powers = torch.full((lheads, 65), 0.97, device=dev) ** torch.arange(65, device=dev)
        o = torch.empty(n, inner, dtype=bf, device=dev)
        need = 0 if dec else ops.lightning_workspace_bytes(batch, lheads, 128, 128, length)
        ws = torch.empty(max(need, 16), dtype=torch.uint8, device=dev)
        add(phase, "lightning attention", lambda: ops.lightning(u, por, state, powers, lheads, 128, 128, o, workspace=ws),
            "decode attention" if dec else "prefill attention", n * inner * 8.0 + batch * lheads * 128 * 128 * 8.0)
        nw = rnd(inner, dtype=f32)
        add(phase, "RMS norm + sigmoid gate", lambda: ops.rms_gate(o, u[:, 3 * inner:], nw, 1e-6), "rope_kv_append", n * inner * 6.0)
        if not dec:  # one long portion alone, in segments
            por1 = ops.Portions(i32([n]), i32([0]), i32([n]), i32([0]), None, n)
            need = ops.lightning_workspace_bytes(1, lheads, 128, 128, n)
            ws = torch.empty(max(need, 16), dtype=torch.uint8, device=dev)
            add(phase, f"lightning attention, one sequence of {n}",
                lambda: ops.lightning(u, por1, state, powers, lheads, 128, 128, o, workspace=ws), "prefill attention",
                n * inner * 8.0 + lheads * 128 * 128 * 8.0)
        del u, state, o
        torch.cuda.empty_cache()
    return rows_out


def bench_hybrid(args, dev) -> int:
    """Prefill and decode throughput of Lotozen-shaped models with random weights beside Llama-shaped ones of equal
    size, and the new kernels against their rooflines.  Not the headline workload."""
    sizes = {}
    steps, warmup = min(args.steps, 20), min(args.warmup, 3)
    for name, shape in HYBRID_SHAPES.items():
        batch, ctx_len = HYBRID_DECODE
        blocks = batch * (ctx_len // 16 + 1)
        entry = {"shape": dict(zip(("width", "heads", "kv_heads", "dim", "vdim", "lightning_heads", "ff", "side"), shape))}
        model = hybrid_model(shape, dev, blocks, batch, ctx_len + 16)
        entry["lotozen"] = hybrid_throughput(model, dev, True, steps, warmup, args.preheat_s)
        del model
        torch.cuda.empty_cache()
        model = llama_model(shape, dev, blocks, ctx_len + 16)
        entry["llama"] = hybrid_throughput(model, dev, False, steps, warmup, args.preheat_s)
        del model
        torch.cuda.empty_cache()
        entry["kernels"] = hybrid_kernels(shape, dev, steps)
        sizes[name] = entry
        print(f"[{name}] done", file=sys.stderr, flush=True)
    main_size = sizes["w4096"]["lotozen"]
    print(json.dumps({
        "metric": "Lotozen prefill tokens/s", "value": main_size["prefill_tokens_per_s"], "unit": "tokens/s", "n_gpus": 1,
        "steps": steps, "warmup": warmup, "ms_per_step": main_size["prefill_ms"], "higher_is_better": True,
        "scaling": "weak", "vs_baseline": None, "dtype": "bf16", "data": "synthetic",
        "config": {"workload": "lotozen", "layers": HYBRID_LAYERS, "window": HYBRID_WINDOW, "prefill": HYBRID_PREFILL,
                   "decode": HYBRID_DECODE}, "sizes": sizes}))
    return 0


# width; attention query heads, kv heads (of 128 x 128), chunk; mLSTM heads, dim, vdim; Mamba-2 heads, vdim, state, groups;
# experts, chosen, groups, kept, inner width, shared inner width; dense feed-forward of the first layer
TEVIRAX_SHAPES = {
    "w2048": dict(width=2048, heads=16, kv_heads=4, chunk=1024, m_heads=4, m_dim=256, m_vdim=512, s_heads=64, s_vdim=64, s_state=128, s_groups=8,
                  experts=64, top=6, groups=8, keep=4, ff=768, shared=1024, dense=5632),
    "w4096": dict(width=4096, heads=32, kv_heads=8, chunk=1024, m_heads=8, m_dim=256, m_vdim=512, s_heads=128, s_vdim=64, s_state=128, s_groups=8,
                  experts=64, top=8, groups=8, keep=4, ff=1408, shared=2816, dense=14336),
}


def tevirax_model(p, dev, num_blocks, slots, max_positions):
    """Mamba-2 layers with a parallel layer (chunk attention and matrix memory) in every fourth place, a dense feed-forward in
    the first layer and experts in the others; random weights."""
    from research_amd.inference import HipPagedAttentionBackend, HybridConfig, HybridDecoder
    from research_amd.inference.hybrid import LayerSpec
    from research_amd.inference.mixers import AttentionSpec, Mamba2Mixer, Mamba2Spec, MlstmMixer, MlstmSpec, ParallelSpec, YarnScaling
    from research_amd.inference.moe import MoESpec

    att = AttentionSpec(heads=p["heads"], kv_heads=p["kv_heads"], dim=128, vdim=128, scale=128 ** -0.5, window=None, taps=0, rot_dims=128,
                        rot_base=500000.0, chunk=p["chunk"], rot_yarn=YarnScaling(4.0, 8192, 32.0, 1.0), rot_halves=True, qk_weights=True, gates=False)
    par = ParallelSpec(att, MlstmSpec(p["m_heads"], p["m_dim"], p["m_vdim"], 15.0), 1.0, 1.0)
    ssd = Mamba2Spec(p["s_heads"], p["s_vdim"], p["s_state"], p["s_groups"], 4, p["s_groups"])
    moe = MoESpec(p["experts"], p["ff"], p["top"], p["groups"], p["keep"], p["shared"])
    cfg = HybridConfig(vocab_size=HYBRID_VOCAB, width=p["width"], norm_eps=1e-6, norm="rms", post_norm=True, embed_scale=p["width"] ** 0.5,
                       positions=max_positions, logit_softcap=30.0,
                       layers=tuple(LayerSpec(par if i % 4 == 3 else ssd, moe if i else p["dense"]) for i in range(HYBRID_LAYERS)))
    backend = HipPagedAttentionBackend(cfg.cache_config(num_blocks, 16, slots, torch.bfloat16, "cuda"))
    model = HybridDecoder(cfg, backend, max_positions)
    with torch.no_grad():
        for q in model.parameters():
            q.normal_(0.0, q.shape[-1] ** -0.5)
        for m in model.modules():
            if isinstance(m, Mamba2Mixer):
                m.rate.uniform_(1.0, 16.0)
                m.dt_bias.fill_(-4.0)
            if isinstance(m, MlstmMixer):
                m.f_bias.fill_(4.0)
    return model.eval()


def tevirax_kernels(p, dev, steps):
    """Every kernel of the design's blocks at the layer's shapes, against its roofline, with the like kernel of the Lotozen or
    Llama block.  Bytes and FLOPs are the algorithmic ones."""
    import torch.nn.functional as F
    from research_amd import ops

    bf, f32 = torch.bfloat16, torch.float32
    rnd = lambda *s, dtype=bf: torch.randn(*s, device=dev, dtype=torch.float32).to(dtype)
    i32 = lambda a: torch.as_tensor(np.ascontiguousarray(a), dtype=torch.int32).to(dev)
    rows_out, add = kernel_table(steps)
    width, heads, kv, d = p["width"], p["heads"], p["kv_heads"], 128
    for phase, (batch, length) in (("prefill", HYBRID_PREFILL), ("decode", HYBRID_DECODE)):
        dec = phase == "decode"
        n = batch if dec else batch * length
        per = length // 16 + (1 if dec else 0)
        tables = np.random.default_rng(5).permutation(batch * per).reshape(batch, per).astype(np.int32)
        ctx = np.full(batch, length + 1 if dec else length)
        pos = np.full((batch, 1), length) if dec else np.tile(np.arange(length), (batch, 1))
        slots = torch.from_numpy((np.take_along_axis(tables, pos // 16, 1).astype(np.int64) * 16 + pos % 16).reshape(-1)).to(dev)
        bt, lens, sslots = i32(tables), i32(ctx), i32(np.arange(batch))
        if dec:
            por = ops.Portions(lens, sslots)
        else:
            first = np.arange(0, length, ops.QKV_TILE_ROWS)
            tiles = np.stack([np.repeat(np.arange(batch), len(first)), np.tile(first, batch)], 1)
            por = ops.Portions(lens, sslots, i32(ctx), i32(np.arange(batch) * length), i32(tiles), length)
        x, y, w = rnd(n, width, dtype=f32), rnd(n, width), rnd(width, dtype=f32)
        add(phase, "residual + RMS-normed branch", lambda: ops.residual_norm(x, bf, y=y, y_weight=w, y_eps=1e-6), "residual + layer norm", n * width * 12.0)
        add(phase, "like: residual + layer norm", lambda: ops.residual_norm(x, bf, y=y, norm="layer", weight=w, bias=w, eps=1e-6), "", n * width * 12.0)
        # experts
        e, top, ff, inner = p["experts"], p["top"], p["ff"], -(-p["ff"] // 64) * 64
        h, router = rnd(n, width), rnd(e + 1, width)
        router *= width ** -0.5
        add(phase, "router logits", lambda: ops.narrow_linear(h, router), "bf16 product of equal size", (n * width + e * width) * 2.0 + n * (e + 1) * 4.0,
            2.0 * n * width * (e + 1))
        add(phase, "like: bf16 product of equal size", lambda: F.linear(h, router), "", (n * width + e * width) * 2.0 + n * (e + 1) * 2.0, 2.0 * n * width * (e + 1))
        logits = ops.narrow_linear(h, router)
        choice = ops.moe_choose(logits, e, top, p["groups"], p["keep"], "gated" if logits.shape[1] > e else None)
        add(phase, "choice of experts and lists", lambda: ops.moe_choose(logits, e, top, p["groups"], p["keep"], "gated" if logits.shape[1] > e else None), "silu(gate) * up",
            n * (e + 1) * 4.0 + n * top * 20.0)
        w_in, w_out = rnd(e, 2 * inner, width), rnd(e, width, inner)
        act, items = rnd(n * top, inner), n * top
        used = int((choice.counts > 0).sum())
        add(phase, "experts: gate, up, silu", lambda: ops.moe_product(h, choice, w_in, inner, width, True), "dense product of equal flops",
            used * 2.0 * inner * width * 2 + n * width * 2.0 + items * inner * 2.0, 4.0 * items * inner * width)
        add(phase, "experts: down", lambda: ops.moe_product(act, choice, w_out, width, inner, False), "dense product of equal flops",
            used * 2.0 * inner * width + items * (inner + width) * 2.0, 2.0 * items * inner * width)
        if not dec:
            dw, dw2 = rnd(2 * top * inner, width), rnd(width, top * inner)
            dact = rnd(n, top * inner)
            add(phase, "like: dense gate and up of equal flops", lambda: F.linear(h, dw), "", 0.0, 4.0 * items * inner * width)
            add(phase, "like: dense down of equal flops", lambda: F.linear(dact, dw2), "", 0.0, 2.0 * items * inner * width)
            del dw, dw2, dact
        else:  # (the same bytes of weights)
            dw, dw2 = rnd(used * 2 * inner, width), rnd(used * width, inner)
            dh = rnd(n * top // used or 1, inner)
            add(phase, "like: dense gate and up of equal bytes", lambda: F.linear(h[: n * top // used or 1], dw), "", used * 2.0 * inner * width * 2)
            add(phase, "like: dense down of equal bytes", lambda: F.linear(dh, dw2), "", used * 2.0 * inner * width)
            del dw, dw2, dh
        del w_in, w_out, act
        eo, shared = rnd(items, width), rnd(n, width)
        add(phase, "residual + RMS-normed sum over experts",
            lambda: ops.residual_norm(x, bf, y=eo, mix=choice.weights, y_extra=shared, y_weight=w, y_eps=1e-6), "residual + layer norm",
            n * width * (10.0 + 2.0 * (top + 1)))
        del eo, shared, x, y
        # attention
        u = rnd(n, (heads + 2 * kv) * d)
        kc, vc = rnd(batch * per * 16, kv, d), rnd(batch * per * 16, kv, d)
        rope, qn = rnd(length + 1, d // 2, 2, dtype=f32), rnd(d, dtype=f32)
        q = torch.empty(n, heads, d, dtype=bf, device=dev)
        add(phase, "q/k norm + rotation + append", lambda: ops.qkv_conv_append(u, por, slots, kc, vc, heads, d, d, 1.0, 1e-6, False, rope, d, None, None,
                                                                               q_out=q, q_norm=qn, k_norm=qn), "rope_kv_append", n * 4.0 * d * (heads + 2 * kv))
        cos, k0, v0, tpos = rnd(length + 1, d), rnd(n, kv, d), rnd(n, kv, d), i32(pos.reshape(-1))
        add(phase, "like: rope_kv_append", lambda: ops.rope_kv_append(q, k0, v0, cos, cos, kc, vc, slots, positions=tpos, q_out=q), "",
            n * 2.0 * d * (2 * heads + 4 * kv))
        o = torch.empty_like(q)
        if dec:
            ws = ops.decode_workspace(q, kc)
            half = i32(np.full(batch, length - p["chunk"] // 2))  # (half a chunk is visible)
            att = lambda win, ln: ops.decode(q, kc, vc, bt, ln, 16, 0.1, ws, out=o, window=win)
            add(phase, "decode attention, half a chunk", lambda: att(-p["chunk"], half), "decode attention, window", 4.0 * kv * d * batch * p["chunk"] / 2)
            add(phase, "like: decode attention, window", lambda: att(p["chunk"] // 2, lens), "", 4.0 * kv * d * batch * p["chunk"] / 2)
        else:
            att = lambda win: ops.prefill_paged(q, kc, vc, bt, lens, por.q_lens, por.q_starts, length, 16, 0.1, out=o, window=win)
            i = np.arange(length)
            add(phase, "prefill attention, chunks", lambda: att(-p["chunk"]), "prefill attention, window", flops=4.0 * d * heads * batch * float((i % p["chunk"] + 1).sum()))
            add(phase, "like: prefill attention, window", lambda: att(p["chunk"]), "",
                flops=4.0 * d * heads * batch * float(np.minimum(i + 1, p["chunk"]).sum()))
        joint = torch.empty(n, heads * d + p["m_heads"] * p["m_vdim"], dtype=bf, device=dev)
        add(phase, "head packing", lambda: ops.head_gate(o, None, d, 1.2, joint[:, : heads * d]), "silu(gate) * up", n * heads * d * 4.0)
        del u, kc, vc, q, o, k0, v0
        # recurrences
        shapes = {"matrix memory": ("mlstm", p["m_heads"], p["m_dim"], p["m_vdim"], p["m_heads"]),
                  "state space": ("ssd", p["s_heads"], p["s_state"], p["s_vdim"], p["s_groups"])}
        for name, (kind, hs, dim, vdim, groups) in shapes.items():
            qk = groups * dim
            u = rnd(n, 2 * qk + hs * vdim + 2 * hs)
            uq, uk, uv, ga, gb = u.split([qk, qk, hs * vdim, hs, hs], 1)
            state = torch.zeros(batch, hs, ops.gated_linear_state_floats(kind, dim, vdim), device=dev)
            out = torch.empty(n, hs * vdim, dtype=bf, device=dev)
            const = (torch.full((hs,), -4.0, device=dev), torch.full((hs,), 4.0, device=dev), torch.ones(hs, device=dev) if kind == "ssd" else None)
            need = 0 if dec else ops.gated_linear_workspace_bytes(batch, hs, dim, vdim, length)
            ws = torch.empty(max(need, 16), dtype=torch.uint8, device=dev)
            run = lambda por, ws: ops.gated_linear(kind, uq, uk, uv, (ga, gb if kind == "mlstm" else None), const, por, state, hs, dim, vdim, out,
                                                   heads_per_group=hs // groups, cap=15.0, q_scale=dim ** -0.5, den_eps=1e-6, workspace=ws)
            n_bytes = n * 2.0 * (2 * qk + 2 * hs * vdim + 2 * hs) + (batch * state[0].numel() * 8.0 if dec else 0.0)
            chunked = n * hs * (4.0 * dim * vdim + 64.0 * (dim + vdim))  # the products of 64-row chunks, one bf16 term each
            add(phase, name, lambda: run(por, ws), "lightning attention", n_bytes, 0.0 if dec else chunked)
            if not dec:
                por1 = ops.Portions(i32([n]), i32([0]), i32([n]), i32([0]), None, n)
                need = ops.gated_linear_workspace_bytes(1, hs, dim, vdim, n)
                ws1 = torch.empty(max(need, 16), dtype=torch.uint8, device=dev)
                add(phase, f"{name}, one sequence of {n}", lambda: run(por1, ws1), "lightning attention, one sequence", n_bytes, chunked)
            nw, z = rnd(hs * vdim, dtype=f32), rnd(n, hs * vdim)
            if kind == "mlstm":
                add(phase, "RMS norm per head + sigmoid gate", lambda: ops.rms_gate(out, z, nw, 1e-6, groups=hs, out=joint[:, heads * d:]), "RMS norm + sigmoid gate",
                    n * hs * vdim * 6.0)
            else:
                add(phase, "silu gate + RMS norm of groups", lambda: ops.rms_gate(out, z, nw, 1e-6, groups=groups, order="silu_first"), "RMS norm + sigmoid gate",
                    n * hs * vdim * 6.0)
                add(phase, "like: RMS norm + sigmoid gate", lambda: ops.rms_gate(out, z, nw, 1e-6), "", n * hs * vdim * 6.0)
                ch = hs * vdim + 2 * qk
                cu, cw, cb = rnd(n, ch), rnd(4, ch, dtype=f32), rnd(ch, dtype=f32)
                cs = torch.zeros(batch, 3, ch, dtype=bf, device=dev)
                add(phase, "short convolution", lambda: ops.short_conv(cu, por, cw, cb, cs, "silu"), "rope_kv_append",
                    n * ch * 4.0 + (batch * 12.0 * ch if dec else 0.0) + ch * 20.0)
                del cu
            del u, state, out, z
        lheads = width // 128
        u = rnd(n, 4 * width)
        state = ops.lightning_state(batch, lheads, 128, 128, dev)
        powers = torch.full((lheads, 65), 0.97, device=dev) ** torch.arange(65, device=dev)
        o = torch.empty(n, width, dtype=bf, device=dev)
        need = 0 if dec else ops.lightning_workspace_bytes(batch, lheads, 128, 128, length)
        ws = torch.empty(max(need, 16), dtype=torch.uint8, device=dev)
        n_bytes, chunked = n * width * 8.0 + (batch * lheads * 128 * 128 * 8.0 if dec else 0.0), n * lheads * (4.0 * 128 * 128 + 64.0 * 256)
        add(phase, "like: lightning attention", lambda: ops.lightning(u, por, state, powers, lheads, 128, 128, o, workspace=ws), "", n_bytes, 0.0 if dec else chunked)
        if not dec:
            need = ops.lightning_workspace_bytes(1, lheads, 128, 128, n)
            ws1 = torch.empty(max(need, 16), dtype=torch.uint8, device=dev)
            add(phase, "like: lightning attention, one sequence", lambda: ops.lightning(u, por1, state, powers, lheads, 128, 128, o, workspace=ws1), "", n_bytes, chunked)
        add(phase, "like: silu(gate) * up", lambda: ops.glu(u[:, :width], u[:, width: 2 * width], "silu"), "", n * width * 6.0)
        del u, state, o, joint
        if dec:
            lg = rnd(n, HYBRID_VOCAB)
            add(phase, "capped logits", lambda: ops.softcap(lg, 30.0), "silu(gate) * up", n * HYBRID_VOCAB * 6.0)
        torch.cuda.empty_cache()
    return rows_out


def bench_tevirax(args, dev) -> int:
    """Prefill and decode throughput of Tevirax-shaped models with random weights beside Lotozen-shaped ones of the same width,
    heads, depth and feed-forward work per token, and the design's kernels against their rooflines.  Not the headline
    workload."""
    sizes = {}
    steps, warmup = min(args.steps, 20), min(args.warmup, 3)
    for name, p in TEVIRAX_SHAPES.items():
        batch, ctx_len = HYBRID_DECODE
        blocks = batch * (ctx_len // 16 + 1)
        model = tevirax_model(p, dev, blocks, batch, ctx_len + 16)
        entry = {"shape": p, "tevirax": hybrid_throughput(model, dev, True, steps, warmup, args.preheat_s)}
        del model
        torch.cuda.empty_cache()
        shape = (p["width"], p["heads"], p["kv_heads"], 128, 128, p["width"] // 128, p["top"] * p["ff"] + p["shared"], 128)
        model = hybrid_model(shape, dev, blocks, batch, ctx_len + 16)
        entry["lotozen"] = hybrid_throughput(model, dev, True, steps, warmup, args.preheat_s)
        del model
        torch.cuda.empty_cache()
        entry["kernels"] = tevirax_kernels(p, dev, steps)
        sizes[name] = entry
        print(f"[{name}] done", file=sys.stderr, flush=True)
    main_size = sizes["w4096"]["tevirax"]
    print(json.dumps({
        "metric": "Tevirax prefill tokens/s", "value": main_size["prefill_tokens_per_s"], "unit": "tokens/s", "n_gpus": 1,
        "steps": steps, "warmup": warmup, "ms_per_step": main_size["prefill_ms"], "higher_is_better": True,
        "scaling": "weak", "vs_baseline": None, "dtype": "bf16", "data": "synthetic",
        "config": {"workload": "tevirax", "layers": HYBRID_LAYERS, "prefill": HYBRID_PREFILL, "decode": HYBRID_DECODE}, "sizes": sizes}))
    return 0


# width; streams; attention query heads, kv heads (of 128 x 128), distance buckets, last distance; latent heads (128 + 64 rotated, values of
# 128), rank; window of both; delta value heads, q/k heads (of 128); experts, identity experts, chosen, groups, kept, inner
# width, shared inner width
VUSALIX_SHAPES = {
    "w2048": dict(width=2048, streams=4, heads=16, kv_heads=4, buckets=32, bias_max=128, l_heads=16, rank=512, window=1024, d_heads=16, d_groups=8,
                  experts=64, identity=8, top=6, groups=8, keep=4, ff=768, shared=1024),
    "w4096": dict(width=4096, streams=4, heads=32, kv_heads=8, buckets=32, bias_max=128, l_heads=32, rank=512, window=1024, d_heads=32, d_groups=16,
                  experts=64, identity=8, top=8, groups=8, keep=4, ff=1408, shared=2816),
}


def vusalix_model(p, dev, num_blocks, slots, max_positions):
    """Two delta layers, a latent-attention layer and a biased-attention layer in turn, experts in every layer; random weights."""
    from research_amd.inference import HipPagedAttentionBackend, HybridConfig, HybridDecoder
    from research_amd.inference.hybrid import LayerSpec, _Streams
    from research_amd.inference.mixers import BiasedAttention, BiasedAttentionSpec, DeltaMixer, DeltaSpec, LatentAttention, LatentSpec, YarnScaling
    from research_amd.inference.moe import MoE, MoESpec

    delta = DeltaSpec(p["d_heads"], p["d_groups"], 128, 128, 4)
    latent = LatentSpec(p["l_heads"], 128, 64, 128, p["rank"], 192 ** -0.5, p["window"], 10000.0, YarnScaling(4.0, 8192, 32.0, 1.0))
    att = BiasedAttentionSpec(p["heads"], p["kv_heads"], 128, 128, 128 ** -0.5, p["window"], 30.0, p["buckets"], p["bias_max"])
    moe = MoESpec(p["experts"], p["ff"], p["top"], p["groups"], p["keep"], p["shared"], shared_gate=False, identity=p["identity"], scores="softmax",
                  group_top=1, correction=True, renormalize=False)
    cfg = HybridConfig(vocab_size=HYBRID_VOCAB, width=p["width"], norm_eps=1e-6, norm="rms", streams=p["streams"],
                       layers=tuple(LayerSpec((delta, delta, latent, att)[i % 4], moe) for i in range(HYBRID_LAYERS)))
    backend = HipPagedAttentionBackend(cfg.cache_config(num_blocks, 16, slots, torch.bfloat16, "cuda"))
    model = HybridDecoder(cfg, backend, max_positions)
    with torch.no_grad():
        for q in model.parameters():
            q.normal_(0.0, q.shape[-1] ** -0.5)
        for m in model.modules():
            if isinstance(m, DeltaMixer):
                m.rate.uniform_(1.0, 16.0)
                m.dt_bias.fill_(-4.0)
            if isinstance(m, LatentAttention):  # (the rotated part passes through)
                m.k_made[:, 128:].zero_()
                m.k_made[:, 128:, p["rank"]:] = torch.eye(64)
            if isinstance(m, _Streams):
                m.between.copy_(torch.eye(p["streams"]))
            if isinstance(m, MoE):
                m.correction.normal_(0.0, 0.01)
    return model.eval()


def vusalix_kernels(p, dev, steps):
    """Every kernel of the design's blocks at the layer's shapes, against its roofline, with the like kernel of the Tevirax
    block.  Bytes and FLOPs are the algorithmic ones (heads unpadded)."""
    import torch.nn.functional as F
    from research_amd import ops

    bf, f32 = torch.bfloat16, torch.float32
    rnd = lambda *s, dtype=bf: torch.randn(*s, device=dev, dtype=torch.float32).to(dtype)
    i32 = lambda a: torch.as_tensor(np.ascontiguousarray(a), dtype=torch.int32).to(dev)
    rows_out, add = kernel_table(steps)
    width, streams, window, d = p["width"], p["streams"], p["window"], 128
    for phase, (batch, length) in (("prefill", HYBRID_PREFILL), ("decode", HYBRID_DECODE)):
        dec = phase == "decode"
        n = batch if dec else batch * length
        per = length // 16 + (1 if dec else 0)
        tables = np.random.default_rng(5).permutation(batch * per).reshape(batch, per).astype(np.int32)
        ctx = np.full(batch, length + 1 if dec else length)
        pos = np.full((batch, 1), length) if dec else np.tile(np.arange(length), (batch, 1))
        slots = torch.from_numpy((np.take_along_axis(tables, pos // 16, 1).astype(np.int64) * 16 + pos % 16).reshape(-1)).to(dev)
        bt, lens, sslots = i32(tables), i32(ctx), i32(np.arange(batch))
        if dec:
            por = ops.Portions(lens, sslots)
        else:
            first = np.arange(0, length, ops.QKV_TILE_ROWS)
            tiles = np.stack([np.repeat(np.arange(batch), len(first)), np.tile(first, batch)], 1)
            por = ops.Portions(lens, sslots, i32(ctx), i32(np.arange(batch) * length), i32(tiles), length)
        seen = np.minimum(np.full(batch, length + 1) if dec else np.tile(np.arange(1, length + 1), batch), window).astype(float).sum()
        # streams
        x, y, w = rnd(n, streams, width, dtype=f32), rnd(n, width), rnd(width, dtype=f32)
        hc = dict(between=torch.eye(streams, device=dev), into=rnd(streams, dtype=f32), sum_weight=rnd(streams, dtype=f32), weight=w, eps=1e-6)
        add(phase, "streams mixed, summed, normed", lambda: ops.hyper_norm(x, bf, y=y, **hc), "residual + RMS-normed branch", n * width * (8.0 * streams + 4))
        x1 = rnd(n, width, dtype=f32)
        add(phase, "like: residual + RMS-normed branch", lambda: ops.residual_norm(x1, bf, y=y, y_weight=w, y_eps=1e-6), "", n * width * 12.0)
        # experts
        e, top, ident = p["experts"], p["top"], p["identity"]
        h, router, corr = rnd(n, width), rnd(e + ident, width), rnd(e + ident, dtype=f32)
        router *= width ** -0.5
        corr *= 0.01
        logits = ops.narrow_linear(h, router)
        add(phase, "router logits", lambda: ops.narrow_linear(h, router), "router logits (65 columns)", (n * width + (e + ident) * width) * 2.0 + n * (e + ident) * 4.0)
        r65 = router[: e + 1].contiguous()
        add(phase, "like: router logits (65 columns)", lambda: ops.narrow_linear(h, r65), "", (n * width + (e + 1) * width) * 2.0 + n * (e + 1) * 4.0)
        pick = lambda: ops.moe_choose(logits, e, top, p["groups"], p["keep"], "plain", ident, "softmax", 1, False, corr)
        add(phase, "choice of experts and lists", pick, "choice by sigmoid scores", n * (e + ident) * 4.0 + n * top * 20.0)
        l65 = logits[:, : e + 1].contiguous()
        add(phase, "like: choice by sigmoid scores", lambda: ops.moe_choose(l65, e, top, p["groups"], p["keep"], "gated"), "", n * (e + 1) * 4.0 + n * top * 20.0)
        choice = pick()
        eo, shared = rnd(n * top, width), rnd(n, width)
        add(phase, "streams + sum over experts", lambda: ops.hyper_norm(x, bf, y=eo, mix=choice.weights, y_extra=shared, y_self=h, **hc),
            "residual + RMS-normed sum over experts", n * width * (8.0 * streams + 2) + (float((choice.weights[:, :top] != 0).sum()) + 2 * n) * width * 2.0)
        mix65 = choice.weights[:, : top + 1].contiguous()
        add(phase, "like: residual + RMS-normed sum over experts", lambda: ops.residual_norm(x1, bf, y=eo, mix=mix65, y_extra=shared, y_weight=w, y_eps=1e-6), "",
            n * width * (10.0 + 2.0 * (top + 1)))
        del eo, shared, x, x1, y
        # attention with distance biases
        heads, kv = p["heads"], p["kv_heads"]
        u = rnd(n, (heads + 2 * kv) * d)
        kc, vc = rnd(batch * per * 16, kv, d), rnd(batch * per * 16, kv, d)
        rope = rnd(length + 1, d // 2, 2, dtype=f32)
        app = lambda rp, rot, norm: ops.qkv_conv_append(u, por, slots, kc, vc, heads, d, d, 1.0, 1e-6, False, rp, rot, None, None, q_norm=norm, k_norm=norm)
        qn = rnd(d, dtype=f32)
        add(phase, "append", lambda: app(None, 0, None), "q/k norm + rotation + append", n * 4.0 * d * (heads + 2 * kv))
        add(phase, "like: q/k norm + rotation + append", lambda: app(rope, d, qn), "", n * 4.0 * d * (heads + 2 * kv))
        q, o = app(None, 0, None), torch.empty(n, heads, d, dtype=bf, device=dev)
        bias, sink = rnd(heads, p["bias_max"] + 1, dtype=f32), rnd(heads, dtype=f32)
        terms = dict(softcap=30.0, bias=bias, sink=sink)
        need = ops.scored_workspace_bytes(batch, heads, kv, d, d, False, per * 16, window) if dec else 0
        ws = torch.empty(max(need, 16), dtype=torch.uint8, device=dev)
        scored = lambda **kw: ops.scored_attention((q,), kc, vc, d, por, bt, 16, d ** -0.5, window, o, workspace=ws, **kw)
        if dec:
            add(phase, "decode attention, cap, biases, sinks", lambda: scored(**terms), "decode attention, window", 4.0 * kv * d * seen)
            dws = ops.decode_workspace(q, kc)
            add(phase, "like: decode attention, window", lambda: ops.decode(q, kc, vc, bt, lens, 16, 0.1, dws, out=o, window=window), "", 4.0 * kv * d * seen)
        else:
            add(phase, "prefill attention, cap, biases, sinks", lambda: scored(**terms), "prefill attention, window", flops=4.0 * d * heads * seen)
            add(phase, "(the same without a cap)", lambda: scored(bias=bias, sink=sink), "prefill attention, window", flops=4.0 * d * heads * seen)
            add(phase, "like: prefill attention, window",
                lambda: ops.prefill_paged(q, kc, vc, bt, lens, por.q_lens, por.q_starts, length, 16, 0.1, out=o, window=window), "", flops=4.0 * d * heads * seen)
        del u, kc, vc, q, o
        # latent attention
        lh, rank, rot = p["l_heads"], p["rank"], 64
        row, size = rank + rot, d + rot
        u, pool, norm = rnd(n, lh * size + row), rnd(batch * per * 16, 1, row), rnd(rank, dtype=f32)
        rope = rnd(length + 1, rot // 2, 2, dtype=f32)
        app = lambda: ops.latent_append(u, por, slots, pool, norm, 1e-6, rope, lh, d, rot, rank, size, 0.1)
        add(phase, "latent norm + rotation + append", app, "q/k norm + rotation + append", n * 4.0 * (lh * size + row))
        q = app()
        if dec:
            over, o = rnd(n, lh, rank), torch.empty(n, lh, rank, dtype=bf, device=dev)
            need = ops.scored_workspace_bytes(batch, lh, 1, row, rank, True, per * 16, window)
            ws = torch.empty(max(need, 16), dtype=torch.uint8, device=dev)
            add(phase, "decode attention over latents", lambda: ops.scored_attention((over, q[..., d:]), pool, pool, rank, por, bt, 16, 0.1, window, o, workspace=ws),
                "decode attention, window", 2.0 * row * seen, 2.0 * (row + rank) * lh * seen)
            lists = (torch.arange(n, dtype=torch.int32, device=dev)[None] * lh + torch.arange(lh, dtype=torch.int32, device=dev)[:, None]).contiguous()
            every = ops.ExpertChoice(lists.view(n, lh), torch.empty(0, device=dev), torch.full((lh,), n, dtype=torch.int32, device=dev), lists)
            wk, wv = rnd(lh, rank, d), rnd(lh, d, rank)
            q2 = q.view(n * lh, size)[:, :d]
            add(phase, "product per head, keys' side", lambda: ops.moe_product(q2, every, wk, rank, d, False), "experts: down of equal flops",
                lh * (rank * d * 2.0 + n * 2.0 * (rank + d)), 2.0 * n * lh * rank * d)
            add(phase, "product per head, values' side", lambda: ops.moe_product(o.view(n * lh, rank), every, wv, d, rank, False), "experts: down of equal flops",
                lh * (rank * d * 2.0 + n * 2.0 * (rank + d)), 2.0 * n * lh * rank * d)
            dw, dx = rnd(lh * d, rank), rnd(n, rank)
            add(phase, "like: dense product of equal flops", lambda: F.linear(dx, dw), "", lh * rank * d * 2.0 + n * 2.0 * (rank + lh * d), 2.0 * n * lh * rank * d)
            del over, o, wk, wv
        else:
            add(phase, "latent rows gathered", lambda: ops.latent_gather(pool, slots), "rope_kv_append", n * row * 4.0)
            wk, wv = rnd(lh * size, row), rnd(lh * d, row)
            lat = ops.latent_gather(pool, slots)
            add(phase, "keys made again (library product)", lambda: F.linear(lat, wk), "dense product of equal flops", flops=2.0 * n * lh * d * rank)
            add(phase, "values made again (library product)", lambda: F.linear(lat, wv), "dense product of equal flops", flops=2.0 * n * lh * d * rank)
            k, v = (F.linear(lat, w).view(n, lh, -1) for w in (wk, wv))
            at = i32(np.arange(n // 16).reshape(batch, -1))
            o = torch.empty(n, lh, d, dtype=bf, device=dev)
            made = ops.Portions(lens, lens, por.q_lens, por.q_starts, None, length)
            add(phase, "prefill attention over made keys", lambda: ops.scored_attention((q,), k, v, d, made, at, 16, 0.1, window, o), "prefill attention, window",
                flops=2.0 * (size + d) * lh * seen)
            del k, v, o, lat
        del u, pool, q
        # delta rule
        hs, groups = p["d_heads"], p["d_groups"]
        qk, inner = groups * d, hs * d
        u = rnd(n, 2 * qk + inner + 2 * hs)
        uq, uk, uv, ga, gb = u.split([qk, qk, inner, hs, hs], 1)
        state, out = torch.zeros(batch, hs, d, d, device=dev), torch.empty(n, inner, dtype=bf, device=dev)
        bias, rate = torch.full((hs,), -4.0, device=dev), torch.full((hs,), 4.0, device=dev)

        def run(por, ws):
            return ops.delta_rule(uq, uk, uv, ga, gb, bias, rate, por, state, hs, d, d, d ** -0.5, out, heads_per_group=hs // groups, workspace=ws)
        need = 0 if dec else ops.delta_workspace_bytes(batch, hs, d, d, length)
        ws = torch.empty(max(need, 16), dtype=torch.uint8, device=dev)
        n_bytes = n * 2.0 * (2 * qk + 2 * inner + 2 * hs) + (batch * state[0].numel() * 8.0 if dec else 0.0)
        # (per row and head: K K^T, Q K^T, T R, C U over 64 columns, half of them; K S, Q S, K^T U; one bf16 term each)
        chunked = n * hs * (6.0 * d * d + 128.0 * 2 * d)
        add(phase, "delta rule", lambda: run(por, ws), "state space", n_bytes, 0.0 if dec else chunked)
        gstate = torch.zeros(batch, hs, ops.gated_linear_state_floats("ssd", d, d), device=dev)
        need = 0 if dec else ops.gated_linear_workspace_bytes(batch, hs, d, d, length)
        gws = torch.empty(max(need, 16), dtype=torch.uint8, device=dev)
        ssd = lambda por, gws: ops.gated_linear("ssd", uq, uk, uv, (ga, None), (bias, rate, rate), por, gstate, hs, d, d, out, heads_per_group=hs // groups, workspace=gws)
        add(phase, "like: state space", lambda: ssd(por, gws), "", n_bytes, 0.0 if dec else n * hs * (4.0 * d * d + 64.0 * 2 * d))
        if not dec:
            por1 = ops.Portions(i32([n]), i32([0]), i32([n]), i32([0]), None, n)
            ws1 = torch.empty(ops.delta_workspace_bytes(1, hs, d, d, n), dtype=torch.uint8, device=dev)
            add(phase, f"delta rule, one sequence of {n}", lambda: run(por1, ws1), "state space, one sequence", n_bytes, chunked)
            gws1 = torch.empty(max(ops.gated_linear_workspace_bytes(1, hs, d, d, n), 16), dtype=torch.uint8, device=dev)
            add(phase, "like: state space, one sequence", lambda: ssd(por1, gws1), "", n_bytes, n * hs * (4.0 * d * d + 64.0 * 2 * d))
        nw, z = rnd(inner, dtype=f32), rnd(n, inner)
        add(phase, "RMS norm per head + silu gate", lambda: ops.rms_gate(out, z, nw, 1e-6, groups=hs, order="silu_last"), "RMS norm per head + sigmoid gate", n * inner * 6.0)
        add(phase, "like: RMS norm per head + sigmoid gate", lambda: ops.rms_gate(out, z, nw, 1e-6, groups=hs), "", n * inner * 6.0)
        ch = 2 * qk + inner
        cw, cs = rnd(4, ch, dtype=f32), torch.zeros(batch, 3, ch, dtype=bf, device=dev)
        add(phase, "short convolution", lambda: ops.short_conv(u[:, :ch], por, cw, None, cs, "silu"), "short convolution (the same kernel)",
            n * ch * 4.0 + (batch * 12.0 * ch if dec else 0.0) + ch * 16.0)
        del u, state, gstate, out, z
        torch.cuda.empty_cache()
    return rows_out


def bench_vusalix(args, dev) -> int:
    """Prefill and decode throughput of Vusalix-shaped models with random weights beside Tevirax-shaped ones of the same width,
    heads, depth and experts, and the design's kernels against their rooflines.  Not the headline workload."""
    sizes = {}
    steps, warmup = min(args.steps, 20), min(args.warmup, 3)
    for name, p in VUSALIX_SHAPES.items():
        batch, ctx_len = HYBRID_DECODE
        blocks = batch * (ctx_len // 16 + 1)
        model = vusalix_model(p, dev, blocks, batch, ctx_len + 16)
        entry = {"shape": p, "vusalix": hybrid_throughput(model, dev, True, steps, warmup, args.preheat_s)}
        del model
        torch.cuda.empty_cache()
        model = tevirax_model(TEVIRAX_SHAPES[name], dev, blocks, batch, ctx_len + 16)
        entry["tevirax"] = hybrid_throughput(model, dev, True, steps, warmup, args.preheat_s)
        del model
        torch.cuda.empty_cache()
        entry["kernels"] = vusalix_kernels(p, dev, steps)
        sizes[name] = entry
        print(f"[{name}] done", file=sys.stderr, flush=True)
    main_size = sizes["w4096"]["vusalix"]
    print(json.dumps({
        "metric": "Vusalix prefill tokens/s", "value": main_size["prefill_tokens_per_s"], "unit": "tokens/s", "n_gpus": 1,
        "steps": steps, "warmup": warmup, "ms_per_step": main_size["prefill_ms"], "higher_is_better": True,
        "scaling": "weak", "vs_baseline": None, "dtype": "bf16", "data": "synthetic",
        "config": {"workload": "vusalix", "layers": HYBRID_LAYERS, "prefill": HYBRID_PREFILL, "decode": HYBRID_DECODE}, "sizes": sizes}))
    return 0


# width; attention and talking-attention query heads, kv heads (of 128 x 128); HGRN2 heads (of 128 x 128); feed-forward without a
# gate: one and a half times the inner width of a gated one is the same work
LOLUZEN_SHAPES = {
    "w2048": dict(width=2048, heads=16, kv_heads=4, r_heads=16, ff=8448),
    "w4096": dict(width=4096, heads=32, kv_heads=8, r_heads=32, ff=21504),
}


def loluzen_model(p, dev, num_blocks, slots, max_positions):
    """Parallel and attention layers in turn, three of five running twice, which makes eight runs; random weights."""
    from research_amd.inference import HipPagedAttentionBackend, HybridConfig, HybridDecoder
    from research_amd.inference.hybrid import LayerSpec, Loop
    from research_amd.inference.mixers import AttentionSpec, Hgrn2Mixer, Hgrn2Spec, LlamaScaling, MLPSpec, ParallelSpec, TalkingAttention, TalkingSpec

    att = AttentionSpec(heads=p["heads"], kv_heads=p["kv_heads"], dim=128, vdim=128, scale=128 ** -0.5, window=None, taps=4, rot_dims=64,
                        rot_base=10000.0, rot_llama=LlamaScaling(8.0, 8192, 1.0, 4.0), qk_weights=True)
    par = ParallelSpec(TalkingSpec(p["heads"], p["kv_heads"], 128, 128, 128 ** -0.5), Hgrn2Spec(p["r_heads"], 128, 128), 0.5, 0.5, norms=True)
    ff = MLPSpec(p["ff"], "relu2")
    cfg = HybridConfig(vocab_size=HYBRID_VOCAB, width=p["width"], norm_eps=1e-6, norm="rms", both_norms=True, norm_offset=1.0, residual_mult=0.5,
                       loop=Loop(1, 4, 2), layers=tuple(LayerSpec(att if i % 2 else par, ff) for i in range(5)))
    if len(cfg.runs()) != HYBRID_LAYERS:
        raise AssertionError("as many runs as the other model has layers")
    backend = HipPagedAttentionBackend(cfg.cache_config(num_blocks, 16, slots, torch.bfloat16, "cuda"))
    model = HybridDecoder(cfg, backend, max_positions)
    with torch.no_grad():
        for q in model.parameters():
            q.normal_(0.0, q.shape[-1] ** -0.5)
        for m in model.modules():
            if isinstance(m, TalkingAttention):
                m.bias_size.uniform_(0.05, 1.5)
                m.bias_rate.uniform_(0.05, 0.6)
                m.talk.copy_((m.talk + torch.eye(p["heads"], device=dev)).to(torch.bfloat16))
            if isinstance(m, Hgrn2Mixer):
                m.lower.uniform_(0.0, 0.9)
                m.f_bias.uniform_(-1.0, 6.0)
    return model.eval()


def loluzen_kernels(p, dev, steps):
    """Every kernel of the design's blocks at the layer's shapes, against its roofline, with the like kernel of the Lotozen
    block.  Bytes and FLOPs are the algorithmic ones: mixed heads add a product of their weights with the matrix."""
    from research_amd import ops

    bf, f32 = torch.bfloat16, torch.float32
    rnd = lambda *s, dtype=bf: torch.randn(*s, device=dev, dtype=torch.float32).to(dtype)
    i32 = lambda a: torch.as_tensor(np.ascontiguousarray(a), dtype=torch.int32).to(dev)
    rows_out, add = kernel_table(steps)
    width, heads, kv, rh, ff, d = p["width"], p["heads"], p["kv_heads"], p["r_heads"], p["ff"], 128
    for phase, (batch, length) in (("prefill", HYBRID_PREFILL), ("decode", HYBRID_DECODE)):
        dec = phase == "decode"
        n = batch if dec else batch * length
        per = length // 16 + (1 if dec else 0)
        tables = np.random.default_rng(5).permutation(batch * per).reshape(batch, per).astype(np.int32)
        ctx = np.full(batch, length + 1 if dec else length)
        pos = np.full((batch, 1), length) if dec else np.tile(np.arange(length), (batch, 1))
        slots = torch.from_numpy((np.take_along_axis(tables, pos // 16, 1).astype(np.int64) * 16 + pos % 16).reshape(-1)).to(dev)
        bt, lens, sslots = i32(tables), i32(ctx), i32(np.arange(batch))
        if dec:
            por = ops.Portions(lens, sslots)
        else:
            first = np.arange(0, length, ops.QKV_TILE_ROWS)
            tiles = np.stack([np.repeat(np.arange(batch), len(first)), np.tile(first, batch)], 1)
            por = ops.Portions(lens, sslots, i32(ctx), i32(np.arange(batch) * length), i32(tiles), length)
        # residual sums
        x, y, z, w = rnd(n, width, dtype=f32), rnd(n, width), rnd(n, width), rnd(width, dtype=f32)
        kw = dict(y_weight=w, y_eps=1e-6, norm="rms", weight=w, eps=1e-6)
        add(phase, "residual + normed sum of two normed branches + norm", lambda: ops.residual_norm(x, bf, y=y, y2=(z, w, w), **kw),
            "residual + RMS-normed branch + layer norm", n * width * 14.0)
        add(phase, "residual + normed branch with bias + norm", lambda: ops.residual_norm(x, bf, y=y, y_bias=w, **kw),
            "residual + RMS-normed branch + layer norm", n * width * 12.0)
        table, ids = rnd(HYBRID_VOCAB, width), torch.randint(0, HYBRID_VOCAB, (n,), device=dev)
        add(phase, "the same + embedding", lambda: ops.residual_norm(x, bf, y=y, y_bias=w, ids=ids, table=table, ids_add=True, **kw),
            "residual + RMS-normed branch + layer norm", n * width * 14.0)
        add(phase, "like: residual + RMS-normed branch + layer norm",
            lambda: ops.residual_norm(x, bf, y=y, y_weight=w, y_eps=1e-6, norm="layer", weight=w, bias=w, eps=1e-6), "", n * width * 12.0)
        del x, y, z, table
        u, b = rnd(n, ff), rnd(ff, dtype=f32)
        add(phase, "bias + square of relu", lambda: ops.bias_act(u, b, "relu2"), "silu(gate) * up", n * ff * 4.0)
        add(phase, "like: silu(gate) * up", lambda: ops.glu(u[:, : ff // 2], u[:, ff // 2:], "silu"), "", n * ff * 3.0)
        del u
        # attention
        chans = (heads + 2 * kv) * d
        u = rnd(n, chans + heads)
        total = batch * per * 16
        kc, vc = rnd(total, kv, d), rnd(total, kv, d)
        conv, cstate, bias = rnd(4, chans, dtype=f32), torch.zeros(batch, 3, chans, dtype=bf, device=dev), rnd(chans, dtype=f32)
        rope, qn = rnd(length + 1, d // 4, 2, dtype=f32), rnd(d, dtype=f32)
        q = torch.empty(n, heads, d, dtype=bf, device=dev)
        lam, vf = rnd(1, dtype=f32), rnd(n, kv * d)
        conv_bytes = n * 4.0 * chans + (batch * 12.0 * chans if dec else 0.0) + chans * 16.0
        add(phase, "conv + q/k norm + rotation + append", lambda: ops.qkv_conv_append(u, por, slots, kc, vc, heads, d, d, 1.0, 1e-6, False, rope, d // 2,
            conv, cstate, q_out=q, q_norm=qn, k_norm=qn), "conv + rotation + unit norm + append", conv_bytes)
        add(phase, "like: conv + rotation + unit norm + append", lambda: ops.qkv_conv_append(u, por, slots, kc, vc, heads, d, d, 1.0, 1e-6, True, rope,
            d // 2, conv, cstate, "mix", vf, lam, q_out=q), "", conv_bytes + n * 2.0 * kv * d)
        add(phase, "biases + append", lambda: ops.qkv_conv_append(u, por, slots, kc, vc, heads, d, d, 1.0, 0.0, False, None, 0, None, None, q_out=q,
            bias=bias), "conv + rotation + unit norm + append", n * 4.0 * chans)
        o = torch.empty_like(q)
        talk = (torch.eye(heads, device=dev) + 0.2 * rnd(heads, heads, dtype=f32)).to(bf).float()
        size, rate = 0.05 + torch.rand(heads, device=dev), 0.05 + 0.5 * torch.rand(heads, device=dev)
        tw = torch.empty(ops.talking_workspace_bytes(n, por, heads, kv, d, per * 16), dtype=torch.uint8, device=dev)
        mixed = lambda: ops.talking_attention(q, kc, vc, d, por, bt, 16, d ** -0.5, talk, o, size, rate, workspace=tw)
        if dec:
            ws = ops.decode_workspace(q, kc)
            moved = 4.0 * kv * d * float(ctx.sum())
            add(phase, "attention, mixed heads", mixed, "decode attention", moved)
            add(phase, "like: decode attention", lambda: ops.decode(q, kc, vc, bt, lens, 16, 0.1, ws, out=o), "", moved)
        else:
            pairs = batch * length * (length + 1) / 2.0
            add(phase, "attention, mixed heads", mixed, "prefill attention", flops=heads * pairs * (4.0 * d + 2.0 * heads))
            need = ops.prefill_workspace_bytes(q, bt, length, 16, kv, 0)
            ws = torch.empty(max(need, 16), dtype=torch.uint8, device=dev)
            add(phase, "like: prefill attention", lambda: ops.prefill_paged(q, kc, vc, bt, lens, por.q_lens, por.q_starts, length, 16, 0.1, out=o,
                workspace=ws if need else None), "", flops=4.0 * d * heads * pairs)
        add(phase, "head gate", lambda: ops.head_gate(o, u[:, chans: chans + heads], d), "the same kernel", n * heads * 2.0 * (2 * d + 1))
        del u, kc, vc, q, o, vf, tw
        # HGRN2
        inner = rh * d
        u = rnd(n, 4 * inner)
        u[:, inner: 2 * inner] += 2.5
        state = torch.zeros(batch, rh, d, d, device=dev)
        lower, fb = 0.9 * torch.rand(inner, device=dev), rnd(inner, dtype=f32)
        powers = torch.full((rh, 65), 0.97, device=dev) ** torch.arange(65, device=dev)
        o = torch.empty(n, inner, dtype=bf, device=dev)
        bytes_r = n * inner * 8.0 + batch * rh * d * d * 8.0

        def hgrn2(portions, rows_bytes, name, like):
            nb = portions.ctx_lens.numel()
            need = 0 if dec else max(ops.channel_linear_workspace_bytes(nb, rh, d, d, portions.max_q_len), ops.lightning_workspace_bytes(nb, rh, d, d, portions.max_q_len))
            ws = torch.empty(max(need, 16), dtype=torch.uint8, device=dev)
            add(phase, name, lambda: ops.channel_linear(u[:, :inner], u[:, inner: 2 * inner], u[:, 2 * inner: 3 * inner], fb, lower, portions, state, rh,
                d, d, o, q_act="silu", workspace=ws), like, rows_bytes)
            add(phase, "like: " + like, lambda: ops.lightning(u, portions, state, powers, rh, d, d, o, workspace=ws), "", rows_bytes)

        hgrn2(por, bytes_r, "HGRN2", "lightning attention")
        if not dec:  # one long portion alone, in segments
            por1 = ops.Portions(i32([n]), i32([0]), i32([n]), i32([0]), None, n)
            hgrn2(por1, n * inner * 8.0 + rh * d * d * 8.0, f"HGRN2, one sequence of {n}", "lightning attention, one sequence")
        nw = rnd(inner, dtype=f32)
        add(phase, "RMS norm per head", lambda: ops.rms_gate(o, None, nw, 1e-6, groups=rh, order=None), "RMS norm + sigmoid gate", n * inner * 4.0)
        add(phase, "like: RMS norm + sigmoid gate", lambda: ops.rms_gate(o, u[:, 3 * inner:], nw, 1e-6), "", n * inner * 6.0)
        del u, state, o
        torch.cuda.empty_cache()
    return rows_out


def bench_loluzen(args, dev) -> int:
    """Prefill and decode throughput of Loluzen-shaped models with random weights beside Lotozen-shaped ones of the same width,
    heads, depth and feed-forward work, and the design's kernels against their rooflines.  Not the headline workload."""
    sizes = {}
    steps, warmup = min(args.steps, 20), min(args.warmup, 3)
    for name, p in LOLUZEN_SHAPES.items():
        batch, ctx_len = HYBRID_DECODE
        blocks = batch * (ctx_len // 16 + 1)
        model = loluzen_model(p, dev, blocks, batch, ctx_len + 16)
        entry = {"shape": p, "loluzen": hybrid_throughput(model, dev, True, steps, warmup, args.preheat_s)}
        del model
        torch.cuda.empty_cache()
        model = hybrid_model(HYBRID_SHAPES[name], dev, blocks, batch, ctx_len + 16)
        entry["lotozen"] = hybrid_throughput(model, dev, True, steps, warmup, args.preheat_s)
        del model
        torch.cuda.empty_cache()
        entry["kernels"] = loluzen_kernels(p, dev, steps)
        sizes[name] = entry
        print(f"[{name}] done", file=sys.stderr, flush=True)
    main_size = sizes["w4096"]["loluzen"]
    print(json.dumps({
        "metric": "Loluzen prefill tokens/s", "value": main_size["prefill_tokens_per_s"], "unit": "tokens/s", "n_gpus": 1,
        "steps": steps, "warmup": warmup, "ms_per_step": main_size["prefill_ms"], "higher_is_better": True,
        "scaling": "weak", "vs_baseline": None, "dtype": "bf16", "data": "synthetic",
        "config": {"workload": "loluzen", "layers": HYBRID_LAYERS, "prefill": HYBRID_PREFILL, "decode": HYBRID_DECODE}, "sizes": sizes}))
    return 0


def secondary(args, dev) -> dict:
    """Short runs of the configurations that are not the headline: what the step costs, the dominant kernel
    against its roofline and a few seconds of the CPU restatement, per workload."""
    import copy

    short = copy.copy(args)
    short.steps, short.warmup, short.preheat_s = 30, 5, 0.3
    short.cpu_seconds = min(args.cpu_seconds, 4.0)
    short.copy_calibration = False
    short.secondary_run = True
    out = {}
    for name in ("c2", "c5", "c3", "c3-d256", "c3-d64", "c3-d96", "dense-64x512", "dense-4x8192", "long-d128", "long-d256"):
        r = (bench_prefill_c3(short, dev) if name == "c3" else bench_prefill_head(short, dev, name) if name in PREFILL_HEAD_SHAPES
             else bench_prefill_dense(short, dev, name) if name in PREFILL_DENSE_SHAPES
             else bench_prefill_long(short, dev, name) if name in PREFILL_LONG_SHAPES else bench_decode(name, short, dev))
        keep = ("metric", "value", "unit", "ms_per_step", "ms_per_step_mean", "steps", "warmup", "tokens_per_s",
                "dtype", "roofline", "cpu_baseline", "append", "pct_of_hbm_peak")
        entry = {k: r[k] for k in keep if k in r}
        entry["workload"] = r["config"]["workload"]
        out[name] = entry
        torch.cuda.empty_cache()
    return out


def main() -> int:
    args = parse_args()
    if args.traffic_from_pmc:
        return traffic_from_pmc(*args.traffic_from_pmc)
    if args.gpus != 1:
        print("bench.py measures one GPU: this build has no multi-GPU path, run with --gpus 1", file=sys.stderr)
        return 2
    from research_amd import _lib

    _lib.load()  # no fallback: raises if the HIP library is missing
    if not torch.cuda.is_available():
        print("bench.py needs a HIP device", file=sys.stderr)
        return 2
    dev = torch.device("cuda:0")
    torch.cuda.set_device(dev)
    if args.workload == "engine":
        return bench_engine(args, dev)
    if args.workload == "lotozen":
        return bench_hybrid(args, dev)
    if args.workload == "tevirax":
        return bench_tevirax(args, dev)
    if args.workload == "vusalix":
        return bench_vusalix(args, dev)
    if args.workload == "loluzen":
        return bench_loluzen(args, dev)
    if args.workload in PREFILL_HEAD_SHAPES:
        result = bench_prefill_head(args, dev, args.workload)
    elif args.workload in PREFILL_LONG_SHAPES:
        result = bench_prefill_long(args, dev, args.workload)
    elif args.workload in PREFILL_DENSE_SHAPES:
        result = bench_prefill_dense(args, dev, args.workload)
    else:
        result = bench_prefill_c3(args, dev) if args.workload == "c3" else bench_decode(args.workload, args, dev)
    if args.workload == "c4" and not args.no_secondary:
        torch.cuda.empty_cache()
        result["secondary"] = secondary(args, dev)
    print(json.dumps(result))
    return 0


if __name__ == "__main__":
    sys.exit(main())
