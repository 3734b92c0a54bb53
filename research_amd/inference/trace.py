"""Replay of a trace: given token ids through a model, step by step, logits to files.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N

Nothing is sampled.  Every line of standard input is a step:

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": ["b"]}

Its entries run as one batch (``InferenceEngine.feed``, the step function that
generation uses): portions of prompts beside single tokens, each continuing
from what earlier steps left in the cache and state.  The logits at the wanted
places go to ``OUT/<step>.f32`` (little-endian float32, in the order of the
entries and of ``want``), ``done <step>`` is printed, and the sequences named in
``end`` give their blocks and slots back.

The pool holds ``--max-tokens`` tokens, each live sequence counted in whole
blocks, and ``--max-sequences`` state slots.  The library is built first when
it is not there.
"""

from __future__ import annotations

import argparse
import json
import os
import sys
from typing import Dict, List, Optional, TextIO

import torch

from .types import EngineConfig, Sequence

BLOCK_SIZE = 16


def parse_args(argv: Optional[List[str]] = None) -> argparse.Namespace:
    ap = argparse.ArgumentParser(prog="trace_run", description="Replay token ids through a model and write logits.")
    ap.add_argument("--model", required=True, help="folder with config.json and safetensors weights")
    ap.add_argument("--dtype", default="bfloat16", choices=["bfloat16", "float32"])
    ap.add_argument("--out", required=True, help="folder for the logits")
    ap.add_argument("--max-tokens", type=int, required=True, help="most tokens that live sequences hold at any time")
    ap.add_argument("--max-sequences", type=int, default=4, help="most sequences that are live at any time")
    return ap.parse_args(argv)


def replay(engine, lines, out_dir: str, report: TextIO) -> None:
    live: Dict[str, Sequence] = {}
    for line in lines:
        if not line.strip():
            continue
        step = json.loads(line)
        entries = [e for e in step["entries"] if e["tokens"]]
        batch = []
        for e in entries:
            if e["id"] not in live:
                live[e["id"]] = engine.open_sequence()
            batch.append((live[e["id"]], list(e["tokens"])))
        if batch:
            hidden, first = engine.feed(batch)
            rows = [at + w for e, at in zip(entries, first) for w in e["want"]]
            if rows:
                with torch.no_grad():
                    logits = engine.model.logits(hidden[torch.tensor(rows, device=hidden.device)]).float()
                logits.cpu().numpy().astype("<f4").tofile(os.path.join(out_dir, f"{step['step']}.f32"))
        for name in step.get("end", ()):
            engine.close_sequence(live.pop(name))
        torch.cuda.synchronize()
        print(f"done {step['step']}", file=report, flush=True)


def main(argv: Optional[List[str]] = None) -> int:
    args = parse_args(argv)
    from .. import _lib, build

    if not os.path.exists(_lib.LIB_PATH):
        build.build(jobs=min(16, os.cpu_count() or 1))
    from .engine import InferenceEngine
    from .registry import model_len

    torch.backends.cuda.matmul.allow_tf32 = False  # float32 means float32
    blocks = max(1, -(-args.max_tokens // BLOCK_SIZE))
    engine = InferenceEngine(EngineConfig(
        model_path=args.model, cache_type="private", block_size=BLOCK_SIZE, max_batch_size=args.max_sequences,
        max_model_len=model_len(args.model, args.max_tokens), num_kv_blocks=blocks, dtype=args.dtype))
    replay(engine, sys.stdin, args.out, sys.stdout)
    return 0
