"""Command line of the inference package.

    python -m research_amd.inference generate --model DIR --prompt-ids 5,17,3 [--prompt-ids ...] [--max-tokens N]
    python -m research_amd.inference trace    --model DIR --out DIR --max-tokens N < steps

``generate`` prints one JSON line per finished sequence.  Any registered design
(registry.py) is loaded by its ``config.json``.
"""

from __future__ import annotations

import argparse
import json
import sys


def generate(argv) -> int:
    ap = argparse.ArgumentParser(prog="python -m research_amd.inference generate")
    ap.add_argument("--model", required=True, help="folder with config.json and safetensors weights")
    ap.add_argument("--dtype", default="bfloat16", choices=["bfloat16", "float32"])
    ap.add_argument("--prompt-ids", action="append", required=True, help="token ids with commas between them; repeatable")
    ap.add_argument("--max-tokens", type=int, default=32)
    ap.add_argument("--temperature", type=float, default=0.0)
    ap.add_argument("--samples", type=int, default=1, help="completions per prompt")
    ap.add_argument("--max-batch-size", type=int, default=32)
    ap.add_argument("--max-model-len", type=int, default=4096)
    ap.add_argument("--cache-type", default="radix", choices=["radix", "paged", "private", "none"])
    ap.add_argument("--prefill-portion", type=int, default=None, help="most tokens of a prompt per step")
    ap.add_argument("--graphs", action="store_true", help="replay decode steps from captured graphs")
    args = ap.parse_args(argv)
    from .engine import InferenceEngine
    from .registry import model_len
    from .types import EngineConfig, SamplingParams

    engine = InferenceEngine(EngineConfig(
        model_path=args.model, cache_type=args.cache_type, max_batch_size=args.max_batch_size,
        max_model_len=model_len(args.model, args.max_model_len), use_graphs=args.graphs, dtype=args.dtype,
        prefill_portion=args.prefill_portion))
    prompts = [[int(t) for t in p.split(",")] for p in args.prompt_ids]
    for sample in engine.generate(prompts, SamplingParams(temperature=args.temperature, max_tokens=args.max_tokens),
                                  args.samples):
        print(json.dumps({"prompt": list(sample.prompt_tokens), "completion": list(sample.completion_tokens),
                          "logprobs": list(sample.logprobs), "finish_reason": sample.finish_reason}), flush=True)
    return 0


def main() -> int:
    if len(sys.argv) > 1 and sys.argv[1] == "generate":
        return generate(sys.argv[2:])
    if len(sys.argv) > 1 and sys.argv[1] == "trace":
        from .trace import main as trace_main

        return trace_main(sys.argv[2:])
    print(__doc__.strip(), file=sys.stderr)
    return 2


if __name__ == "__main__":
    sys.exit(main())
