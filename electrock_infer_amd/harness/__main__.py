"""Generate from a model directory:

    python -m electrock_infer_amd.harness --model DIR --prompt 5,17,3 [--prompt ...] [--max-tokens N] [--temperature T]

Prompts are token ids (there is no tokenizer here); one JSON line per prompt is printed, {"prompt": [...], "token_ids": [...]}."""
import argparse
import json
import sys

from .config import SamplingParams
from .engine import LLMEngine
from .registry import DTYPES, REGISTRY, ensure_libraries, load_config


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="python -m electrock_infer_amd.harness", description="generate tokens with a model",
                                 epilog=f"architectures: {', '.join(sorted(REGISTRY))}")
    ap.add_argument("--model", required=True, help="folder with config.json and safetensors files")
    ap.add_argument("--prompt", action="append", required=True, help="token ids with commas between them; may be repeated")
    ap.add_argument("--dtype", choices=sorted(DTYPES), default="bfloat16")
    ap.add_argument("--max-tokens", type=int, default=16)
    ap.add_argument("--temperature", type=float, default=0.0, help="0: greedy")
    ap.add_argument("--eos", type=int, default=-1, help="token that ends a request")
    ap.add_argument("--prefill-portion", type=int, default=0, help="compute prompts in portions of at most so many tokens")
    ap.add_argument("--max-num-seqs", type=int, default=16)
    args = ap.parse_args(argv)
    prompts = [[int(t) for t in p.split(",")] for p in args.prompt]
    longest = max(map(len, prompts)) + args.max_tokens
    ensure_libraries(load_config(args.model, args.dtype))
    engine = LLMEngine(args.model, dtype=args.dtype, eos=args.eos, prefill_portion=args.prefill_portion,
                       max_num_seqs=args.max_num_seqs, max_model_len=longest + 1, max_num_batched_tokens=max(longest, 2048))
    sp = SamplingParams(temperature=args.temperature, max_tokens=args.max_tokens, ignore_eos=args.eos < 0)
    for prompt, out in zip(prompts, engine.generate(prompts, sp)):
        print(json.dumps({"prompt": prompt, "token_ids": out["token_ids"]}))
    return 0


if __name__ == "__main__":
    sys.exit(main())
