"""Replay of a token trace: steps that feed given tokens to requests through the engine's own runner, cache pool and
state slots, and read logits at chosen places.  Nothing is sampled.

    python -m electrock_infer_amd.harness.trace --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N

reads one JSON object a line from standard input,

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": []}

('want': places among the entry's tokens; 'end': requests that are finished behind this step) and writes the wanted
logits, little-endian float32 [wanted, vocab] in the order of the entries, to DIR/<step>.f32.  'done <step>' is printed
behind every step.  Exit code 3: the model does not run in the asked type.
"""
import argparse
import json
import os
import sys
from typing import Dict, List, Optional

import torch

from .batch_planner import BatchPlanner
from .config import EngineConfig, SamplingParams
from .model_runner import ModelRunner
from .registry import ensure_libraries, load_config
from .sequence import Sequence


class TraceReplay:
    """Live requests and the engine parts that hold them."""

    MAX_REQUESTS = 256

    def __init__(self, config: EngineConfig):
        self.config = config
        Sequence.block_size = config.kvcache_block_size
        self.runner = ModelRunner(config)
        self.planner = BatchPlanner(config)
        self.live: Dict[str, Sequence] = {}

    @classmethod
    def for_model(cls, model_dir: str, dtype: str, max_tokens: int) -> "TraceReplay":
        model = load_config(model_dir, dtype)
        ensure_libraries(model)
        requests, block = min(max(max_tokens, 1), cls.MAX_REQUESTS), EngineConfig.kvcache_block_size
        return cls(EngineConfig(model=model, model_dir=model_dir, reuse_prefix=False, max_num_seqs=requests, decode_graphs=False,
                                num_kvcache_blocks=max(max_tokens, 1) // block + 1 + requests,
                                max_num_batched_tokens=max(max_tokens, 1)))

    def _portion(self, request: str, tokens: List[int]) -> Sequence:
        """The request with its next tokens planned."""
        if not tokens or not all(isinstance(t, int) and 0 <= t < self.config.model.vocab_size for t in tokens):
            raise ValueError("an entry needs tokens of the vocabulary")
        seq = self.live.get(request)
        if seq is None:
            seq = Sequence(tokens, SamplingParams())
            self.planner.pool.admit(seq)
            if self.planner.slots is not None:
                self.planner.slots.take(seq)
            self.live[request] = seq
        else:
            seq.token_ids.extend(tokens)
            if not self.planner.pool.can_extend(seq):
                raise RuntimeError("the cache is too small for the trace")
            self.planner.pool.extend(seq)
        seq.num_scheduled_tokens = len(tokens)
        return seq

    def step(self, entries: List[dict], end: List[str]) -> Optional[torch.Tensor]:
        """Float32 logits [wanted, vocab] on the host, or None if nothing is wanted."""
        seqs, rows, at = [], [], 0
        for e in entries:
            seqs.append(self._portion(e["id"], e["tokens"]))
            if not all(0 <= w < len(e["tokens"]) for w in e["want"]):
                raise ValueError("'want' counts through the entry's tokens")
            rows += [at + w for w in e["want"]]
            at += len(e["tokens"])
        logits = None
        if seqs:
            out = self.runner.portion_logits(seqs, rows)
            logits = out.float().cpu() if rows else None
            torch.cuda.synchronize()
        for s in seqs:
            s.num_computed_tokens += s.num_scheduled_tokens
            s.num_scheduled_tokens = 0
        for request in end:
            self.planner.release(self.live.pop(request))
        return logits


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description="feed a token trace to a model and write logits")
    ap.add_argument("--model", required=True, help="folder with config.json and safetensors files")
    ap.add_argument("--dtype", required=True, choices=["bfloat16", "float32"])
    ap.add_argument("--out", required=True, help="folder for <step>.f32")
    ap.add_argument("--max-tokens", type=int, required=True, help="most tokens that live requests hold at any time")
    args = ap.parse_args(argv)
    try:
        load_config(args.model, args.dtype)
    except ValueError as e:
        print(e, file=sys.stderr)
        return 3 if args.dtype == "float32" else 2
    replay = TraceReplay.for_model(args.model, args.dtype, args.max_tokens)
    for line in sys.stdin:
        if not line.strip():
            continue
        step = json.loads(line)
        logits = replay.step(step["entries"], step.get("end", []))
        if logits is not None:
            logits.numpy().astype("<f4").tofile(os.path.join(args.out, f"{step['step']}.f32"))
        print(f"done {step['step']}", flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
