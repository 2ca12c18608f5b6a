"""The Nunivik model on the GPU through the engine's own runner, pool, slots and planner, against the oracle: whole
prompts, token by token, portions, batches, reused pages and slots, long decoding, greedy generation, the trace replay."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

from electrock_infer_amd.harness import LLMEngine, SamplingParams
from electrock_infer_amd.harness.trace import TraceReplay
from oracle import nunivik_oracle as N
from tests.feguvik_util import draw_tokens, row_errors
from tests.gpu_util import announce
from tests.nunivik_util import CONFIGS, make_model, oracle_logits
from tests.test_gpu_feguvik import F32_TOL, ROOT, assert_close, feed

pytestmark = pytest.mark.gpu


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    base, cache = tmp_path_factory.mktemp("nunivik"), {}
    def get(name):
        if name not in cache:
            cache[name] = make_model(base / name, name, seed=3)
        return cache[name]
    return get


def fill_with_nan(replay):
    """Pages and slots as an earlier request might leave them, only worse."""
    for cache in replay.runner.model.caches:
        for t in cache if isinstance(cache, tuple) else (cache,):
            t.fill_(float("nan"))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_prompts_decoding_and_portions(models, name, dtype):
    """The logits of a position do not depend on how the tokens were cut."""
    announce(f"nunivik {name} {dtype}: whole, one by one, portions")
    path, cfg, w = models(name)
    toks = draw_tokens(cfg, 150, seed=1)
    want = oracle_logits(toks, w, cfg)
    replay = TraceReplay.for_model(path, dtype, 200)
    for sizes in ([150], [1], [2], [149, 1], [3, 2, 16, 1, 33], [64, 22], [37, 3], [100, 2]):
        fill_with_nan(replay)
        assert_close(feed(replay, "r", toks, sizes), want, dtype, f"{name} {sizes}")
    assert not replay.live


@pytest.mark.parametrize("name", ["odd", "plain"])
def test_long_prompts(models, name):
    """Several chunks of the recurrences, many pages, windows far behind; then decoding."""
    announce(f"nunivik {name}: 700 tokens")
    path, cfg, w = models(name)
    toks = draw_tokens(cfg, 700, seed=7)
    want = oracle_logits(toks, w, cfg)
    for dtype in ("float32", "bfloat16"):
        replay = TraceReplay.for_model(path, dtype, 700)
        for sizes in ([700], [300, 2, 256, 1], [690, 1]):
            assert_close(feed(replay, "r", toks, sizes), want, dtype, f"{name} {sizes}")


@pytest.mark.parametrize("name", ["odd", "wide"])
def test_stream_behind_every_layer(models, name):
    announce(f"nunivik {name}: streams")
    path, cfg, w = models(name)
    toks, want, got = draw_tokens(cfg, 40, seed=2), [], []
    N.forward(toks, w, cfg, torch.float64, want)
    replay = TraceReplay.for_model(path, "float32", 64)
    replay.runner.model.layer_hook = lambda r, x: got.append((r, x.double().cpu()))
    replay.step([{"id": "a", "tokens": toks, "want": []}], ["a"])
    assert [r for r, _ in got] == list(range(len(want)))
    for (r, x), y in zip(got, want):
        assert float((x - y).abs().max() / y.abs().max()) < 2e-5, r


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["odd", "wide", "recurrent"])
def test_batches_reused_pages_and_slots(models, name, dtype):
    """Unequal requests in one step, each against itself alone; then requests that end in between and new ones that take
    their pages and slots over (the pool is small enough that nothing else is left)."""
    announce(f"nunivik {name} {dtype}: batches")
    path, cfg, w = models(name)
    lens = {"a": 90, "b": 1, "c": 41, "d": 64}
    toks = {k: draw_tokens(cfg, n + 40, seed=10 + n) for k, n in lens.items()}
    want = {k: oracle_logits(t, w, cfg) for k, t in toks.items()}
    replay = TraceReplay.for_model(path, dtype, 240)
    at = dict.fromkeys(toks, 0)
    def step(counts, end=()):
        out = replay.step([{"id": k, "tokens": toks[k][at[k]:at[k] + n], "want": list(range(n))} for k, n in counts.items()], list(end))
        for (k, n), part in zip(counts.items(), out.split(list(counts.values()))):
            # (a few rows have no spread of their own: measured against the whole request's)
            padded = want[k].clone()
            padded[at[k]:at[k] + n] = part
            assert_close(padded, want[k], dtype, f"{k} {at[k]} + {n}")
            at[k] += n
    fill_with_nan(replay)
    step(lens)                                            # four prompts of unequal length
    for _ in range(3):
        step(dict.fromkeys(toks, 1))                      # decoding together
    step({"a": 2, "c": 7, "d": 1}, end=["a"])            # portions beside decoding; a leaves
    slot, blocks = replay.planner.slots.free[-1], replay.planner.pool.free_ids()
    at["a"] = 0
    step({"a": 33, "b": 5})                               # a again, from the start, where others have been
    assert replay.live["a"].state_slot == slot and set(replay.live["a"].block_table) <= set(blocks)
    step({"a": 57, "b": 1, "c": 1, "d": 19}, end=["b", "c"])
    at["b"], at["c"] = 0, 0
    step({"c": 41, "b": 1, "a": 1})
    step({"b": 40, "c": 16}, end=["a", "b", "c", "d"])
    assert replay.planner.pool.num_free == replay.planner.pool.num_blocks


def test_long_decoding(models):
    announce("nunivik odd, plain: 300 decoded tokens")
    for name in ("odd", "plain"):
        path, cfg, w = models(name)
        toks = draw_tokens(cfg, 320, seed=4)
        replay = TraceReplay.for_model(path, "float32", 320)
        assert_close(feed(replay, "r", toks, [20] + [1] * 300), oracle_logits(toks, w, cfg), "float32", f"{name} long decoding")


@pytest.mark.parametrize("name,portion", [("odd", 0), ("odd", 17), ("plain", 33), ("attention", 0)])
def test_greedy_generation_through_the_engine(models, name, portion):
    """The entry point, planner and sampler: prompts of unequal length in a cache so small that a request is preempted and
    computed again, with and without prompt portions; every token is the oracle's arg-max (float32)."""
    announce(f"nunivik {name}: generate, portion {portion}")
    path, cfg, w = models(name)
    prompts = [draw_tokens(cfg, n, seed=20 + n) for n in (70, 5, 33, 1, 50)]
    max_tokens = [40, 40, 39, 30, 35]
    engine = LLMEngine(path, dtype="float32", num_kvcache_blocks=7, max_num_seqs=4, max_num_batched_tokens=96, max_model_len=200,
                       prefill_portion=portion)
    outs = engine.generate(prompts, [SamplingParams(temperature=0.0, max_tokens=m, ignore_eos=True) for m in max_tokens])
    for p, o, m in zip(prompts, outs, max_tokens):
        assert len(o["token_ids"]) == m
        full = p + o["token_ids"]
        lg = oracle_logits(full, w, cfg)[len(p) - 1:-1]
        picked = lg.gather(1, torch.tensor(o["token_ids"])[:, None])[:, 0]
        assert float((lg.max(-1).values - picked).max()) < 1e-3          # the arg-max, or within rounding of it
    assert engine.stats["preemptions"] >= 1, engine.stats
    assert engine.planner.pool.num_free == 7 and (engine.planner.slots is None or engine.planner.slots.num_free == 4)
    assert (engine.planner.slots is None) == (name == "attention")


def test_sampled_generation_in_bfloat16(models):
    announce("nunivik wide: sampled generation")
    path, cfg, _ = models("wide")
    engine = LLMEngine(path, num_kvcache_blocks=40, max_num_seqs=4, max_num_batched_tokens=256, max_model_len=200)
    outs = engine.generate([draw_tokens(cfg, n) for n in (9, 80)], SamplingParams(temperature=0.8, max_tokens=7, ignore_eos=True))
    assert all(len(o["token_ids"]) == 7 and all(0 <= t < cfg["vocab"] for t in o["token_ids"]) for o in outs)


def test_trace_runner_and_command_line(models, tmp_path):
    announce("nunivik: bin/trace_run and python -m electrock_infer_amd.harness")
    path, cfg, w = models("plain")
    toks = draw_tokens(cfg, 30, seed=6)
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": toks[:20], "want": [3, 19]}], "end": []},
             {"step": 1, "entries": [{"id": "x", "tokens": toks[20:21], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "x", "tokens": toks[21:], "want": [8]}], "end": ["x"]}]
    p = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", path, "--dtype", "float32", "--out", str(tmp_path),
                        "--max-tokens", "30"], input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=100)
    assert p.returncode == 0, p.stderr[-2000:]
    assert [l for l in p.stdout.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    got = np.concatenate([np.fromfile(tmp_path / f"{i}.f32", dtype="<f4") for i in (0, 2)]).reshape(-1, cfg["vocab"])
    want = oracle_logits(toks, w, cfg)
    assert float(row_errors(torch.from_numpy(got), want[[3, 19, 29]]).max()) < F32_TOL
    p = subprocess.run([sys.executable, "-m", "electrock_infer_amd.harness", "--model", path, "--dtype", "float32", "--max-tokens", "3",
                        "--prompt", ",".join(map(str, toks))], capture_output=True, text=True, timeout=100, cwd=ROOT)
    assert p.returncode == 0, p.stderr[-2000:]
    lines = [json.loads(l) for l in p.stdout.splitlines() if l.startswith("{")]
    assert len(lines) == 1 and lines[0]["token_ids"][0] == int(want[-1].argmax())


@pytest.mark.parametrize("name,dtype", [("odd", "float32"), ("wide", "bfloat16"), ("plain", "bfloat16")])
def test_recorded_decode_steps_equal_eager_ones(models, name, dtype):
    """Every decode step of a batch whose size and contexts change, replayed from the recorded graphs, against the same
    step run eagerly and (float32) against the oracle; eager prompts of new requests run between the replays."""
    announce(f"nunivik {name} {dtype}: decode graphs")
    path, cfg, w = models(name)
    prompts = [draw_tokens(cfg, n, seed=40 + n) for n in (3, 60, 21, 9, 30)]
    params = [SamplingParams(temperature=0.0, max_tokens=m, ignore_eos=True) for m in (60, 10, 25, 30, 8)]
    logits = {}
    for graphs in (True, False):
        engine = LLMEngine(path, dtype=dtype, num_kvcache_blocks=40, max_num_seqs=3, max_num_batched_tokens=96, max_model_len=200,
                           decode_graphs=graphs)
        seen, first = {}, {}
        def hook(seqs, is_prefill, rows):
            for s, row in zip(seqs, rows.float().cpu()):
                seen[(first.setdefault(s.seq_id, len(first)), len(s))] = (list(s.token_ids), row)
        engine.step_hook = hook
        engine.generate(prompts, params)
        logits[graphs] = seen
        if graphs:
            g = engine.model_runner.graphs
            assert g.replays >= 59 and g.recorded and all(r is not None for r in g.recorded.values()), g.recorded
            assert len(g.recorded) >= 3                    # one, two and three sequences (padded to four)
    close = 0
    for key, (toks, row) in logits[True].items():
        if dtype == "float32":
            want = oracle_logits(toks, w, cfg)[-1]
            assert float((row - want).abs().max() / want.std()) < F32_TOL * 5, key
        other = logits[False].get(key)
        if other is not None and other[0] == toks:
            close += 1
            assert float((row - other[1]).abs().max() / row.std()) < (1e-3 if dtype == "float32" else 0.5), key
    assert close > len(logits[True]) // 2
