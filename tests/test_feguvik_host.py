"""Host side of the Feguvik model and of what it brought to the engine (no GPU): registry and configuration, weight
loading, ragged batches, state slots, prompt portions, the trace replay's bookkeeping, the decoder library's C surface."""
import ctypes
import json
import os
import re

import pytest
import torch

from electrock_infer_amd import _lib
from electrock_infer_amd.harness import LLMEngine, ModelConfig, SamplingParams
from electrock_infer_amd.harness import trace as trace_module
from electrock_infer_amd.harness.batch import make_ragged
from electrock_infer_amd.harness.batch_planner import BatchPlanner
from electrock_infer_amd.harness.config import EngineConfig
from electrock_infer_amd.harness.feguvik import FeguvikConfig, FeguvikForCausalLM
from electrock_infer_amd.harness.kv_pool import KVBlockPool, StateSlotPool
from electrock_infer_amd.harness.registry import checkpoint_shapes, load_config
from electrock_infer_amd.harness.sequence import Sequence
from electrock_infer_amd.utils import load_model
from tests.feguvik_util import CONFIGS, make_model, write_checkpoint

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
BS = 4


@pytest.fixture(autouse=True)
def small_blocks():
    old, Sequence.block_size = Sequence.block_size, BS
    yield
    Sequence.block_size = old


def seq(n, first=0, **kw):
    return Sequence(list(range(first, first + n)), SamplingParams(**kw))


# ---- registry, configuration, weights ----
def test_config_is_read_from_the_checkpoint(tmp_path):
    path, raw, _ = make_model(tmp_path / "m", "odd")
    cfg = load_config(path, "float32")
    assert isinstance(cfg, FeguvikConfig) and cfg.torch_dtype == torch.float32
    assert (cfg.vocab_size, cfg.width, cfg.side_dim, cfg.norm_eps, cfg.embedding_scale) == (101, 90, 5, 1e-5, 1.7)
    assert [l.ff for l in cfg.layers] == [70, 0, 33, 50] and [l.decay_rank for l in cfg.layers] == [0, 7, 0, 7]
    assert cfg.runs() == [(0, None), (1, 0), (2, 0), (1, 1), (2, 1), (1, 2), (2, 2), (3, None)] and cfg.has_recurrent_state
    assert load_config(make_model(tmp_path / "p", "plain")[0]).loop is None
    shapes = checkpoint_shapes(path)
    assert shapes["l1.mix.a2"] == (38, 7) and shapes["loop.in"] == (90, 180)


@pytest.mark.parametrize("edit,what", [(lambda c: c.update(architecture="Nothing"), "no registered"),
                                       (lambda c: c["layers"][0].update(type="conv"), "unknown mixer"),
                                       (lambda c: c["layers"][0]["mlp"].update(kind="moe"), "unknown feed-forward")])
def test_unknown_designs_are_refused(tmp_path, edit, what):
    path, raw, _ = make_model(tmp_path / "m", "odd")
    raw = json.loads(json.dumps(raw))
    edit(raw)
    (tmp_path / "m" / "config.json").write_text(json.dumps(raw))
    with pytest.raises(ValueError, match=what):
        load_config(path)


def test_mixtral_is_registered_too(tmp_path):
    (tmp_path / "config.json").write_text(json.dumps({"architectures": ["MixtralForCausalLM"], "hidden_size": 512, "vocab_size": 77,
                                                       "num_hidden_layers": 3, "something_else": 1}))
    cfg = load_config(str(tmp_path))
    assert isinstance(cfg, ModelConfig) and (cfg.hidden_size, cfg.vocab_size, cfg.num_hidden_layers) == (512, 77, 3)
    with pytest.raises(ValueError, match="bfloat16"):
        load_config(str(tmp_path), "float32")


@pytest.mark.parametrize("name", sorted(CONFIGS))
@pytest.mark.parametrize("dtype", ["bfloat16", "float32"])
def test_weights_reach_their_parameters(tmp_path, name, dtype):
    path, raw, w = make_model(tmp_path / "m", name)
    model = FeguvikForCausalLM(load_config(path, dtype))
    assert sorted(load_model(model, path)) == sorted(w)
    assert torch.equal(model.head.float(), w["head"]) and model.head.dtype == getattr(torch, dtype)
    for i, layer in enumerate(model.layers):
        p = layer.mix.in_proj
        for section in p.rows:
            a = p.offset[section]
            assert a % 8 == 0 and torch.equal(p.weight[a:a + p.rows[section]].float(), w[f"l{i}.mix.{section}"])
        assert torch.equal(layer.post1, w[f"l{i}.norm1b"] * w[f"l{i}.ls1"]) and layer.norm1.dtype == torch.float32
        assert (layer.mlp is None) == (raw["layers"][i]["mlp"] is None)
        if raw["layers"][i]["type"] == "latent_attention":
            m = raw["layers"][i]["mixer"]
            t = layer.mix.uk_t
            assert t.shape == (m["heads"], m["kv_rank"], -(-m["dim"] // 32) * 32) and not t[:, :, m["dim"]:].any()
            uk = w[f"l{i}.mix.uk"].view(m["heads"], m["dim"], m["kv_rank"])
            assert torch.equal(t[:, :, :m["dim"]].float(), uk.transpose(1, 2))


def test_missing_unknown_and_misshapen_tensors_are_errors(tmp_path):
    path, cfg, w = make_model(tmp_path / "m", "plain")
    bf = {k: v.to(torch.bfloat16) for k, v in w.items()}
    def load(tensors):
        return load_model(FeguvikForCausalLM(load_config(path)), write_checkpoint(tmp_path / "x", cfg, tensors))
    with pytest.raises(KeyError, match="lacks.*l1.mix.sink"):
        load({k: v for k, v in bf.items() if k != "l1.mix.sink"})
    with pytest.raises(KeyError, match="l1.mix.w"):
        load({**bf, "l1.mix.w": bf["head"].clone()})
    with pytest.raises(ValueError, match="l0.mlp.up"):
        load({**bf, "l0.mlp.up": bf["l0.mlp.up"][:-1].contiguous()})
    with pytest.raises(ValueError, match="projection 'q'"):
        load({**bf, "l0.mix.q": bf["l0.mix.q"][:-1].contiguous()})


# ---- batches, slots, portions ----
def test_ragged_batch_describes_portions():
    pool = KVBlockPool(32, BS, reuse_prefix=False)
    a, b, c = seq(11), seq(3, 50), seq(9, 100)
    for i, (s, start, n) in enumerate(((a, 4, 7), (b, 0, 3), (c, 8, 1))):
        pool.admit(s)
        s.num_computed_tokens, s.num_scheduled_tokens, s.state_slot = start, n, 5 + i
    r = make_ragged([a, b, c], BS, 3, "cpu")
    assert r.tokens.tolist() == [4, 5, 6, 7, 8, 9, 10, 50, 51, 52, 108] and r.positions.tolist() == [4, 5, 6, 7, 8, 9, 10, 0, 1, 2, 8]
    assert r.q_begin.tolist() == [0, 7, 10, 11] and r.starts.tolist() == [4, 0, 8] and r.state_slots.tolist() == [5, 6, 7]
    assert (r.max_q, r.max_context, r.table_width, r.n_chunks) == (7, 11, 3, 5)
    assert r.chunks.tolist() == [[0, 0, 3, 0], [0, 3, 3, 0], [0, 6, 1, 0], [1, 7, 3, 0], [2, 10, 1, 0]]
    assert r.seq_chunks.tolist() == [0, 3, 4, 5] and r.logit_rows.tolist() == [6, 9, 10]
    assert r.cache_rows.tolist()[:7] == [a.block_table[p // BS] * BS + p % BS for p in range(4, 11)]
    assert r.tables[1].tolist() == b.block_table + [0, 0] and r.k_lens.tolist() == [11, 3, 9]
    assert r.k_begin.tolist() == [0, 64, 128, 192] and r.padded_keys == 192
    assert make_ragged([b], BS, 3, "cpu", rows=[0, 2]).logit_rows.tolist() == [0, 2]
    b.num_scheduled_tokens = 4
    with pytest.raises(ValueError, match="blocks"):
        make_ragged([b], BS, 3, "cpu")


def test_state_slots_and_blocks_without_reuse():
    slots = StateSlotPool(2)
    a, b = seq(4), seq(4)
    slots.take(a), slots.take(b)
    assert {a.state_slot, b.state_slot} == {0, 1} and slots.num_free == 0
    slots.give_back(a)
    slots.give_back(a)                                  # nothing held: nothing happens
    assert slots.num_free == 1 and a.state_slot == -1
    pool = KVBlockPool(8, BS, reuse_prefix=False)
    pool.admit(a), pool.admit(b)
    assert not set(a.block_table) & set(b.block_table) and b.num_cached_tokens == 0      # equal prompts share nothing
    a.token_ids += [1] * 6
    assert pool.can_extend(a)
    pool.extend(a)
    assert len(a.block_table) == 3 and pool.num_free == 4


def config_for(blocks, **kw):
    model = FeguvikConfig(vocab_size=1000, width=8, layers=[], norm_eps=1e-6)
    model.layers = [type("L", (), {"kind": "gla"})()]
    return EngineConfig(model=model, num_kvcache_blocks=blocks, kvcache_block_size=BS, **kw)


def test_portions_slots_and_preemption_in_the_planner():
    cfg = config_for(8, max_num_seqs=2, max_num_batched_tokens=10, prefill_portion=6)
    assert not cfg.reuse_prefix and cfg.num_state_slots == 2
    pl = BatchPlanner(cfg)
    a, b, c = seq(13, max_tokens=9, ignore_eos=True), seq(5, max_tokens=3, ignore_eos=True), seq(3, max_tokens=3, ignore_eos=True)
    for s in (a, b, c):
        pl.submit(s)
    p = pl.plan()                                       # 6 of a's 13 tokens, then the rest of the budget for b; c has no slot
    assert p.is_prefill and [(s is a, s.num_scheduled_tokens) for s in p.seqs] == [(True, 6), (False, 4)] and pl.slots.num_free == 0
    assert pl.commit(p.seqs, [9, 9]) == [] and len(a) == 13 and len(b) == 5             # no token sampled in mid-prompt
    p = pl.plan()
    assert p.is_prefill and [(s.num_computed_tokens, s.num_scheduled_tokens) for s in p.seqs] == [(6, 6), (4, 1)]
    pl.commit(p.seqs, [9, 77])
    assert len(a) == 13 and b.token_ids[-1] == 77
    p = pl.plan()                                       # a's last portion goes before b's decoding
    assert p.is_prefill and p.seqs == [a] and a.num_scheduled_tokens == 1
    pl.commit(p.seqs, [88])
    p = pl.plan()
    assert not p.is_prefill and p.seqs == [a, b] and all(s.num_scheduled_tokens == 1 for s in p.seqs)
    assert a.num_computed_tokens == 13 and b.num_computed_tokens == 5
    pl.commit(p.seqs, [1, 2])
    pl._evict(pl.running.pop())                          # b gives its place: slot and blocks go back, it starts over
    assert b.state_slot == -1 and b.num_computed_tokens == 0 and pl.slots.num_free == 1 and not b.block_table
    p = pl.plan()
    assert p.is_prefill and p.seqs == [b] and b.num_scheduled_tokens == 6 and len(b) == 7   # prompt and completion again
    pl.commit(p.seqs, [5])
    p = pl.plan()                                       # its last token is a completion token, and still prefill
    assert p.is_prefill and b.num_scheduled_tokens == 1 and b.num_computed_tokens == 6
    assert pl.commit(p.seqs, [6]) == [b] and pl.slots.num_free == 1
    while not pl.idle():
        p = pl.plan()
        pl.commit(p.seqs, [0] * len(p.seqs))
    assert pl.pool.num_free == 8 and pl.slots.num_free == 2 and len(c) == 6


class _CountingRunner:
    """Next token = number of tokens computed so far; checks that portions join up."""

    def __init__(self):
        self.seen = {}

    def run(self, seqs, is_prefill, return_logits=False):
        for s in seqs:
            assert self.seen.get(s.seq_id, 0) == s.num_computed_tokens and s.num_scheduled_tokens > 0
            self.seen[s.seq_id] = s.num_computed_tokens + s.num_scheduled_tokens
        return [self.seen[s.seq_id] for s in seqs]


@pytest.mark.parametrize("portion", [1, 2, 5, 64])
def test_engine_generates_with_portions(portion):
    runner = _CountingRunner()
    eng = LLMEngine(ModelConfig(), model_runner=runner, num_kvcache_blocks=64, kvcache_block_size=BS, max_num_seqs=4,
                    max_num_batched_tokens=16, prefill_portion=portion)
    outs = eng.generate([list(range(40)), [7], list(range(9))], SamplingParams(temperature=0.0, max_tokens=3, ignore_eos=True))
    assert [o["token_ids"] for o in outs] == [[40, 41, 42], [1, 2, 3], [9, 10, 11]]
    with pytest.raises(ValueError, match="vocabulary"):
        eng.add_request([1, 32000], SamplingParams())


# ---- trace replay ----
class _EchoRunner:
    def __init__(self, config):
        self.config = config

    def portion_logits(self, seqs, rows):
        flat = [float(t) for s in seqs for t in s.token_ids[s.num_computed_tokens:s.num_computed_tokens + s.num_scheduled_tokens]]
        return torch.tensor(flat)[rows].unsqueeze(1).expand(-1, 3)


def test_trace_replay_books_portions_and_gives_everything_back(monkeypatch):
    monkeypatch.setattr(trace_module, "ModelRunner", _EchoRunner)
    monkeypatch.setattr(torch.cuda, "synchronize", lambda: None)
    r = trace_module.TraceReplay(config_for(6, max_num_seqs=3, reuse_prefix=False))
    out = r.step([{"id": "a", "tokens": [5, 6, 7], "want": [0, 2]}, {"id": "b", "tokens": [9], "want": [0]}], [])
    assert out[:, 0].tolist() == [5, 7, 9] and r.live["a"].num_computed_tokens == 3
    assert r.step([{"id": "a", "tokens": [1, 2, 3, 4], "want": []}], ["b"]) is None
    assert len(r.live["a"].block_table) == 2 and set(r.live) == {"a"}
    with pytest.raises(ValueError, match="vocabulary"):
        r.step([{"id": "c", "tokens": [1000], "want": []}], [])
    with pytest.raises(ValueError, match="want"):
        r.step([{"id": "a", "tokens": [1], "want": [1]}], [])
    r.step([], ["a"])
    assert not r.live and r.planner.pool.num_free == 6 and r.planner.slots.num_free == 3


# ---- C surface of the decoder library ----
def _header():
    return re.sub(r"/\*.*?\*/", "", open(os.path.join(ROOT, "include", "electrock_decoder.h")).read(), flags=re.S)


def test_decoder_library_exports_what_its_header_declares():
    names = sorted(set(re.findall(r"\b(ed_[a-z0-9_]+)\s*\(", _header())))
    assert names == sorted(_lib.DECODER_SYMBOLS)
    lib = _lib.load_decoder()
    assert all(getattr(lib, n) is not None for n in names) and lib.ed_version() >= 100


def test_argument_structs_match_the_header():
    for struct, mirror in (("ed_gla_args", _lib.GlaArgs), ("ed_latent_args", _lib.LatentArgs),
                           ("ed_latent_prompt_args", _lib.LatentPromptArgs)):
        body = re.search(r"typedef struct %s \{(.*?)\} %s;" % (struct, struct), _header(), flags=re.S).group(1)
        fields = []
        for decl in body.split(";"):
            m = re.match(r"\s*(?:const\s+)?(void|float|int32_t|int64_t)\s*(.*)$", decl.strip(), flags=re.S)
            if m:
                for item in m.group(2).split(","):
                    star = "*" in item
                    ctype = ctypes.c_void_p if star else {"float": ctypes.c_float, "int32_t": ctypes.c_int32,
                                                          "int64_t": ctypes.c_int64}[m.group(1)]
                    fields.append((item.replace("*", "").strip(), ctype))
        assert fields == list(mirror._fields_), struct


def test_decoder_argument_errors_are_reported_before_any_launch():
    lib, F32, BF16, F16 = _lib.load_decoder(), 0, 1, 2
    assert lib.ed_embed(None, None, 1.0, None, None, 0, 4, 8, F16, None) == -3
    assert lib.ed_embed(None, None, 1.0, None, None, 0, 4, 1 << 20, BF16, None) == -2
    assert lib.ed_embed(None, None, 1.0, None, None, 0, 4, 8, BF16, None) == -1
    assert lib.ed_residual_norm(3, None, None, BF16, 1, None, None, None, 0, 1, 8, 1e-6, BF16, None) == -2
    assert lib.ed_residual_norm(1, None, None, BF16, 1, None, None, None, 0, 1, 8, 1e-6, F32, None) == -3
    assert lib.ed_token_gate(None, None, None, None, 8, 4, None, 1, 16, 5, BF16, None) == -2           # columns 4 .. 8 of 8
    assert lib.ed_residual_norm(1, None, None, BF16, 2, None, None, None, 0, 1, 8, 1e-6, BF16, None) == -2    # partial sums are float32
    assert lib.ed_relu_squared(None, 0, BF16, None) == 0
    assert lib.ed_skinny_gemm_splits(65, 64, 64) == 0 and lib.ed_skinny_gemm_splits(33, 4096, 4096) == 0 and lib.ed_skinny_gemm_splits(4, 64, 100) == 0
    assert lib.ed_skinny_gemm_splits(64, 2048, 2048) > 1 and lib.ed_skinny_gemm_splits(64, 64, 64) == 1
    assert lib.ed_skinny_gemm(None, None, None, BF16, 2, 4, 64, 128, 0, None) == -2
    assert lib.ed_skinny_gemm(None, None, None, BF16, 1, 4, 64, 128, 0, None) == -1
    assert lib.ed_skinny_gemm(None, None, None, BF16, 1, 4, 64, 100, 0, None) == -4
    g = _lib.GlaArgs(n_seqs=1, heads=2, dim=300, vdim=8, rank=4, a2_stride=4, dtype=BF16, tau=1.0)
    assert lib.ed_gla_step(ctypes.byref(g), None) == -4
    g.dim = 8
    assert lib.ed_gla_step(ctypes.byref(g), None) == -1 and lib.ed_gla_prefill(ctypes.byref(g), None) == -1
    g.tau = 0.0
    assert lib.ed_gla_step(ctypes.byref(g), None) == -2
    l = _lib.LatentArgs(T=1, heads=2, dim=8, rot=3, rank=8, dtype=BF16)
    assert lib.ed_latent_prepare(ctypes.byref(l), None) == -4                          # odd rotation
    l.rot = 4
    assert lib.ed_latent_prepare(ctypes.byref(l), None) == -1 and lib.ed_latent_paged(ctypes.byref(l), None) == -2
    assert lib.ed_latent_row_elems(9, 2) == 24 and lib.ed_latent_row_elems(16, 0) == 16
    assert lib.ed_latent_prompt_supported(64, 32, 64) == 1 and lib.ed_latent_prompt_supported(22, 6, 20) == 0
    assert lib.ed_head_gemm(None, 1, 1, None, None, 1, 1, 1, 0, 1, 1, BF16, None) == -2


def test_missing_decoder_library_fails_loudly(monkeypatch, tmp_path):
    monkeypatch.setattr(_lib, "_decoder_lib", None)
    monkeypatch.setattr(_lib, "DECODER_LIB_PATH", str(tmp_path / "nope.so"))
    with pytest.raises(RuntimeError, match="no fallback"):
        _lib.load_decoder()
