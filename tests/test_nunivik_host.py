"""Host side of the Nunivik model (no GPU): registry and configuration, weight loading, what it asks of cache and state,
argument checks of its kernels."""
import ctypes
import json
import re

import pytest
import torch

from electrock_infer_amd import _lib
from electrock_infer_amd.harness.config import EngineConfig
from electrock_infer_amd.harness.nunivik import NunivikConfig, NunivikForCausalLM
from electrock_infer_amd.harness.registry import build_model, load_config
from electrock_infer_amd.layers.attention import SoftmaxAttention
from electrock_infer_amd.layers.latent_attention import rotary_frequencies
from electrock_infer_amd.layers.recurrent import GatedDeltaRule, StateSpaceMixer
from electrock_infer_amd.utils import load_model
from tests.feguvik_util import write_checkpoint
from tests.nunivik_util import CONFIGS, make_model
from tests.test_feguvik_host import _header


def test_config_is_read_from_the_checkpoint(tmp_path):
    path, raw, _ = make_model(tmp_path / "m", "odd")
    cfg = load_config(path, "float32")
    assert isinstance(cfg, NunivikConfig) and cfg.torch_dtype == torch.float32
    assert (cfg.vocab_size, cfg.width, cfg.norm_eps, cfg.embedding_scale) == (101, 90, 1e-5, 1.7)
    assert [l.ff for l in cfg.layers] == [70, 0, 0, 33, 50, 0] and [l.kind for l in cfg.layers][:2] == ["attention", "delta"]
    model = build_model(EngineConfig(model=cfg))
    a, d, b, m, e, _ = (l.mix for l in model.layers)
    assert (a.heads, a.kv_heads, a.dim, a.vdim, a.window, a.softcap, a.rot, a.rotary_base, a.rotary_factor, a.mix_values) == \
        (6, 2, 22, 19, 7, 5.0, 10, 500.0, 1.5, False)
    assert (b.window, b.softcap, b.rotary_factor, b.mix_values) == (40, 0.0, 1.0, True) and (e.window, e.rot) == (0, 0)
    assert (d.heads, d.kv_heads, d.dim, d.vdim, d.taps, d.eps) == (6, 3, 19, 27, 5, 1e-5)
    assert (m.heads, m.kv_heads, m.dim, m.vdim, m.taps, m.norm_groups) == (6, 2, 21, 10, 2, 3)


@pytest.mark.parametrize("edit,what", [(lambda c: c.update(architecture="Nothing"), "no registered"),
                                       (lambda c: c["layers"][0].update(type="rwkv"), "unknown mixer"),
                                       (lambda c: c["layers"][0]["mlp"].update(kind="moe"), "unknown feed-forward"),
                                       (lambda c: c["layers"][4]["mixer"].update(vdim=9), "another size")])
def test_unknown_designs_are_refused(tmp_path, edit, what):
    path, raw, _ = make_model(tmp_path / "m", "odd")
    raw = json.loads(json.dumps(raw))
    edit(raw)
    (tmp_path / "m" / "config.json").write_text(json.dumps(raw))
    with pytest.raises(ValueError, match=what):
        load_config(path)


def test_impossible_sizes_are_refused():
    with pytest.raises(ValueError, match="share"):
        SoftmaxAttention(8, 3, 2, 4, 4, 1.0, 1e-6, torch.float32)
    with pytest.raises(ValueError, match="share"):
        GatedDeltaRule(8, 3, 2, 4, 4, 3, 1e-6, torch.float32)
    with pytest.raises(ValueError, match="equal parts"):
        StateSpaceMixer(8, 2, 1, 4, 5, 3, 3, 1e-6, torch.float32)


@pytest.mark.parametrize("name", sorted(CONFIGS))
@pytest.mark.parametrize("dtype", ["bfloat16", "float32"])
def test_weights_reach_their_parameters(tmp_path, name, dtype):
    path, raw, w = make_model(tmp_path / "m", name)
    cfg = load_config(path, dtype)
    model = NunivikForCausalLM(cfg)
    assert sorted(load_model(model, path)) == sorted(w) == sorted(model.expected_tensors())
    assert torch.equal(model.head.float(), w["head"]) and model.head.dtype == getattr(torch, dtype)
    kinds = {l["type"] for l in raw["layers"]}
    block, slot = model.cache_bytes(32)
    assert (block > 0) == ("attention" in kinds) and (slot > 0) == cfg.has_recurrent_state == bool(kinds & {"delta", "mamba2"})
    for i, layer in enumerate(model.layers):
        p, mix, m, kind = f"l{i}.", layer.mix, raw["layers"][i]["mixer"], raw["layers"][i]["type"]
        section = lambda n: mix.in_proj.weight[mix.in_proj.offset[n]:mix.in_proj.offset[n] + mix.in_proj.rows[n]].float()
        assert all(at % 8 == 0 for at in mix.in_proj.offset.values()) and torch.equal(layer.norm1, w[p + "norm1"])
        if layer.mlp is not None:
            assert torch.equal(layer.mlp.up.float(), torch.cat((w[p + "mlp.gate"], w[p + "mlp.up"])))
        if kind == "mamba2":
            inner, shared = m["heads"] * m["vdim"], m["groups"] * m["state"]
            z, x, B, C, dt = w[p + "mix.in"].split([inner, inner, shared, shared, m["heads"]])
            for n, want in (("z", z), ("v", x), ("k", B), ("q", C), ("decay", dt)):
                assert torch.equal(section(n), want)
            x, B, C = w[p + "mix.conv"].split([inner, shared, shared])
            assert torch.equal(mix.conv, torch.cat((C, B, x))) and mix.conv.dtype == torch.float32
            x, B, C = w[p + "mix.conv.b"].split([inner, shared, shared])
            assert torch.equal(mix.conv_bias, torch.cat((C, B, x))) and torch.equal(mix.skip, w[p + "mix.D"])
        elif kind == "delta":
            for n, want in (("q", "q"), ("k", "k"), ("v", "v"), ("gate", "g"), ("decay", "a"), ("beta", "b")):
                assert torch.equal(section(n), w[p + "mix." + want])
            assert torch.equal(mix.conv, torch.cat([w[p + f"mix.{x}.conv"] for x in "qkv"])) and mix.conv_bias is None
            assert torch.equal(mix.a_log, w[p + "mix.A_log"]) and torch.equal(mix.dt_bias, w[p + "mix.dt_bias"])
        else:
            rot = m.get("rot", {"dims": 0, "base": 1.0})
            want = rotary_frequencies(rot["dims"], rot["base"]) / rot.get("scaling", {"factor": 1.0})["factor"]
            assert torch.allclose(mix.inv_freq, want, rtol=1e-6)
            if m["v_mix"]:
                assert mix.vmix.shape == () and torch.equal(mix.vmix, w[p + "mix.vmix"])


def test_missing_unknown_and_misshapen_tensors_are_errors(tmp_path):
    path, cfg, w = make_model(tmp_path / "m", "plain")
    bf = {k: v.to(torch.bfloat16) for k, v in w.items()}
    def load(tensors):
        return load_model(NunivikForCausalLM(load_config(path)), write_checkpoint(tmp_path / "x", cfg, tensors))
    for name in ("l0.mix.in", "l0.mix.D", "l1.mix.k.conv", "l2.mix.vmix", "l3.mlp.gate", "final.norm"):
        with pytest.raises(KeyError, match=f"lacks.*{name}"):
            load({k: v for k, v in bf.items() if k != name})
    for name in ("l2.mix.sink", "l2.mlp.up", "l9.norm1", "l0.mix.q"):
        with pytest.raises(KeyError, match=name):
            load({**bf, name: bf["head"].clone()})
    for name in ("l0.mix.in", "l1.mix.v.conv", "l3.mlp.up", "l3.mix.o", "l1.mix.A_log"):
        with pytest.raises(ValueError, match="expected"):
            load({**bf, name: bf[name][:-1].contiguous()})


def test_argument_structs_match_the_header():
    types = {"float": ctypes.c_float, "int32_t": ctypes.c_int32, "int64_t": ctypes.c_int64}
    for struct, mirror in (("ed_recur_args", _lib.RecurArgs), ("ed_attn_args", _lib.AttnArgs)):
        body = re.search(r"typedef struct %s \{(.*?)\} %s;" % (struct, struct), _header(), flags=re.S).group(1)
        fields = []
        for decl in body.split(";"):
            m = re.match(r"\s*(?:const\s+)?(void|float|int32_t|int64_t)\s*(.*)$", decl.strip(), flags=re.S)
            if m:
                fields += [(item.replace("*", "").strip(), ctypes.c_void_p if "*" in item else types[m.group(1)]) for item in m.group(2).split(",")]
        assert fields == list(mirror._fields_), struct


def test_argument_errors_are_reported_before_any_launch():
    lib, F32, BF16, F16 = _lib.load_decoder(), 0, 1, 2
    r = _lib.RecurArgs(n_seqs=1, heads=4, kv_heads=3, dim=16, vdim=16, taps=4, dtype=BF16)
    assert lib.ed_recur_step(ctypes.byref(r), None) == -4                       # heads that cannot be shared
    r.kv_heads = 2
    assert lib.ed_recur_step(ctypes.byref(r), None) == -1 and lib.ed_recur_prefill(ctypes.byref(r), None) == -1
    for field, bad in (("dim", 257), ("vdim", 300), ("taps", 17), ("taps", 0)):
        old = getattr(r, field)
        setattr(r, field, bad)
        assert lib.ed_recur_prefill(ctypes.byref(r), None) == -4, field
        setattr(r, field, old)
    r.dtype = F16
    assert lib.ed_recur_step(ctypes.byref(r), None) == -3
    a = _lib.AttnArgs(T=1, n_seqs=1, max_q=1, heads=4, kv_heads=2, dim=16, vdim=16, rot=6, splits=1, block_size=8, table_width=1, dtype=BF16)
    assert lib.ed_attn_prepare(ctypes.byref(a), None) == -1 and lib.ed_attn_paged(ctypes.byref(a), None) == -1
    for field, bad, code in (("rot", 5, -4), ("rot", 18, -4), ("kv_heads", 3, -4), ("dim", 260, -4), ("window", -1, -2), ("softcap", -1.0, -2), ("dtype", F16, -3)):
        old = getattr(a, field)
        setattr(a, field, bad)
        assert lib.ed_attn_paged(ctypes.byref(a), None) == code, field
        setattr(a, field, old)
    assert lib.ed_attn_row_elems(3, 9, 4) == 3 * 24 and lib.ed_recur_record(1) > lib.ed_recur_record(0) > 0
    assert lib.ed_attn_prompt_supported(256, 128) == 1 and lib.ed_attn_prompt_supported(64, 129) == 0
    assert lib.ed_silu_gate(None, None, 4, 8, F16, None) == -3 and lib.ed_silu_gate(None, None, 4, 8, BF16, None) == -1
    assert lib.ed_gated_norm(None, None, 15, None, 1, 2, 8, 1e-6, BF16, None) == -2       # rows of z shorter than y's
    assert lib.ed_gated_norm(None, None, 16, None, 1, 2, 8, 1e-6, BF16, None) == -1
    assert lib.ed_skinny_gemm(None, None, None, F32, 1, 4, 64, 128, 2, None) == -2        # the gated form stores bf16
