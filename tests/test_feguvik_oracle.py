"""The oracle of the Feguvik decoder against other formulations of the same equations (CPU)."""
import math

import pytest
import torch

from oracle import feguvik_oracle as F
from tests.feguvik_util import CONFIGS, draw_tokens, random_weights

torch.manual_seed(0)


def test_norm_and_activations_against_torch():
    x, w = torch.randn(5, 48), torch.randn(48)
    assert torch.allclose(F.rms_norm(x, w, 1e-3), torch.nn.functional.rms_norm(x, (48,), w, 1e-3), atol=1e-6)
    tiny = torch.full((1, 4), 1e-4)                     # eps inside the root decides
    assert torch.allclose(F.rms_norm(tiny, torch.ones(4), 1e-6), tiny / math.sqrt(1e-8 + 1e-6))
    assert torch.allclose(F.gelu_tanh(x), torch.nn.functional.gelu(x, approximate="tanh"), atol=1e-6)
    assert torch.equal(F.relu_squared(torch.tensor([-2.0, 0.0, 3.0])), torch.tensor([0.0, 0.0, 9.0]))


def test_recurrence_against_its_quadratic_form():
    """o_t = sum_s<=t sum_d q_td (prod of alpha between) k_sd v_s"""
    n, H, d, v = 9, 2, 5, 3
    q, k, val, a = torch.randn(n, H, d), torch.randn(n, H, d), torch.randn(n, H, v), torch.rand(n, H, d)
    want = torch.zeros(n, H, v)
    for t in range(n):
        for s in range(t + 1):
            gap = torch.ones(H, d)
            for u in range(s + 1, t + 1):
                gap = gap * a[u]
            want[t] += (q[t] * gap * k[s]).sum(-1, keepdim=True) * val[s]
    assert torch.allclose(F.gated_linear_recurrence(q, k, val, a), want, atol=1e-5)
    assert torch.allclose(F.decay_per_channel(torch.tensor([0.0, 30.0]), 4.0), torch.tensor([0.5 ** 0.25, 1.0]))


def test_rotation_is_complex_multiplication():
    x, pos = torch.randn(6, 2, 8, dtype=torch.float64), torch.tensor([0, 1, 2, 7, 100, 5000])
    z = torch.complex(x[..., :4], x[..., 4:])
    freq = 300.0 ** (-torch.arange(4, dtype=torch.float64) / 4)
    turned = z * torch.exp(1j * pos[:, None, None] * freq)
    want = torch.cat((turned.real, turned.imag), -1)
    assert torch.allclose(F.rotate_half(x, pos, 300.0), want)
    assert torch.equal(F.rotate_half(x, pos, 300.0)[0], x[0])


def test_sink_is_a_key_without_a_value():
    s = torch.randn(4, 7)
    p = F.softmax_with_sink(s, 0.7)
    full = torch.softmax(torch.cat((s, torch.full((4, 1), 0.7)), -1), -1)
    assert torch.allclose(p, full[:, :-1]) and torch.allclose(1 - p.sum(-1), full[:, -1])
    assert F.softmax_with_sink(torch.full((1, 2), -500.0), 400.0).sum() == 0          # no overflow either way
    assert torch.allclose(F.softmax_with_sink(torch.tensor([[300.0, 300.0]]), -400.0), torch.tensor([[0.5, 0.5]]))


def test_latent_attention_against_library_attention():
    """With the keys and values written out it is attention with one more key of score `sink` and value zero."""
    n, W, H, d, r, v, c = 11, 24, 3, 6, 4, 5, 9
    m = {"heads": H, "dim": d, "rot_dim": r, "vdim": v, "kv_rank": c, "scale": 0.3, "rot": {"base": 100.0, "dims": r}}
    w = {"m." + k: torch.randn(*s) for k, s in {"q": (H * (d + r), W), "dkv": (c + r, W), "dkv.norm": (c,), "uk": (H * d, c),
                                               "uv": (H * v, c), "sink": (H,), "o": (W, H * v)}.items()}
    h = torch.randn(n, W)
    got = F.latent_attention(h, w, "m.", m, 1e-5)
    pos = torch.arange(n)
    q = (h @ w["m.q"].t()).view(n, H, d + r)
    q = torch.cat((q[..., :d], F.rotate_half(q[..., d:], pos, 100.0)), -1)
    down = h @ w["m.dkv"].t()
    lat = torch.nn.functional.rms_norm(down[:, :c], (c,), w["m.dkv.norm"], 1e-5)
    k = torch.cat(((lat @ w["m.uk"].t()).view(n, H, d), F.rotate_half(down[:, c:], pos, 100.0)[:, None].expand(n, H, r)), -1)
    val = (lat @ w["m.uv"].t()).view(n, H, v)
    bias = torch.zeros(H, n, n + 1).masked_fill(torch.ones(n, n + 1).triu(1).bool(), float("-inf"))
    bias[:, :, n] = w["m.sink"][:, None]
    k = torch.cat((k, torch.zeros(1, H, d + r)))
    val = torch.cat((val, torch.zeros(1, H, v)))
    o = torch.nn.functional.scaled_dot_product_attention(q.transpose(0, 1), k.transpose(0, 1), val.transpose(0, 1), bias, scale=0.3)
    assert torch.allclose(got, o.transpose(0, 1).reshape(n, H * v) @ w["m.o"].t(), atol=1e-4)


def test_order_of_layer_runs():
    layers = [None] * 5
    assert F.layer_runs({"layers": layers}) == [(i, None) for i in range(5)]
    assert F.layer_runs({"layers": layers, "loop": {"start": 1, "stop": 3, "times": 2}}) == [
        (0, None), (1, 0), (2, 0), (1, 1), (2, 1), (3, None), (4, None)]


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_model_is_causal_and_every_weight_matters(name):
    cfg, rank = CONFIGS[name]
    w = {k: v.double() for k, v in random_weights(cfg, rank).items()}
    toks = draw_tokens(cfg, 14)
    layers = []
    full = F.forward(toks, w, cfg, torch.float64, layers)
    assert len(layers) == len(F.layer_runs(cfg)) and full.shape == (14, cfg["vocab"])
    assert torch.allclose(F.forward(toks[:9], w, cfg, torch.float64), full[:9])
    for key in w:
        # (the only head's sink scales the mixer's whole output, which the norm behind it takes out again)
        lone_sink = key.endswith("sink") and w[key].numel() == 1
        if not key.startswith(("embed", "side.embed")) and not lone_sink:
            changed = dict(w)
            changed[key] = w[key] * 1.5 + 0.01
            assert not torch.allclose(F.forward(toks, changed, cfg, torch.float64)[-1], full[-1], atol=1e-6), key
