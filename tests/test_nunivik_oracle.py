"""The oracle of the Nunivik decoder against other formulations of the same equations (CPU)."""
import math

import pytest
import torch
import torch.nn.functional as F

from oracle import nunivik_oracle as N
from tests.feguvik_util import draw_tokens
from tests.nunivik_util import CONFIGS, random_weights

torch.manual_seed(0)
F64 = torch.float64


def rnd(*shape):
    return torch.randn(shape, dtype=F64)


def test_norms_and_activations_against_torch():
    x, w = rnd(5, 48), rnd(48)
    assert torch.allclose(N.rms_norm(x, w, 1e-3), F.rms_norm(x, (48,), w, 1e-3))
    assert torch.allclose(N.rms_norm(torch.full((1, 4), 1e-4, dtype=F64), torch.ones(4), 1e-6), torch.tensor(1e-4 / math.sqrt(1e-8 + 1e-6), dtype=F64))
    assert torch.allclose(N.silu(x), F.silu(x)) and torch.allclose(N.softplus(x * 20), F.softplus(x * 20), atol=1e-6)
    assert torch.allclose(N.unit(x), F.normalize(x, dim=-1), atol=1e-6)
    assert torch.allclose(N.unit(torch.full((1, 4), 1e-3, dtype=F64)), torch.tensor(1e-3 / math.sqrt(4e-6 + 1e-6), dtype=F64))
    y, z = rnd(5, 48), rnd(5, 48)
    want = F.rms_norm((y * F.silu(z)).view(5, 3, 16), (16,), None, 1e-3).view(5, 48) * w
    assert torch.allclose(N.gated_group_norm(y, z, w, 3, 1e-3), want)


def test_rotation_is_complex_multiplication_of_neighbours():
    x, pos = rnd(6, 2, 11), torch.tensor([0, 1, 2, 7, 100, 5000])
    got = N.rotate_pairs(x, pos, {"base": 300.0, "dims": 8, "scaling": {"factor": 2.5}})
    z = torch.complex(x[..., 0:8:2], x[..., 1:8:2])
    turned = z * torch.exp(1j * pos[:, None, None] * (300.0 ** (-torch.arange(4, dtype=F64) / 4) / 2.5))
    assert torch.allclose(torch.stack((turned.real, turned.imag), -1).flatten(-2), got[..., :8])
    assert torch.equal(got[..., 8:], x[..., 8:]) and torch.equal(N.rotate_pairs(x, pos, None), x)
    assert not torch.allclose(N.rotate_pairs(x, pos, {"base": 300.0, "dims": 8}), got)


def test_window_and_soft_cap():
    see = N.visible(6, 3)
    assert see.tolist() == [[0 <= i - j <= 2 for j in range(6)] for i in range(6)]
    assert torch.equal(N.visible(6, None), torch.ones(6, 6).tril().bool()) and torch.equal(N.visible(4, 1), torch.eye(4).bool())
    s = torch.tensor([-1e4, -3.0, 1e-3, 3.0, 1e4])
    assert torch.allclose(N.soft_cap(s, 2.0), torch.tensor([-2.0, -2 * math.tanh(1.5), 1e-3, 2 * math.tanh(1.5), 2.0]))
    assert torch.equal(N.soft_cap(s, None), s)


def test_attention_against_library_attention():
    n, W, H, G, d, v = 11, 24, 6, 2, 8, 5
    m = {"heads": H, "kv_heads": G, "dim": d, "vdim": v, "scale": 0.3, "rot": {"base": 100.0, "dims": 6}, "mask": {"size": 4}, "v_mix": True}
    w = {"m." + k: rnd(*s) for k, s in {"q": (H * d, W), "k": (G * d, W), "v": (G * v, W), "q.norm": (d,), "k.norm": (d,), "o": (W, H * v),
                                       "vmix": ()}.items()}
    h, first, carried = rnd(n, W), rnd(n, G, v), {}
    def library(values):
        pos = torch.arange(n)
        q = N.rotate_pairs(F.rms_norm((h @ w["m.q"].t()).view(n, H, d), (d,), w["m.q.norm"], 1e-5), pos, m["rot"])
        k = N.rotate_pairs(F.rms_norm((h @ w["m.k"].t()).view(n, G, d), (d,), w["m.k.norm"], 1e-5), pos, m["rot"])
        see = torch.tensor([[0 <= i - j < 4 for j in range(n)] for i in range(n)])
        rep = lambda t: t.repeat_interleave(H // G, 1).transpose(0, 1)
        o = F.scaled_dot_product_attention(q.transpose(0, 1), rep(k), rep(values), see, scale=0.3)
        return o.transpose(0, 1).reshape(n, H * v) @ w["m.o"].t()
    own = (h @ w["m.v"].t()).view(n, G, v)
    assert torch.allclose(N.attention(h, w, "m.", m, 1e-5, carried), library(own)) and torch.equal(carried["v"], own)
    lam = w["m.vmix"]
    assert torch.allclose(N.attention(h, w, "m.", m, 1e-5, {"v": first}), library((1 - lam) * own + lam * first))


def test_short_convolution_against_library_convolution():
    for taps, n in ((1, 5), (4, 9), (5, 3)):
        x, w, b = rnd(n, 7), rnd(7, taps), rnd(7)
        want = F.conv1d(F.pad(x.t()[None], (taps - 1, 0)), w[:, None], b, groups=7)[0].t()
        assert torch.allclose(N.short_convolution(x, w, b), want) and torch.allclose(N.short_convolution(x, w), want - b)


def test_delta_rule_against_its_triangular_system():
    """u solves (I + A) u = beta v with A_ts = beta_t (decay between) k_t . k_s; o_t = sum (decay between) (q_t . k_s) u_s"""
    n, H, d, v = 9, 2, 5, 3
    q, k, val, g, beta = rnd(n, H, d), rnd(n, H, d), rnd(n, H, v), torch.rand(n, H, dtype=F64), torch.rand(n, H, dtype=F64)
    got = N.gated_delta_recurrence(q, k, val, g, beta)
    for h in range(H):
        between = torch.tensor([[float(g[s + 1:t + 1, h].prod()) if s <= t else 0.0 for s in range(n)] for t in range(n)], dtype=F64)
        A = (beta[:, h, None] * between * (k[:, h] @ k[:, h].t())).tril(-1)
        u = torch.linalg.solve(torch.eye(n, dtype=F64) + A, beta[:, h, None] * val[:, h])
        assert torch.allclose(got[:, h], (between * (q[:, h] @ k[:, h].t())).tril() @ u)


def test_state_space_recurrence_against_its_quadratic_form():
    n, H, d, v = 9, 2, 5, 3
    C, B, x, a, dt, D = rnd(n, H, d), rnd(n, H, d), rnd(n, H, v), torch.rand(n, H, dtype=F64), torch.rand(n, H, dtype=F64), rnd(H)
    got = N.state_space_recurrence(C, B, x, a, dt, D)
    for h in range(H):
        between = torch.tensor([[float(a[s + 1:t + 1, h].prod()) if s <= t else 0.0 for s in range(n)] for t in range(n)], dtype=F64)
        assert torch.allclose(got[:, h], (between * (C[:, h] @ B[:, h].t())).tril() @ (dt[:, h, None] * x[:, h]) + D[h] * x[:, h])


def test_delta_mixer_writes_before_it_reads():
    """The first token's read-out is its own write: o = beta (k . q) v."""
    W, m = 12, {"heads": 2, "kv_heads": 1, "dim": 4, "vdim": 3, "conv": 2}
    w = {"m." + k: rnd(*s) for k, s in {"q": (4, W), "k": (4, W), "v": (6, W), "q.conv": (4, 2), "k.conv": (4, 2), "v.conv": (6, 2), "b": (2, W),
                                       "a": (2, W), "A_log": (2,), "dt_bias": (2,), "norm": (3,), "g": (6, W), "o": (W, 6)}.items()}
    h = rnd(1, W)
    conv = lambda x: F.silu((h @ w["m." + x].t()) * w[f"m.{x}.conv"][:, -1])
    q, k, v = F.normalize(conv("q"), dim=-1) / 2, F.normalize(conv("k"), dim=-1), conv("v").view(2, 3)
    o = torch.sigmoid(h @ w["m.b"].t()).view(2, 1) * (q * k).sum() * v
    o = F.rms_norm(o, (3,), w["m.norm"], 1e-9) * F.silu(h @ w["m.g"].t()).view(2, 3)
    assert torch.allclose(N.delta(h, w, "m.", m, 1e-9), o.reshape(1, 6) @ w["m.o"].t(), rtol=1e-3, atol=1e-4)


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_model_is_causal_and_every_weight_matters(name):
    cfg = CONFIGS[name]
    w = {k: v.double() for k, v in random_weights(cfg).items()}
    toks, layers = draw_tokens(cfg, 14), []
    full = N.forward(toks, w, cfg, F64, layers)
    assert len(layers) == len(cfg["layers"]) and full.shape == (14, cfg["vocab"])
    assert torch.allclose(N.forward(toks[:9], w, cfg, F64), full[:9])
    first_mix = next((i for i, l in enumerate(cfg["layers"]) if l["mixer"].get("v_mix")), None)
    for key in w:
        i = int(key[1:key.index(".")]) if key[0] == "l" else -1
        spec = cfg["layers"][i] if i >= 0 else None
        idle = key.endswith("vmix") and i == first_mix                     # nothing to mix with
        # a query that sees one key, and the decay of a head whose scale the norm behind it takes out again
        idle = idle or (spec and (spec["mixer"].get("mask") or {}).get("size") == 1 and key.split("mix.")[-1] in ("q", "k", "q.norm", "k.norm"))
        if not key.startswith("embed") and not idle:
            changed = dict(w)
            changed[key] = w[key] * 1.5 + 0.01
            assert not torch.allclose(N.forward(toks, changed, cfg, F64), full, atol=1e-7), key
