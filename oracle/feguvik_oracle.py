"""CPU restatement, in plain float32 (or float64) torch, of the Feguvik decoder.  TEST INFRASTRUCTURE ONLY: imported by
tests/ (and by nothing in the product path).

One function per mechanism, each written from its equation and sharing no code with the kernels' callers.  There is no
cache and no portioning here: every call computes a whole sequence from position 0, token by token where the mechanism
is a recurrence, which is what cached, portioned and batched execution must be equivalent to.

Weights are a dict of tensors under the checkpoint's names ('embed', 'l0.mix.q', 'loop.in', ...); `cfg` is the parsed
config.json (a dict).
"""
import math
from typing import Dict, List, Optional

import torch

Weights = Dict[str, torch.Tensor]


def rms_norm(x: torch.Tensor, weight: torch.Tensor, eps: float) -> torch.Tensor:
    """x / sqrt(mean(x^2) + eps) * w over the last dimension."""
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps) * weight


def gelu_tanh(z: torch.Tensor) -> torch.Tensor:
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def relu_squared(z: torch.Tensor) -> torch.Tensor:
    return torch.where(z > 0, z * z, torch.zeros_like(z))


def decay_per_channel(z: torch.Tensor, tau: float) -> torch.Tensor:
    """alpha = sigmoid(z)^(1/tau)."""
    return torch.pow(torch.sigmoid(z), 1.0 / tau)


def gated_linear_recurrence(q, k, v, alpha) -> torch.Tensor:
    """q, k, alpha [n, heads, dim], v [n, heads, vdim]: S_t = diag(alpha_t) S_(t-1) + k_t v_t^T, o_t = S_t^T q_t,
    starting from S = 0."""
    n, heads, dim = q.shape
    state = torch.zeros(heads, dim, v.shape[-1], dtype=q.dtype)
    out = torch.empty_like(v)
    for t in range(n):
        state = alpha[t][:, :, None] * state + k[t][:, :, None] * v[t][:, None, :]
        out[t] = (state * q[t][:, :, None]).sum(dim=1)
    return out


def gated_linear_attention(h: torch.Tensor, w: Weights, prefix: str, m: dict, eps: float) -> torch.Tensor:
    """The whole 'gla' mixer on h [n, width]; `prefix` is '<layer>.mix.'."""
    n = h.shape[0]
    heads, dim, vdim = m["heads"], m["dim"], m["vdim"]
    q = (h @ w[prefix + "q"].t()).view(n, heads, dim) * dim ** -0.5
    k = (h @ w[prefix + "k"].t()).view(n, heads, dim)
    v = (h @ w[prefix + "v"].t()).view(n, heads, vdim)
    z = (h @ w[prefix + "a1"].t()) @ w[prefix + "a2"].t() + w[prefix + "a2.b"]
    o = gated_linear_recurrence(q, k, v, decay_per_channel(z, m["tau"]).view(n, heads, dim))
    o = rms_norm(o, w[prefix + "norm"], eps).reshape(n, heads * vdim)
    g = h @ w[prefix + "g"].t()
    return (o * (g * torch.sigmoid(g))) @ w[prefix + "o"].t()


def rotate_half(x: torch.Tensor, positions: torch.Tensor, base: float) -> torch.Tensor:
    """x [n, ..., dims]: the pair (x[i], x[i + dims/2]) turns by the angle position * base^(-2i/dims)."""
    dims = x.shape[-1]
    out = torch.empty_like(x)
    for i in range(dims // 2):
        a = positions.to(x.dtype) * (base ** (-2.0 * i / dims))
        c, s = torch.cos(a), torch.sin(a)
        c, s = (t.view([-1] + [1] * (x.dim() - 2)) for t in (c, s))
        u, v = x[..., i], x[..., i + dims // 2]
        out[..., i] = u * c - v * s
        out[..., i + dims // 2] = v * c + u * s
    return out


def softmax_with_sink(scores: torch.Tensor, sink: float) -> torch.Tensor:
    """Row-wise exp(s_j) / (sum_j exp(s_j) + exp(sink)): the sink takes weight and has no value."""
    top = torch.clamp(scores.max(dim=-1, keepdim=True).values, min=sink)
    e = torch.exp(scores - top)
    return e / (e.sum(dim=-1, keepdim=True) + torch.exp(torch.as_tensor(sink, dtype=scores.dtype) - top))


def latent_attention(h: torch.Tensor, w: Weights, prefix: str, m: dict, eps: float,
                     first_position: int = 0) -> torch.Tensor:
    """The whole 'latent_attention' mixer on h [n, width], with the keys and values of every head written out."""
    n = h.shape[0]
    heads, dim, rot, vdim, rank = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    pos = torch.arange(first_position, first_position + n)
    q = (h @ w[prefix + "q"].t()).view(n, heads, dim + rot)
    q_rot = rotate_half(q[..., dim:], pos, m["rot"]["base"])
    down = h @ w[prefix + "dkv"].t()
    c = rms_norm(down[:, :rank], w[prefix + "dkv.norm"], eps)
    k_rot = rotate_half(down[:, rank:], pos, m["rot"]["base"])
    k = (c @ w[prefix + "uk"].t()).view(n, heads, dim)
    v = (c @ w[prefix + "uv"].t()).view(n, heads, vdim)
    unseen = torch.ones(n, n, dtype=torch.bool).triu(1)
    outs = []
    for i in range(heads):
        s = (q[:, i, :dim] @ k[:, i].t() + q_rot[:, i] @ k_rot.t()) * m["scale"]
        p = softmax_with_sink(s.masked_fill(unseen, float("-inf")), float(w[prefix + "sink"][i]))
        outs.append(p @ v[:, i])
    return torch.cat(outs, dim=-1) @ w[prefix + "o"].t()


MIXERS = {"gla": gated_linear_attention, "latent_attention": latent_attention}


def feed_forward(h: torch.Tensor, w: Weights, prefix: str, m: dict) -> torch.Tensor:
    assert m["kind"] == "dense"
    return relu_squared(h @ w[prefix + "up"].t()) @ w[prefix + "down"].t()


def token_side_input(x: torch.Tensor, tokens: torch.Tensor, w: Weights, layer: int, dim: int, eps: float) -> torch.Tensor:
    """What layer `layer` adds to the stream from its slice of the tokens' side embedding."""
    e = w["side.embed"][tokens][:, layer * dim:(layer + 1) * dim]
    g = gelu_tanh(x @ w[f"l{layer}.side.gate"].t()) * e
    return rms_norm(g @ w[f"l{layer}.side.proj"].t(), w[f"l{layer}.side.norm"], eps)


def loop_entry(x: torch.Tensor, x0: torch.Tensor, w: Weights, t: int) -> torch.Tensor:
    """In front of pass t of the looped layers."""
    return torch.cat((x, x0), dim=-1) @ w["loop.in"].t() + w["loop.step"][t]


def layer_runs(cfg: dict) -> List[tuple]:
    """(layer, pass or None) in the order in which layers run."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    runs = [(i, None) for i in range(loop["start"])]
    for t in range(loop["times"]):
        runs += [(i, t) for i in range(loop["start"], loop["stop"])]
    return runs + [(i, None) for i in range(loop["stop"], n)]


def layer(x: torch.Tensor, tokens: torch.Tensor, w: Weights, cfg: dict, i: int) -> torch.Tensor:
    spec, eps, name = cfg["layers"][i], cfg["norm"]["eps"], f"l{i}."
    y = MIXERS[spec["type"]](rms_norm(x, w[name + "norm1"], eps), w, name + "mix.", spec["mixer"], eps)
    x = x + rms_norm(y, w[name + "norm1b"], eps) * w[name + "ls1"]
    if spec["mlp"] is not None:
        y = feed_forward(rms_norm(x, w[name + "norm2"], eps), w, name + "mlp.", spec["mlp"])
        x = x + rms_norm(y, w[name + "norm2b"], eps) * w[name + "ls2"]
    return x + token_side_input(x, tokens, w, i, cfg["token_side"]["dim"], eps)


def forward(tokens, w: Weights, cfg: dict, dtype=torch.float32, layers_out: Optional[list] = None) -> torch.Tensor:
    """Logits [n, vocab] of every position; the stream after every layer run is appended to `layers_out`."""
    w = {k: v.to(dtype) for k, v in w.items()}
    tokens = torch.as_tensor(tokens)
    x = w["embed"][tokens] * cfg["embedding"]["scale"]
    x0 = x
    for i, t in layer_runs(cfg):
        if t is not None and i == cfg["loop"]["start"]:
            x = loop_entry(x, x0, w, t)
        x = layer(x, tokens, w, cfg, i)
        if layers_out is not None:
            layers_out.append(x)
    return rms_norm(x, w["final.norm"], cfg["norm"]["eps"]) @ w["head"].t()
