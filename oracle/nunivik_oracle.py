"""CPU restatement, in plain float32 (or float64) torch, of the Nunivik decoder.  TEST INFRASTRUCTURE ONLY: imported by
tests/ (and by nothing in the product path).

One function per mechanism, each written from its equation and sharing no code with the kernels' callers.  There is no
cache and no portioning here: every call computes a whole sequence from position 0, token by token where the mechanism
is a recurrence, which is what cached, portioned and batched execution must be equivalent to.

Weights are a dict of tensors under the checkpoint's names ('embed', 'l0.mix.q', ...); `cfg` is the parsed config.json.
"""
from typing import Dict, List, Optional

import torch

Weights = Dict[str, torch.Tensor]
UNIT_EPS = 1e-6      # under the root of the recurrent mixers' unit vectors


def rms_norm(x: torch.Tensor, weight: torch.Tensor, eps: float) -> torch.Tensor:
    """x / sqrt(mean(x^2) + eps) * w over the last dimension."""
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps) * weight


def silu(z: torch.Tensor) -> torch.Tensor:
    return z / (1.0 + torch.exp(-z))


def softplus(z: torch.Tensor) -> torch.Tensor:
    """log(1 + e^z)"""
    return torch.logaddexp(z, torch.zeros_like(z))


def unit(x: torch.Tensor) -> torch.Tensor:
    return x / torch.sqrt((x * x).sum(dim=-1, keepdim=True) + UNIT_EPS)


def head_of(i: int, heads: int, groups: int) -> int:
    """Which of `groups` shared heads serves head i of `heads`."""
    return i // (heads // groups)


# ---- attention ----
def rotate_pairs(x: torch.Tensor, positions: torch.Tensor, rot: Optional[dict]) -> torch.Tensor:
    """x [n, heads, dim]: of the first rot.dims elements the pair (x[2i], x[2i + 1]) turns by the angle
    position * base^(-2i/dims) / factor."""
    if rot is None:
        return x
    dims, out = rot["dims"], x.clone()
    factor = rot["scaling"]["factor"] if rot.get("scaling") else 1.0
    for i in range(dims // 2):
        a = positions.to(x.dtype) * (rot["base"] ** (-2.0 * i / dims) / factor)
        c, s = torch.cos(a)[:, None], torch.sin(a)[:, None]
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * c - v * s
        out[..., 2 * i + 1] = v * c + u * s
    return out


def soft_cap(scores: torch.Tensor, cap: Optional[float]) -> torch.Tensor:
    return scores if cap is None else cap * torch.tanh(scores / cap)


def visible(n: int, size: Optional[int]) -> torch.Tensor:
    """[query, key]: 0 <= query - key < size (any distance for None)."""
    gap = torch.arange(n)[:, None] - torch.arange(n)[None, :]
    return (gap >= 0) & (gap < (size if size is not None else n + 1))


def attention(h: torch.Tensor, w: Weights, prefix: str, m: dict, eps: float, carried: dict,
              first_position: int = 0) -> torch.Tensor:
    """The whole 'attention' mixer on h [n, width].  `carried` keeps the values of the first value-mixing layer for the
    later ones."""
    n = h.shape[0]
    H, G, dim, vdim = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    pos = torch.arange(first_position, first_position + n)
    q = rms_norm((h @ w[prefix + "q"].t()).view(n, H, dim), w[prefix + "q.norm"], eps)
    k = rms_norm((h @ w[prefix + "k"].t()).view(n, G, dim), w[prefix + "k.norm"], eps)
    v = (h @ w[prefix + "v"].t()).view(n, G, vdim)
    q, k = rotate_pairs(q, pos, m.get("rot")), rotate_pairs(k, pos, m.get("rot"))
    if m.get("v_mix"):
        if "v" in carried:
            lam = w[prefix + "vmix"]
            v = (1.0 - lam) * v + lam * carried["v"]
        else:
            carried["v"] = v
    see = visible(n, m["mask"]["size"] if m.get("mask") else None)
    outs = []
    for i in range(H):
        g = head_of(i, H, G)
        s = soft_cap(q[:, i] @ k[:, g].t() * m["scale"], m.get("softcap"))
        outs.append(torch.softmax(s.masked_fill(~see, float("-inf")), dim=-1) @ v[:, g])
    return torch.cat(outs, dim=-1) @ w[prefix + "o"].t()


# ---- recurrent mixers ----
def short_convolution(x: torch.Tensor, taps: torch.Tensor, bias: Optional[torch.Tensor] = None) -> torch.Tensor:
    """x [n, channels], taps [channels, K]: y[t] = sum_j taps[:, j] x[t - (K - 1) + j], zeros in front of the start."""
    n, K = x.shape[0], taps.shape[1]
    y = torch.zeros_like(x) if bias is None else bias.expand_as(x).clone()
    for j in range(K):
        back = K - 1 - j
        if back < n:
            y[back:] += x[:n - back] * taps[:, j]
    return y


def gated_delta_recurrence(q, k, v, g, beta) -> torch.Tensor:
    """q, k [n, heads, dim], v [n, heads, vdim], g, beta [n, heads], from S = 0: S <- g S; u = beta (v - S^T k);
    S <- S + k u^T; o = S^T q."""
    n, heads, dim = q.shape
    S, out = torch.zeros(heads, dim, v.shape[-1], dtype=q.dtype), torch.empty_like(v)
    for t in range(n):
        S = S * g[t][:, None, None]
        u = beta[t][:, None] * (v[t] - (S * k[t][:, :, None]).sum(1))
        S = S + k[t][:, :, None] * u[:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(1)
    return out


def delta(h: torch.Tensor, w: Weights, prefix: str, m: dict, eps: float, carried: Optional[dict] = None) -> torch.Tensor:
    """The whole 'delta' mixer on h [n, width]."""
    n = h.shape[0]
    H, G, dim, vdim = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (silu(short_convolution(h @ w[prefix + x].t(), w[prefix + x + ".conv"])) for x in "qkv")
    q, k = unit(q.view(n, G, dim)) * dim ** -0.5, unit(k.view(n, G, dim))
    per_head = torch.tensor([head_of(i, H, G) for i in range(H)])
    beta = torch.sigmoid(h @ w[prefix + "b"].t())
    g = torch.exp(-torch.exp(w[prefix + "A_log"]) * softplus(h @ w[prefix + "a"].t() + w[prefix + "dt_bias"]))
    o = gated_delta_recurrence(q[:, per_head], k[:, per_head], v.view(n, H, vdim), g, beta)
    o = rms_norm(o, w[prefix + "norm"], eps) * silu(h @ w[prefix + "g"].t()).view(n, H, vdim)
    return o.reshape(n, H * vdim) @ w[prefix + "o"].t()


def state_space_recurrence(C, B, x, decay, dt, D) -> torch.Tensor:
    """C, B [n, heads, state], x [n, heads, vdim], decay, dt [n, heads], D [heads], from S = 0:
    S <- decay S + dt B x^T; y = S^T C + D x."""
    n, heads, N = B.shape
    S, out = torch.zeros(heads, N, x.shape[-1], dtype=x.dtype), torch.empty_like(x)
    for t in range(n):
        S = S * decay[t][:, None, None] + dt[t][:, None, None] * B[t][:, :, None] * x[t][:, None, :]
        out[t] = (S * C[t][:, :, None]).sum(1) + D[:, None] * x[t]
    return out


def gated_group_norm(y: torch.Tensor, z: torch.Tensor, weight: torch.Tensor, groups: int, eps: float) -> torch.Tensor:
    """y silu(z), normed in `groups` equal parts."""
    n, inner = y.shape
    y = (y * silu(z)).view(n, groups, inner // groups)
    return (y / torch.sqrt((y * y).mean(-1, keepdim=True) + eps)).reshape(n, inner) * weight


def mamba2(h: torch.Tensor, w: Weights, prefix: str, m: dict, eps: float, carried: Optional[dict] = None) -> torch.Tensor:
    """The whole 'mamba2' mixer on h [n, width]."""
    n = h.shape[0]
    H, vdim, N, G = m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * vdim
    z, xBC, dt = torch.split(h @ w[prefix + "in"].t(), [inner, inner + 2 * G * N, H], dim=-1)
    x, B, C = torch.split(silu(short_convolution(xBC, w[prefix + "conv"], w[prefix + "conv.b"])), [inner, G * N, G * N], dim=-1)
    dt = softplus(dt + w[prefix + "dt_bias"])
    group = torch.tensor([head_of(i, H, G) for i in range(H)])
    y = state_space_recurrence(C.view(n, G, N)[:, group], B.view(n, G, N)[:, group], x.view(n, H, vdim),
                               torch.exp(-torch.exp(w[prefix + "A_log"]) * dt), dt, w[prefix + "D"])
    return gated_group_norm(y.reshape(n, inner), z, w[prefix + "norm"], m["norm_groups"], eps) @ w[prefix + "o"].t()


MIXERS = {"attention": attention, "delta": delta, "mamba2": mamba2}


# ---- the model ----
def feed_forward(h: torch.Tensor, w: Weights, prefix: str, m: dict) -> torch.Tensor:
    assert m["kind"] == "dense"
    return (silu(h @ w[prefix + "gate"].t()) * (h @ w[prefix + "up"].t())) @ w[prefix + "down"].t()


def layer(x: torch.Tensor, w: Weights, cfg: dict, i: int, carried: dict) -> torch.Tensor:
    spec, eps, name = cfg["layers"][i], cfg["norm"]["eps"], f"l{i}."
    x = x + rms_norm(MIXERS[spec["type"]](x, w, name + "mix.", spec["mixer"], eps, carried), w[name + "norm1"], eps)
    if spec.get("mlp") is not None:
        x = x + rms_norm(feed_forward(x, w, name + "mlp.", spec["mlp"]), w[name + "norm2"], eps)
    return x


def forward(tokens, w: Weights, cfg: dict, dtype=torch.float32, layers_out: Optional[List[torch.Tensor]] = None) -> torch.Tensor:
    """Logits [n, vocab] of every position; the stream after every layer is appended to `layers_out`."""
    w = {k: v.to(dtype) for k, v in w.items()}
    x, carried = w["embed"][torch.as_tensor(tokens)] * cfg["embedding"]["scale"], {}
    for i in range(len(cfg["layers"])):
        x = layer(x, w, cfg, i, carried)
        if layers_out is not None:
            layers_out.append(x)
    return rms_norm(x, w["final.norm"], cfg["norm"]["eps"]) @ w["head"].t()
