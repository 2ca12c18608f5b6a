"""Small Nunivik models with random weights for the tests, as checkpoint directories."""
import math

import torch

from oracle import nunivik_oracle as N
from tests.feguvik_util import write_checkpoint


def attn(heads, kv, dim, vdim, size=None, cap=None, rot=None, base=10000.0, factor=None, mix=False, scale=None):
    m = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale or dim ** -0.5, "v_mix": mix}
    if rot:
        m["rot"] = {"base": base, "dims": rot, **({"scaling": {"factor": factor}} if factor else {})}
    if size:
        m["mask"] = {"size": size}
    if cap:
        m["softcap"] = cap
    return {"type": "attention", "mixer": m}


def delta(heads, kv, dim, vdim, taps):
    return {"type": "delta", "mixer": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "conv": taps}}


def mamba(heads, groups, state, vdim, taps, norm_groups=1):
    return {"type": "mamba2", "mixer": {"heads": heads, "groups": groups, "state": state, "vdim": vdim, "conv": taps,
                                        "norm_groups": norm_groups}}


def config(width, vocab, layers, eps=1e-6, scale=1.0):
    """``layers``: (mixer entry, ff or None) pairs."""
    return {"architecture": "Nunivik", "width": width, "vocab": vocab, "norm": {"eps": eps}, "embedding": {"scale": scale},
            "layers": [{**m, "mlp": {"kind": "dense", "ff": ff} if ff else None} for m, ff in layers]}


CONFIGS = {
    # nothing is a multiple of eight; the values that are mixed come from a layer in the middle; five and two taps
    "odd": config(90, 101, [(attn(6, 2, 22, 19, size=7, cap=5.0, rot=10, base=500.0, factor=1.5), 70), (delta(6, 3, 19, 27, 5), None),
                            (attn(3, 3, 11, 13, size=40, mix=True, rot=4, base=90.0), None), (mamba(6, 2, 21, 10, 2, norm_groups=3), 33),
                            (attn(6, 3, 10, 13, cap=3.0, mix=True), 50), (mamba(5, 1, 9, 7, 1), None)], eps=1e-5, scale=1.7),
    # recurrences in front, a feed-forward behind each kind
    "plain": config(128, 300, [(mamba(4, 4, 48, 32, 4, norm_groups=4), 96), (delta(4, 1, 64, 48, 3), 192),
                               (attn(8, 2, 48, 40, size=33, cap=30.0, rot=48, base=1e5, factor=4.0, mix=True), None),
                               (attn(4, 2, 64, 40, size=64, rot=32, mix=True), 160)]),
    # sizes of wide heads; the window is longer than a page and a tile, a cap that no constant can stand for
    "wide": config(256, 384, [(attn(4, 1, 128, 96, size=100, cap=60.0, rot=64, base=3e5, factor=8.0, mix=True), 320),
                              (delta(2, 2, 96, 128, 4), None), (mamba(2, 1, 128, 144, 3), 256),
                              (attn(2, 1, 160, 96, size=70, cap=12.0, rot=160, mix=True), None)], scale=0.7),
    # ones wherever there can be ones
    "tiny": config(32, 50, [(attn(1, 1, 8, 8, size=1, rot=2, mix=True), 40), (delta(1, 1, 16, 16, 1), 40), (mamba(1, 1, 1, 4, 1), None)]),
    # attention alone: no recurrent state, no slots
    "attention": config(64, 77, [(attn(4, 2, 16, 24, size=20, cap=9.0, rot=16), 64), (attn(4, 4, 16, 16), None)]),
    # no attention: no cache
    "recurrent": config(64, 77, [(delta(2, 1, 32, 32, 4), None), (mamba(4, 2, 16, 16, 4, norm_groups=2), 64)]),
}


def random_weights(cfg, seed=0):
    """bfloat16 tensors under the checkpoint's names.  Head norms are scaled up so that attention is not flat, decays reach
    from a few tokens to hundreds, values are mixed by a half and more."""
    g = torch.Generator().manual_seed(seed)
    W, V, w = cfg["width"], cfg["vocab"], {}
    mat = lambda n, k, s=1.0: torch.randn(n, k, generator=g) * s / math.sqrt(k)
    vec = lambda n, mean=1.0, s=0.2: mean + torch.randn(n, generator=g) * s
    w["embed"], w["head"], w["final.norm"] = torch.randn(V, W, generator=g), mat(V, W), vec(W)
    for i, spec in enumerate(cfg["layers"]):
        p, m = f"l{i}.", spec["mixer"]
        H, v = m["heads"], m["vdim"]
        w[p + "norm1"] = vec(W)
        if spec["type"] == "attention":
            G, d = m["kv_heads"], m["dim"]
            w.update({p + "mix.q": mat(H * d, W), p + "mix.k": mat(G * d, W), p + "mix.v": mat(G * v, W), p + "mix.q.norm": vec(d, 1.7),
                      p + "mix.k.norm": vec(d, 1.5)})
            if m["v_mix"]:
                w[p + "mix.vmix"] = vec((), 0.6, 0.2)
        elif spec["type"] == "delta":
            G, d = m["kv_heads"], m["dim"]
            w.update({p + "mix.q": mat(G * d, W), p + "mix.k": mat(G * d, W), p + "mix.v": mat(H * v, W), p + "mix.g": mat(H * v, W),
                      p + "mix.a": mat(H, W), p + "mix.b": mat(H, W), p + "mix.norm": vec(v)})
            w.update({p + f"mix.{x}.conv": vec((n, m["conv"]), 0.3, 0.5) for x, n in (("q", G * d), ("k", G * d), ("v", H * v))})
        else:
            G, n = m["groups"], m["state"]
            channels = H * v + 2 * G * n
            w.update({p + "mix.in": mat(channels + H * v + H, W), p + "mix.conv": vec((channels, m["conv"]), 0.3, 0.5),
                      p + "mix.conv.b": vec(channels, 0.1), p + "mix.D": vec(H), p + "mix.norm": vec(H * v)})
        if spec["type"] != "attention":
            w.update({p + "mix.A_log": vec(H, -1.0, 1.0), p + "mix.dt_bias": vec(H, -2.0, 1.5)})
        w[p + "mix.o"] = mat(W, H * v)
        if spec["mlp"]:
            w.update({p + "norm2": vec(W), p + "mlp.gate": mat(spec["mlp"]["ff"], W), p + "mlp.up": mat(spec["mlp"]["ff"], W),
                      p + "mlp.down": mat(W, spec["mlp"]["ff"])})
    return {k: t.to(torch.bfloat16).contiguous() for k, t in w.items()}


def make_model(path, name, seed=0):
    """(directory, config, float32 weights)"""
    cfg = CONFIGS[name]
    w = random_weights(cfg, seed)
    return write_checkpoint(path, cfg, w), cfg, {k: v.float() for k, v in w.items()}


def oracle_logits(tokens, w, cfg):
    return N.forward(tokens, w, cfg, torch.float64).float()
