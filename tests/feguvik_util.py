"""Small Feguvik models with random weights for the tests, as checkpoint directories."""
import json
import math
import os

import torch
from safetensors.torch import save_file

from oracle import feguvik_oracle as F


def gla(heads, dim, vdim, tau):
    return {"type": "gla", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau}}


def mla(heads, dim, rot, vdim, rank, base=10000.0, scale=None):
    return {"type": "latent_attention",
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": rank,
                      "rot": {"base": base, "dims": rot}, "scale": scale or (dim + rot) ** -0.5}}


def config(width, vocab, layers, side, loop=None, eps=1e-6, scale=1.0):
    """``layers``: (mixer entry, ff or None) pairs."""
    out = {"architecture": "Feguvik", "width": width, "vocab": vocab, "norm": {"eps": eps}, "embedding": {"scale": scale},
           "token_side": {"dim": side},
           "layers": [{**m, "mlp": {"kind": "dense", "ff": ff} if ff else None} for m, ff in layers]}
    if loop:
        out["loop"] = dict(zip(("start", "stop", "times"), loop))
    return out


CONFIGS = {
    # nothing is a multiple of eight; a layer without feed-forward; the loop in the middle
    "odd": (config(90, 101, [(mla(3, 22, 6, 20, 37, base=500.0), 70), (gla(2, 19, 27, 5.0), None),
                             (mla(2, 10, 4, 12, 21, base=500.0), 33), (gla(3, 33, 17, 1.0), 50)], side=5, loop=(1, 3, 3),
                   eps=1e-5, scale=1.7), 7),
    # no loop, one layer of each, heads of different sizes
    "plain": (config(128, 300, [(gla(4, 64, 48, 16.0), 192), (mla(5, 48, 16, 40, 72), 160)], side=24), 12),
    # sizes of the written-out prompt kernel and of the wide state tiles; the loop runs over everything
    "wide": (config(256, 384, [(mla(4, 64, 32, 64, 128, scale=0.13), 320), (gla(2, 96, 128, 8.0), 256)], side=32,
                    loop=(0, 2, 2), scale=0.7), 32),
    # one latent layer with a single head and a one-layer model's other extremes
    "tiny": (config(32, 50, [(mla(1, 8, 2, 8, 9), 40), (gla(1, 16, 16, 2.0), 40)], side=1, loop=(0, 1, 1)), 1),
}


def random_weights(cfg, decay_rank, seed=0):
    """bfloat16 tensors under the checkpoint's names.  Queries are scaled up so that attention is not flat, decays reach
    from a few tokens to hundreds, sinks matter."""
    g = torch.Generator().manual_seed(seed)
    W, V, w = cfg["width"], cfg["vocab"], {}
    mat = lambda n, k, s=1.0: torch.randn(n, k, generator=g) * s / math.sqrt(k)
    vec = lambda n, mean=1.0, s=0.2: mean + torch.randn(n, generator=g) * s
    w["embed"], w["head"] = torch.randn(V, W, generator=g), mat(V, W)
    w["final.norm"] = vec(W)
    side = cfg["token_side"]["dim"]
    w["side.embed"] = torch.randn(V, side * len(cfg["layers"]), generator=g)
    if "loop" in cfg:
        w["loop.in"], w["loop.step"] = mat(W, 2 * W), torch.randn(cfg["loop"]["times"], W, generator=g) * 0.3
    for i, spec in enumerate(cfg["layers"]):
        p, m = f"l{i}.", spec["mixer"]
        for n in ("norm1", "norm1b", "ls1") + (("norm2", "norm2b", "ls2") if spec["mlp"] else ()):
            w[p + n] = vec(W)
        if spec["type"] == "gla":
            h, d, v = m["heads"], m["dim"], m["vdim"]
            w.update({p + "mix.q": mat(h * d, W), p + "mix.k": mat(h * d, W), p + "mix.v": mat(h * v, W),
                      p + "mix.g": mat(h * v, W), p + "mix.o": mat(W, h * v), p + "mix.norm": vec(v),
                      p + "mix.a1": mat(decay_rank, W), p + "mix.a2": mat(h * d, decay_rank),
                      p + "mix.a2.b": vec(h * d, 2.0 + math.log(m["tau"] + 1.0), 1.5)})
        else:
            h, d, r, v, c = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
            w.update({p + "mix.q": mat(h * (d + r), W, 2.0), p + "mix.dkv": mat(c + r, W), p + "mix.dkv.norm": vec(c),
                      p + "mix.uk": mat(h * d, c), p + "mix.uv": mat(h * v, c), p + "mix.sink": vec(h, 0.5, 1.0),
                      p + "mix.o": mat(W, h * v)})
        if spec["mlp"]:
            w[p + "mlp.up"], w[p + "mlp.down"] = mat(spec["mlp"]["ff"], W), mat(W, spec["mlp"]["ff"])
        w.update({p + "side.gate": mat(side, W), p + "side.proj": mat(W, side), p + "side.norm": vec(W)})
    return {k: v.to(torch.bfloat16).contiguous() for k, v in w.items()}


def write_checkpoint(path, cfg, weights):
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file(weights, os.path.join(path, "model.safetensors"))
    return str(path)


def make_model(path, name, seed=0):
    """(directory, config, float32 weights)"""
    cfg, rank = CONFIGS[name]
    w = random_weights(cfg, rank, seed)
    return write_checkpoint(path, cfg, w), cfg, {k: v.float() for k, v in w.items()}


def draw_tokens(cfg, n, seed=0):
    return torch.randint(0, cfg["vocab"], (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def oracle_logits(tokens, w, cfg):
    return F.forward(tokens, w, cfg, torch.float64).float()


def row_errors(got, want):
    """Per row: root mean square of the difference of two logit rows, their means taken off, relative to the spread of
    the expected logits."""
    d = got.double() - want.double()
    d = d - d.mean(-1, keepdim=True)
    return d.pow(2).mean(-1).sqrt() / want.double().std()
