"""Feguvik: a decoder whose layers mix gated linear attention (recurrent state) and latent attention (paged cache), with
norms in front of and behind every sublayer, layer scales, a per-layer token input, and a range of layers that runs
several times with the same weights, each pass with its own cache and state.

The residual stream is float32; projections run in the configuration's compute type (bfloat16, or float32 throughout).
"""
from dataclasses import dataclass, field
from typing import List, Optional, Tuple

import torch
import torch.nn.functional as F
from torch import nn

from ..layers.decoder_ops import ADD_NORMED, KEEP, REPLACE, embed_rows, linear_parts, residual_norm
from ..layers.dense_mlp import DenseMLP
from ..layers.gla import GatedLinearAttention
from ..layers.latent_attention import LatentAttention
from ..layers.token_side import TokenSideInput
from .batch import RaggedBatch
from .decoder_model import DecoderModel


@dataclass
class LayerSpec:
    """One entry of config.json's 'layers'; ``ff`` is 0 for a layer without a feed-forward."""
    kind: str                       # 'gla' | 'latent_attention'
    mixer: dict
    ff: int = 0
    decay_rank: int = 0             # 'gla': inner size of the decay's two factors (not in config.json: a tensor's shape)


@dataclass
class LoopSpec:
    start: int
    stop: int
    times: int


@dataclass
class FeguvikConfig:
    vocab_size: int
    width: int
    layers: List[LayerSpec]
    norm_eps: float
    embedding_scale: float = 1.0
    side_dim: int = 0               # per-layer token input; 0: none
    loop: Optional[LoopSpec] = None
    max_position_embeddings: int = 1 << 24      # positions are exact in float32 up to here; there is no table
    torch_dtype: torch.dtype = field(default=torch.bfloat16)

    @property
    def has_recurrent_state(self) -> bool:
        return any(l.kind == "gla" for l in self.layers)

    @classmethod
    def from_checkpoint(cls, config: dict, shapes: dict, dtype: torch.dtype) -> "FeguvikConfig":
        layers = []
        for i, entry in enumerate(config["layers"]):
            if entry["type"] not in ("gla", "latent_attention"):
                raise ValueError(f"layer {i}: unknown mixer '{entry['type']}'")
            mlp = entry.get("mlp")
            if mlp is not None and mlp["kind"] != "dense":
                raise ValueError(f"layer {i}: unknown feed-forward '{mlp['kind']}'")
            rot = entry["mixer"].get("rot")
            if rot is not None and rot["dims"] != entry["mixer"]["rot_dim"]:
                raise ValueError(f"layer {i}: rot.dims differs from rot_dim")
            layers.append(LayerSpec(entry["type"], dict(entry["mixer"]), mlp["ff"] if mlp is not None else 0,
                                    shapes[f"l{i}.mix.a1"][0] if entry["type"] == "gla" else 0))
        loop, side = config.get("loop"), config.get("token_side")
        return cls(vocab_size=config["vocab"], width=config["width"], layers=layers, norm_eps=config["norm"]["eps"],
                   embedding_scale=config["embedding"]["scale"], side_dim=side["dim"] if side else 0,
                   loop=LoopSpec(loop["start"], loop["stop"], loop["times"]) if loop else None, torch_dtype=dtype)

    def runs(self) -> List[Tuple[int, Optional[int]]]:
        """(layer, pass or None) in running order."""
        every = range(len(self.layers))
        if self.loop is None:
            return [(i, None) for i in every]
        a, b = self.loop.start, self.loop.stop
        return ([(i, None) for i in every[:a]] + [(i, t) for t in range(self.loop.times) for i in every[a:b]] +
                [(i, None) for i in every[b:]])


class FeguvikLayer(nn.Module):

    def __init__(self, cfg: FeguvikConfig, index: int):
        super().__init__()
        spec, dtype, m = cfg.layers[index], cfg.torch_dtype, cfg.layers[index].mixer
        vector = lambda: nn.Parameter(torch.ones(cfg.width, dtype=torch.float32), requires_grad=False)
        if spec.kind == "gla":
            self.mix = GatedLinearAttention(cfg.width, m["heads"], m["dim"], m["vdim"], m["tau"], spec.decay_rank,
                                            cfg.norm_eps, dtype)
        else:
            self.mix = LatentAttention(cfg.width, m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"], m["scale"],
                                       m["rot"]["base"], cfg.norm_eps, dtype)
        self.norm1, self.norm1b, self.ls1 = vector(), vector(), vector()
        self.mlp = None
        if spec.ff:
            self.norm2, self.norm2b, self.ls2 = vector(), vector(), vector()
            self.mlp = DenseMLP(cfg.width, spec.ff, dtype)
        self.side = TokenSideInput(cfg.width, cfg.side_dim, index * cfg.side_dim, dtype) if cfg.side_dim else None
        self.post1 = self.post2 = None

    def tensor_names(self) -> List[str]:
        names = ["norm1", "norm1b", "ls1"] + [f"mix.{n}" for n in self.mix.TENSORS]
        names += ["norm2", "norm2b", "ls2"] + [f"mlp.{n}" for n in self.mlp.TENSORS] if self.mlp is not None else []
        return names + (["side.gate", "side.proj", "side.norm"] if self.side is not None else [])

    def finish_loading(self) -> None:
        """The output norm's weight and the layer scale multiply the same vector: one factor."""
        self.post1 = (self.norm1b * self.ls1).contiguous()
        if self.mlp is not None:
            self.post2 = (self.norm2b * self.ls2).contiguous()
        if hasattr(self.mix, "finish_loading"):
            self.mix.finish_loading()


class FeguvikForCausalLM(DecoderModel):

    NAMES = {"embed": "embed", "side.embed": "side_embed", "loop.in": "loop_in", "loop.step": "loop_step",
             "final.norm": "final_norm", "head": "head"}
    ZEROS = ("sink", "a2_bias")

    def __init__(self, cfg: FeguvikConfig):
        super().__init__()
        self.cfg = cfg
        W, dtype = cfg.width, cfg.torch_dtype
        matrix = lambda *shape: nn.Parameter(torch.zeros(*shape, dtype=dtype), requires_grad=False)
        self.embed = matrix(cfg.vocab_size, W)
        if cfg.side_dim:
            self.side_embed = matrix(cfg.vocab_size, len(cfg.layers) * cfg.side_dim)
        if cfg.loop is not None:
            self.loop_in = matrix(W, 2 * W)
            self.loop_step = nn.Parameter(torch.zeros(cfg.loop.times, W, dtype=torch.float32), requires_grad=False)
        self.layers = nn.ModuleList([FeguvikLayer(cfg, i) for i in range(len(cfg.layers))])
        self.final_norm = nn.Parameter(torch.ones(W, dtype=torch.float32), requires_grad=False)
        self.head = matrix(cfg.vocab_size, W)
        self.runs = cfg.runs()

    # ---- forward ----
    def forward(self, batch: RaggedBatch) -> torch.Tensor:
        """Normed output [T, width] of every token of the batch."""
        cfg, dtype, dev = self.cfg, self.head.dtype, self.head.device
        T, W, eps = batch.tokens.numel(), cfg.width, cfg.norm_eps
        rows = lambda: torch.empty(T, W, dtype=dtype, device=dev)
        both = torch.empty(T, 2 * W, dtype=dtype, device=dev) if cfg.loop is not None else None   # [stream | embedding]
        x = embed_rows(batch.tokens, self.embed, cfg.embedding_scale, both[:, W:] if both is not None else None)
        h = rows()
        n_runs = len(self.runs)
        opens_pass = lambda r: r < n_runs and self.runs[r][1] is not None and self.runs[r][0] == cfg.loop.start

        def open_run(r, update):
            """``update(out, norm)`` changes the stream and writes x / rms(x) * norm, or x for None: what run ``r`` reads."""
            norm = self.layers[self.runs[r][0]].norm1 if r < n_runs else self.final_norm
            if not opens_pass(r):
                update(h, norm)
            else:
                update(both[:, :W], None)
            if self.layer_hook is not None and r > 0:
                self.layer_hook(r - 1, x)
            if opens_pass(r):
                residual_norm(REPLACE, x, linear_parts(both, self.loop_in, exact=True), self.loop_step[self.runs[r][1]], eps, h, norm)

        open_run(0, lambda out, norm: residual_norm(KEEP, x, None, None, eps, out, norm))
        for r, (i, _) in enumerate(self.runs):
            layer = self.layers[i]
            y, post = layer.mix(h, batch, self.caches[r]), layer.post1
            if layer.mlp is not None:
                residual_norm(ADD_NORMED, x, y, post, eps, h, layer.norm2)
                y, post = layer.mlp(h), layer.post2
            if layer.side is not None:
                open_run(r + 1, lambda out, norm: layer.side.close_layer(x, y, post, batch.tokens, self.side_embed, eps, out, norm))
            else:
                open_run(r + 1, lambda out, norm: residual_norm(ADD_NORMED, x, y, post, eps, out, norm))
        return h
