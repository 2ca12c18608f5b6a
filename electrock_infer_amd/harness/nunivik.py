"""Nunivik: a decoder whose layers have one of three mixers -- softmax attention (grouped heads, sliding window, soft cap,
mixed values), the gated delta rule, or the state-space form -- and perhaps a gated feed-forward.  A sublayer reads the
residual stream as it is; only its result is normed before it is added.

The residual stream is float32; projections run in the configuration's compute type (bfloat16, or float32 throughout).
"""
from dataclasses import dataclass, field
from typing import List

import torch
from torch import nn

from ..layers.attention import CarriedValues, SoftmaxAttention
from ..layers.decoder_ops import ADD_NORMED, embed_rows, residual_norm
from ..layers.dense_mlp import DenseMLP
from ..layers.recurrent import GatedDeltaRule, StateSpaceMixer
from .batch import RaggedBatch
from .decoder_model import DecoderModel


@dataclass
class MixerSpec:
    """One entry of config.json's 'layers'; ``ff`` is 0 for a layer without a feed-forward."""
    kind: str                       # 'attention' | 'delta' | 'mamba2'
    mixer: dict
    ff: int = 0


def _attention(width, m, eps, dtype):
    rot = m.get("rot") or {}
    return SoftmaxAttention(width, m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["scale"], eps, dtype, rot_dims=rot.get("dims", 0),
                            rotary_base=rot.get("base", 1.0), rotary_factor=(rot.get("scaling") or {}).get("factor", 1.0),
                            softcap=m.get("softcap") or 0.0, window=(m.get("mask") or {}).get("size") or 0,
                            mix_values=bool(m.get("v_mix")))


def _delta(width, m, eps, dtype):
    return GatedDeltaRule(width, m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"], eps, dtype)


def _mamba2(width, m, eps, dtype):
    return StateSpaceMixer(width, m["heads"], m["groups"], m["state"], m["vdim"], m["conv"], m["norm_groups"], eps, dtype)


MIXERS = {"attention": _attention, "delta": _delta, "mamba2": _mamba2}


@dataclass
class NunivikConfig:
    vocab_size: int
    width: int
    layers: List[MixerSpec]
    norm_eps: float
    embedding_scale: float = 1.0
    max_position_embeddings: int = 1 << 24      # positions are exact in float32 up to here; there is no table
    torch_dtype: torch.dtype = field(default=torch.bfloat16)

    @property
    def has_recurrent_state(self) -> bool:
        return any(l.kind != "attention" for l in self.layers)

    @classmethod
    def from_checkpoint(cls, config: dict, shapes: dict, dtype: torch.dtype) -> "NunivikConfig":
        """From config.json; ``shapes`` (tensor name -> shape) is not needed."""
        layers, mixed = [], None
        for i, entry in enumerate(config["layers"]):
            if entry["type"] not in MIXERS:
                raise ValueError(f"layer {i}: unknown mixer '{entry['type']}'")
            mlp, m = entry.get("mlp"), dict(entry["mixer"])
            if mlp is not None and mlp["kind"] != "dense":
                raise ValueError(f"layer {i}: unknown feed-forward '{mlp['kind']}'")
            if m.get("v_mix"):
                mixed = mixed or (m["kv_heads"], m["vdim"])
                if mixed != (m["kv_heads"], m["vdim"]):
                    raise ValueError(f"layer {i}: its values cannot be mixed with those of another size")
            layers.append(MixerSpec(entry["type"], m, mlp["ff"] if mlp is not None else 0))
        return cls(vocab_size=config["vocab"], width=config["width"], layers=layers, norm_eps=config["norm"]["eps"],
                   embedding_scale=config["embedding"]["scale"], torch_dtype=dtype)


class NunivikLayer(nn.Module):

    def __init__(self, cfg: NunivikConfig, index: int):
        super().__init__()
        spec, dtype = cfg.layers[index], cfg.torch_dtype
        vector = lambda: nn.Parameter(torch.ones(cfg.width, dtype=torch.float32), requires_grad=False)
        self.mix = MIXERS[spec.kind](cfg.width, spec.mixer, cfg.norm_eps, dtype)
        self.norm1 = vector()
        self.mlp = None
        if spec.ff:
            self.norm2 = vector()
            self.mlp = DenseMLP(cfg.width, spec.ff, dtype, "silu_gate")

    def tensor_names(self) -> List[str]:
        names = ["norm1"] + [f"mix.{n}" for n in self.mix.TENSORS]
        return names + (["norm2"] + [f"mlp.{n}" for n in self.mlp.TENSORS] if self.mlp is not None else [])

    def finish_loading(self) -> None:
        if hasattr(self.mix, "finish_loading"):
            self.mix.finish_loading()


class NunivikForCausalLM(DecoderModel):

    ZEROS = ("a_log", "dt_bias", "conv_bias", "vmix")

    def __init__(self, cfg: NunivikConfig):
        super().__init__()
        self.cfg = cfg
        matrix = lambda *shape: nn.Parameter(torch.zeros(*shape, dtype=cfg.torch_dtype), requires_grad=False)
        self.embed = matrix(cfg.vocab_size, cfg.width)
        self.layers = nn.ModuleList([NunivikLayer(cfg, i) for i in range(len(cfg.layers))])
        self.final_norm = nn.Parameter(torch.ones(cfg.width, dtype=torch.float32), requires_grad=False)
        self.head = matrix(cfg.vocab_size, cfg.width)
        self.runs = [(i,) for i in range(len(cfg.layers))]

    def chunk_tokens(self, tokens: int) -> int:
        """Fewer, longer chunks where there are enough of them to fill the chip: the scan over them is sequential."""
        return 512 if tokens >= 8192 else 256 if tokens >= 4096 else 128 if tokens >= 1024 else 64

    def forward(self, batch: RaggedBatch) -> torch.Tensor:
        """Normed output [T, width] of every token of the batch."""
        cfg, eps = self.cfg, self.cfg.norm_eps
        h = torch.empty(batch.tokens.numel(), cfg.width, dtype=self.head.dtype, device=self.head.device)
        x = embed_rows(batch.tokens, self.embed, cfg.embedding_scale, h)        # h: the stream in the compute type
        carried = CarriedValues()
        for i, layer in enumerate(self.layers):
            last = self.final_norm if i + 1 == len(self.layers) else None
            y = layer.mix(h, batch, self.caches[i], carried)
            residual_norm(ADD_NORMED, x, y, layer.norm1, eps, h, last if layer.mlp is None else None)
            if layer.mlp is not None:
                residual_norm(ADD_NORMED, x, layer.mlp(h), layer.norm2, eps, h, last)
            if self.layer_hook is not None:
                self.layer_hook(i, x)
        return h
