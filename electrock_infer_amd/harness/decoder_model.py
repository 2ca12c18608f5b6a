"""What decoder models on the kernels of libelectrock_decoder.so share: names of checkpoint tensors, random weights, cache
and state, logits.  A model lists its layers, each with a mixer (``mix``) and perhaps a feed-forward (``mlp``) whose
``TENSORS`` map checkpoint names to parameters."""
from typing import List, Tuple

import torch
from torch import nn

from ..layers.decoder_ops import linear_f32
from .batch import RaggedBatch


class DecoderModel(nn.Module):

    ragged_batches = True
    NAMES = {"embed": "embed", "final.norm": "final_norm", "head": "head"}     # tensors outside the layers
    ZEROS: Tuple[str, ...] = ()       # ends of vectors' names that random weights leave at zero (the others are ones)

    layers: nn.ModuleList     # of modules with ``mix``, ``mlp`` (or None) and LAYER_TENSORS
    runs: List[Tuple]         # running order: (layer, ...)

    def __init__(self):
        super().__init__()
        self.caches: List = []            # per run: what its mixer's new_cache made
        self.layer_hook = None            # called as hook(run index, stream) behind every layer run when set

    def chunk_tokens(self, tokens: int) -> int:
        """Tokens that one workgroup of the recurrent mixers' prompt kernels takes in a step of ``tokens``."""
        return 256

    # ---- weights ----
    def checkpoint_target(self, name: str):
        """(parameter name, section or None) of a checkpoint tensor, or None."""
        if name in self.NAMES:
            return self.NAMES[name], None
        first, _, rest = name.partition(".")
        if not (first[:1] == "l" and first[1:].isdigit() and int(first[1:]) < len(self.layers)):
            return None
        prefix, layer = f"layers.{first[1:]}.", self.layers[int(first[1:])]
        part, _, inner = rest.partition(".")
        module = getattr(layer, part, None) if inner else layer
        if module is None:
            return None
        if inner and hasattr(module, "TENSORS"):
            entry = module.TENSORS.get(inner)
            return (f"{prefix}{part}.{entry[0]}", entry[1]) if entry is not None else None
        return prefix + rest, None

    def expected_tensors(self) -> List[str]:
        """Checkpoint names of every parameter (section)."""
        out = [n for n, p in self.NAMES.items() if hasattr(self, p)]
        for i, layer in enumerate(self.layers):
            out += [f"l{i}.{n}" for n in layer.tensor_names()]
        return out

    def finish_loading(self) -> None:
        for layer in self.layers:
            layer.finish_loading()

    @torch.no_grad()
    def init_random_weights(self, seed: int = 0, std: float = 0.02) -> None:
        """N(0, std) for every matrix; ones or zeros for vectors."""
        g = torch.Generator(device=self.head.device).manual_seed(seed)
        for name, p in self.named_parameters():
            if p.dim() >= 2:
                p.copy_(torch.randn(p.shape, generator=g, device=p.device, dtype=torch.float32) * std)
            else:
                p.fill_(0.0 if name.endswith(self.ZEROS) else 1.0)
        self.finish_loading()

    # ---- cache and state ----
    def cache_bytes(self, block_size: int) -> Tuple[int, int]:
        """(bytes of a cache block, bytes of a state slot), over all layer runs."""
        sizes = [self.layers[run[0]].mix.cache_bytes(block_size) for run in self.runs]
        return sum(b for b, _ in sizes), sum(s for _, s in sizes)

    def allocate_cache(self, num_blocks: int, block_size: int, num_slots: int, device) -> None:
        self.caches = [self.layers[run[0]].mix.new_cache(num_blocks, block_size, num_slots, device) for run in self.runs]

    # ---- forward ----
    def compute_logits(self, hidden: torch.Tensor, batch: RaggedBatch) -> torch.Tensor:
        """float32 logits of the batch's wanted rows."""
        return linear_f32(hidden.index_select(0, batch.logit_rows), self.head)
