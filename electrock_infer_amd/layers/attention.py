"""Softmax attention over a paged cache (csrc/decoder/attention.hip): grouped heads, with an RMS norm per query and key
head, rotation of neighbouring pairs, a soft cap on the scores, a sliding window and values mixed with an earlier
layer's -- each of them optional."""
from typing import Optional

import torch
from torch import nn

from .. import _lib
from .decoder_ops import StackedLinear, byref, linear_parts
from .latent_attention import rotary_frequencies


class CarriedValues:
    """The values of the first value-mixing layer, on their way through one forward pass."""

    def __init__(self):
        self.rows: Optional[torch.Tensor] = None      # that layer's projections (kept alive)
        self.ptr, self.stride = 0, 0


class SoftmaxAttention(nn.Module):

    PROMPT_TOKENS = 48           # portions from this length on go to the kernel for prompts, if it takes the sizes
    TARGET_WORKGROUPS = 768      # the keys are shared out over workgroups until a launch has about this many
    SPLIT_KEYS = 128             # fewest keys of a workgroup

    def __init__(self, width: int, heads: int, kv_heads: int, dim: int, vdim: int, scale: float, eps: float, dtype,
                 rot_dims: int = 0, rotary_base: float = 10000.0, rotary_factor: float = 1.0, softcap: float = 0.0, window: int = 0,
                 mix_values: bool = False, head_norms: bool = True):
        """``window``: keys that a query sees, itself included (0: all); ``softcap`` 0: none."""
        super().__init__()
        if heads % kv_heads:
            raise ValueError(f"{heads} heads cannot share {kv_heads} keys and values")
        self.heads, self.kv_heads, self.dim, self.vdim, self.scale, self.eps = heads, kv_heads, dim, vdim, scale, eps
        self.rot, self.rotary_base, self.rotary_factor = rot_dims, rotary_base, rotary_factor
        self.softcap, self.window, self.mix_values = softcap, window, mix_values
        self.in_proj = StackedLinear(width, {"q": heads * dim, "k": kv_heads * dim, "v": kv_heads * vdim}, dtype)
        vector = lambda n: nn.Parameter(torch.ones(n, dtype=torch.float32), requires_grad=False)
        self.q_norm, self.k_norm = (vector(dim), vector(dim)) if head_norms else (None, None)
        self.vmix = nn.Parameter(torch.zeros((), dtype=torch.float32), requires_grad=False) if mix_values else None
        self.o = nn.Parameter(torch.zeros(width, heads * vdim, dtype=dtype), requires_grad=False)
        self.register_buffer("inv_freq", torch.zeros(rot_dims // 2, dtype=torch.float32), persistent=False)
        # checkpoint tensor (behind '<layer>.mix.') -> (parameter, section)
        self.TENSORS = {**{n: ("in_proj.weight", n) for n in "qkv"}, "o": ("o", None),
                        **({"q.norm": ("q_norm", None), "k.norm": ("k_norm", None)} if head_norms else {}),
                        **({"vmix": ("vmix", None)} if mix_values else {})}

    def finish_loading(self) -> None:
        self.inv_freq.copy_(rotary_frequencies(self.rot, self.rotary_base, self.rotary_factor))

    def row_elems(self) -> int:
        """Elements that one token takes in the cache."""
        return self.kv_heads * (-(-self.dim // 8) * 8 + -(-self.vdim // 8) * 8)

    def cache_bytes(self, block_size: int):
        """(bytes of a cache block, bytes of a state slot)"""
        return block_size * self.row_elems() * self.o.element_size(), 0

    def new_cache(self, num_blocks: int, block_size: int, num_slots: int, device) -> torch.Tensor:
        return torch.zeros(num_blocks, block_size, self.row_elems(), dtype=self.o.dtype, device=device)

    def splits(self, batch) -> int:
        groups = -(-batch.max_q * (self.heads // self.kv_heads) // 16) * batch.n_seqs * self.kv_heads
        keys = min(batch.max_context, self.window + batch.max_q) if self.window else batch.max_context
        return max(1, min(-(-self.TARGET_WORKGROUPS // groups), -(-keys // self.SPLIT_KEYS), 64))

    def forward(self, h: torch.Tensor, batch, cache: torch.Tensor, carried: Optional[CarriedValues] = None) -> torch.Tensor:
        """h [T, width] -> [T, width] (as ``linear_parts`` has it); ``cache`` [blocks, block_size, row_elems] receives the
        new tokens' rows first."""
        T, dev, H = h.shape[0], h.device, self.heads
        p, ptr = self.in_proj(h), lambda t: None if t is None else t.data_ptr()
        sec = lambda n: self.in_proj.section_ptr(p, n)
        q_rows = torch.empty(T, H, -(-self.dim // 8) * 8, dtype=h.dtype, device=dev)
        o = torch.empty(T, H * self.vdim, dtype=h.dtype, device=dev)
        a = _lib.AttnArgs(q=sec("q"), k=sec("k"), v=sec("v"), stride=p.stride(0), q_norm=ptr(self.q_norm), k_norm=ptr(self.k_norm),
                          inv_freq=self.inv_freq.data_ptr(), positions=batch.positions.data_ptr(), cache_rows=batch.cache_rows.data_ptr(),
                          cache=cache.data_ptr(), q_rows=q_rows.data_ptr(), out=o.data_ptr(), q_begin=batch.q_begin.data_ptr(),
                          starts=batch.starts.data_ptr(), tables=batch.tables.data_ptr(), T=T, n_seqs=batch.n_seqs, max_q=batch.max_q,
                          table_width=batch.table_width, block_size=cache.shape[1], splits=1, heads=H, kv_heads=self.kv_heads,
                          dim=self.dim, vdim=self.vdim, rot=self.rot, window=self.window, dtype=_lib.dtype_code(h.dtype),
                          scale=self.scale, softcap=self.softcap, eps=self.eps)
        if self.mix_values:
            if carried.rows is None:
                carried.rows, carried.ptr, carried.stride = p, sec("v"), p.stride(0)
            else:
                a.mix, a.v_first, a.v_first_stride = self.vmix.data_ptr(), carried.ptr, carried.stride
        lib, stream = _lib.load_decoder(), _lib.current_stream(dev)
        _lib.check_decoder(lib.ed_attn_prepare(byref(a), stream), "attn_prepare")
        if batch.max_q >= self.PROMPT_TOKENS and h.dtype == torch.bfloat16 and lib.ed_attn_prompt_supported(self.dim, self.vdim) == 1:
            _lib.check_decoder(lib.ed_attn_prompt(byref(a), stream), "attn_prompt")
            return linear_parts(o, self.o)
        a.splits = self.splits(batch)
        if a.splits > 1:
            part_o = torch.empty(T * H * a.splits * self.vdim, dtype=torch.float32, device=dev)
            part_ml = torch.empty(T * H * a.splits * 2, dtype=torch.float32, device=dev)
            a.part_o, a.part_ml = part_o.data_ptr(), part_ml.data_ptr()
        _lib.check_decoder(lib.ed_attn_paged(byref(a), stream), "attn_paged")
        return linear_parts(o, self.o)
