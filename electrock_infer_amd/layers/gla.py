"""Gated linear attention (csrc/decoder/gla.hip): a recurrent mixer with one decay per key channel, a float32 state per
head and sequence, a norm over every head's output and a SiLU gate."""
import torch
from torch import nn

from .. import _lib
from .decoder_ops import StackedLinear, byref, linear_parts


class GatedLinearAttention(nn.Module):
    """Projections stacked in one matrix: q, k, v, the output gate g and the first factor a1 of the decay."""

    def __init__(self, width: int, heads: int, dim: int, vdim: int, tau: float, decay_rank: int, eps: float, dtype):
        super().__init__()
        self.heads, self.dim, self.vdim, self.tau, self.rank, self.eps = heads, dim, vdim, tau, decay_rank, eps
        self.in_proj = StackedLinear(width, {"q": heads * dim, "k": heads * dim, "v": heads * vdim, "g": heads * vdim,
                                             "a1": decay_rank}, dtype)
        self.a2 = nn.Parameter(torch.zeros(heads * dim, decay_rank, dtype=dtype), requires_grad=False)
        self.a2_bias = nn.Parameter(torch.zeros(heads * dim, dtype=torch.float32), requires_grad=False)
        self.norm = nn.Parameter(torch.ones(vdim, dtype=torch.float32), requires_grad=False)
        self.o = nn.Parameter(torch.zeros(width, heads * vdim, dtype=dtype), requires_grad=False)

    # checkpoint tensor (behind '<layer>.mix.') -> (parameter, section)
    TENSORS = {**{n: ("in_proj.weight", n) for n in ("q", "k", "v", "g", "a1")}, "a2": ("a2", None),
               "a2.b": ("a2_bias", None), "norm": ("norm", None), "o": ("o", None)}

    def cache_bytes(self, block_size: int):
        """(bytes of a cache block, bytes of a state slot)"""
        return 0, self.heads * self.dim * self.vdim * 4

    def new_cache(self, num_blocks: int, block_size: int, num_slots: int, device) -> torch.Tensor:
        return torch.zeros(num_slots, *self.state_shape(), dtype=torch.float32, device=device)

    def state_shape(self):
        return (self.heads, self.dim, self.vdim)

    def forward(self, h: torch.Tensor, batch, states: torch.Tensor) -> torch.Tensor:
        """h [T, width] -> [T, width] (as ``linear_parts`` has it); ``states`` float32 [slots, heads, dim, vdim] is updated in place."""
        T = h.shape[0]
        p = self.in_proj(h)
        out = torch.empty(T, self.heads * self.vdim, dtype=h.dtype, device=h.device)
        sec = self.in_proj.section_ptr
        a = _lib.GlaArgs(q=sec(p, "q"), k=sec(p, "k"), v=sec(p, "v"), g=sec(p, "g"), a1=sec(p, "a1"), stride=p.stride(0),
                         a2=self.a2.data_ptr(), bias=self.a2_bias.data_ptr(), norm_w=self.norm.data_ptr(), out=out.data_ptr(),
                         slots=batch.state_slots.data_ptr(), starts=batch.starts.data_ptr(), states=states.data_ptr(),
                         n_seqs=batch.n_seqs, heads=self.heads, dim=self.dim, vdim=self.vdim, rank=self.rank,
                         a2_stride=self.a2.stride(0), dtype=_lib.dtype_code(h.dtype), tau=self.tau, q_scale=self.dim ** -0.5,
                         eps=self.eps)
        lib, stream = _lib.load_decoder(), _lib.current_stream(h.device)
        if batch.max_q == 1:
            _lib.check_decoder(lib.ed_gla_step(byref(a), stream), "gla_step")
        else:
            log_decay = torch.empty(T, self.heads * self.dim, dtype=torch.float32, device=h.device)
            a.log_decay, a.chunks, a.seq_chunks = log_decay.data_ptr(), batch.chunks.data_ptr(), batch.seq_chunks.data_ptr()
            a.n_chunks, a.chunk_tokens = batch.n_chunks, batch.chunk_tokens
            if batch.n_chunks > batch.n_seqs:
                cs = torch.empty(batch.n_chunks, *self.state_shape(), dtype=torch.float32, device=h.device)
                cd = torch.empty(batch.n_chunks, self.heads * self.dim, dtype=torch.float32, device=h.device)
                a.chunk_states, a.chunk_decay = cs.data_ptr(), cd.data_ptr()
            _lib.check_decoder(lib.ed_gla_prefill(byref(a), stream), "gla_prefill")
        return linear_parts(out, self.o)
