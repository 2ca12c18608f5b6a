"""Recurrent mixers with one decay per head and token behind short causal convolutions (csrc/decoder/recurrence.hip): the
gated delta rule and the state-space form.  A sequence carries a float32 state per head and its last projections."""
from typing import Dict, NamedTuple, Optional

import torch
from torch import nn

from .. import _lib
from .decoder_ops import StackedLinear, StackedRows, byref, gated_norm_, linear_parts

UNIT_EPS = 1e-6      # under the root of the delta rule's unit vectors


class RecurrentCache(NamedTuple):
    states: torch.Tensor      # float32 [slots, heads, dim, vdim]
    ring: torch.Tensor        # [slots, taps, channels]: the projection of position p in row p % taps


class DecayedRecurrence(nn.Module):
    """What both mixers share: q, k [kv_heads, dim] and v [heads, vdim] from convolutions over ``in_proj``'s sections of
    these names, decay inputs in its section ``decay``, and the recurrence itself."""

    def __init__(self, width: int, heads: int, kv_heads: int, dim: int, vdim: int, taps: int, eps: float, sections: Dict[str, int],
                 conv_bias: bool, dtype):
        super().__init__()
        if heads % kv_heads:
            raise ValueError(f"{heads} heads cannot share {kv_heads} keys")
        self.heads, self.kv_heads, self.dim, self.vdim, self.taps, self.eps = heads, kv_heads, dim, vdim, taps, eps
        self.in_proj = StackedLinear(width, sections, dtype)
        channels = StackedRows({"q": kv_heads * dim, "k": kv_heads * dim, "v": heads * vdim})
        self.channels = channels.total
        vector = lambda n, value: nn.Parameter(torch.full((n,), value, dtype=torch.float32), requires_grad=False)
        self.conv = channels.parameter(taps, dtype=torch.float32)
        self.conv_bias = channels.parameter(dtype=torch.float32) if conv_bias else None
        self.a_log, self.dt_bias = vector(heads, 0.0), vector(heads, 0.0)
        self.o = nn.Parameter(torch.zeros(width, heads * vdim, dtype=dtype), requires_grad=False)

    def state_shape(self):
        return (self.heads, self.dim, self.vdim)

    def cache_bytes(self, block_size: int):
        """(bytes of a cache block, bytes of a state slot)"""
        return 0, self.heads * self.dim * self.vdim * 4 + self.taps * self.channels * self.o.element_size()

    def new_cache(self, num_blocks: int, block_size: int, num_slots: int, device) -> RecurrentCache:
        return RecurrentCache(torch.zeros(num_slots, *self.state_shape(), dtype=torch.float32, device=device),
                              torch.zeros(num_slots, self.taps, self.channels, dtype=self.o.dtype, device=device))

    def recur(self, p: torch.Tensor, batch, cache: RecurrentCache, beta: Optional[str] = None, gate: Optional[str] = None,
              norm: Optional[torch.Tensor] = None, skip: Optional[torch.Tensor] = None, q_scale: float = 1.0,
              unit_eps: float = 0.0) -> torch.Tensor:
        """[T, heads * vdim] of the projections ``p``; ``cache`` is updated in place.  ``beta`` and ``gate`` name sections of
        ``in_proj``: with them it is the delta rule with its normed and gated output."""
        T, dev, delta = p.shape[0], p.device, beta is not None
        out = torch.empty(T, self.heads * self.vdim, dtype=p.dtype, device=dev)
        sec, ptr = lambda n: self.in_proj.section_ptr(p, n) if n else None, lambda t: None if t is None else t.data_ptr()
        a = _lib.RecurArgs(q=sec("q"), k=sec("k"), v=sec("v"), decay_in=sec("decay"), beta_in=sec(beta), gate=sec(gate),
                           stride=p.stride(0), conv_w=self.conv.data_ptr(), conv_b=ptr(self.conv_bias), a_log=self.a_log.data_ptr(),
                           dt_bias=self.dt_bias.data_ptr(), skip=ptr(skip), norm_w=ptr(norm), ring=cache.ring.data_ptr(),
                           states=cache.states.data_ptr(), out=out.data_ptr(), slots=batch.state_slots.data_ptr(),
                           starts=batch.starts.data_ptr(), n_seqs=batch.n_seqs, heads=self.heads, kv_heads=self.kv_heads,
                           dim=self.dim, vdim=self.vdim, taps=self.taps, dtype=_lib.dtype_code(p.dtype), q_scale=q_scale,
                           unit_eps=unit_eps, eps=self.eps)
        lib, stream = _lib.load_decoder(), _lib.current_stream(dev)
        if batch.max_q == 1:
            _lib.check_decoder(lib.ed_recur_step(byref(a), stream), "recur_step")
            return out
        f32 = lambda *shape: torch.empty(*shape, dtype=torch.float32, device=dev)
        H, padded, chunks = self.heads, -(-self.dim // 16) * 16, batch.n_chunks
        scratch = {"q_rows": f32(T, self.kv_heads, padded), "k_rows": f32(T, self.kv_heads, padded), "v_rows": torch.empty_like(out),
                   "rates": f32(T, H, 2), "blocks": f32(chunks, batch.chunk_tokens // 16, H, lib.ed_recur_record(int(delta)))}
        if chunks > batch.n_seqs:
            scratch["chunk_states"] = f32(chunks, *self.state_shape())
            scratch["chunk_trans"] = f32(chunks, H, padded, padded) if delta else f32(chunks, H)
        for name, t in scratch.items():
            setattr(a, name, t.data_ptr())
        a.q_begin, a.chunks, a.seq_chunks = batch.q_begin.data_ptr(), batch.chunks.data_ptr(), batch.seq_chunks.data_ptr()
        a.n_chunks, a.chunk_tokens = chunks, batch.chunk_tokens
        _lib.check_decoder(lib.ed_recur_prefill(byref(a), stream), "recur_prefill")
        return out


class GatedDeltaRule(DecayedRecurrence):

    def __init__(self, width: int, heads: int, kv_heads: int, dim: int, vdim: int, taps: int, eps: float, dtype):
        super().__init__(width, heads, kv_heads, dim, vdim, taps, eps,
                         {"q": kv_heads * dim, "k": kv_heads * dim, "v": heads * vdim, "gate": heads * vdim, "decay": heads,
                          "beta": heads}, False, dtype)
        self.norm = nn.Parameter(torch.ones(vdim, dtype=torch.float32), requires_grad=False)

    # checkpoint tensor (behind '<layer>.mix.') -> (parameter, section)
    TENSORS = {**{n: ("in_proj.weight", s) for n, s in (("q", "q"), ("k", "k"), ("v", "v"), ("g", "gate"), ("a", "decay"), ("b", "beta"))},
               **{n + ".conv": ("conv", n) for n in "qkv"}, "A_log": ("a_log", None), "dt_bias": ("dt_bias", None),
               "norm": ("norm", None), "o": ("o", None)}

    def forward(self, h: torch.Tensor, batch, cache: RecurrentCache, carried=None) -> torch.Tensor:
        """h [T, width] -> [T, width] (as ``linear_parts`` has it)"""
        return linear_parts(self.recur(self.in_proj(h), batch, cache, "beta", "gate", self.norm, q_scale=self.dim ** -0.5,
                                       unit_eps=UNIT_EPS), self.o)


class StateSpaceMixer(DecayedRecurrence):
    """Mamba-2: q, k and v are C, B and x; a skip per head; the gated output is normed in ``norm_groups`` parts."""

    def __init__(self, width: int, heads: int, groups: int, state: int, vdim: int, taps: int, norm_groups: int, eps: float, dtype):
        inner, shared = heads * vdim, groups * state
        if inner % norm_groups:
            raise ValueError(f"{inner} channels cannot be normed in {norm_groups} equal parts")
        super().__init__(width, heads, groups, state, vdim, taps, eps,
                         {"z": inner, "v": inner, "k": shared, "q": shared, "decay": heads}, True, dtype)
        self.norm_groups = norm_groups
        self.skip = nn.Parameter(torch.ones(heads, dtype=torch.float32), requires_grad=False)
        self.norm = nn.Parameter(torch.ones(inner, dtype=torch.float32), requires_grad=False)

    TENSORS = {"in": ("in_proj.weight", "z|v|k|q|decay"), "conv": ("conv", "v|k|q"), "conv.b": ("conv_bias", "v|k|q"),
               "dt_bias": ("dt_bias", None), "A_log": ("a_log", None), "D": ("skip", None), "norm": ("norm", None), "o": ("o", None)}

    def forward(self, h: torch.Tensor, batch, cache: RecurrentCache, carried=None) -> torch.Tensor:
        """h [T, width] -> [T, width] (as ``linear_parts`` has it)"""
        p = self.in_proj(h)
        y = self.recur(p, batch, cache, skip=self.skip)
        return linear_parts(gated_norm_(y, self.in_proj.section_ptr(p, "z"), p.stride(0), self.norm, self.norm_groups, self.eps), self.o)
