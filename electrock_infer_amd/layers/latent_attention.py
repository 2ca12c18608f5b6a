"""Latent attention (csrc/decoder/latent_attention.hip): keys and values of all heads are projections of one cached
latent per token; a rotated key part is shared by the heads; the softmax has a learned sink per head."""
import torch
import torch.nn.functional as F
from torch import nn

from .. import _lib
from .decoder_ops import StackedLinear, byref, head_gemm, linear_parts, pad_k


def rotary_frequencies(dims: int, base: float, factor: float = 1.0) -> torch.Tensor:
    """base^(-2i / dims) / factor for i < dims / 2, rounded once to float32."""
    return (float(base) ** (-torch.arange(0, dims, 2, dtype=torch.float64) / max(dims, 1)) / factor).float()


class LatentAttention(nn.Module):

    PROMPT_TOKENS = 64           # portions from this length on write their keys and values out, if the kernel takes the sizes
    TARGET_WORKGROUPS = 768      # the keys are shared out over workgroups until a launch has about this many

    def __init__(self, width: int, heads: int, dim: int, rot_dim: int, vdim: int, kv_rank: int, scale: float,
                 rotary_base: float, eps: float, dtype):
        super().__init__()
        self.heads, self.dim, self.rot, self.vdim, self.rank = heads, dim, rot_dim, vdim, kv_rank
        self.scale, self.rotary_base, self.eps = scale, rotary_base, eps
        self.pitch = (kv_rank + 7) // 8 * 8
        self.in_proj = StackedLinear(width, {"q": heads * (dim + rot_dim), "dkv": kv_rank + rot_dim}, dtype)
        self.latent_norm = nn.Parameter(torch.ones(kv_rank, dtype=torch.float32), requires_grad=False)
        self.uk = nn.Parameter(torch.zeros(heads * dim, kv_rank, dtype=dtype), requires_grad=False)
        self.uv = nn.Parameter(torch.zeros(heads * vdim, kv_rank, dtype=dtype), requires_grad=False)
        self.sink = nn.Parameter(torch.zeros(heads, dtype=torch.float32), requires_grad=False)
        self.o = nn.Parameter(torch.zeros(width, heads * vdim, dtype=dtype), requires_grad=False)
        self.register_buffer("inv_freq", torch.zeros(rot_dim // 2, dtype=torch.float32), persistent=False)
        self.uk_t = self.uv_p = None

    TENSORS = {"q": ("in_proj.weight", "q"), "dkv": ("in_proj.weight", "dkv"), "dkv.norm": ("latent_norm", None),
               "uk": ("uk", None), "uv": ("uv", None), "sink": ("sink", None), "o": ("o", None)}

    def finish_loading(self) -> None:
        """Forms of the weights that the kernels read."""
        self.inv_freq.copy_(rotary_frequencies(self.rot, self.rotary_base))
        self.uk_t = pad_k(self.uk.data.view(self.heads, self.dim, self.rank).transpose(1, 2))
        self.uv_p = pad_k(self.uv.data.view(self.heads, self.vdim, self.rank))

    def cache_bytes(self, block_size: int):
        """(bytes of a cache block, bytes of a state slot)"""
        return block_size * self.row_elems() * self.uk.element_size(), 0

    def new_cache(self, num_blocks: int, block_size: int, num_slots: int, device) -> torch.Tensor:
        return torch.zeros(num_blocks, block_size, self.row_elems(), dtype=self.uk.dtype, device=device)

    def row_elems(self) -> int:
        """Elements that one token takes in the cache."""
        return self.pitch + (self.rot + 7) // 8 * 8

    def splits(self, batch) -> int:
        groups = -(-batch.max_q * self.heads // 16) * batch.n_seqs
        return max(1, min(-(-self.TARGET_WORKGROUPS // groups), -(-batch.max_context // 128), 64))

    def forward(self, h: torch.Tensor, batch, cache: torch.Tensor) -> torch.Tensor:
        """h [T, width] -> [T, width] (as ``linear_parts`` has it); ``cache`` [blocks, block_size, row_elems] receives the new tokens' rows first."""
        T, dev = h.shape[0], h.device
        p = self.in_proj(h)
        a = _lib.LatentArgs(q=self.in_proj.section_ptr(p, "q"), q_stride=p.stride(0), down=self.in_proj.section_ptr(p, "dkv"),
                            down_stride=p.stride(0), latent_w=self.latent_norm.data_ptr(), inv_freq=self.inv_freq.data_ptr(),
                            positions=batch.positions.data_ptr(), cache_rows=batch.cache_rows.data_ptr(),
                            cache=cache.data_ptr(), sink=self.sink.data_ptr(), q_begin=batch.q_begin.data_ptr(),
                            starts=batch.starts.data_ptr(), tables=batch.tables.data_ptr(), T=T, n_seqs=batch.n_seqs,
                            max_q=batch.max_q, table_width=batch.table_width, block_size=cache.shape[1], splits=1,
                            heads=self.heads, dim=self.dim, rot=self.rot, rank=self.rank, dtype=_lib.dtype_code(h.dtype),
                            scale=self.scale, eps=self.eps)
        _lib.check_decoder(_lib.load_decoder().ed_latent_prepare(byref(a), _lib.current_stream(dev)), "latent_prepare")
        o = torch.empty(T, self.heads * self.vdim, dtype=h.dtype, device=dev)
        if self.writes_out(batch, h.dtype):
            self._attend_written_out(p, batch, cache, o)
        else:
            self._attend_paged(a, p, batch, o)
        return linear_parts(o, self.o)

    def writes_out(self, batch, dtype) -> bool:
        """A long portion: the up-projections of its context cost less than attending over the latents."""
        return (batch.max_q >= self.PROMPT_TOKENS and dtype == torch.bfloat16 and self.scale > 0 and
                _lib.load_decoder().ed_latent_prompt_supported(self.dim, self.rot, self.vdim) == 1)

    def _attend_paged(self, a, p: torch.Tensor, batch, o: torch.Tensor) -> None:
        T, H, dev = o.shape[0], self.heads, o.device
        q_lat = torch.empty(T, H, self.pitch, dtype=o.dtype, device=dev)
        o_lat = torch.empty_like(q_lat)
        a.q_latent, a.out, a.splits = q_lat.data_ptr(), o_lat.data_ptr(), self.splits(batch)
        if a.splits > 1:
            part_o = torch.empty(T * H * a.splits * self.pitch, dtype=torch.float32, device=dev)
            part_ml = torch.empty(T * H * a.splits * 2, dtype=torch.float32, device=dev)
            a.part_o, a.part_ml = part_o.data_ptr(), part_ml.data_ptr()
        head_gemm(p, p.stride(0), self.dim + self.rot, self.uk_t, self.dim, q_lat, H * self.pitch, self.pitch, T)
        _lib.check_decoder(_lib.load_decoder().ed_latent_paged(byref(a), _lib.current_stream(dev)), "latent_paged")
        head_gemm(o_lat, H * self.pitch, self.pitch, self.uv_p, self.rank, o, H * self.vdim, self.vdim, T)

    def _attend_written_out(self, p: torch.Tensor, batch, cache: torch.Tensor, o: torch.Tensor) -> None:
        dev, row, lib, stream = o.device, self.row_elems(), _lib.load_decoder(), _lib.current_stream(o.device)
        rows = torch.empty(batch.padded_keys, row, dtype=o.dtype, device=dev)
        _lib.check_decoder(lib.ed_latent_gather(cache.data_ptr(), batch.tables.data_ptr(), batch.table_width, cache.shape[1],
                                                batch.k_begin.data_ptr(), batch.k_lens.data_ptr(), batch.n_seqs,
                                                -(-batch.max_context // 64) * 64, row, rows.data_ptr(),
                                                _lib.dtype_code(o.dtype), stream), "latent_gather")
        latents = rows[:, :self.rank]
        k = F.linear(latents, self.uk)
        vt = torch.mm(self.uv, latents.t())
        a = _lib.LatentPromptArgs(q=self.in_proj.section_ptr(p, "q"), q_stride=p.stride(0), k=k.data_ptr(), k_stride=k.stride(0),
                                  k_rot=rows.data_ptr() + self.pitch * rows.element_size(), k_rot_stride=row, vt=vt.data_ptr(),
                                  v_stride=vt.stride(0), out=o.data_ptr(), sink=self.sink.data_ptr(),
                                  q_begin=batch.q_begin.data_ptr(), starts=batch.starts.data_ptr(),
                                  k_begin=batch.k_begin.data_ptr(), n_seqs=batch.n_seqs, max_q=batch.max_q, heads=self.heads,
                                  dim=self.dim, rot=self.rot, vdim=self.vdim, scale=self.scale)
        _lib.check_decoder(lib.ed_latent_prompt(byref(a), stream), "latent_prompt")
