"""Latent attention (csrc/decoder/latent_attention.hip): keys and values of all heads are projections of one cached
latent per token; a rotated key part is shared by the heads; the softmax has a learned sink per head."""
import torch
import torch.nn.functional as F
from torch import nn

from .. import _lib
from .decoder_ops import StackedLinear, byref, head_gemm, pad_k


def rotary_frequencies(dims: int, base: float) -> torch.Tensor:
    """base^(-2i / dims) for i < dims / 2, rounded once to float32."""
    return (float(base) ** (-torch.arange(0, dims, 2, dtype=torch.float64) / max(dims, 1))).float()


class LatentAttention(nn.Module):

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

    def row_elems(self) -> int:
        """Elements that one token takes in the cache."""
        return self.pitch + (self.rot + 7) // 8 * 8

    def splits(self, batch) -> int:
        groups = -(-batch.max_q * self.heads // 16) * batch.n_seqs
        return max(1, min(-(-self.TARGET_WORKGROUPS // groups), -(-batch.max_context // 128), 64))

    def forward(self, h: torch.Tensor, batch, cache: torch.Tensor) -> torch.Tensor:
        """h [T, width] -> [T, width]; ``cache`` [blocks, block_size, row_elems] receives the new tokens' rows first."""
        T, H, dev = h.shape[0], self.heads, h.device
        p = self.in_proj(h)
        q_lat = torch.empty(T, H, self.pitch, dtype=h.dtype, device=dev)
        o_lat = torch.empty_like(q_lat)
        splits = self.splits(batch)
        a = _lib.LatentArgs(q=self.in_proj.section_ptr(p, "q"), q_stride=p.stride(0), down=self.in_proj.section_ptr(p, "dkv"),
                            down_stride=p.stride(0), latent_w=self.latent_norm.data_ptr(), inv_freq=self.inv_freq.data_ptr(),
                            positions=batch.positions.data_ptr(), cache_rows=batch.cache_rows.data_ptr(),
                            cache=cache.data_ptr(), q_latent=q_lat.data_ptr(), out=o_lat.data_ptr(), sink=self.sink.data_ptr(),
                            q_begin=batch.q_begin.data_ptr(), starts=batch.starts.data_ptr(), tables=batch.tables.data_ptr(),
                            T=T, n_seqs=batch.n_seqs, max_q=batch.max_q, table_width=batch.table_width,
                            block_size=cache.shape[1], splits=splits, heads=H, dim=self.dim, rot=self.rot, rank=self.rank,
                            dtype=_lib.dtype_code(h.dtype), scale=self.scale, eps=self.eps)
        if splits > 1:
            part_o = torch.empty(T * H * splits * self.pitch, dtype=torch.float32, device=dev)
            part_ml = torch.empty(T * H * splits * 2, dtype=torch.float32, device=dev)
            a.part_o, a.part_ml = part_o.data_ptr(), part_ml.data_ptr()
        lib, stream = _lib.load_decoder(), _lib.current_stream(dev)
        _lib.check_decoder(lib.ed_latent_prepare(byref(a), stream), "latent_prepare")
        head_gemm(p, p.stride(0), self.dim + self.rot, self.uk_t, self.dim, q_lat, H * self.pitch, self.pitch, T)
        _lib.check_decoder(lib.ed_latent_paged(byref(a), stream), "latent_paged")
        o = torch.empty(T, H * self.vdim, dtype=h.dtype, device=dev)
        head_gemm(o_lat, H * self.pitch, self.pitch, self.uv_p, self.rank, o, H * self.vdim, self.vdim, T)
        return F.linear(o, self.o)
