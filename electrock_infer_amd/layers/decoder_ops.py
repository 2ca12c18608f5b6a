"""Row operations of a decoder whose residual stream is float32 (libelectrock_decoder.so), and the two matrix products
around them.  Every function takes and returns GPU tensors; there is no other path."""
import ctypes
from typing import Optional

import torch
import torch.nn.functional as F

from .. import _lib


def _ptr(t: Optional[torch.Tensor]) -> Optional[int]:
    return None if t is None else t.data_ptr()


def _skinny(x: torch.Tensor, weight: torch.Tensor, out: torch.Tensor, splits: int, act: int) -> torch.Tensor:
    (T, K), N = x.shape, weight.shape[0]
    code = _lib.load_decoder().ed_skinny_gemm(x.data_ptr(), weight.data_ptr(), out.data_ptr(), _lib.dtype_code(out.dtype), splits,
                                              T, N, K, act, _lib.current_stream(x.device))
    _lib.check_decoder(code, "skinny_gemm")
    return out


def _skinny_splits(x: torch.Tensor, weight: torch.Tensor) -> int:
    """For a decode batch that the weight-streaming kernel takes: how many ranges of K fill the chip; else 0."""
    if x.dtype != torch.bfloat16 or x.shape[0] > 64 or not x.is_contiguous():
        return 0
    return _lib.load_decoder().ed_skinny_gemm_splits(x.shape[0], weight.shape[0], x.shape[1])


def linear(x: torch.Tensor, weight: torch.Tensor, act: Optional[str] = None) -> torch.Tensor:
    """act(x @ weight^T) in x's type: a weight-streaming kernel for a decode batch, a library product otherwise;
    ``act``: None or 'relu_squared'."""
    if _skinny_splits(x, weight):
        return _skinny(x, weight, torch.empty(x.shape[0], weight.shape[0], dtype=x.dtype, device=x.device), 1, int(act is not None))
    out = F.linear(x, weight)
    return relu_squared_(out) if act is not None else out


def linear_silu_gate(x: torch.Tensor, weight: torch.Tensor) -> torch.Tensor:
    """silu(x @ gate^T) * (x @ up^T) for ``weight`` = [gate; up]: one launch for a decode batch."""
    (T, _), ff = x.shape, weight.shape[0] // 2
    out = torch.empty(T, ff, dtype=x.dtype, device=x.device)
    if _skinny_splits(x, weight):
        code = _lib.load_decoder().ed_skinny_gemm(x.data_ptr(), weight.data_ptr(), out.data_ptr(), _lib.dtype_code(out.dtype), 1, T, ff,
                                                  x.shape[1], 2, _lib.current_stream(x.device))
        _lib.check_decoder(code, "skinny_gemm")
        return out
    u = F.linear(x, weight)
    _lib.check_decoder(_lib.load_decoder().ed_silu_gate(u.data_ptr(), out.data_ptr(), T, ff, _lib.dtype_code(x.dtype),
                                                        _lib.current_stream(x.device)), "silu_gate")
    return out


def linear_f32(x: torch.Tensor, weight: torch.Tensor) -> torch.Tensor:
    """x @ weight^T with the float32 accumulators as the result, for sums that stay float32."""
    if x.dtype == torch.float32:
        return F.linear(x, weight)
    if _skinny_splits(x, weight):
        return _skinny(x, weight, torch.empty(x.shape[0], weight.shape[0], dtype=torch.float32, device=x.device), 1, 0)
    return torch.mm(x, weight.t(), out_dtype=torch.float32)


def linear_parts(x: torch.Tensor, weight: torch.Tensor, exact: bool = False) -> torch.Tensor:
    """x @ weight^T as ``residual_norm`` takes it: [T, N], or float32 partial sums [parts, T, N] of a decode batch.
    ``exact``: not rounded to the compute type on the way."""
    splits = _skinny_splits(x, weight)
    if splits > 1:
        return _skinny(x, weight, torch.empty(splits, x.shape[0], weight.shape[0], dtype=torch.float32, device=x.device), splits, 0)
    return linear_f32(x, weight) if exact else linear(x, weight)


def embed_rows(tokens: torch.Tensor, table: torch.Tensor, scale: float, copy: Optional[torch.Tensor] = None) -> torch.Tensor:
    """float32 rows table[tokens] * scale; ``copy`` (rows may be strided) receives them in the table's type."""
    T, W = tokens.numel(), table.shape[1]
    x = torch.empty(T, W, dtype=torch.float32, device=table.device)
    code = _lib.load_decoder().ed_embed(tokens.data_ptr(), table.data_ptr(), float(scale), x.data_ptr(), _ptr(copy),
                                        copy.stride(0) if copy is not None else 0, T, W, _lib.dtype_code(table.dtype),
                                        _lib.current_stream(table.device))
    _lib.check_decoder(code, "embed_rows")
    return x


KEEP, ADD_NORMED, REPLACE = 0, 1, 2


def residual_norm(update: int, x: torch.Tensor, y: Optional[torch.Tensor], post_w: Optional[torch.Tensor], eps: float,
                  out: Optional[torch.Tensor], next_w: Optional[torch.Tensor] = None) -> None:
    """Update the stream ``x`` in place (KEEP; ADD_NORMED: x += y / rms(y) * post_w; REPLACE: x = y + post_w) and write
    the next sublayer's input into ``out`` (rows may be strided): x / rms(x) * next_w, or x itself, in out's type.
    ``y`` [T, W] or partial sums [parts, T, W] (``linear_parts``)."""
    T, W = x.shape
    parts = y.shape[0] if y is not None and y.dim() == 3 else 1
    dtype = out.dtype if out is not None else (y.dtype if y is not None else x.dtype)
    code = _lib.load_decoder().ed_residual_norm(
        update, x.data_ptr(), _ptr(y), _lib.dtype_code(y.dtype if y is not None else dtype), parts, _ptr(post_w), _ptr(next_w),
        _ptr(out), out.stride(0) if out is not None else 0, T, W, float(eps), _lib.dtype_code(dtype),
        _lib.current_stream(x.device))
    _lib.check_decoder(code, "residual_norm")


def relu_squared_(u: torch.Tensor) -> torch.Tensor:
    code = _lib.load_decoder().ed_relu_squared(u.data_ptr(), u.numel(), _lib.dtype_code(u.dtype), _lib.current_stream(u.device))
    _lib.check_decoder(code, "relu_squared")
    return u


def gated_norm_(y: torch.Tensor, z_ptr: int, z_stride: int, weight: torch.Tensor, parts: int, eps: float) -> torch.Tensor:
    """y = y * silu(z), RMS-normed in equal parts of a row, times ``weight``; in place."""
    T, inner = y.shape
    code = _lib.load_decoder().ed_gated_norm(y.data_ptr(), z_ptr, z_stride, weight.data_ptr(), T, parts, inner // parts, float(eps),
                                             _lib.dtype_code(y.dtype), _lib.current_stream(y.device))
    _lib.check_decoder(code, "gated_norm")
    return y


def token_gate(x: torch.Tensor, gate: torch.Tensor, tokens: torch.Tensor, table: torch.Tensor, column0: int) -> torch.Tensor:
    """gelu_tanh(x @ gate^T) * table[tokens, column0 : column0 + dim]"""
    (T, W), dim = x.shape, gate.shape[0]
    g = torch.empty(T, dim, dtype=x.dtype, device=x.device)
    code = _lib.load_decoder().ed_token_gate(x.data_ptr(), gate.data_ptr(), tokens.data_ptr(), table.data_ptr(), table.stride(0),
                                             column0, g.data_ptr(), T, W, dim, _lib.dtype_code(x.dtype), _lib.current_stream(x.device))
    _lib.check_decoder(code, "token_gate")
    return g


def pad_k(w: torch.Tensor) -> torch.Tensor:
    """[heads, N, K] with K zero-padded to a multiple of 32: the operand form of ``head_gemm``."""
    return F.pad(w, (0, -w.shape[-1] % 32)).contiguous()


def head_gemm(a: torch.Tensor, a_row: int, a_head: int, b: torch.Tensor, K: int, out: torch.Tensor, out_row: int,
              out_head: int, T: int) -> None:
    """out[t, h, n] = sum_k a[t, h, k] b[h, n, k] (strides in elements; ``b`` from ``pad_k``)."""
    heads, N, _ = b.shape
    code = _lib.load_decoder().ed_head_gemm(a.data_ptr(), a_row, a_head, b.data_ptr(), out.data_ptr(), out_row, out_head, T,
                                            heads, N, K, _lib.dtype_code(b.dtype), _lib.current_stream(b.device))
    _lib.check_decoder(code, "head_gemm")


class StackedRows:
    """Places of several named sections in one parameter: ``sections`` name -> rows, every section starting at a multiple of
    ``align`` rows.  A checkpoint tensor that holds several sections one behind the other is loaded as 'first|second|...'."""

    def __init__(self, sections, align: int = 1):
        self.offset, self.rows, at = {}, dict(sections), 0
        for name, rows in self.rows.items():
            self.offset[name] = at
            at += -(-rows // align) * align
        self.total = at

    def parameter(self, *columns, dtype) -> torch.nn.Parameter:
        p = torch.nn.Parameter(torch.zeros(self.total, *columns, dtype=dtype), requires_grad=False)
        p.weight_loader = self.load
        return p

    def load(self, param, loaded: torch.Tensor, names: str) -> None:
        names = names.split("|")
        if loaded.shape != (sum(self.rows[n] for n in names), *param.shape[1:]):
            raise ValueError(f"projection '{'|'.join(names)}' is {tuple(loaded.shape)}, expected "
                             f"{(sum(self.rows[n] for n in names), *param.shape[1:])}")
        at = 0
        for n in names:
            param.data[self.offset[n]:self.offset[n] + self.rows[n]].copy_(loaded[at:at + self.rows[n]])
            at += self.rows[n]


class StackedLinear(torch.nn.Module):
    """Several projections of one input as a single matrix.  A section starts at a multiple of eight rows (zeros between),
    so that vector loads of its outputs are aligned."""

    def __init__(self, width: int, sections, dtype):
        super().__init__()
        self.places = StackedRows(sections, 8)
        self.offset, self.rows, self.out_rows = self.places.offset, self.places.rows, self.places.total
        self.weight = self.places.parameter(width, dtype=dtype)

    def forward(self, x: torch.Tensor) -> torch.Tensor:
        return linear(x, self.weight)

    def section_ptr(self, out: torch.Tensor, name: str) -> int:
        return out.data_ptr() + self.offset[name] * out.element_size()


byref = ctypes.byref
