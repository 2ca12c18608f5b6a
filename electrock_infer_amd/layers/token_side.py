"""A per-layer input of the token: the stream gates a slice of a second embedding of the token, and the projected result
is normed and added to the stream."""
import torch
from torch import nn

from .. import _lib
from .decoder_ops import ADD_NORMED, linear, residual_norm, token_gate


class TokenSideInput(nn.Module):

    ONE_LAUNCH_ROWS = 2     # in widths: fewer rows do not fill the chip with the one-launch kernel's workgroups

    def __init__(self, width: int, dim: int, column0: int, dtype):
        super().__init__()
        self.column0 = column0
        self.gate = nn.Parameter(torch.zeros(dim, width, dtype=dtype), requires_grad=False)
        self.proj = nn.Parameter(torch.zeros(width, dim, dtype=dtype), requires_grad=False)
        self.norm = nn.Parameter(torch.ones(width, dtype=torch.float32), requires_grad=False)

    def forward(self, x: torch.Tensor, tokens: torch.Tensor, table: torch.Tensor) -> torch.Tensor:
        """x [T, width] (the stream in the compute type) -> what is to be normed with ``norm`` and added."""
        return linear(token_gate(x, self.gate, tokens, table, self.column0), self.proj)

    def close_layer(self, x: torch.Tensor, y: torch.Tensor, post_w: torch.Tensor, tokens: torch.Tensor, table: torch.Tensor,
                    eps: float, out: torch.Tensor, next_w) -> None:
        """Everything from the feed-forward's result ``y`` to the next layer's input: the stream ``x`` takes the normed y,
        then the token's input; ``out`` (rows may be strided) = x / rms(x) * next_w, or x.  One launch for a bfloat16
        prompt of a width its kernel takes; a few rows are better spread over the chip in four."""
        T, W = x.shape
        lib, dim = _lib.load_decoder(), self.gate.shape[0]
        if T >= self.ONE_LAUNCH_ROWS * W and y.dim() == 2 and y.dtype == torch.bfloat16 and out.stride(0) % 4 == 0 and lib.ed_token_side_supported(W, dim) == 1:
            code = lib.ed_token_side(x.data_ptr(), y.data_ptr(), post_w.data_ptr(), self.gate.data_ptr(), self.proj.data_ptr(),
                                     tokens.data_ptr(), table.data_ptr(), table.stride(0), self.column0, self.norm.data_ptr(),
                                     None if next_w is None else next_w.data_ptr(), out.data_ptr(), out.stride(0), T, W, dim,
                                     float(eps), _lib.current_stream(x.device))
            _lib.check_decoder(code, "token_side")
            return
        rows = torch.empty(T, W, dtype=out.dtype, device=x.device)
        residual_norm(ADD_NORMED, x, y, post_w, eps, rows)
        residual_norm(ADD_NORMED, x, self(rows, tokens, table), self.norm, eps, out, next_w)
