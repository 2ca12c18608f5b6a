"""A per-layer input of the token: the stream gates a slice of a second embedding of the token, and the projected result
is normed and added to the stream."""
import torch
import torch.nn.functional as F
from torch import nn

from .decoder_ops import token_gate_


class TokenSideInput(nn.Module):

    def __init__(self, width: int, dim: int, column0: int, dtype):
        super().__init__()
        self.column0 = column0
        self.gate = nn.Parameter(torch.zeros(dim, width, dtype=dtype), requires_grad=False)
        self.proj = nn.Parameter(torch.zeros(width, dim, dtype=dtype), requires_grad=False)
        self.norm = nn.Parameter(torch.ones(width, dtype=torch.float32), requires_grad=False)

    def forward(self, x: torch.Tensor, tokens: torch.Tensor, table: torch.Tensor) -> torch.Tensor:
        """x [T, width] (the stream in the compute type) -> what is to be normed with ``norm`` and added."""
        return F.linear(token_gate_(F.linear(x, self.gate), tokens, table, self.column0), self.proj)
