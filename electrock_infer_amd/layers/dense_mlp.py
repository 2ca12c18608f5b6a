"""Dense feed-forward: down(act(up(h)))."""
import torch
import torch.nn.functional as F
from torch import nn

from .decoder_ops import relu_squared_


class DenseMLP(nn.Module):
    """``activation``: 'relu_squared'."""

    ACTIVATIONS = {"relu_squared": relu_squared_}

    def __init__(self, width: int, ff: int, dtype, activation: str = "relu_squared"):
        super().__init__()
        self.act_ = self.ACTIVATIONS[activation]
        self.up = nn.Parameter(torch.zeros(ff, width, dtype=dtype), requires_grad=False)
        self.down = nn.Parameter(torch.zeros(width, ff, dtype=dtype), requires_grad=False)

    def forward(self, h: torch.Tensor) -> torch.Tensor:
        return F.linear(self.act_(F.linear(h, self.up)), self.down)
