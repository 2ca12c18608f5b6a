"""Dense feed-forward: down(act(up(h)))."""
import torch
from torch import nn

from .decoder_ops import linear, linear_parts


class DenseMLP(nn.Module):
    """``activation``: 'relu_squared'."""

    ACTIVATIONS = ("relu_squared",)

    def __init__(self, width: int, ff: int, dtype, activation: str = "relu_squared"):
        super().__init__()
        if activation not in self.ACTIVATIONS:
            raise ValueError(f"unknown activation '{activation}'")
        self.activation = activation
        self.up = nn.Parameter(torch.zeros(ff, width, dtype=dtype), requires_grad=False)
        self.down = nn.Parameter(torch.zeros(width, ff, dtype=dtype), requires_grad=False)

    def forward(self, h: torch.Tensor) -> torch.Tensor:
        """-> [T, width] (as ``linear_parts`` has it)"""
        return linear_parts(linear(h, self.up, self.activation), self.down)
