"""Dense feed-forward: down(act(up(h))), or down(act(gate(h)) * up(h))."""
import torch
from torch import nn

from .decoder_ops import StackedRows, linear, linear_parts, linear_silu_gate


class DenseMLP(nn.Module):
    """``activation``: 'relu_squared', or 'silu_gate' for a gated one, whose two input matrices are stacked in ``up``."""

    ACTIVATIONS = ("relu_squared", "silu_gate")

    def __init__(self, width: int, ff: int, dtype, activation: str = "relu_squared"):
        super().__init__()
        if activation not in self.ACTIVATIONS:
            raise ValueError(f"unknown activation '{activation}'")
        self.activation = activation
        if activation == "silu_gate":
            self.up = StackedRows({"gate": ff, "up": ff}).parameter(width, dtype=dtype)
            self.TENSORS = {"gate": ("up", "gate"), "up": ("up", "up"), "down": ("down", None)}
        else:
            self.up = nn.Parameter(torch.zeros(ff, width, dtype=dtype), requires_grad=False)
            self.TENSORS = {"up": ("up", None), "down": ("down", None)}
        self.down = nn.Parameter(torch.zeros(width, ff, dtype=dtype), requires_grad=False)

    def forward(self, h: torch.Tensor) -> torch.Tensor:
        """-> [T, width] (as ``linear_parts`` has it)"""
        u = linear_silu_gate(h, self.up) if self.activation == "silu_gate" else linear(h, self.up, self.activation)
        return linear_parts(u, self.down)
