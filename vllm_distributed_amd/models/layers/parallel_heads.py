"""Two sequence mixers side by side on one input, their output projections fused into one."""
from __future__ import annotations

import torch
import torch.nn as nn

from .linear import RowParallelLinear


class ParallelHeads(nn.Module):
    """``left`` and ``right`` read the same input and write their (already scaled) heads into neighbouring columns; one
    projection over ``[left heads | right heads]`` gives the sum of both halves.  Each half has ``out_cols`` and
    ``forward(h, index, out)``; ``index`` counts the runs of a layer that runs several times in a forward pass."""

    def __init__(self, left: nn.Module, right: nn.Module, width: int, dtype: torch.dtype):
        super().__init__()
        self.left, self.right, self.dtype = left, right, dtype
        self.o = RowParallelLinear(left.out_cols + right.out_cols, width, False, dtype)

    def load_output_half(self, half: int, w: torch.Tensor) -> None:
        """A half's own output projection ``[width, out_cols]`` into its columns of the fused one."""
        lo, n = (0, self.left.out_cols) if half == 0 else (self.left.out_cols, self.right.out_cols)
        assert tuple(w.shape) == (self.o.weight.shape[0], n), (tuple(w.shape), n)
        self.o.weight.data[:, lo:lo + n].copy_(w)

    def forward(self, h: torch.Tensor, index: int = 0) -> torch.Tensor:
        nl = self.left.out_cols
        heads = torch.empty((h.shape[0], nl + self.right.out_cols), dtype=self.dtype, device=h.device)
        self.left(h, index, heads[:, :nl])
        self.right(h, index, heads[:, nl:])
        return self.o(heads)
