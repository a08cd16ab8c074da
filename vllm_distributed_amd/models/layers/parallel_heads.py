"""Two sequence mixers side by side on one input: their output projections fused into one, or their input projections fused
and their outputs kept apart (each is normed before they meet)."""
from __future__ import annotations

import torch
import torch.nn as nn

from .linear import GroupedColumnLinear, RowParallelLinear


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


class ParallelNormed(nn.Module):
    """``left`` and ``right`` read the same input through ONE projection; their outputs, each ``o(heads)`` in the model
    width, are RMS-normed on their own (gains ``left_out`` / ``right_out``) before they join the residual stream, which the
    caller does in the launch that also adds the feed-forward (``layers.attention.ResidualRMSNorm.after_pair``).  Each
    half has ``sizes`` (its sub-matrices of the projection), ``out_cols`` and ``forward(columns) -> heads``."""

    def __init__(self, left: nn.Module, right: nn.Module, width: int, dtype: torch.dtype):
        super().__init__()
        self.left, self.right = left, right
        self.proj = GroupedColumnLinear(width, [left.sizes, right.sizes], dtype)
        self.left_o = RowParallelLinear(left.out_cols, width, False, dtype)
        self.right_o = RowParallelLinear(right.out_cols, width, False, dtype)
        f32 = torch.float32
        self.left_out = nn.Parameter(torch.zeros(width, dtype=f32), requires_grad=False)
        self.right_out = nn.Parameter(torch.zeros(width, dtype=f32), requires_grad=False)

    def forward(self, h: torch.Tensor):
        x = self.proj(h)
        (l0, l1), (r0, r1) = self.proj.columns(0), self.proj.columns(1)
        return self.left_o(self.left(x[:, l0:l1])), self.right_o(self.right(x[:, r0:r1]))
