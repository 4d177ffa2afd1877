"""Two sequence mixers side by side on the same input (layer type 'parallel')."""

from __future__ import annotations

import torch
import torch.nn as nn

from ..parallel.layers import MergedColumnParallelLinear
from .forward_meta import ForwardMeta


class ParallelMixer(nn.Module):
    """Two mixers over the same input. The input projections of both are one
    GEMM; the two results stay apart (forward returns both) so that the
    caller's residual kernel scales (left_scale, right_scale: for it to use),
    norms and adds them in fp32. Both mixers are built with own_proj=False;
    the left one's mix() takes its projections as a list, the right one's as
    one column range of the merged result."""

    def __init__(self, hidden_size: int, left: nn.Module, right: nn.Module,
                 left_scale: float = 1.0, right_scale: float = 1.0):
        super().__init__()
        self.left, self.right = left, right
        self.left_scale, self.right_scale = float(left_scale), float(right_scale)
        self.n_left = len(left.proj_sizes)
        self.in_proj = MergedColumnParallelLinear(
            hidden_size, list(left.proj_sizes) + list(right.proj_sizes))
        self._right_width = sum(right.proj_sizes)

    def invalidate_constants(self) -> None:
        self.left.invalidate_constants()
        self.right.invalidate_constants()

    def forward(self, h: torch.Tensor, meta: ForwardMeta):
        y = self.in_proj(h)
        parts = self.in_proj.split_output(y)
        a = self.left.o_proj(self.left.mix(parts[: self.n_left], meta, h.dtype))
        # the right mixer's projections are adjacent columns of y
        b = self.right.o_proj(
            self.right.mix(y[:, y.shape[1] - self._right_width:], meta))
        return a, b
