"""Hyper-connections: the residual stream as several copies that every sublayer
reads as one weighted sum and writes back to with a matrix.

With streams x_1 .. x_s and a sublayer F,

    u = sum_s read[s] x_s,    y = F(norm(u)),
    x_t <- sum_s mix[s, t] x_s + write[t] y     (all streams from the old ones),

mix indexed [from, to]. The streams are fp32 whatever the activation dtype and
lie side by side in one row per token, [x_1 | x_2 | ...]. Writing one
sublayer's result and reading the next one's input is a single kernel
(ops.hyper_rmsnorm), so a HyperConnection only holds the coefficients.
"""

from __future__ import annotations

import torch
import torch.nn as nn


class HyperConnection(nn.Module):
    """The coefficients of one sublayer."""

    def __init__(self, streams: int):
        super().__init__()
        self.streams = int(streams)
        self.read = nn.Parameter(torch.empty(streams), requires_grad=False)
        self.write = nn.Parameter(torch.empty(streams), requires_grad=False)
        self.mix = nn.Parameter(torch.empty(streams, streams), requires_grad=False)
        self._f32 = None

    def invalidate_constants(self) -> None:
        self._f32 = None

    def f32(self, device):
        """(read, write, mix) as fp32 on the run device."""
        if self._f32 is None or self._f32[0].device != device:
            self._f32 = tuple(p.detach().float().contiguous().to(device)
                              for p in (self.read, self.write, self.mix))
        return self._f32
