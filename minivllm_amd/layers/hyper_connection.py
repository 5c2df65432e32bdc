"""Hyper-connections: several residual streams in place of one.

A token carries S streams x_1 .. x_S (fp32).  A sublayer reads u = sum_a read[a] x_a, and its
output y is written back while the streams are mixed, all new ones from the old ones:
x_b <- sum_a mix[a, b] x_a + mult write[b] y.  With one stream and all numbers 1 this is the
ordinary residual sum x <- x + mult y.

The update, the next sublayer's read and its (element-wise) norm are one kernel
(``ops.hyper_update_norm``), so a sublayer costs one read and one write of the streams.
"""
from __future__ import annotations

import torch
import torch.nn as nn

MAX_STREAMS = 8                  # what the kernels keep in registers per thread


class HyperConnection(nn.Module):
    def __init__(self, streams: int, mult: float = 1.0):
        super().__init__()
        if not 1 <= streams <= MAX_STREAMS:
            raise ValueError(f"between 1 and {MAX_STREAMS} residual streams")
        self.streams, self.mult = int(streams), float(mult)
        f32 = dict(dtype=torch.float32)
        self.read = nn.Parameter(torch.ones(streams, **f32), requires_grad=False)
        # ``write`` holds the learned numbers times ``mult``
        self.write = nn.Parameter(torch.full((streams,), self.mult, **f32), requires_grad=False)
        self.mix = nn.Parameter(torch.eye(streams, **f32), requires_grad=False)

    @torch.no_grad()
    def load(self, read: torch.Tensor, write: torch.Tensor, mix: torch.Tensor) -> None:
        """``mix`` is indexed [from, to]."""
        self.read.copy_(read)
        self.write.copy_(write.to(device=self.write.device, dtype=torch.float32) * self.mult)
        self.mix.copy_(mix)
