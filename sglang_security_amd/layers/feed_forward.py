"""Un-gated feed-forward: down(act(up x)), the activation applied where the up product's split sums are added."""
from __future__ import annotations

import torch

from ..ops_hybrid import ACT_RELU2, source_act
from .linear import Linear, pad, padded


class FeedForward:
    def __init__(self, up: torch.Tensor, down: torch.Tensor, pitch: int, act: int = ACT_RELU2):
        """up [ff, width], down [width, ff]; rows of the residual stream are `pitch` long."""
        ff = pad(up.shape[0], 128)
        self.act, self.ff = act, ff
        self.up = Linear(padded(up, ff, pitch))
        self.down = Linear(padded(down, pitch, ff))

    def bytes(self) -> int:
        """Bytes of matrix weights one step reads."""
        return sum(x.bytes() for x in (self.up, self.down))

    def forward(self, h):
        src = self.up.source(h)
        a = torch.empty(h.shape[0], self.ff, dtype=h.dtype, device=h.device) if src.f32 else src.data
        return self.down.source(source_act(src, a, self.act))
