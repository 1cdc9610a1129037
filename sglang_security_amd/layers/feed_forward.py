"""Feed-forwards, plain down(act(up x)) and gated down(act(gate x) * up x); the activation is applied where the first
product's split sums are added."""
from __future__ import annotations

import torch

from ..ops_hybrid import ACT_RELU2, ACT_SILU, source_act, source_gated_act
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


class GatedFeedForward:
    def __init__(self, gate: torch.Tensor, up: torch.Tensor, down: torch.Tensor, pitch: int, act: int = ACT_SILU):
        """gate, up [ff, width], down [width, ff]; rows of the residual stream are `pitch` long."""
        ff = pad(up.shape[0], 128)
        self.act, self.ff = act, ff
        self.gate_up = Linear(torch.cat([padded(gate, ff, pitch), padded(up, ff, pitch)]))
        self.down = Linear(padded(down, pitch, ff))

    def bytes(self) -> int:
        """Bytes of matrix weights one step reads."""
        return sum(x.bytes() for x in (self.gate_up, self.down))

    def forward(self, h):
        a = torch.empty(h.shape[0], self.ff, dtype=h.dtype, device=h.device)
        return self.down.source(source_gated_act(self.gate_up.source(h), a, self.act))
