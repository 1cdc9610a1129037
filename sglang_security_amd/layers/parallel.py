"""Mixers side by side on the same input, their results added: one product makes every mixer's inputs and one product
takes all their results back to the residual width.

A mixer has `w_in` [inputs, pitch], `w_out` [pitch, results] (rows and columns padded to multiples of eight), an optional
`b_out` [pitch] in fp32, a `cache_spec`, and mix(source of its inputs, batch, pool, out [rows, results]).
"""
from __future__ import annotations

import torch

from .linear import Linear, pad, padded


class Parallel:
    def __init__(self, mixers, pitch: int, dtype):
        self.mixers, self.dtype = list(mixers), dtype
        self.inputs, self.results, ni, nr = [], [], 0, 0
        for m in self.mixers:
            self.inputs.append((ni, ni + m.w_in.shape[0]))
            self.results.append((nr, nr + m.w_out.shape[1]))
            ni, nr = self.inputs[-1][1], self.results[-1][1]
        self.nr = nr
        w_in, w_out = torch.cat([m.w_in for m in self.mixers]), torch.cat([m.w_out for m in self.mixers], 1)
        self.w_in, self.w_out = Linear(padded(w_in, pad(ni, 128), pitch)), Linear(padded(w_out, pitch, pad(nr, 128)))
        biases = [m.b_out for m in self.mixers if m.b_out is not None]
        self.bias = sum(biases) if biases else None      # joins the residual stream beside the product
        for m in self.mixers:
            m.w_in = m.w_out = None                      # they live in the stacked products from here on

    def bytes(self) -> int:
        """Bytes of matrix weights one step reads."""
        return self.w_in.bytes() + self.w_out.bytes()

    @property
    def cache_spec(self):
        return ("parallel", [m.cache_spec for m in self.mixers])

    def forward(self, h, batch, pools):
        """Returns the output product's source (without `bias`)."""
        T = h.shape[0]
        src = self.w_in.source(h)
        out = (torch.zeros if self.w_out.K != self.nr else torch.empty)(T, self.w_out.K, dtype=self.dtype, device=h.device)
        for m, pool, (i0, i1), (r0, r1) in zip(self.mixers, pools, self.inputs, self.results):
            m.mix(src.columns(i0, i1), batch, pool, out[:, r0:r1])
        return self.w_out.source(out)
