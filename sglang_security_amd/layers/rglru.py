"""Recurrent mixer: two branches, a short causal convolution and a real-gated linear recurrent unit on one of them, gelu on
the other, their product projected out.  Channels are kept block by block, each block padded to a multiple of 32."""
from __future__ import annotations

import torch

from .. import ops_hybrid as hops
from .linear import Linear, pad, padded

MAX_TILE_BLOCK = 1024   # channels of a gate block that fit the tile kernels' LDS rows


class Rglru:
    def __init__(self, c: dict, weight, pitch: int, dtype):
        """c: width, blocks, conv (taps); weight(name): the tensor of that name in the activation type."""
        wx, wy, o = weight("x"), weight("y"), weight("o")
        self.width, self.blocks, D = wx.shape[0], c["blocks"], wx.shape[1]
        bw = self.width // self.blocks
        self.bwp = pad(bw, 32)
        used = self.blocks * self.bwp
        self.W = pad(used, 128)
        self.dtype = dtype
        self.tiles = dtype == torch.bfloat16 and self.bwp <= MAX_TILE_BLOCK
        ch = torch.arange(self.width, device=wx.device)
        place = ch // bw * self.bwp + ch % bw                # where a channel lives

        def channels(t, dim=0):
            """channel axis `dim` of t spread to its padded places, W long"""
            shape = list(t.shape)
            shape[dim] = self.W
            return t.new_zeros(shape).index_copy_(dim, place, t.contiguous())

        xy = wx.new_zeros(2, self.W, pitch)
        xy[0, :, :D], xy[1, :, :D] = channels(wx), channels(wy)
        self.xy = Linear(xy.view(2 * self.W, pitch))
        self.o = Linear(padded(channels(o, 1), pitch, self.W))
        f = lambda name: channels(weight(name).float().reshape(self.width))
        gates = [padded(weight(n), self.blocks, self.bwp, self.bwp) for n in ("ra", "ri")]
        if self.tiles:
            gates = [hops.pack_heads(g) for g in gates]
        sp = torch.nn.functional.softplus(weight("lam").double()).float()
        self.w = hops.RglruWeights(bx=f("x.b"), by=f("y.b"), conv=channels(weight("conv").float()).t().contiguous(),
                                   conv_b=f("conv.b"), wr=gates[0], wi=gates[1], br=f("ra.b"), bi=f("ri.b"), sp=channels(sp),
                                   blocks=self.blocks, bwp=self.bwp)

    def bytes(self) -> int:
        """Bytes of matrix weights one step reads."""
        return sum(x.bytes() for x in (self.xy, self.o)) + sum(t.numel() * t.element_size() for t in (self.w.wr, self.w.wi))

    def forward(self, h, batch, cache):
        """cache: the layer's mem_cache.RecurrentStatePool.  Returns the output product's source."""
        T = h.shape[0]
        w, seqs = self.w, batch.seqs
        src = self.xy.source(h)
        u = torch.empty(T, self.W, dtype=self.dtype, device=h.device)
        y = torch.empty_like(u)
        out = (torch.zeros_like if self.W != w.used else torch.empty_like)(u)
        n1 = batch.singles if self.tiles else 0
        hops.rglru_conv(src, w, u, y, cache.conv, seqs, n1)
        if not self.tiles:
            hops.rglru_rows(src, u, y, w, cache.conv, cache.state, seqs, out)
        else:
            if n1:
                hops.rglru_step(u, y, w, cache.state, seqs, out, n1)
            if n1 < T:
                hops.rglru_scan(src, u, y, w, cache.conv, cache.state, seqs, out, n1, n1, batch.tile_row, batch.tile_rows,
                                batch.tile0)
        return self.o.source(out)
