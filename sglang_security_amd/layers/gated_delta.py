"""Gated delta rule: heads with a matrix state that is decayed, corrected towards the current value along the current key,
and read by the query; short convolutions with silu in front, a gated norm per head behind.

Rows that are a sequence's only row of the step are walked one by one, longer portions in tiles of 64 rows; types or sizes
without a tile kernel are walked row after row.  Key and value sizes are padded to multiples of 32 and 16 (zeros).  The mixer owns rows of a stacked input product (`w_in`)
and columns of a stacked output product (`w_out`): see layers/parallel.py.
"""
from __future__ import annotations

import torch

from .. import ops_hybrid as hops
from .linear import pad, padded, vector


class GatedDelta:
    b_out = None

    def __init__(self, c: dict, weight, pitch: int, eps: float, dtype, out_scale: float = 1.0):
        """c: heads, kv_heads, dim, vdim, conv (taps); weight(name, type=None): the tensor of that name, in the activation
        type unless another is asked for; out_scale: factor on the result."""
        H, K, dim, vdim = c["heads"], c["kv_heads"], c["dim"], c["vdim"]
        if H % K:
            raise ValueError(f"{H} heads over {K} query/key heads")
        dp, vp, Hp = pad(dim, 32), pad(vdim, 16), pad(H, 8)
        self.dtype, self.out_scale, self.taps = dtype, out_scale, c["conv"]
        self.tiles = dtype == torch.bfloat16 and hops.delta_chunk_supported(dp, vp)
        f32 = lambda name: weight(name, torch.float32)

        def heads(t, n, d, to):
            return padded(t.reshape(n, d, -1), n, to, t.numel() // (n * d)).reshape(n * to, -1)

        sizes = {"q": (K, dim, dp), "k": (K, dim, dp), "v": (H, vdim, vp)}
        q = weight("q")
        width = q.shape[1]
        rows = [heads(weight(n), *sizes[n]) for n in "qkv"] + [heads(weight("g"), H, vdim, vp), padded(weight("b"), Hp, width),
                                                               padded(weight("a"), Hp, width)]
        self.w_in = padded(torch.cat(rows), sum(r.shape[0] for r in rows), pitch)
        self.conv = torch.cat([heads(f32(n + ".conv"), *sizes[n]) for n in "qkv"]).t().contiguous()
        self.w_out = padded(weight("o").view(width, H, vdim), pitch, H, vp).view(pitch, H * vp)
        self.w = hops.DeltaWeights(rate=f32("A_log").double().exp().float(), dt=f32("dt_bias").contiguous(),
                                   norm=vector(f32("norm"), vp), heads=H, kv_heads=K, dp=dp, vp=vp, dim=dim, vdim=vdim,
                                   b_col=H * vp, a_col=H * vp + Hp, eps=eps)

    @property
    def cache_spec(self):
        return ("matrix", self.w.channels, self.taps, (self.w.heads, self.w.dp, self.w.vp))

    def mix(self, src, batch, pool, out):
        """src: the rows' columns of the stacked input product; pool: the layer's RecurrentStatePool; out [rows, H * vp]."""
        T, n1, w, seqs = out.shape[0], batch.singles, self.w, batch.seqs
        u = torch.empty(T, w.channels, dtype=self.dtype, device=out.device)
        hops.short_conv(src.columns(0, w.channels), self.conv, u, pool.conv, seqs, n1, hops.ACT_SILU)
        gates = src.columns(w.channels, src.cols)
        n = seqs.rows.numel()
        step_to = n1 if self.tiles else n                # sequences that are walked row after row
        if step_to:
            hops.delta_step(u, gates, w, pool.state, seqs, out, self.out_scale, 0, step_to)
        if step_to < n:
            hops.delta_chunk(u, gates, w, pool.state, seqs, out, self.out_scale, n1, n1, batch.tile_row, batch.tile_rows, batch.tile0)
