"""Causal grouped-query attention whose values are its keys before their norm, with norms over whole projections, a
learned bias by distance, a temperature on the query and a sink; every size a parameter.

A token caches one row of all key/value heads and one number, the key norm's factor: the norm's weight is folded into the
query (with the scale and log2(e); the kernels work in base 2).  Rows that are a sequence's only row of the step run
split over the context, longer runs in blocks of rows, both over the pool through the request table.  Sizes or types
without a tile kernel take one wave per row and head.

The mixer owns rows of a stacked input product (`w_in`) and columns of a stacked output product (`w_out`, `b_out`): see
layers/parallel.py.
"""
from __future__ import annotations

import torch

from .. import ops_hybrid as hops
from .linear import pad, padded, vector
from .position_bias import LOG2E, distance_table

TILE_SIZES = (32, 64, 96, 128, 192, 256)


def head_pitch(dim: int) -> int:
    return next((s for s in TILE_SIZES if s >= dim), pad(dim, 32))


class TiedAttention:
    def __init__(self, c: dict, weight, pitch: int, eps: float, dtype, factor: torch.Tensor, max_context: int,
                 out_scale: float = 1.0):
        """c: heads, kv_heads, dim, scale, bias_max; weight(name, type=None): the tensor of that name, in the activation
        type unless another is asked for; factor: the query's temperature by position; out_scale: factor on the result."""
        H, G, dim = self.H, self.G, self.dim = c["heads"], c["kv_heads"], c["dim"]
        if H % G:
            raise ValueError(f"{H} query heads over {G} key/value heads")
        D = self.D = head_pitch(dim)
        self.eps, self.dtype, self.factor, self.out_scale = eps, dtype, factor, out_scale
        self.tiles = dtype == torch.bfloat16 and hops.tied_supported(D)
        f32 = lambda name: weight(name, torch.float32)
        heads = lambda t, n: padded(t.reshape(n, dim, -1), n, D, t.numel() // (n * dim)).reshape(n * D, -1)
        width = weight("q").shape[1]
        self.w_in = padded(torch.cat([heads(weight("q"), H), heads(weight("k"), G)]), (H + G) * D, pitch)
        self.bias = torch.cat([heads(f32("q.b"), H), heads(f32("k.b"), G)]).reshape(-1).contiguous()
        wk = f32("k.norm").double().view(G, 1, dim).expand(G, H // G, dim).reshape(H, dim)
        wq = f32("q.norm").double().view(H, dim) * wk * (c["scale"] * LOG2E)
        self.wq = vector(padded(wq.float(), H, D), H * D)
        o = weight("o")
        self.w_out = padded(o.view(width, H, dim), pitch, H, D).view(pitch, H * D)
        self.b_out = vector(f32("o.b") * out_scale, pitch)
        self.w = hops.TiedWeights(bias=distance_table(f32("rel"), c["bias_max"], max_context),
                                  sink=(f32("sink").double() * LOG2E).float().contiguous(), heads=H, kv_heads=G, D=D)

    @property
    def cache_spec(self):
        return ("tied", self.G * self.D)

    def _splits(self, rows: int, max_context: int) -> int:
        """Splits of a row's context: two blocks for every unit of the chip, a tile for each of a block's waves."""
        blocks = rows * self.G * ((self.H // self.G + 15) // 16)
        return max(1, min(64, (512 + blocks - 1) // blocks, (max_context + 127) // 128))

    def mix(self, src, batch, pool, out):
        """src: the rows' columns of the stacked input product; pool: the layer's TiedKVPool; out [rows, H * D]."""
        T, n1 = out.shape[0], batch.singles
        q = torch.empty(T, self.H * self.D, dtype=self.dtype, device=out.device)
        hops.tied_prep(src, self.bias, self.wq, self.factor, q, pool.rows, pool.rms, batch.loc, batch.positions, self.H * self.dim,
                       self.G * self.dim, self.eps)
        kv = (pool.rows, pool.rms, batch.req_to_token)
        if not self.tiles:
            hops.tied_rows(q, *kv, batch.row_req, batch.positions, self.w, out, self.out_scale)
            return
        if n1:
            S = self._splits(n1, batch.max_context)
        if n1 and S == 1:
            hops.tied_decode(q[:n1], *kv, batch.row_req, batch.positions, self.w, out=out[:n1], out_scale=self.out_scale)
        elif n1:
            part = torch.empty(n1, self.H, S, self.D, dtype=torch.float32, device=out.device)
            lse = torch.empty(n1, self.H, S, dtype=torch.float32, device=out.device)
            hops.tied_decode(q[:n1], *kv, batch.row_req, batch.positions, self.w, part, lse)
            hops.tied_merge(part, lse, self.w, out[:n1], self.out_scale)
        if n1 < T:
            s = batch.seqs
            hops.tied_prefill(q, *kv, s.row0[n1:], s.rows[n1:], s.start[n1:], s.slot[n1:], int(batch.host["rows"].max()), self.w, out,
                              self.out_scale)
