"""Latent attention under an optional sliding window, with every size a parameter.

A token caches one row: its normalised key/value latent (padded to a multiple of 64) and one rotated key part shared by
the heads (padded to 64).  Rows that are a sequence's only row of the step run in the absorbed form -- the key
projection folded into the query, the value projection applied to the mixed latents -- over the pool; longer runs
expand the keys and values of the tokens they can see once and attend over those.  Sizes or types without a tile kernel
take the absorbed form one wave per row and head.
"""
from __future__ import annotations

import torch

from .. import ops_hybrid as hops
from .linear import Linear, pad, padded, vector


class LatentAttention:
    def __init__(self, c: dict, weight, pitch: int, eps: float, dtype, device, cos_sin: torch.Tensor):
        """c: heads, dim, rot_dim, vdim, q_rank, kv_rank, scale, mask (None or {"size"}), rot {"dims"}; weight(name): the
        tensor of that name in the activation type; cos_sin: the rotary table."""
        self.H, self.dim, self.rot_dim, self.vdim = c["heads"], c["dim"], c["rot_dim"], c["vdim"]
        self.R = c["kv_rank"]
        dq, dkv, uq, uk, uv, o = (weight(n) for n in ("dq", "dkv", "uq", "uk", "uv", "o"))
        self.q_rank = dq.shape[0]
        self.rot_dims = c["rot"]["dims"]
        self.scale = c["scale"]
        self.window = c["mask"]["size"] if c.get("mask") else 0
        self.eps, self.dtype, self.cos_sin = eps, dtype, cos_sin
        H, D = self.H, dq.shape[1]
        self.Rp, self.rotp = pad(self.R, 64), pad(self.rot_dim, 64)
        self.Qp, self.kp, self.vp = pad(self.q_rank, 128), pad(self.dim, 64), pad(self.vdim, 64)
        self.op = pad(H * self.vdim, 128)
        # one product for the query latent, the key/value latent and the rotated key part
        down = dq.new_zeros(self.Qp + self.Rp + self.rotp, pitch)
        down[: self.q_rank, :D] = dq
        down[self.Qp: self.Qp + self.R, :D] = dkv[: self.R]
        down[self.Qp + self.Rp: self.Qp + self.Rp + self.rot_dim, :D] = dkv[self.R:]
        self.down = Linear(down)
        self.wq, self.wkv = vector(weight("dq.norm"), self.Qp), vector(weight("dkv.norm"), self.Rp)
        q = uq.new_zeros(H, self.kp + self.rotp, self.Qp)
        uqh = uq.view(H, self.dim + self.rot_dim, self.q_rank)
        q[:, : self.dim, : self.q_rank] = uqh[:, : self.dim]
        q[:, self.kp: self.kp + self.rot_dim, : self.q_rank] = uqh[:, self.dim:]
        self.uq = Linear(q.view(H * (self.kp + self.rotp), self.Qp))
        ukh, uvh = uk.view(H, self.dim, self.R), uv.view(H, self.vdim, self.R)
        wk = padded(ukh.transpose(1, 2), H, self.Rp, self.kp)          # absorbed: [H, latent, key element]
        self.vn = pad(self.vdim, 16)
        wv = padded(uvh, H, self.vn, self.Rp)
        tile = dtype == torch.bfloat16
        self.wk, self.wv = (hops.pack_heads(wk), hops.pack_heads(wv)) if tile else (wk, wv)
        self.decode_tiles = tile and hops.latent_decode_supported(self.Rp, self.rotp)
        self.prefill_tiles = tile and self.rotp == 64 and hops.latent_prefill_supported(self.kp, self.vp)
        if self.prefill_tiles:
            self.w_expand = torch.cat([padded(ukh, H, self.kp, self.Rp).view(H * self.kp, self.Rp),
                                       padded(uvh, H, self.vp, self.Rp).view(H * self.vp, self.Rp)]).contiguous()
        self.o = Linear(padded(o, pitch, self.op))

    def bytes(self) -> int:
        """Bytes of matrix weights one step reads."""
        return sum(x.bytes() for x in (self.down, self.uq, self.o)) + sum(t.numel() * t.element_size() for t in (self.wk, self.wv))

    @property
    def cache_row(self):
        """(latent, rotated part) elements of a cached row."""
        return self.Rp, self.rotp

    def _splits(self, rows: int, max_context: int) -> int:
        """Splits of a row's visible range: enough blocks for two rounds of the chip, at least two tiles each."""
        tiles = (self.H + (31 if self.H >= 32 else 15)) // (32 if self.H >= 32 else 16)
        longest = min(self.window or max_context, max_context)
        return max(1, min(8, (512 + rows * tiles - 1) // (rows * tiles), (longest + 63) // 64))

    def _absorbed(self, q, batch, pool, lo, hi, attn, tiles):
        """Rows [lo, hi) of the step: q [rows, H, kp + rotp] (unrotated) -> attn [rows, H, vdim]."""
        M, H = hi - lo, self.H
        pos, req = batch.positions[lo:hi], batch.row_req[lo:hi]
        qa = torch.empty(M, H, self.Rp + self.rotp, dtype=self.dtype, device=q.device)
        hops.head_gemm(q[..., : self.kp], self.wk, qa[..., : self.Rp], self.kp, self.Rp)
        hops.latent_rope_q(q[..., self.kp:], qa[..., self.Rp:], self.cos_sin, pos, self.rot_dims)
        mixed = torch.empty(M, H, self.Rp, dtype=self.dtype, device=q.device)
        if tiles:
            S = self._splits(M, batch.max_context)
            part = torch.empty(M, H, S, self.Rp, dtype=torch.float32, device=q.device)
            lse = torch.empty(M, H, S, dtype=torch.float32, device=q.device)
            hops.latent_decode(qa, pool, batch.req_to_token, req, pos, part, lse, self.Rp, self.window, self.scale)
            hops.latent_merge(part, lse, mixed)
        else:
            hops.latent_attention_rows(qa, pool, batch.req_to_token, req, pos, mixed, self.window, self.scale)
        hops.head_gemm(mixed, self.wv, attn, self.Rp, self.vn)

    def _expanded(self, q, batch, pool, out):
        """Rows from batch.singles on: q, out are the whole step's rows."""
        n1, H = batch.singles, self.H
        qm = q[n1:].view(-1, H, self.kp + self.rotp)[..., self.kp:]
        hops.latent_rope_q(qm, qm, self.cos_sin, batch.positions[n1:], self.rot_dims)
        e = batch.expansion(self.window)
        seen = pool.index_select(0, batch.req_to_token.view(-1).index_select(0, e.table_index))
        kv = torch.matmul(seen[:, : self.Rp], self.w_expand.t())
        nk = H * self.kp
        hops.latent_prefill(q, kv[:, :nk], kv[:, nk:], seen[:, self.Rp:], out, e.row0, e.rows, e.tok0, e.ahead, e.max_rows, H,
                            self.kp, self.vp, self.vdim, self.window, self.scale)

    def forward(self, h, batch, pool):
        """pool: the layer's rows [slots, Rp + rotp].  Returns the output product's source."""
        T, H = h.shape[0], self.H
        cq = torch.empty(T, self.Qp, dtype=self.dtype, device=h.device)
        hops.latent_prep(self.down.source(h), self.wq, self.wkv, cq, pool, batch.loc, self.cos_sin, batch.positions, self.q_rank,
                         self.R, self.Rp, self.rot_dim, self.rot_dims, self.eps)
        q = self.uq.rows(cq)
        attn = (torch.zeros if self.op != H * self.vdim else torch.empty)(T, self.op, dtype=self.dtype, device=h.device)
        q3 = q.view(T, H, self.kp + self.rotp)
        a3 = attn[:, : H * self.vdim].unflatten(1, (H, self.vdim))
        n1 = batch.singles
        if n1:
            self._absorbed(q3[:n1], batch, pool, 0, n1, a3[:n1], self.decode_tiles)
        if n1 < T:
            if self.prefill_tiles:
                self._expanded(q, batch, pool, attn)
            else:
                self._absorbed(q3[n1:], batch, pool, n1, T, a3[n1:], False)
        return self.o.source(attn)
