"""Entry points over the C ABI for decoders with an fp32 residual stream, latent or tied attention, gated linear recurrences
or delta rules: argument checks and launches on torch's current stream, in the manner of ops.py.

A `Source` is a product's result on its way to the kernel that consumes it: fp32 split sums that nobody has added up yet,
or finished rows of the activation type.
"""
from __future__ import annotations

import dataclasses
from typing import Optional

import torch

from ._lib import SglkError, check, dtype_code, lib
from .ops import _need_gpu, _ptr, _stream

ACT_NONE, ACT_RELU2, ACT_GELU_TANH, ACT_SILU = 0, 1, 2, 3


@dataclasses.dataclass
class Source:
    data: torch.Tensor         # [splits, rows, cols] fp32, or [rows, cols] rows of the activation type
    f32: bool

    @property
    def rows(self):
        return self.data.shape[-2]

    @property
    def cols(self):
        return self.data.shape[-1]

    def args(self):
        d = self.data
        if d.stride(-1) != 1:
            raise SglkError("a product's rows must have unit inner stride")
        if self.f32:
            return _ptr(d), 1, d.shape[0], d.stride(0), d.stride(1)
        return _ptr(d), 0, 1, 0, d.stride(0)

    def columns(self, lo: int, hi: int) -> "Source":
        """The same rows, columns [lo, hi) only (lo a multiple of eight)."""
        return Source(self.data[..., lo:hi], self.f32)


_NO_SOURCE = (0, 0, 1, 0, 0)


def _f32(t, n, what):
    if t is not None and (t.dtype != torch.float32 or t.numel() < n or not t.is_contiguous()):
        raise SglkError(f"{what} must be a contiguous float32 tensor of at least {n} elements")


def _i32(t, n, what):
    if t is not None and (t.dtype != torch.int32 or t.numel() < n or not t.is_contiguous()):
        raise SglkError(f"{what} must be a contiguous int32 tensor of at least {n} elements")


def _src_ok(src: Source, rows, cols, dtype, what):
    _need_gpu(src.data)
    if src.rows < rows or src.cols < cols or src.data.dtype != (torch.float32 if src.f32 else dtype):
        raise SglkError(f"{what}: the product's rows {tuple(src.data.shape)} {src.data.dtype} do not fit [{rows}, {cols}]")


def residual_norm(x, width, eps, h=None, w_next=None, src: Optional[Source] = None, w_post=None, embed=None, ids=None,
                  embed_scale=1.0, x0=None, add_x0=False, step=None, rows=None, store_x=True, dtype=torch.bfloat16):
    """x (fp32 [rows, pitch], in place) += norm(src) * w_post (+ x0, + step); h = norm(x) * w_next.  With `embed`, x starts
    as embed[ids] * embed_scale and is saved to x0.  `rows` picks rows for h (x is not written then)."""
    _need_gpu(x, h, embed)
    pitch = x.shape[1]
    M = x.shape[0] if rows is None else rows.numel()
    _f32(x, x.shape[0] * pitch, "residual_norm: x")
    _f32(x0, x.shape[0] * pitch if x0 is not None else 0, "residual_norm: x0")
    for t, what in ((w_post, "w_post"), (step, "step"), (w_next, "w_next")):
        _f32(t, pitch, f"residual_norm: {what}")
    _i32(ids, x.shape[0], "residual_norm: ids")
    _i32(rows, 0, "residual_norm: rows")
    if src is not None:
        _src_ok(src, x.shape[0], pitch, dtype, "residual_norm")
    if w_next is not None and (h is None or h.dtype != dtype or h.shape[0] < M or h.shape[1] < pitch or h.stride(1) != 1):
        raise SglkError("residual_norm: h does not fit")
    if embed is not None and (embed.dtype != dtype or embed.shape[1] < pitch or embed.stride(1) != 1):
        raise SglkError("residual_norm: embedding table does not fit")
    check(lib().sglk_residual_norm(
        _ptr(x), _ptr(embed), _ptr(ids), 0 if embed is None else embed.stride(0), float(embed_scale),
        *(_NO_SOURCE if src is None else src.args()), _ptr(w_post), _ptr(x0), int(add_x0), _ptr(step), _ptr(w_next), _ptr(h),
        0 if h is None else h.stride(0), _ptr(rows), int(store_x and rows is None), M, width, pitch, float(eps),
        dtype_code(dtype), _stream(x)), "residual_norm")


def source_act(src: Source, out, act, bias=None):
    """out = act(src + bias), rounded once to the type of out."""
    M, N = out.shape
    _src_ok(src, M, N, out.dtype, "source_act")
    _f32(bias, N, "source_act: bias")
    check(lib().sglk_source_act(*src.args(), _ptr(bias), _ptr(out), M, N, out.stride(0), int(act), dtype_code(out.dtype),
                                _stream(out)), "source_act")
    return out


def source_gated_act(src: Source, out, act):
    """out = act(first half of src's columns) * second half."""
    M, N = out.shape
    _src_ok(src, M, 2 * N, out.dtype, "source_gated_act")
    check(lib().sglk_source_gated_act(*src.args(), _ptr(out), M, N, out.stride(0), int(act), dtype_code(out.dtype), _stream(out)),
          "source_gated_act")
    return out


def capped_logits(src: Source, out, cap, dtype):
    """fp32 out [M, V] = cap * tanh(src / cap); cap None or 0: src."""
    M, V = out.shape
    _src_ok(src, M, V, dtype, "capped_logits")
    _f32(out, M * V, "capped_logits: out")
    check(lib().sglk_capped_logits(*src.args(), _ptr(out), M, src.cols, V, out.stride(0), float(cap or 0.0), dtype_code(dtype),
                                   _stream(out)), "capped_logits")
    return out


def assign_slots(req_to_token, row_seq, seq_req, positions, loc):
    T = loc.numel()
    for t, what in ((row_seq, "row_seq"), (positions, "positions"), (loc, "loc")):
        _i32(t, T, f"assign_slots: {what}")
    _i32(seq_req, 1, "assign_slots: seq_req")
    if req_to_token.dtype != torch.int32:
        raise SglkError("assign_slots: req_to_token must be int32")
    check(lib().sglk_assign_slots(_ptr(req_to_token), req_to_token.stride(0), _ptr(row_seq), _ptr(seq_req), _ptr(positions),
                                  _ptr(loc), T, _stream(req_to_token)), "assign_slots")


# ------------------------------------------------------------------------------------------------ latent attention
def pack_heads(w):
    """[H, N, K] -> the operand order head_gemm streams (N a multiple of 16, K of 32)."""
    H, N, K = w.shape
    return w.view(H, N // 16, 16, K // 32, 4, 8).permute(0, 1, 3, 4, 2, 5).contiguous()


def latent_prep(src: Source, wq, wkv, cq, pool, loc, cos_sin, positions, q_rank, kv_rank, r_pitch, rot_dim, rot_dims, eps):
    M, q_pitch = cq.shape
    rot_pitch = pool.shape[-1] - r_pitch
    _src_ok(src, M, q_pitch + r_pitch + rot_pitch, cq.dtype, "latent_prep")
    _f32(wq, q_pitch, "latent_prep: wq")
    _f32(wkv, r_pitch, "latent_prep: wkv")
    _i32(loc, M, "latent_prep: loc")
    _i32(positions, M, "latent_prep: positions")
    _f32(cos_sin, rot_dims, "latent_prep: cos_sin")
    if pool.dtype != cq.dtype or pool.stride(-1) != 1:
        raise SglkError("latent_prep: the pool must be of the activation type")
    check(lib().sglk_latent_prep(*src.args(), _ptr(wq), _ptr(wkv), _ptr(cq), cq.stride(0), _ptr(pool), pool.stride(0),
                                 _ptr(loc), _ptr(cos_sin), _ptr(positions), M, q_rank, q_pitch, kv_rank, r_pitch, rot_dim,
                                 rot_pitch, rot_dims, float(eps), dtype_code(cq.dtype), _stream(cq)), "latent_prep")


def latent_rope_q(src, out, cos_sin, positions, rot_dims):
    """src, out [M, H, rot_pitch] views (they may be the same)."""
    M, H, rot_pitch = src.shape
    _need_gpu(src, out)
    _i32(positions, M, "latent_rope_q: positions")
    if out.shape != src.shape or out.dtype != src.dtype or src.stride(2) != 1 or out.stride(2) != 1:
        raise SglkError("latent_rope_q: src and out must be [M, H, n] views with unit inner stride")
    check(lib().sglk_latent_rope_q(_ptr(src), src.stride(0), src.stride(1), _ptr(out), out.stride(0), out.stride(1),
                                   _ptr(cos_sin), _ptr(positions), M, H, rot_pitch, rot_dims, dtype_code(src.dtype),
                                   _stream(src)), "latent_rope_q")


def head_gemm(a, w, out, K, Np):
    """out [M, H, N] = a [M, H, K] . w^T per head."""
    M, H, N = out.shape
    _need_gpu(a, w, out)
    if a.shape[0] != M or a.shape[1] != H or a.shape[2] < K or a.stride(2) != 1 or out.stride(2) != 1 or w.numel() != H * Np * K:
        raise SglkError("head_gemm: shapes do not match")
    if not (a.dtype == out.dtype == w.dtype):
        raise SglkError("head_gemm: a, w and out must be of one type")
    check(lib().sglk_head_gemm(_ptr(a), a.stride(0), a.stride(1), _ptr(w), _ptr(out), M, H, N, Np, K, out.stride(0), out.stride(1),
                               dtype_code(out.dtype), _stream(out)), "head_gemm")
    return out


def latent_merge(part, lse, out):
    """Split partials [M, H, S, K] and their log-sum-exps [M, H, S] -> out [M, H, K] contiguous."""
    M, H, S, K = part.shape
    _f32(part, M * H * S * K, "latent_merge: part")
    _f32(lse, M * H * S, "latent_merge: lse")
    if out.shape != (M, H, K) or not out.is_contiguous():
        raise SglkError("latent_merge: out must be contiguous [M, H, K]")
    check(lib().sglk_latent_merge(_ptr(part), _ptr(lse), S, _ptr(out), M * H, K, dtype_code(out.dtype), _stream(out)), "latent_merge")
    return out


def latent_decode_supported(r_pitch, rot_pitch) -> bool:
    return bool(lib().sglk_latent_decode_supported(r_pitch, rot_pitch))


def latent_prefill_supported(k_pitch, v_pitch) -> bool:
    return bool(lib().sglk_latent_prefill_supported(k_pitch, v_pitch))


def _check_rows(q, pool, req, positions, what):
    _need_gpu(q, pool)
    M = q.shape[0]
    _i32(req, M, f"{what}: req")
    _i32(positions, M, f"{what}: positions")
    if q.dtype != pool.dtype or q.stride(2) != 1 or pool.stride(-1) != 1 or q.shape[2] > pool.shape[-1]:
        raise SglkError(f"{what}: query and pool rows do not match")


def latent_decode(q, pool, req_to_token, req, positions, part, lse, r_pitch, window, scale):
    """q [M, H, r_pitch + rot_pitch] over the pool -> part [M, H, S, r_pitch], lse [M, H, S]."""
    _check_rows(q, pool, req, positions, "latent_decode")
    M, H, D = q.shape
    S = lse.shape[2]
    _f32(part, M * H * S * r_pitch, "latent_decode: part")
    _f32(lse, M * H * S, "latent_decode: lse")
    check(lib().sglk_latent_decode(_ptr(q), q.stride(0), q.stride(1), _ptr(pool), pool.stride(0), _ptr(req_to_token),
                                   req_to_token.stride(0), _ptr(req), _ptr(positions), _ptr(part), _ptr(lse), M, H, r_pitch,
                                   D - r_pitch, int(window or 0), S, float(scale), _stream(q)), "latent_decode")


def latent_attention_rows(q, pool, req_to_token, req, positions, out, window, scale):
    """q [M, H, D] over the pool -> out [M, H, DV]: any size and float type."""
    _check_rows(q, pool, req, positions, "latent_attention_rows")
    M, H, D = q.shape
    if out.shape[:2] != (M, H) or out.dtype != q.dtype or out.stride(2) != 1:
        raise SglkError("latent_attention_rows: out does not match")
    check(lib().sglk_latent_attention_rows(
        _ptr(q), q.stride(0), q.stride(1), _ptr(pool), pool.stride(0), _ptr(req_to_token), req_to_token.stride(0), _ptr(req),
        _ptr(positions), _ptr(out), out.stride(0), out.stride(1), M, H, D, out.shape[2], int(window or 0), float(scale),
        dtype_code(q.dtype), _stream(q)), "latent_attention_rows")


def latent_prefill(q, k, v, kr, o, row0, rows, tok0, ahead, max_rows, H, k_pitch, v_pitch, vdim, window, scale):
    """q [T, H * (k_pitch + 64)], k [N, H * k_pitch], v [N, H * v_pitch], kr [N, 64], o [T, >= H * vdim] (bf16)."""
    _need_gpu(q, k, v, kr, o)
    n = rows.numel()
    for t, what in ((row0, "row0"), (rows, "rows"), (tok0, "tok0"), (ahead, "ahead")):
        _i32(t, n, f"latent_prefill: {what}")
    if not (q.dtype == k.dtype == v.dtype == kr.dtype == o.dtype == torch.bfloat16):
        raise SglkError("latent_prefill: bf16 only")
    if kr.shape[1] != 64 or k.shape[1] < H * k_pitch or v.shape[1] < H * v_pitch or o.shape[1] < H * vdim:
        raise SglkError("latent_prefill: rows too short")
    check(lib().sglk_latent_prefill(_ptr(q), q.stride(0), _ptr(k), k.stride(0), _ptr(v), v.stride(0), _ptr(kr), kr.stride(0),
                                    _ptr(o), o.stride(0), vdim, _ptr(row0), _ptr(rows), _ptr(tok0), _ptr(ahead), n,
                                    int(max_rows), H, k_pitch, v_pitch, vdim, int(window or 0), float(scale), _stream(q)),
          "latent_prefill")


# ----------------------------------------------------------------------------------------- gated linear recurrence
@dataclasses.dataclass
class RglruWeights:
    """One mixer's parameters in the kernels' layout (channels block by block, bwp per block, rows of W)."""
    bx: torch.Tensor
    by: torch.Tensor
    conv: torch.Tensor       # [taps, W]
    conv_b: torch.Tensor
    wr: torch.Tensor
    wi: torch.Tensor
    br: torch.Tensor
    bi: torch.Tensor
    sp: torch.Tensor         # softplus(lambda)
    blocks: int
    bwp: int

    @property
    def W(self):
        return self.conv.shape[1]

    @property
    def taps(self):
        return self.conv.shape[0]

    @property
    def used(self):
        return self.blocks * self.bwp


@dataclasses.dataclass
class RowSeqs:
    """Which sequence every row belongs to, and per sequence: first row, rows, position of the first row, state slot."""
    row_seq: torch.Tensor
    row0: torch.Tensor
    rows: torch.Tensor
    start: torch.Tensor
    slot: torch.Tensor


def _conv_args(src, w: RglruWeights, u, y, conv_state, seqs: RowSeqs, singles):
    M = u.shape[0]
    _src_ok(src, M, 2 * w.W, u.dtype, "rglru")
    n = seqs.rows.numel()
    _i32(seqs.row_seq, M, "rglru: row_seq")
    for t in (seqs.row0, seqs.rows, seqs.start, seqs.slot):
        _i32(t, n, "rglru: sequence arrays")
    for t in (w.bx, w.by, w.conv_b, w.br, w.bi, w.sp):
        _f32(t, w.W, "rglru: channel vectors")
    _f32(w.conv, w.taps * w.W, "rglru: conv")
    if u.shape != (M, w.W) or y.shape != u.shape or y.dtype != u.dtype or not (u.is_contiguous() and y.is_contiguous()):
        raise SglkError("rglru: u and y must be contiguous [rows, W]")
    if conv_state.shape[1:] != (w.taps - 1, w.W) or conv_state.dtype != u.dtype or not conv_state.is_contiguous():
        raise SglkError("rglru: convolution state does not match")
    return (*src.args(), _ptr(w.bx), _ptr(w.by), _ptr(w.conv), _ptr(w.conv_b), _ptr(u), _ptr(y), _ptr(conv_state),
            _ptr(seqs.row_seq), _ptr(seqs.row0), _ptr(seqs.rows), _ptr(seqs.start), _ptr(seqs.slot), M, w.W, w.taps,
            int(singles), n)


def rglru_conv(src, w, u, y, conv_state, seqs, singles):
    check(lib().sglk_rglru_conv(*_conv_args(src, w, u, y, conv_state, seqs, singles), dtype_code(u.dtype), _stream(u)),
          "rglru_conv")


def _gate_ok(u, w):
    if u.dtype != torch.bfloat16 or w.wr.dtype != torch.bfloat16 or w.wr.numel() != w.blocks * w.bwp ** 2 or w.wi.numel() != w.wr.numel():
        raise SglkError("rglru: the tile kernels take bf16 gate weights in operand order")


def rglru_step(u, y, w, state, seqs, out, M):
    """The first M rows, each a sequence of its own (sequence m is row m)."""
    _gate_ok(u, w)
    _f32(state, state.shape[0] * w.W, "rglru_step: state")
    _i32(seqs.start, M, "rglru_step: start")
    if u.shape[0] < M or y.shape[0] < M or out.shape[0] < M or out.dtype != u.dtype or state.shape[1] != w.W:
        raise SglkError("rglru_step: rows do not match")
    check(lib().sglk_rglru_step(_ptr(u), _ptr(w.wr), _ptr(w.wi), _ptr(w.br), _ptr(w.bi), _ptr(w.sp), _ptr(y), _ptr(state),
                                _ptr(seqs.start), _ptr(seqs.slot), _ptr(out), out.stride(0), M, w.W, w.bwp, w.blocks,
                                _stream(u)), "rglru_step")


def rglru_scan(src, u, y, w, conv_state, state, seqs, out, singles, seq0, tile_row, tile_rows, tile0):
    """Rows from `singles` on (sequences from seq0 on), in tiles of 64 rows of one sequence."""
    _gate_ok(u, w)
    tiles = tile_row.numel()
    _i32(tile_rows, tiles, "rglru_scan: tile_rows")
    _i32(tile0, seqs.rows.numel(), "rglru_scan: tile0")
    M = u.shape[0]
    if out.shape[0] < M or out.dtype != u.dtype or out.shape[1] < w.used or state.shape[1] != w.W or state.dtype != torch.float32:
        raise SglkError("rglru_scan: rows do not match")
    hloc = torch.empty(M, w.W, dtype=torch.float32, device=u.device)
    prod = torch.empty_like(hloc)
    carry = torch.empty(tiles, w.W, dtype=torch.float32, device=u.device)
    check(lib().sglk_rglru_gates(_ptr(u), _ptr(w.wr), _ptr(w.wi), _ptr(w.br), _ptr(w.bi), _ptr(w.sp), _ptr(tile_row),
                                 _ptr(tile_rows), tiles, _ptr(hloc), _ptr(prod), w.W, w.bwp, w.blocks, _stream(u)), "rglru_gates")
    check(lib().sglk_rglru_carry(*_conv_args(src, w, u, y, conv_state, seqs, singles), _ptr(hloc), _ptr(prod), _ptr(carry),
                                 _ptr(state), _ptr(tile0), int(seq0), w.used, dtype_code(u.dtype), _stream(u)), "rglru_carry")
    check(lib().sglk_rglru_apply(_ptr(hloc), _ptr(prod), _ptr(carry), _ptr(y), _ptr(out), out.stride(0), _ptr(seqs.row_seq),
                                 _ptr(seqs.row0), _ptr(tile0), int(singles), M, w.W, w.used, dtype_code(u.dtype), _stream(u)),
          "rglru_apply")


def rglru_rows(src, u, y, w, conv_state, state, seqs, out):
    """All rows, any float type: gate weights row-major [blocks, bwp, bwp]."""
    if w.wr.dtype != u.dtype or w.wr.numel() != w.blocks * w.bwp ** 2 or state.shape[1] != w.W or state.dtype != torch.float32:
        raise SglkError("rglru_rows: weights or state do not match")
    if out.shape[0] < u.shape[0] or out.dtype != u.dtype or out.shape[1] < w.used:
        raise SglkError("rglru_rows: out does not match")
    da = torch.empty(u.shape, dtype=torch.float32, device=u.device)
    db = torch.empty_like(da)
    check(lib().sglk_rglru_rows(*_conv_args(src, w, u, y, conv_state, seqs, 0), _ptr(w.wr), _ptr(w.wi), _ptr(w.br), _ptr(w.bi),
                                _ptr(w.sp), _ptr(da), _ptr(db), _ptr(state), _ptr(out), out.stride(0), w.bwp, w.blocks,
                                dtype_code(u.dtype), _stream(u)), "rglru_rows")


# -------------------------------------------------------------------------------------------------- tied attention
@dataclasses.dataclass
class TiedWeights:
    """What tied attention adds to the products of its queries and rows (everything in the base-2 domain)."""
    bias: torch.Tensor       # [H, nb] by distance
    sink: torch.Tensor       # [H]
    heads: int
    kv_heads: int
    D: int                   # padded head size


def tied_prep(src: Source, bias, wq, factor, q, pool, rms, loc, positions, q_size, k_size, eps):
    """src [rows, q_cols + k_cols] -> q [rows, q_cols]; key rows to pool [slots, k_cols], their norms' factors to rms."""
    M, q_cols = q.shape
    k_cols = pool.shape[1]
    _src_ok(src, M, q_cols + k_cols, q.dtype, "tied_prep")
    _f32(bias, q_cols + k_cols, "tied_prep: bias")
    _f32(wq, q_cols, "tied_prep: wq")
    _f32(factor, 1, "tied_prep: factor")
    _f32(rms, pool.shape[0], "tied_prep: rms")
    _i32(loc, M, "tied_prep: loc")
    _i32(positions, M, "tied_prep: positions")
    if pool.dtype != q.dtype or pool.stride(1) != 1 or not q.is_contiguous():
        raise SglkError("tied_prep: queries and pool rows do not match")
    check(lib().sglk_tied_prep(*src.args(), _ptr(bias), _ptr(wq), _ptr(factor), _ptr(q), _ptr(pool), pool.stride(0), _ptr(rms),
                               _ptr(loc), _ptr(positions), M, q_cols, k_cols, q_size, k_size, float(eps), dtype_code(q.dtype),
                               _stream(q)), "tied_prep")


def tied_supported(D) -> bool:
    return bool(lib().sglk_tied_supported(D))


def _tied_args(q, pool, rms, req_to_token, w: TiedWeights, what):
    _need_gpu(q, pool, rms, req_to_token)
    if q.dtype != pool.dtype or not q.is_contiguous() or q.shape[1] != w.heads * w.D or pool.stride(1) != 1 or \
            pool.shape[1] < w.kv_heads * w.D or w.heads % w.kv_heads:
        raise SglkError(f"{what}: query and pool rows do not match")
    _f32(rms, pool.shape[0], f"{what}: rms")
    _f32(w.bias, w.heads, f"{what}: bias")
    _f32(w.sink, w.heads, f"{what}: sink")
    if req_to_token.dtype != torch.int32 or w.bias.shape[0] != w.heads:
        raise SglkError(f"{what}: request table or bias table do not match")
    return (_ptr(q), _ptr(pool), pool.stride(0), _ptr(rms), _ptr(req_to_token), req_to_token.stride(0), _ptr(w.bias),
            w.bias.shape[1], _ptr(w.sink), w.heads, w.kv_heads, w.D)


def _tied_out(out, q, w, what):
    if out.shape != (q.shape[0], w.heads * w.D) or out.dtype != q.dtype or out.stride(1) != 1:
        raise SglkError(f"{what}: out must be [rows, heads * D]")


def tied_decode(q, pool, rms, req_to_token, req, positions, w: TiedWeights, part=None, lse=None, out=None, out_scale=1.0):
    """q [M, H * D], every row a request's last one -> part [M, H, S, D], lse [M, H, S]; or, unsplit, finished rows out."""
    M = q.shape[0]
    if q.dtype != torch.bfloat16:
        raise SglkError("tied_decode: bf16 only")
    args = _tied_args(q, pool, rms, req_to_token, w, "tied_decode")
    _i32(req, M, "tied_decode: req")
    _i32(positions, M, "tied_decode: positions")
    S = 1
    if out is not None:
        _tied_out(out, q, w, "tied_decode")
        part = lse = None
    else:
        S = lse.shape[2]
        _f32(part, M * w.heads * S * w.D, "tied_decode: part")
        _f32(lse, M * w.heads * S, "tied_decode: lse")
    check(lib().sglk_tied_decode(*args, _ptr(req), _ptr(positions), _ptr(part), _ptr(lse), M, S, float(out_scale), _ptr(out),
                                 0 if out is None else out.stride(0), _stream(q)), "tied_decode")


def tied_merge(part, lse, w: TiedWeights, out, out_scale=1.0):
    M, H, S, D = part.shape
    _f32(part, M * H * S * D, "tied_merge: part")
    _f32(lse, M * H * S, "tied_merge: lse")
    if out.shape != (M, H * D) or out.stride(1) != 1 or (H, D) != (w.heads, w.D):
        raise SglkError("tied_merge: out must be [rows, heads * D]")
    check(lib().sglk_tied_merge(_ptr(part), _ptr(lse), _ptr(w.sink), S, float(out_scale), _ptr(out), out.stride(0), M, H, D,
                                dtype_code(out.dtype), _stream(out)), "tied_merge")


def tied_prefill(q, pool, rms, req_to_token, row0, rows, start, req, max_rows, w: TiedWeights, out, out_scale=1.0):
    """Runs of rows (row0, rows, position of the first row, request per sequence); q, out: all rows of the step."""
    n = rows.numel()
    if q.dtype != torch.bfloat16:
        raise SglkError("tied_prefill: bf16 only")
    args = _tied_args(q, pool, rms, req_to_token, w, "tied_prefill")
    _tied_out(out, q, w, "tied_prefill")
    for t in (row0, rows, start, req):
        _i32(t, n, "tied_prefill: sequence arrays")
    check(lib().sglk_tied_prefill(*args, _ptr(row0), _ptr(rows), _ptr(start), _ptr(req), n, int(max_rows), float(out_scale),
                                  _ptr(out), out.stride(0), _stream(q)), "tied_prefill")


def tied_rows(q, pool, rms, req_to_token, req, positions, w: TiedWeights, out, out_scale=1.0):
    """Every row of q by itself: any size and float type."""
    M = q.shape[0]
    args = _tied_args(q, pool, rms, req_to_token, w, "tied_rows")
    _tied_out(out, q, w, "tied_rows")
    _i32(req, M, "tied_rows: req")
    _i32(positions, M, "tied_rows: positions")
    check(lib().sglk_tied_rows(*args, _ptr(req), _ptr(positions), float(out_scale), _ptr(out), out.stride(0), M,
                               dtype_code(q.dtype), _stream(q)), "tied_rows")


# ------------------------------------------------------------------------------------------------ gated delta rule
def short_conv(src: Source, conv, u, conv_state, seqs: RowSeqs, singles, act=ACT_NONE, bias=None, conv_b=None):
    """u [rows, W] = act(convolution); conv [taps, W]; conv_state [slots, taps - 1, W]."""
    M, W = u.shape
    taps, n = conv.shape[0], seqs.rows.numel()
    _src_ok(src, M, W, u.dtype, "short_conv")
    _f32(conv, taps * W, "short_conv: conv")
    _f32(bias, W, "short_conv: bias")
    _f32(conv_b, W, "short_conv: conv_b")
    _i32(seqs.row_seq, M, "short_conv: row_seq")
    for t in (seqs.row0, seqs.rows, seqs.start, seqs.slot):
        _i32(t, n, "short_conv: sequence arrays")
    if conv.shape[1] != W or not u.is_contiguous():
        raise SglkError("short_conv: filters or rows do not match")
    if conv_state.shape[1:] != (taps - 1, W) or conv_state.dtype != u.dtype or not conv_state.is_contiguous():
        raise SglkError("short_conv: convolution state does not match")
    check(lib().sglk_short_conv(*src.args(), _ptr(bias), _ptr(conv), _ptr(conv_b), _ptr(u), _ptr(conv_state), _ptr(seqs.row_seq),
                                _ptr(seqs.row0), _ptr(seqs.rows), _ptr(seqs.start), _ptr(seqs.slot), M, W, taps, int(singles), n,
                                int(act), dtype_code(u.dtype), _stream(u)), "short_conv")


@dataclasses.dataclass
class DeltaWeights:
    """One gated delta mixer's parameters and sizes in the kernels' layout."""
    rate: torch.Tensor       # [heads] exp(A_log)
    dt: torch.Tensor         # [heads]
    norm: torch.Tensor       # [vp]
    heads: int
    kv_heads: int
    dp: int                  # padded key and value sizes, then the true ones
    vp: int
    dim: int
    vdim: int
    b_col: int               # columns of the step sizes and decays behind the gates
    a_col: int
    eps: float

    @property
    def channels(self):
        return 2 * self.kv_heads * self.dp + self.heads * self.vp


def _delta_args(u, src: Source, w: DeltaWeights, state, seqs: RowSeqs, out, out_scale, what):
    M = u.shape[0]
    _src_ok(src, M, w.a_col + w.heads, u.dtype, what)
    _f32(w.rate, w.heads, f"{what}: rate")
    _f32(w.dt, w.heads, f"{what}: dt")
    _f32(w.norm, w.vp, f"{what}: norm")
    _f32(state, 0, f"{what}: state")
    n = seqs.rows.numel()
    _i32(seqs.row_seq, M, f"{what}: row_seq")
    for t in (seqs.row0, seqs.rows, seqs.start, seqs.slot):
        _i32(t, n, f"{what}: sequence arrays")
    if u.shape[1] != w.channels or u.stride(1) != 1 or state.shape[1:] != (w.heads, w.dp, w.vp):
        raise SglkError(f"{what}: channels or state do not match")
    if out.shape != (M, w.heads * w.vp) or out.dtype != u.dtype or out.stride(1) != 1:
        raise SglkError(f"{what}: out must be [rows, heads * vp]")
    return (_ptr(u), u.stride(0), *src.args(), w.b_col, w.a_col, _ptr(w.rate), _ptr(w.dt), _ptr(w.norm), _ptr(state), _ptr(out),
            out.stride(0), _ptr(seqs.row_seq), _ptr(seqs.row0), _ptr(seqs.rows), _ptr(seqs.start), _ptr(seqs.slot), M, w.kv_heads,
            w.heads, w.dp, w.vp, w.dim, w.vdim, float(out_scale), float(w.eps))


def delta_step(u, src, w: DeltaWeights, state, seqs, out, out_scale, seq0, n_seqs):
    """Sequences seq0 .. n_seqs - 1, row after row; u, src, out: all rows of the step."""
    if n_seqs > seqs.rows.numel():
        raise SglkError("delta_step: sequence range")
    check(lib().sglk_delta_step(*_delta_args(u, src, w, state, seqs, out, out_scale, "delta_step"), int(seq0), int(n_seqs),
                                dtype_code(u.dtype), _stream(u)), "delta_step")


def delta_chunk_supported(dp, vp) -> bool:
    return bool(lib().sglk_delta_chunk_supported(dp, vp))


def delta_chunk(u, src, w: DeltaWeights, state, seqs, out, out_scale, first_row, seq0, tile_row, tile_rows, tile0):
    """Rows from first_row on (sequences from seq0 on), in tiles of 64 rows of one sequence."""
    M, tiles, n = u.shape[0], tile_row.numel(), seqs.rows.numel()
    if u.dtype != torch.bfloat16:
        raise SglkError("delta_chunk: bf16 only")
    _i32(tile_row, tiles, "delta_chunk: tile_row")
    _i32(tile_rows, tiles, "delta_chunk: tile_rows")
    _i32(tile0, n, "delta_chunk: tile0")
    size = lib().sglk_delta_chunk_workspace_bytes(tiles, w.heads)
    ws = torch.empty(size, dtype=torch.uint8, device=u.device)
    o = torch.empty(M, w.heads * w.vp, dtype=torch.float32, device=u.device)
    check(lib().sglk_delta_chunk(*_delta_args(u, src, w, state, seqs, out, out_scale, "delta_chunk"), _ptr(tile_row), _ptr(tile_rows),
                                 _ptr(tile0), tiles, _ptr(ws), size, _ptr(o), int(first_row), int(seq0), n, _stream(u)), "delta_chunk")
