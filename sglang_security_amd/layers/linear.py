"""Unquantised linear layers padded for the matrix kernels."""
from __future__ import annotations

import torch

from .. import ops
from ..ops_hybrid import Source

LIBRARY_MIN_ROWS = 129   # more rows than this read the weights from the row-major copy through the library product


def pad(n: int, to: int) -> int:
    return (n + to - 1) // to * to


def padded(t: torch.Tensor, *shape: int) -> torch.Tensor:
    """t in the leading corner of a zero tensor of the given shape."""
    if tuple(t.shape) == tuple(shape):
        return t.contiguous()
    out = t.new_zeros(shape)
    out[tuple(slice(0, n) for n in t.shape)] = t
    return out


class Linear:
    """y = x W^T for W [N, K] given with N and K already padded (N to 16, K to 128; zeros in the padding).

    bf16: up to LIBRARY_MIN_ROWS - 1 rows stream the operand-order copy (split sums left to the consumer), larger
    batches multiply by the row-major copy through the library.  fp32: the library in full precision."""

    def __init__(self, weight: torch.Tensor):
        self.N, self.K = weight.shape
        if self.N % 16 or self.K % 128:
            raise ValueError(f"linear weight [{self.N}, {self.K}] is not padded")
        self.weight = weight.contiguous()
        self.bf16 = weight.dtype == torch.bfloat16
        self.packed = ops.dense_repack(self.weight) if self.bf16 else None

    def bytes(self) -> int:
        return self.weight.numel() * self.weight.element_size()

    def source(self, x: torch.Tensor) -> Source:
        """The product in the form the consumer kernels take."""
        M = x.shape[0]
        if not self.bf16:
            return Source(torch.matmul(x, self.weight.t()).unsqueeze(0), True)
        if M >= LIBRARY_MIN_ROWS:
            return Source(torch.matmul(x, self.weight.t()), False)
        splits = ops.dense_gemm_partial_splits(M, self.N, self.K)
        p = torch.empty(splits, M, self.N, dtype=torch.float32, device=x.device)
        ops.dense_gemm_packed_partial(x, self.packed, p)
        return Source(p, True)

    def rows(self, x: torch.Tensor) -> torch.Tensor:
        """Finished rows of the activation type."""
        M = x.shape[0]
        if not self.bf16 or M >= LIBRARY_MIN_ROWS:
            return torch.matmul(x, self.weight.t())
        out = torch.empty(M, self.N, dtype=x.dtype, device=x.device)
        splits = ops.dense_gemm_partial_splits(M, self.N, self.K)
        ws = torch.empty(splits * M * self.N, dtype=torch.float32, device=x.device) if splits > 1 else None
        return ops.dense_gemm_packed_ws(x, self.packed, None, out, ws)


def vector(t: torch.Tensor, n: int) -> torch.Tensor:
    """fp32, zero-padded to n elements."""
    return padded(t.reshape(-1).float(), n)
