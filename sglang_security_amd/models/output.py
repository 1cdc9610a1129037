"""The output matrix of checkpoint-loaded decoders."""
from __future__ import annotations

from typing import Optional

import torch

from .. import ops_hybrid as hops

LOGIT_ROWS = 64   # rows of the output product at a time: its split sums are vocab-wide


def output_logits(head, h: torch.Tensor, rows: int, vocab: int, cap: Optional[float] = None) -> torch.Tensor:
    """fp32 logits [rows, vocab] of the first rows of h; cap: cap * tanh(logit / cap)."""
    logits = torch.empty(rows, vocab, dtype=torch.float32, device=h.device)
    for i in range(0, rows, LOGIT_ROWS):
        out = logits[i: i + LOGIT_ROWS]
        hops.capped_logits(head.source(h[i: i + out.shape[0]]), out, cap, h.dtype)
    return logits
