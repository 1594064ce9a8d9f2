"""One product for everything that reads a mixer's rows: matrices stacked along their rows, every segment starting at a multiple
of 8 rows (zero rows between), so that slices of the product's result stay aligned to 16 bytes."""
from __future__ import annotations

from typing import List, Sequence, Tuple

import torch


def stacked_rows(segments: Sequence[torch.Tensor]) -> Tuple[torch.Tensor, List[int]]:
    """-> the stacked matrix (its number of rows a multiple of 8) and the row that every segment starts at."""
    rows, offsets, at = [], [], 0
    for seg in segments:
        offsets.append(at)
        rows.append(seg)
        pad = -seg.shape[0] % 8
        if pad:
            rows.append(torch.zeros((pad, seg.shape[1]), dtype=seg.dtype, device=seg.device))
        at += seg.shape[0] + pad
    return torch.cat(rows, dim=0).contiguous(), offsets
