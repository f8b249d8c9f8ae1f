"""What a sequence keeps between steps in the layers of mixers.py.

`LatentCache` holds one row per position that all heads of a latent attention share.
`ChunkRing` holds the keys and values of the chunk a sequence is in: position p in
row p % chunk, so a decode step's visible keys are the first p % chunk + 1 rows and
memory does not grow past one chunk.  `RecurrentState` holds a recurrence's fp32
state and the last inputs of its short convolution.  Both are filled by the kernels
(csrc/latent.hip, csrc/chunk_attend.hip, csrc/recurrence.hip); a portion at position 0 starts them
anew, so a slot can be used again without being cleared.
"""
from __future__ import annotations

from typing import List

import torch
from torch import Tensor


class ChunkRing:
    def __init__(self, batch: int, max_seq_length: int, kv_heads: int, dim: int, chunk: int, dtype, device):
        rows = min(chunk, max_seq_length)
        self.chunk = chunk
        self.k = torch.zeros(batch, kv_heads, rows, dim, dtype=dtype, device=device)
        self.v = torch.zeros_like(self.k)
        self.len = torch.zeros(batch, dtype=torch.int32, device=device)    # visible rows of the last decode step

    def tensors(self) -> List[Tensor]:
        return [self.k, self.v, self.len]

    def overwritten_by_a_step(self) -> List[Tensor]:
        """Tensors whose old contents a decode step needs again to be repeated: none (a step
        writes its own row and reads it back)."""
        return []


class LatentCache:
    """Row p: the normed latent of position p, zeros up to a multiple of 8, the rotated key part,
    zeros up to a multiple of 8."""

    def __init__(self, batch: int, max_seq_length: int, rank: int, rot: int, dtype, device):
        self.rank, self.rot = rank, rot
        self.rot_at = (rank + 7) // 8 * 8
        self.width = self.rot_at + (rot + 7) // 8 * 8
        self.rows = torch.zeros(batch, max_seq_length, self.width, dtype=dtype, device=device)

    def tensors(self) -> List[Tensor]:
        return [self.rows]

    def overwritten_by_a_step(self) -> List[Tensor]:
        """None: a step writes its own row and reads it back."""
        return []


class RecurrentState:
    def __init__(self, batch: int, heads: int, dim: int, vdim: int, conv_inputs: int, conv_channels: int, dtype, device):
        self.s = torch.zeros(batch, heads, dim, vdim, dtype=torch.float32, device=device)
        # two halves, taken in turn by the parity of the position: heads that share q / k
        # channels can all read the old inputs while one of them stores the new ones
        self.conv = torch.zeros(2, batch, max(conv_inputs, 0), conv_channels, dtype=dtype, device=device)

    def tensors(self) -> List[Tensor]:
        return [self.s, self.conv]

    def overwritten_by_a_step(self) -> List[Tensor]:
        return [self.s, self.conv]
