"""What a decoder keeps of one sequence: preallocated key/value caches, latent rows and recurrent states, per layer run."""
from __future__ import annotations

from typing import List, Tuple

import torch


class SequenceCache:
    """Key/value caches and latent rows are written at absolute positions and need no clearing; recurrent states start at zero and only move
    forward, so a model with states continues where the last call ended (``begin``) or starts over at position 0."""

    def __init__(self, device):
        self.device = torch.device(device)
        self.length = 0                              # positions held
        self.kv: List[Tuple[torch.Tensor, torch.Tensor]] = []
        self.rows: List[torch.Tensor] = []
        self.states: List[torch.Tensor] = []

    def add_kv(self, heads: int, ctx: int, k_dim: int, v_dim: int) -> Tuple[torch.Tensor, torch.Tensor]:
        f32 = dict(dtype=torch.float32, device=self.device)
        pair = (torch.zeros((heads, ctx, k_dim), **f32), torch.zeros((heads, ctx, v_dim), **f32))
        self.kv.append(pair)
        return pair

    def add_rows(self, ctx: int, width: int, dtype: torch.dtype) -> torch.Tensor:
        """One row per position that all heads share (latents); layers may attend to another layer's rows."""
        t = torch.zeros((ctx, width), dtype=dtype, device=self.device)
        self.rows.append(t)
        return t

    def add_state(self, *shape: int) -> torch.Tensor:
        s = torch.zeros(shape, dtype=torch.float32, device=self.device)
        self.states.append(s)
        return s

    def reset(self) -> None:
        """Give the sequence back: the next one starts at position 0 from zero states."""
        self.length = 0
        for s in self.states:
            s.zero_()

    def begin(self, pos: int) -> None:
        """A call that starts at position ``pos``."""
        if pos == 0 and self.length:
            self.reset()
        if self.states and pos != self.length:
            raise ValueError(f"position {pos} does not continue a sequence of {self.length} tokens (recurrent states cannot move back)")

    def nbytes(self) -> int:
        return sum(t.numel() * t.element_size() for t in [x for p in self.kv for x in p] + self.rows + self.states)
