"""Recurrent state of a stage's recurrent layers, one slot per session row.

A recurrent layer's state replaces its KV cache: a fixed fp32 block per session ([heads, dim, vdim], and
what else the mixer carries) instead of
pages that grow with the context.  Slots are the session manager's rows: a row that is handed out again needs no
clearing, because a sequence's first token starts from a zero state whatever the slot holds.  State cannot be
rewound: a session continues from its length or starts over.
"""
from __future__ import annotations

from typing import List, Sequence, Tuple

import torch


class RecurrentState:
    def __init__(self, shapes: Sequence[Sequence[Tuple[int, ...]]], max_sessions: int, device="cpu"):
        """``shapes``: the shapes of every recurrent layer's tensors (the state matrix [heads, dim, vdim] first)."""
        self.states: List[torch.Tensor] = []
        self._layers: List[Tuple[torch.Tensor, ...]] = []
        for lay in shapes:
            made = tuple(torch.zeros((max_sessions,) + tuple(s), dtype=torch.float32, device=device) for s in lay)
            self.states += made
            self._layers.append(made)

    def layer(self, i: int) -> Tuple[torch.Tensor, ...]:
        return self._layers[i]

    def copy_row(self, src: int, dst: int) -> None:
        for s in self.states:
            s[dst].copy_(s[src])

    @property
    def nbytes(self) -> int:
        return sum(s.numel() * 4 for s in self.states)
