"""The description of one step's batch, on the host and on the device."""
from dataclasses import dataclass, field
from typing import NamedTuple

import numpy as np
import torch


class StepEntry(NamedTuple):
    """A request's next tokens and the places among them whose logits are wanted.  (A named tuple: a serving loop
    makes one per request and step, and a frozen dataclass costs several times as much to construct.)"""
    request: object
    tokens: tuple
    want: tuple = ()


@dataclass
class StepContext:
    """What parts see of a step.  Device tensors are int32.

    Rows are the step's tokens, packed request after request in the order of ``requests``: the step function puts
    the requests that bring several tokens first (``tile_seqs`` of them) and keeps the caller's order otherwise;
    ``cu_seqlens[s] .. cu_seqlens[s + 1]`` are the rows of sequence s.  ``logit_rows`` follow the caller's order.
    """
    n_tokens: int
    n_seqs: int
    n_logit_rows: int
    token_ids: torch.Tensor        # [N]
    positions: torch.Tensor        # [N] absolute position of each row
    row_seq: torch.Tensor          # [N] sequence index of each row
    cu_seqlens: torch.Tensor       # [S + 1]
    seq_starts: torch.Tensor       # [S] position of each sequence's first row (cached length before the step)
    seq_slots: torch.Tensor        # [S] state slot of each sequence's request
    logit_rows: torch.Tensor       # [M] rows whose logits are wanted
    single_rows: torch.Tensor      # rows that are alone in their sequence; None if every row is (max_query == 1)
    max_query: int                 # most rows of one sequence
    max_context: int               # largest position + 1
    host_cu_seqlens: list = field(default_factory=list)
    host_starts: list = field(default_factory=list)
    host_slots: list = field(default_factory=list)
    requests: list = field(default_factory=list)
    previous_tokens: torch.Tensor = None   # [N] the token before each row's in its sequence (-1: none), for embeddings
                                           # that ask for it (``needs_previous_tokens``)
    tile_seqs: int = None          # sequences 0 .. tile_seqs - 1 are those of two or more rows; None: any may be


class StepPieces:
    """The integer arrays that describe a step, by name, and where each lies once they are laid end to end into
    the one int32 array that goes to the device.  Names: ``tokens``, ``positions``, ``row_seq``, ``cu_seqlens``,
    ``starts``, ``slots``, ``logit_rows``, ``single_rows``, ``previous`` (if the embedding asks for it), and per page group g ``tables<g>`` (the block tables,
    row-major) and ``token_slots<g>`` (the cache slot of every new token)."""

    def __init__(self):
        self.names, self.arrays = [], []

    def add(self, name, array):
        if name in self.names:
            raise ValueError(f'piece {name!r} twice')
        self.names.append(name)
        self.arrays.append(np.asarray(array))

    def sizes(self):
        return [len(a) for a in self.arrays]

    def spans(self):
        """name -> (first, one past the last) index in the flat array."""
        ends = np.cumsum([0] + self.sizes()).tolist()
        return {name: (ends[i], ends[i + 1]) for i, name in enumerate(self.names)}

    def flat(self):
        return np.concatenate(self.arrays).astype(np.int32)
