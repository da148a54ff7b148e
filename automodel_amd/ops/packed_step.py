"""Where the packed tokens of one step belong."""

from __future__ import annotations

from dataclasses import dataclass, field

import numpy as np
import torch


@dataclass
class PackedStep:
    """Where the packed tokens of one step belong.

    ``positions``/``slots`` are int32 ``[T]``. A prompt step also carries the
    sequence bounds; in a decode step every token attends the cached prefix of
    its slot up to its own position.
    """

    positions: torch.Tensor
    slots: torch.Tensor | None = None
    prompt: bool = True
    cu_seqlens: torch.Tensor | None = None      # int32 [n + 1], prompt steps
    doc_start: torch.Tensor | None = None       # int32 [rows padded to 256]
    seq_end: torch.Tensor | None = None         # int32 [T], end of the token's sequence
    logit_rows: torch.Tensor | None = None      # rows whose logits are wanted
    n_seqs: int = 1
    max_len: int = 1                            # longest sequence of a prompt step
    _chunk_start: dict = field(default_factory=dict, repr=False)

    @classmethod
    def for_prompts(cls, lengths: list[int], device, slots: list[int] | None = None,
                    logit_rows: list[int] | None = None) -> "PackedStep":
        lens = np.asarray(lengths, dtype=np.int32)
        cu = np.concatenate([[0], np.cumsum(lens)]).astype(np.int32)
        total = int(cu[-1])
        start = np.repeat(cu[:-1], lens)
        parts = {
            "positions": np.arange(total, dtype=np.int32) - start,
            # padding rows form a document of their own after the last one
            "doc_start": np.concatenate([start, np.full((-total) % 256, total, np.int32)]),
            "cu_seqlens": cu,
            "seq_end": np.repeat(cu[1:], lens),
            "slots": None if slots is None else np.repeat(np.asarray(slots, np.int32), lens),
            "logit_rows": None if logit_rows is None else np.asarray(logit_rows, np.int32),
        }
        parts = {k: v for k, v in parts.items() if v is not None}
        flat = torch.from_numpy(np.concatenate(list(parts.values())).astype(np.int32)).to(device)
        views = dict(zip(parts, flat.split([len(v) for v in parts.values()])))
        return cls(**views, n_seqs=len(lengths), max_len=int(lens.max()))

    def chunk_start(self, chunk: int) -> torch.Tensor:
        """``doc_start`` with every sequence cut into chunks of ``chunk`` tokens,
        counted from its first: the first row that a prompt token's chunk has."""
        if self.max_len <= chunk:
            return self.doc_start
        if chunk not in self._chunk_start:
            start = self.doc_start.clone()
            n = self.positions.numel()
            start[:n] += self.positions - self.positions % chunk
            self._chunk_start[chunk] = start
        return self._chunk_start[chunk]
