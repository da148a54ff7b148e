"""Grouped-head attention (chunks, sink, partial rotation) as a module."""

from __future__ import annotations

import torch
import torch.nn as nn

from automodel_amd.ops.grouped_attention import (
    GroupedAttentionSpec,
    grouped_attention_decode,
    grouped_attention_prompt,
)
from automodel_amd.ops.packed_step import PackedStep
from automodel_amd.serving.decode_linear import project


class GroupedAttention(nn.Module):
    """From projected rows that begin with [q | k | v] (``spec.in_width``
    columns; the projection belongs to the caller, who may stack more onto it)
    to [T, width]."""

    def __init__(self, width: int, spec: GroupedAttentionSpec, sink: bool = False):
        super().__init__()
        self.spec = spec
        self.sink = nn.Parameter(torch.zeros(spec.heads)) if sink else None
        self.o_proj = nn.Linear(spec.heads * spec.vdim, width, bias=False)

    def make_state(self, n_slots: int, max_len: int, device, dtype) -> dict[str, torch.Tensor]:
        return self.spec.make_state(n_slots, max_len, device, dtype)

    def forward(self, proj: torch.Tensor, step: PackedStep, rope, state=None) -> torch.Tensor:
        attend = grouped_attention_prompt if step.prompt else grouped_attention_decode
        return project(self.o_proj, attend(proj, self.sink, self.spec, rope, step, state))
