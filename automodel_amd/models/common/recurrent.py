"""Recurrent mixers as modules: state space (scalar decay per head) and time
mixing (wkv, decay per channel), for packed tokens, with or without a state."""

from __future__ import annotations

from dataclasses import dataclass

import torch
import torch.nn as nn

from automodel_amd.ops.linear_scan import (
    causal_conv_silu,
    gated_group_norm,
    ssd_scan,
    token_shift,
    wkv_decode,
    wkv_scan,
)
from automodel_amd.ops.packed_step import PackedStep
from automodel_amd.serving.decode_linear import (
    DecodeLinear,
    grouped_rows,
    project,
    project_grouped,
)


@dataclass(frozen=True)
class StateSpaceSpec:
    heads: int
    vdim: int                       # channels per head
    state: int                      # state size per channel
    groups: int                     # heads share B and C in equal groups
    norm_groups: int
    conv: int                       # taps of the short convolution
    eps: float

    def __post_init__(self):
        if self.heads % self.groups or self.inner % self.norm_groups:
            raise ValueError("heads and channels divide into equal groups")

    @property
    def inner(self) -> int:
        return self.heads * self.vdim

    @property
    def conv_width(self) -> int:
        return self.inner + 2 * self.groups * self.state

    @property
    def in_width(self) -> int:
        return self.inner + self.conv_width + self.heads


class StateSpace(nn.Module):
    """From projected rows [z | x | B | C | dt] (``spec.in_width`` columns, which
    may be a slice of wider rows) to [T, width]. The gate silu(z) comes before
    the group norm."""

    def __init__(self, width: int, spec: StateSpaceSpec):
        super().__init__()
        self.spec = spec
        self.conv_weight = nn.Parameter(torch.zeros(spec.conv_width, spec.conv))
        self.conv_bias = nn.Parameter(torch.zeros(spec.conv_width))
        self.dt_bias = nn.Parameter(torch.zeros(spec.heads))
        self.A_log = nn.Parameter(torch.zeros(spec.heads))
        self.D = nn.Parameter(torch.ones(spec.heads))
        self.norm_weight = nn.Parameter(torch.ones(spec.inner))
        self.o_proj = nn.Linear(spec.inner, width, bias=False)

    def make_state(self, n_slots: int, max_len: int, device, dtype) -> dict[str, torch.Tensor]:
        s = self.spec
        return {"conv": torch.zeros(n_slots, s.conv - 1, s.conv_width, device=device, dtype=dtype),
                "ssm": torch.zeros(n_slots, s.heads, s.state, s.vdim, device=device)}

    def forward(self, proj: torch.Tensor, step: PackedStep, state=None) -> torch.Tensor:
        s = self.spec
        conv_state, ssm = (state["conv"], state["ssm"]) if state else (None, None)
        z, xbc, dt = proj.split([s.inner, s.conv_width, s.heads], dim=-1)
        xbc = causal_conv_silu(xbc, self.conv_weight, self.conv_bias, step, conv_state)
        y = ssd_scan(xbc, dt, self.dt_bias, self.A_log, self.D, s.groups, s.state, step, ssm)
        y = gated_group_norm(y, z, self.norm_weight, s.norm_groups, s.eps, gate_first=True)
        return project(self.o_proj, y)


class TimeMixing(nn.Module):
    """h [T, width] -> [T, width]. Every projection reads its own mix of the
    token and the one before; ``in_proj`` stacks r, k, v, the gate and the
    decay's down-projection, ``mu`` their mixes in this order."""

    def __init__(self, width: int, heads: int, dim: int, rank: int, eps: float):
        super().__init__()
        self.heads, self.dim, self.rank, self.eps = heads, dim, rank, eps
        n = heads * dim
        self.mu = nn.Parameter(torch.full((5, width), 0.5))
        self.in_proj = nn.Linear(width, 4 * n + rank, bias=False)
        self.decay_proj = nn.Linear(rank, n, bias=False)
        self.decay_bias = nn.Parameter(torch.full((n,), -3.0))
        self.bonus = nn.Parameter(torch.zeros(heads, dim))
        self.norm_weight = nn.Parameter(torch.ones(n))
        self.o_proj = nn.Linear(n, width, bias=False)

    def make_state(self, n_slots: int, max_len: int, device, dtype) -> dict[str, torch.Tensor]:
        return {"shift": torch.zeros(n_slots, self.mu.shape[1], device=device, dtype=dtype),
                "wkv": torch.zeros(n_slots, self.heads, self.dim, self.dim, device=device)}

    def forward(self, h: torch.Tensor, step: PackedStep, state=None) -> torch.Tensor:
        shift, wkv = (state["shift"], state["wkv"]) if state else (None, None)
        sizes = [self.heads * self.dim] * 4 + [self.rank]
        xs = token_shift(h, self.mu, step, shift)
        if not step.prompt:
            if type(self.decay_proj) not in (nn.Linear, DecodeLinear):
                # the decode kernel multiplies by the raw weight
                raise RuntimeError("merge adapters on decay_proj before decoding with a cache")
            proj = grouped_rows(self.in_proj, xs, sizes)
            if proj is None:
                proj = torch.cat(project_grouped(self.in_proj, xs, sizes), dim=-1)
            o = wkv_decode(proj, self.decay_proj.weight, self.decay_bias, self.bonus,
                           self.norm_weight, self.eps, step, wkv)
            return project(self.o_proj, o)
        r, k, v, g, low = project_grouped(self.in_proj, xs, sizes)
        low = project(self.decay_proj, torch.tanh(low), out_f32=True)
        o = wkv_scan(r, k, v, low, self.decay_bias, self.bonus, step, wkv)
        o = gated_group_norm(o, g, self.norm_weight, self.heads, self.eps, gate_first=False)
        return project(self.o_proj, o)
