"""Latent attention as a module, for packed tokens, with or without a cache."""

from __future__ import annotations

import torch
import torch.nn as nn

from automodel_amd.ops.latent_attention import (
    LatentAttentionSpec,
    PackedStep,
    latent_attention_decode,
    latent_attention_prompt,
)
from automodel_amd.ops.rms_norm import RMSNorm
from automodel_amd.serving.decode_linear import project


class LatentAttention(nn.Module):
    """h [T, width] -> [T, width].

    ``q_kv_a_proj`` stacks the query projection and the latent/rotated-key
    down-projection (one GEMM per layer); ``kv_b_proj`` stacks the key and the
    value up-projection.
    """

    def __init__(self, width: int, spec: LatentAttentionSpec, norm_backend: str = "hip"):
        super().__init__()
        self.spec = spec
        self.q_kv_a_proj = nn.Linear(width, spec.q_width + spec.kv_rank + spec.rot_dim, bias=False)
        self.kv_a_layernorm = RMSNorm(spec.kv_rank, spec.eps, norm_backend)
        self.kv_b_proj = nn.Linear(spec.kv_rank, spec.heads * (spec.dim + spec.vdim), bias=False)
        self.o_proj = nn.Linear(spec.heads * spec.vdim, width, bias=False)

    def forward(self, h: torch.Tensor, step: PackedStep, rope: tuple[torch.Tensor, torch.Tensor],
                cache: torch.Tensor | None = None) -> torch.Tensor:
        if type(self.kv_b_proj) is not nn.Linear and cache is not None:
            # the cached path multiplies by the raw weight (absorbed form)
            raise RuntimeError("merge adapters on kv_b_proj before decoding with a cache")
        qkv = project(self.q_kv_a_proj, h)
        attend = latent_attention_prompt if step.prompt else latent_attention_decode
        o = attend(qkv, self.kv_a_layernorm.weight, self.kv_b_proj.weight, self.spec, rope,
                   step, cache)
        return project(self.o_proj, o)
