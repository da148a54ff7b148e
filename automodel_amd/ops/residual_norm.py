"""RMS norms, scaled adds and casts around a 32-bit residual stream.

The HIP kernels (csrc/residual_norm.hip) run on the GPU when no gradient is
recorded; the torch expressions below them are the differentiable form (used
for training) and the CPU reference. The residual is always float32; weights
and sublayer inputs/outputs keep the model's dtype.
"""

from __future__ import annotations

import torch

from automodel_amd.ops._backend import hip_ops


def use_hip(x: torch.Tensor) -> bool:
    return x.is_cuda and not torch.is_grad_enabled()


def rms_f32(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    """x / sqrt(mean(x^2) + eps) * w, computed and returned in float32."""
    x = x.float()
    return x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps) * w.float()


def embed_rms_norm(ids: torch.Tensor, table: torch.Tensor, w: torch.Tensor,
                   eps: float) -> torch.Tensor:
    """ids [T] -> normed embedding rows [T, W], float32."""
    if use_hip(table):
        return hip_ops().embed_rms_norm(ids.contiguous(), table, w, eps)
    return rms_f32(torch.nn.functional.embedding(ids, table), w, eps)


def residual_rms_norm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    """Sublayer input from the residual: rms(x) * w in the weight's dtype."""
    if use_hip(x):
        return hip_ops().residual_rms_norm(x, w, eps)
    return rms_f32(x, w, eps).to(w.dtype)


def residual_add_norm(
    x: torch.Tensor, y: torch.Tensor, w_post: torch.Tensor, mult: float, eps: float,
    w_next: torch.Tensor | None = None,
) -> tuple[torch.Tensor, torch.Tensor | None]:
    """(x + mult * rms(y) * w_post, the next sublayer's normed input or None).

    The HIP path updates ``x`` in place and reads each row once for both norms.
    """
    if use_hip(x):
        h = hip_ops().residual_add_norm(x, y, w_post, mult, eps, w_next, eps)
        return x, (h if w_next is not None else None)
    x = x + mult * rms_f32(y, w_post, eps)
    return x, (rms_f32(x, w_next, eps).to(w_next.dtype) if w_next is not None else None)


def concat_cast(a: torch.Tensor, b: torch.Tensor, dtype: torch.dtype) -> torch.Tensor:
    """[a ; b] along the last dim, cast from float32 to ``dtype``."""
    if use_hip(a):
        return hip_ops().concat_cast(a, b, dtype == torch.bfloat16)
    return torch.cat([a, b], dim=-1).to(dtype)


def relu2(x: torch.Tensor) -> torch.Tensor:
    """max(x, 0)^2; the HIP path overwrites ``x``."""
    if use_hip(x):
        return hip_ops().relu2_(x)
    return torch.relu(x).square()
