"""Hyper-connections: several float32 residual streams around the sublayers.

A sublayer reads a weighted sum of the streams, normed; afterwards every stream
becomes a mix of all the old ones plus its share of the sublayer's output. The
HIP kernels (csrc/hyper.hip) do an update, the next input and its norm in one
pass over the streams; the torch expressions are the differentiable form and
the CPU reference.
"""

from __future__ import annotations

from typing import NamedTuple

import torch

from automodel_amd.ops._backend import hip_ops
from automodel_amd.ops.residual_norm import rms_f32, use_hip


class NormedPair(NamedTuple):
    """A sublayer's output as two branches: (rms(a) * wa + rms(b) * wb) / 2."""

    a: torch.Tensor
    b: torch.Tensor
    wa: torch.Tensor
    wb: torch.Tensor

    def rows(self, index: torch.Tensor) -> "NormedPair":
        return self._replace(a=self.a[index], b=self.b[index])


def _read(x, w_in, w_norm, eps):
    u = x.sum(1) if w_in is None else torch.einsum("s,tsw->tw", w_in.float(), x)
    return rms_f32(u, w_norm, eps).to(w_norm.dtype)


def hyper_embed(ids: torch.Tensor, table: torch.Tensor, scale: float, w_in: torch.Tensor,
                w_norm: torch.Tensor, eps: float) -> tuple[torch.Tensor, torch.Tensor]:
    """ids [T] -> (streams [T, S, W] float32, all the scaled embedding; the first
    sublayer's input [T, W])."""
    if use_hip(table):
        return hip_ops().hyper_embed(ids.contiguous(), table, scale, w_in, w_norm, eps)
    x = torch.nn.functional.embedding(ids, table).float() * scale
    x = x[:, None].expand(-1, w_in.numel(), -1)
    return x, _read(x, w_in, w_norm, eps)


def hyper_step(x: torch.Tensor, y: torch.Tensor | NormedPair, w_mix: torch.Tensor,
               w_out: torch.Tensor, w_in: torch.Tensor | None, w_norm: torch.Tensor,
               eps: float, keep: bool = True) -> tuple[torch.Tensor, torch.Tensor]:
    """Streams x [T, S, W] after a sublayer's output y [T, W], and the next
    sublayer's input: x_t <- sum_s mix[s, t] x_s + out[t] y, then
    rms(sum_t in[t] x_t) * w_norm (``w_in`` None: the plain sum).

    The HIP path updates ``x`` in place, or leaves it as it was if the new
    streams are of no further use (``keep`` False).
    """
    if use_hip(x):
        a, b, wa, wb = y if isinstance(y, NormedPair) else (y, None, None, None)
        return x, hip_ops().hyper_step(x, a, b, wa, wb, w_mix, w_out, w_in, w_norm, eps, keep)
    if isinstance(y, NormedPair):
        y = 0.5 * (rms_f32(y.a, y.wa, eps) + rms_f32(y.b, y.wb, eps))
    x = torch.einsum("st,nsw->ntw", w_mix.float(), x) \
        + w_out.float()[None, :, None] * y.float()[:, None]
    return x, _read(x, w_in, w_norm, eps)


def clamped_glu(gu: torch.Tensor, limit: float, alpha: float = 1.702) -> torch.Tensor:
    """Rows [g | u] -> g' sigmoid(alpha g') (u' + 1), g' = min(g, limit),
    u' = u clamped to [-limit, limit]."""
    if use_hip(gu):
        return hip_ops().clamped_glu(gu, limit, alpha)
    g, u = gu.float().chunk(2, dim=-1)
    g, u = g.clamp(max=limit), u.clamp(-limit, limit)
    return (g * torch.sigmoid(alpha * g) * (u + 1)).to(gu.dtype)
