"""Decode-path linear: route skinny (rows<=16) matmuls to the HIP GEMV.

Reference behavior: serving engines (which the reference defers to for
deployment) special-case decode GEMVs; here the kernel is in-tree
(ops/csrc/gemv.hip — wave-per-row bf16 row streaming) and DecodeLinear
swaps in for inference. Training paths are untouched: the GEMV route only
fires under no_grad with a 3-D [B, 1, K] or 2-D [<=16, K] bf16 input on
GPU; everything else falls through to F.linear (hipBLASLt)."""

from __future__ import annotations

import torch
import torch.nn as nn
import torch.nn.functional as F

_PAD_TO = {5: 8, 6: 8, 7: 8, 9: 16, 10: 16, 11: 16, 12: 16, 13: 16, 14: 16, 15: 16}


def gemv_bf16(x2d: torch.Tensor, w: torch.Tensor, bias: torch.Tensor | None = None,
              relu2: bool = False, out_f32: bool = False) -> torch.Tensor:
    """y = x2d @ w.T via the HIP kernel; pads odd batch sizes to a
    compiled template instance. Epilogues: max(y, 0)^2, f32 output."""
    from automodel_amd.ops._backend import hip_ops

    B = x2d.shape[0]
    tgt = _PAD_TO.get(B, B)
    if tgt != B:
        x2d = F.pad(x2d, (0, 0, 0, tgt - B))
    y = hip_ops().gemv_bf16(x2d, w, bias, relu2, out_f32)
    return y[:B] if tgt != B else y


def _gemv_eligible(x: torch.Tensor, w: torch.Tensor) -> bool:
    if torch.is_grad_enabled() or not x.is_cuda:
        return False
    if x.dtype != torch.bfloat16 or w.dtype != torch.bfloat16:
        return False
    rows = x.numel() // x.shape[-1]
    # measured on MI355X (profiles/README.md): the wave-per-row GEMV beats
    # hipBLASLt up to ~4 rows; above that the library's m-tiled path wins
    return rows <= 4 and x.shape[-1] % 512 == 0


def project(lin: nn.Module, x: torch.Tensor, relu2: bool = False,
            out_f32: bool = False) -> torch.Tensor:
    """``lin(x)`` for packed rows x [T, K], optionally followed by max(y, 0)^2
    and optionally in float32 (a residual input or logits must not be rounded
    to bf16 on the way out of the accumulator).

    Inference on the GPU: up to 4 bf16 rows take the GEMV, up to 64 the skinny
    MFMA GEMM, both with fused epilogues; more take the library GEMM. Wrapped layers (adapters) and autograd take the
    module itself."""
    from automodel_amd.ops import residual_norm as rn

    if type(lin) not in (nn.Linear, DecodeLinear) or lin.bias is not None or not rn.use_hip(x):
        y = lin(x)
        y = rn.relu2(y) if relu2 else y
        return y.float() if out_f32 else y
    w = lin.weight
    if x.shape[0] == 0:
        return x.new_empty(0, w.shape[0], dtype=torch.float32 if out_f32 else x.dtype)
    if x.dtype == torch.bfloat16 and x.shape[0] <= 64 and x.shape[1] % 8 == 0:
        if x.shape[0] <= 4:
            return gemv_bf16(x, w, None, relu2, out_f32)
        from automodel_amd.ops._backend import hip_ops

        return hip_ops().gemm_skinny_bf16(x, w, relu2, out_f32)
    if out_f32 and x.dtype == torch.bfloat16:
        y = torch.mm(x, w.t(), out_dtype=torch.float32)
    else:
        y = F.linear(x, w)
    return rn.relu2(y) if relu2 else y


def project_grouped(lin: nn.Module, xs: torch.Tensor, sizes: list[int]) -> list[torch.Tensor]:
    """Several inputs through one stacked projection: the weight's rows, split by
    ``sizes``, apply to xs[i] each, xs [n, T, K]. -> the n outputs [T, sizes[i]].

    Up to 64 bf16 rows on the GPU are one launch (the outputs are slices of one
    [T, N] tensor then, see ``grouped_rows``); more take a GEMM each. A wrapped
    layer (adapters) sees every input as a whole."""
    y = grouped_rows(lin, xs, sizes)
    if y is not None:
        return list(y.split(sizes, dim=1))
    if type(lin) not in (nn.Linear, DecodeLinear):
        return [lin(x).split(sizes, dim=-1)[i] for i, x in enumerate(xs)]
    return [F.linear(x, w) for x, w in zip(xs, lin.weight.split(sizes))]


def grouped_rows(lin: nn.Module, xs: torch.Tensor, sizes: list[int]) -> torch.Tensor | None:
    """The one-launch form of ``project_grouped``, [T, N], if it applies: equal
    sizes, of which the last may be smaller."""
    from automodel_amd.ops import residual_norm as rn

    n, T, K = xs.shape
    group = sizes[0]
    if not (rn.use_hip(xs) and xs.dtype == torch.bfloat16 and 1 <= T <= 64 and K % 8 == 0
            and type(lin) in (nn.Linear, DecodeLinear) and lin.bias is None
            and sizes[:-1] == [group] * (n - 1) and 1 <= sizes[-1] <= group
            and group % (2 if T <= 4 else 16) == 0):
        return None
    w = lin.weight
    from automodel_amd.ops._backend import hip_ops

    x = xs.reshape(n * T, K)
    if T <= 4:
        return hip_ops().gemv_bf16(x, w, None, False, False, group)
    return hip_ops().gemm_skinny_bf16(x, w, False, False, group)


class DecodeLinear(nn.Linear):
    """nn.Linear that runs decode-shaped inputs on the in-tree GEMV."""

    @classmethod
    def from_linear(cls, lin: nn.Linear) -> "DecodeLinear":
        m = cls(lin.in_features, lin.out_features, bias=lin.bias is not None,
                device=lin.weight.device, dtype=lin.weight.dtype)
        with torch.no_grad():
            m.weight.copy_(lin.weight)
            if lin.bias is not None:
                m.bias.copy_(lin.bias)
        return m

    def forward(self, x: torch.Tensor) -> torch.Tensor:
        if _gemv_eligible(x, self.weight):
            lead = x.shape[:-1]
            y = gemv_bf16(x.reshape(-1, x.shape[-1]), self.weight, self.bias)
            return y.reshape(*lead, self.out_features)
        return F.linear(x, self.weight, self.bias)


def swap_linears_for_decode(model: nn.Module) -> int:
    """Swap every nn.Linear for DecodeLinear (weights shared by copy).
    Returns count. Call on an inference model before generate_graphed."""
    n = 0
    for name, parent in list(model.named_modules()):
        for child_name, child in list(parent.named_children()):
            if type(child) is nn.Linear:
                setattr(parent, child_name, DecodeLinear.from_linear(child))
                n += 1
    return n
