"""Linear recurrences with a matrix state per head, over packed prompts and one
token at a time: the state-space recurrence with a scalar decay per head, and
the wkv recurrence with a decay per key channel and a bonus for the current
token; with the short convolution, the token shift and the gated group norm
around them.

The HIP kernels (csrc/linear_scan.hip) walk prompts in blocks of 16 tokens on
the f32 matrix cores. States are float32. The torch expressions run token by
token; they serve autograd and CPU tests.
"""

from __future__ import annotations

import torch
import torch.nn.functional as F

from automodel_amd.ops._backend import hip_ops
from automodel_amd.ops.packed_step import PackedStep
from automodel_amd.ops.residual_norm import use_hip


def _slots(step: PackedStep, state) -> torch.Tensor | None:
    return step.slots if state is not None else None


def _seq_bounds(step: PackedStep) -> list[tuple[int, int, int | None]]:
    """(begin, end, slot) per sequence of a prompt step."""
    cu = step.cu_seqlens.tolist()
    return [(a, b, None if step.slots is None else int(step.slots[a]))
            for a, b in zip(cu, cu[1:])]


def causal_conv_silu(x: torch.Tensor, w: torch.Tensor, bias: torch.Tensor, step: PackedStep,
                     state: torch.Tensor | None) -> torch.Tensor:
    """x [T, C] (rows may be strided) -> silu of the causal convolution per
    channel, w [C, taps] (last: the current token). ``state`` [slots, taps - 1, C]
    keeps the last inputs, row = position modulo (taps - 1)."""
    if use_hip(x):
        return hip_ops().causal_conv_silu(x, w, bias, step.positions, _slots(step, state),
                                          step.seq_end if step.prompt else None, state)
    taps = w.shape[1]
    wf = w.float()
    if step.prompt:
        out = []
        for a, b, slot in _seq_bounds(step):
            xs = x[a:b].float()
            xs = F.pad(xs, (0, 0, taps - 1, 0))
            out.append(sum(xs[j:j + b - a] * wf[:, j] for j in range(taps)) + bias.float())
            if state is not None:
                for t in range(max(a, b - taps + 1), b):
                    state[slot, (t - a) % (taps - 1)] = x[t]
        return F.silu(torch.cat(out)).to(x.dtype)
    out = bias.float() + x.float() * wf[:, -1]
    for r, (p, slot) in enumerate(zip(step.positions.tolist(), step.slots.tolist())):
        for back in range(1, min(p, taps - 1) + 1):
            out[r] += state[slot, (p - back) % (taps - 1)].float() * wf[:, taps - 1 - back]
        if taps > 1:
            state[slot, p % (taps - 1)] = x[r]
    return F.silu(out).to(x.dtype)


def token_shift(h: torch.Tensor, mu: torch.Tensor, step: PackedStep,
                state: torch.Tensor | None) -> torch.Tensor:
    """h [T, W], mu [n, W] -> [n, T, W]: h + (h' - h) * mu, h' the token before
    (zeros for the first). ``state`` [slots, W] keeps the last token's h."""
    if use_hip(h):
        return hip_ops().token_shift(h, mu, step.positions, _slots(step, state),
                                     step.seq_end if step.prompt else None, state)
    hf = h.float()
    if step.prompt:
        before = torch.cat([torch.zeros_like(hf[:1]), hf[:-1]])
    else:
        before = state[step.slots.long()].float()
    before = before * (step.positions > 0)[:, None]
    if state is not None:
        if step.prompt:
            ends = step.cu_seqlens[1:].long() - 1
            state[step.slots[ends].long()] = h[ends].detach()
        else:
            state[step.slots.long()] = h
    return (hf + (before - hf) * mu.float()[:, None]).to(h.dtype)


def gated_group_norm(y: torch.Tensor, z: torch.Tensor, w: torch.Tensor, groups: int,
                     eps: float, gate_first: bool) -> torch.Tensor:
    """RMS norm of y [T, I] in equal parts, times w and silu(z); ``gate_first``
    norms y * silu(z) instead of y."""
    if use_hip(y):
        return hip_ops().gated_group_norm(y, z, w, groups, eps, gate_first)
    a, gate = y.float(), F.silu(z.float())
    if gate_first:
        a = a * gate
    a = a.view(a.shape[0], groups, -1)
    a = (a / torch.sqrt(a.pow(2).mean(-1, keepdim=True) + eps)).view(y.shape) * w.float()
    return (a if gate_first else a * gate).to(y.dtype)


def _run(step: PackedStep, n_tok: int, fn, state) -> torch.Tensor:
    """``fn(begin, end, S or None) -> (outputs, S)`` per sequence, the final
    state kept in its slot."""
    if step.prompt:
        spans = _seq_bounds(step)
    else:
        spans = [(r, r + 1, s) for r, s in enumerate(step.slots.tolist())]
    out = []
    for a, b, slot in spans:
        o, S = fn(a, b, None if step.prompt else state[slot].clone())
        out.extend(o)
        if state is not None:
            state[slot] = S.detach()
    return torch.stack(out)


def ssd_scan(xbc: torch.Tensor, dt: torch.Tensor, dt_bias: torch.Tensor, a_log: torch.Tensor,
             d_skip: torch.Tensor, groups: int, n_state: int, step: PackedStep,
             state: torch.Tensor | None) -> torch.Tensor:
    """xbc [T, H*P + 2*G*N] = [x | B | C], dt [T, H] before bias and softplus ->
    [T, H*P]: S_t = exp(-exp(A_log) dt) S + dt B x^T, y = S_t^T C + D x.
    ``state`` [slots, H, N, P] float32."""
    if use_hip(xbc):
        if step.prompt:
            return hip_ops().ssd_prompt(xbc, dt, dt_bias, a_log, d_skip, step.cu_seqlens,
                                        _slots(step, state), state, groups, n_state,
                                        step.max_len)
        return hip_ops().ssd_decode(xbc, dt, dt_bias, a_log, d_skip, step.slots, state, groups,
                                    n_state)
    T, H = dt.shape
    gn = groups * n_state
    x, B, C = xbc.float().split([xbc.shape[1] - 2 * gn, gn, gn], dim=-1)
    x = x.reshape(T, H, -1)
    B, C = (t.reshape(T, groups, n_state).repeat_interleave(H // groups, dim=1) for t in (B, C))
    dt = F.softplus(dt.float() + dt_bias.float(), threshold=80.0)
    decay = torch.exp(-torch.exp(a_log.float()) * dt)
    skip = d_skip.float()[:, None]

    def one(a, b, S):
        S = x.new_zeros(H, n_state, x.shape[2]) if S is None else S
        out = []
        for t in range(a, b):
            S = decay[t, :, None, None] * S + (dt[t, :, None] * B[t])[..., None] * x[t][:, None]
            out.append((torch.einsum("hnp,hn->hp", S, C[t]) + skip * x[t]).reshape(-1))
        return out, S

    return _run(step, T, one, state).to(xbc.dtype)


def wkv_scan(r: torch.Tensor, k: torch.Tensor, v: torch.Tensor, low: torch.Tensor,
             w0: torch.Tensor, u: torch.Tensor, step: PackedStep,
             state: torch.Tensor | None) -> torch.Tensor:
    """r, k, v [T, H*n], low [T, H*n] float32 (may be overwritten), u [H, n] ->
    [T, H*n]: o = (S + diag(u) k v^T)^T r, S <- diag(w) S + k v^T with
    w = exp(-exp(low + w0)). ``state`` [slots, H, n, n] float32."""
    if use_hip(r) and step.prompt:
        return hip_ops().wkv_prompt(r, k, v, low, w0, u, step.cu_seqlens, _slots(step, state),
                                    state, step.max_len)
    T, (H, n) = r.shape[0], u.shape
    dtype = r.dtype
    r, k, v, low = (t.float().reshape(T, H, n) for t in (r, k, v, low + w0.float()))
    decay, bonus = torch.exp(-torch.exp(low)), u.float()[..., None]

    def one(a, b, S):
        S = r.new_zeros(H, n, n) if S is None else S
        out = []
        for t in range(a, b):
            kv = k[t][..., None] * v[t][:, None]
            out.append(torch.einsum("hkv,hk->hv", S + bonus * kv, r[t]).reshape(-1))
            S = decay[t][..., None] * S + kv
        return out, S

    return _run(step, T, one, state).to(dtype)


def wkv_decode(proj: torch.Tensor, w2: torch.Tensor, w0: torch.Tensor, u: torch.Tensor,
               w_norm: torch.Tensor, eps: float, step: PackedStep,
               state: torch.Tensor) -> torch.Tensor:
    """One token per row from proj [R, 4*H*n + rank] = [r | k | v | g | low]:
    decay, recurrence, norm per head and gate -> [R, H*n]."""
    if use_hip(proj):
        return hip_ops().wkv_decode(proj, w2, w0, u, w_norm, eps, step.slots, state)
    hn = w0.numel()
    r, k, v, g, low = proj.split([hn, hn, hn, hn, w2.shape[1]], dim=-1)
    low = torch.tanh(low.float()) @ w2.float().T
    o = wkv_scan(r, k, v, low, w0, u, step, state)
    return gated_group_norm(o, g, w_norm, u.shape[0], eps, gate_first=False)
