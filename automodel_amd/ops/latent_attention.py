"""Latent attention over packed sequences and over a latent KV cache.

A token's keys and values of all heads are functions of one small latent
vector plus one rotated key shared by the heads; only those two are cached.
Two ways to compute the same attention:

* prompts (``latent_attention_prompt``): keys and values are up-projected for
  the tokens of the step and the flash kernel runs over the packed sequences;
* decoding (``latent_attention_decode``): the up-projections are absorbed into
  query and output, and the kernels read cache rows only.

Sequences are packed without padding: a step is ``[T]`` tokens plus a
``PackedStep`` that says where each token belongs. In bf16 within the flash
kernel's head sizes and rank <= 512 the MFMA kernels run; 32-bit models and
other sizes take the row-parallel HIP kernel (``attn_rows``). Torch
expressions serve autograd and CPU tests.
"""

from __future__ import annotations

from dataclasses import dataclass

import torch
import torch.nn.functional as F

from automodel_amd.ops._backend import hip_ops
from automodel_amd.ops.attention import (
    _target_dims,
    flash_attention_varlen,
)
from automodel_amd.ops.packed_step import PackedStep
from automodel_amd.ops.residual_norm import rms_f32, use_hip
from automodel_amd.ops.rope import rope_half_tables  # noqa: F401  (callers import it from here)

FLASH_MAX_HEAD_DIM = 256
MFMA_MAX_RANK = 512
MFMA_MAX_CACHE_WIDTH = 832
_KEYS_PER_TILE = 64                 # latent_decode.hip LD_KEYS
_TARGET_WORKGROUPS = 256            # one per CU: a staged tile fills most of its LDS


def pad32(n: int) -> int:
    return (n + 31) // 32 * 32


@dataclass(frozen=True)
class LatentAttentionSpec:
    """Sizes and constants of one latent-attention layer."""

    heads: int
    dim: int                        # unrotated query/key dims per head
    rot_dim: int                    # rotated query/key dims (key shared by heads)
    vdim: int                       # value dims per head
    kv_rank: int                    # latent size
    scale: float
    rope_base: float = 10000.0
    eps: float = 1e-6               # latent norm

    @property
    def q_width(self) -> int:
        return self.heads * (self.dim + self.rot_dim)

    @property
    def cache_width(self) -> int:
        """Elements of a cache row: latent and rotated key, each padded to 32."""
        return pad32(self.kv_rank) + pad32(self.rot_dim)


def _rotate(x: torch.Tensor, cos: torch.Tensor, sin: torch.Tensor) -> torch.Tensor:
    """x [T, ..., rot]; cos/sin [T, rot/2]. Pairs (i, i + rot/2), in float32."""
    for _ in range(x.dim() - 2):
        cos, sin = cos.unsqueeze(1), sin.unsqueeze(1)
    u, v = x.float().chunk(2, dim=-1)
    return torch.cat([u * cos - v * sin, v * cos + u * sin], dim=-1).to(x.dtype)


def _split_torch(qkv, norm_w, spec, rope, positions):
    """-> q_unrot [T,H,dim], q_rot [T,H,rot], latent [T,rank], key_rot [T,rot]."""
    cos, sin = rope[0][positions.long()], rope[1][positions.long()]
    q, c, kr = qkv.split([spec.q_width, spec.kv_rank, spec.rot_dim], dim=-1)
    q = q.reshape(q.shape[0], spec.heads, spec.dim + spec.rot_dim)
    c = rms_f32(c, norm_w, spec.eps).to(qkv.dtype)
    return (q[..., :spec.dim], _rotate(q[..., spec.dim:], cos, sin), c,
            _rotate(kr, cos, sin))


def _write_cache_torch(cache, step, c, kr, spec):
    slots, pos = step.slots.long(), step.positions.long()
    cache[slots, pos, :spec.kv_rank] = c
    start = pad32(spec.kv_rank)
    cache[slots, pos, start:start + spec.rot_dim] = kr


def latent_attention_prompt(qkv, norm_w, w_kv_b, spec: LatentAttentionSpec, rope,
                            step: PackedStep, cache: torch.Tensor | None = None) -> torch.Tensor:
    """qkv [T, q_width + rank + rot] of whole prompts -> [T, heads * vdim].

    ``w_kv_b`` stacks the key then the value up-projection, [H*dim + H*vdim, rank].
    """
    T, H, dn, dv = qkv.shape[0], spec.heads, spec.dim, spec.vdim
    if use_hip(qkv):
        ops = hip_ops()
        flash = (qkv.dtype == torch.bfloat16 and dn + spec.rot_dim <= FLASH_MAX_HEAD_DIM
                 and dv <= FLASH_MAX_HEAD_DIM)
        kd, vd = _target_dims(dn + spec.rot_dim, dv) if flash else (dn + spec.rot_dim, dv)
        # rows in whole workgroups of the flash kernel: 8 waves of 32, 4 if few
        rows = T + (-T) % (256 if T > 1024 else 128) if flash else T
        q, c, kr = ops.latent_prep(
            qkv, norm_w, spec.eps, rope[0], rope[1], step.positions,
            step.slots if cache is not None else None, cache,
            H, dn, spec.rot_dim, kd, rows)
        k, v = ops.latent_assemble(F.linear(c[:T], w_kv_b), kr, H, dn, dv, kd, vd, T)
        if flash:
            # one sequence needs no document bounds: padding rows come last
            o, _ = ops.flash_attn_fwd(q[None], k[None], v[None], spec.scale, True, 0,
                                      step.doc_start if step.n_seqs > 1 else None)
            return o[0, :T, :, :dv].reshape(T, H * dv)
        o = ops.attn_rows(q, k, v, step.doc_start[:T].long(), step.positions + 1, spec.scale,
                          False)
        return o.view(T, H * dv)

    qn, qr, c, kr = _split_torch(qkv, norm_w, spec, rope, step.positions)
    if cache is not None:
        _write_cache_torch(cache, step, c, kr, spec)
    kn, v = F.linear(c, w_kv_b).split([H * dn, H * dv], dim=-1)
    q = torch.cat([qn, qr], dim=-1)
    k = torch.cat([kn.reshape(T, H, dn), kr[:, None].expand(T, H, spec.rot_dim)], dim=-1)
    v = v.reshape(T, H, dv)
    if qkv.is_cuda and qkv.dtype == torch.bfloat16:
        o = flash_attention_varlen(q[None], k[None], v[None].contiguous(), step.cu_seqlens,
                                   spec.scale, "hip")[0]
    else:
        i = torch.arange(T, device=qkv.device)
        start = step.doc_start[:T].to(i)
        keep = (i[None] <= i[:, None]) & (i[None] >= start[:, None])
        s = torch.einsum("ihd,jhd->hij", q.float(), k.float()) * spec.scale
        p = torch.softmax(s.masked_fill(~keep, float("-inf")), dim=-1)
        o = torch.einsum("hij,jhd->ihd", p, v.float()).to(qkv.dtype)
    return o.reshape(T, H * dv)


def decode_splits(rows: int, heads: int, max_len: int) -> int:
    """KV splits per (row, head group): enough workgroups for the chip, no more
    than there are key tiles. Depends on capacities only, so that it is the
    same on every replay of a captured step."""
    groups = -(-heads // (16 if heads <= 16 else 32))
    want = _TARGET_WORKGROUPS // max(1, rows * groups)
    return max(1, min(want, -(-max_len // _KEYS_PER_TILE), 64))


def latent_attention_decode(qkv, norm_w, w_kv_b, spec: LatentAttentionSpec, rope,
                            step: PackedStep, cache: torch.Tensor) -> torch.Tensor:
    """One token per row, each against its slot's cached prefix (which this
    call extends by the row's own token) -> [R, heads * vdim]."""
    H, dn, dv, rank = spec.heads, spec.dim, spec.vdim, spec.kv_rank
    w_uk, w_uv = w_kv_b[:H * dn], w_kv_b[H * dn:]
    R = qkv.shape[0]
    if use_hip(qkv):
        ops = hip_ops()
        q = ops.latent_decode_prep(qkv, w_uk, norm_w, spec.eps, rope[0], rope[1],
                                   step.positions, step.slots, cache, H, dn, spec.rot_dim)
        if (qkv.dtype == torch.bfloat16 and rank <= MFMA_MAX_RANK
                and spec.cache_width <= MFMA_MAX_CACHE_WIDTH):
            part, ml = ops.latent_decode_attn(
                q, cache, step.slots, step.positions, rank, spec.rot_dim, spec.scale,
                decode_splits(R, H, cache.shape[1]))
            return ops.latent_decode_combine(part, ml, w_uv, dv)
        rows = cache.view(-1, 1, cache.shape[2])
        o = ops.attn_rows(q, rows, rows[..., :rank], step.slots.long() * cache.shape[1],
                          step.positions + 1, spec.scale, True)
        return ops.latent_decode_combine(o.view(R, H, 1, rank), None, w_uv, dv)

    qn, qr, c, kr = _split_torch(qkv, norm_w, spec, rope, step.positions)
    _write_cache_torch(cache, step, c, kr, spec)
    out = qkv.new_empty(R, H * dv)
    off = pad32(rank)
    for r in range(R):
        keys = cache[int(step.slots[r]), :int(step.positions[r]) + 1]
        lat, rot = keys[:, :rank].float(), keys[:, off:off + spec.rot_dim].float()
        q_lat = torch.einsum("hd,hdr->hr", qn[r].float(), w_uk.float().view(H, dn, rank))
        s = (q_lat @ lat.T + qr[r].float() @ rot.T) * spec.scale
        o = torch.softmax(s, dim=-1) @ lat
        out[r] = torch.einsum("hr,hvr->hv", o, w_uv.float().view(H, dv, rank)) \
            .reshape(-1).to(out.dtype)
    return out
