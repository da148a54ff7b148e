"""Grouped-head attention over packed sequences and a slot cache.

Query heads share key/value heads in equal groups, part of a head may turn with
the position, keys may be limited to the token's own chunk of the sequence
(counted from its first token), and the softmax may have a sink: one learned
logit per head, without key or value, in the denominator.

* prompts (``grouped_attention_prompt``): the flash kernel, chunks as document
  bounds;
* decoding (``grouped_attention_decode``): split-KV kernel over the cache, which
  keeps one chunk per slot (row = position modulo chunk).

In bf16 with heads of up to 256 the MFMA kernels run on the blocked cache;
32-bit models and larger heads take the row-parallel HIP kernel (``attn_rows``)
on the plain one (layouts: csrc/gqa_attn.hip). Torch expressions serve autograd
and CPU tests.
"""

from __future__ import annotations

from dataclasses import dataclass

import torch

from automodel_amd.ops._backend import hip_ops
from automodel_amd.ops.attention import _target_dims
from automodel_amd.ops.packed_step import PackedStep
from automodel_amd.ops.residual_norm import use_hip
from automodel_amd.ops.rope import rope_half_tables

MFMA_MAX_HEAD_DIM = 256
NO_CHUNK = 2**31 - 1
_KEYS_PER_BLOCK = 32                # gqa_attn.hip: keys per step of a wave
_TARGET_WAVES = 2048                # two per SIMD


def _up(n: int, m: int) -> int:
    return (n + m - 1) // m * m


@dataclass(frozen=True)
class GroupedAttentionSpec:
    """Sizes and constants of one layer. ``chunk`` None: every earlier key;
    ``rope_scaling``: items of a ``build_rope_cache`` scaling dict."""

    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot_dim: int
    rope_base: float = 10000.0
    rope_scaling: tuple | None = None
    chunk: int | None = None

    def __post_init__(self):
        if self.heads % self.kv_heads:
            raise ValueError("query heads share key/value heads in equal groups")
        if self.rot_dim % 2 or not 0 <= self.rot_dim <= self.dim:
            raise ValueError("rotated dims come in pairs within a head")
        if self.chunk is not None and self.chunk < 1:
            raise ValueError("a chunk has at least one token")

    @property
    def in_width(self) -> int:
        return self.heads * self.dim + self.kv_heads * (self.dim + self.vdim)

    @property
    def chunk_size(self) -> int:
        return self.chunk or NO_CHUNK

    @property
    def rope_key(self) -> tuple:
        return self.rot_dim, self.rope_base, self.rope_scaling

    def rope_tables(self, n: int, device):
        return rope_half_tables(self.rot_dim, n, self.rope_base, device,
                                dict(self.rope_scaling) if self.rope_scaling else None)

    def blocked(self, device, dtype) -> bool:
        return (torch.device(device).type == "cuda" and dtype == torch.bfloat16
                and max(self.dim, self.vdim) <= MFMA_MAX_HEAD_DIM)

    def make_state(self, n_slots: int, max_len: int, device, dtype) -> dict[str, torch.Tensor]:
        rows, G = min(self.chunk_size, max_len), self.kv_heads
        if self.blocked(device, dtype):
            rows = _up(rows, _KEYS_PER_BLOCK)
            shapes = {"k": (n_slots, G, rows, _up(self.dim, 32)),
                      "v": (n_slots, G, rows // 32, _up(self.vdim, 16), 32)}
        else:
            shapes = {"k": (n_slots, rows, G, self.dim), "v": (n_slots, rows, G, self.vdim)}
        # zeros: what a kernel reads beyond a sequence's keys must be finite
        return {n: torch.zeros(s, device=device, dtype=dtype) for n, s in shapes.items()}


def _rotate(x: torch.Tensor, cos: torch.Tensor, sin: torch.Tensor) -> torch.Tensor:
    """x [T, heads, dim]: the first 2 * cos.shape[1] dims in pairs, in float32."""
    half = cos.shape[1]
    cos, sin = cos[:, None], sin[:, None]
    xf = x.float()
    u, v, rest = xf[..., :half], xf[..., half:2 * half], xf[..., 2 * half:]
    return torch.cat([u * cos - v * sin, v * cos + u * sin, rest], dim=-1).to(x.dtype)


def _split_torch(proj, spec, rope, positions):
    T, H, G = proj.shape[0], spec.heads, spec.kv_heads
    cos, sin = rope[0][positions.long()], rope[1][positions.long()]
    q, k, v = proj[:, :spec.in_width].split([H * spec.dim, G * spec.dim, G * spec.vdim], dim=-1)
    return (_rotate(q.reshape(T, H, spec.dim), cos, sin),
            _rotate(k.reshape(T, G, spec.dim), cos, sin), v.reshape(T, G, spec.vdim))


def _softmax_sink(s: torch.Tensor, sink: torch.Tensor | None) -> torch.Tensor:
    """Softmax over the last dim of s [heads, ..., keys] with the sink's share left out."""
    if sink is None:
        return torch.softmax(s, dim=-1)
    extra = sink.float().view(-1, *[1] * (s.dim() - 1)).expand(*s.shape[:-1], 1)
    return torch.softmax(torch.cat([s, extra], dim=-1), dim=-1)[..., :-1]


def grouped_attention_prompt(proj, sink, spec: GroupedAttentionSpec, rope, step: PackedStep,
                             state: dict | None = None) -> torch.Tensor:
    """proj [T, >= in_width], beginning with [q | k | v] of whole prompts
    -> [T, heads * vdim]."""
    T, H, G, d, dv = proj.shape[0], spec.heads, spec.kv_heads, spec.dim, spec.vdim
    chunk = spec.chunk_size
    start = step.chunk_start(chunk)
    if use_hip(proj):
        ops = hip_ops()
        flash = proj.dtype == torch.bfloat16 and max(d, dv) <= MFMA_MAX_HEAD_DIM
        kd, vd = _target_dims(d, dv) if flash else (d, dv)
        # rows in whole workgroups of the flash kernel: 8 waves of 32, 4 if few
        rows = _up(T, 256 if T > 1024 else 128) if flash else T
        k_cache, v_cache = (state["k"], state["v"]) if state else (None, None)
        q, k, v = ops.gqa_prep(proj, rope[0], rope[1], step.positions,
                               step.slots if state else None, step.seq_end, step.cu_seqlens,
                               k_cache, v_cache, chunk, H, G, d, dv, kd, vd, rows, False)
        if flash:
            # one sequence in one chunk needs no bounds: padding rows come last
            whole = step.n_seqs == 1 and step.max_len <= chunk
            o, _ = ops.flash_attn_fwd(q[None], k[None], v[None], spec.scale, True, 0,
                                      None if whole else start, sink)
            o = o[0, :T]
            return (o if vd == dv else o[..., :dv]).reshape(T, H * dv)
        count = (step.positions % chunk + 1).int()
        return ops.attn_rows(q, k, v, start[:T].long(), count, spec.scale, False,
                             sink).view(T, H * dv)

    q, k, v = _split_torch(proj, spec, rope, step.positions)
    if state is not None:
        last = step.positions + step.seq_end - 1 - torch.arange(T, device=proj.device)
        keep = (last // chunk == step.positions // chunk).nonzero()[:, 0]
        slots, rows = step.slots[keep].long(), (step.positions[keep] % chunk).long()
        state["k"][slots, rows], state["v"][slots, rows] = k[keep], v[keep]
    k, v = (t.repeat_interleave(H // G, dim=1).float() for t in (k, v))
    i = torch.arange(T, device=proj.device)
    keep = (i[None] <= i[:, None]) & (i[None] >= start[:T].to(i)[:, None])
    s = torch.einsum("ihd,jhd->hij", q.float(), k) * spec.scale
    p = _softmax_sink(s.masked_fill(~keep, float("-inf")), sink)
    return torch.einsum("hij,jhd->ihd", p, v).to(proj.dtype).reshape(T, H * dv)


def decode_splits(rows: int, spec: GroupedAttentionSpec, cache_rows: int) -> int:
    """KV splits per (row, head group), from capacities only, so that it is the
    same on every replay of a captured step."""
    groups = spec.kv_heads * -(-(spec.heads // spec.kv_heads) // 16)
    want = _TARGET_WAVES // max(1, rows * groups)
    return max(1, min(want, cache_rows // _KEYS_PER_BLOCK, 64))


def grouped_attention_decode(proj, sink, spec: GroupedAttentionSpec, rope, step: PackedStep,
                             state: dict) -> torch.Tensor:
    """One token per row against what its slot's cache has of its chunk (which
    this call extends by the row's own token) -> [R, heads * vdim]."""
    R, H, G, d, dv = proj.shape[0], spec.heads, spec.kv_heads, spec.dim, spec.vdim
    k_cache, v_cache, chunk = state["k"], state["v"], spec.chunk_size
    if use_hip(proj):
        ops = hip_ops()
        blocked = v_cache.dim() == 5
        kd = k_cache.shape[3] if blocked else d
        q, _, _ = ops.gqa_prep(proj, rope[0], rope[1], step.positions, step.slots, None, None,
                               k_cache, v_cache, chunk, H, G, d, dv, kd, dv, R, True)
        if blocked:
            return ops.gqa_decode_attn(q, k_cache, v_cache, step.slots, step.positions, sink,
                                       chunk, dv, spec.scale,
                                       decode_splits(R, spec, k_cache.shape[2]))
        base = step.slots.long() * k_cache.shape[1]
        return ops.attn_rows(q, k_cache.view(-1, G, d), v_cache.view(-1, G, dv), base,
                             (step.positions % chunk + 1).int(), spec.scale, False,
                             sink).view(R, H * dv)

    q, k, v = _split_torch(proj, spec, rope, step.positions)
    slots, rows = step.slots.long(), (step.positions % chunk).long()
    k_cache[slots, rows], v_cache[slots, rows] = k, v
    out = []
    for r in range(R):
        n = int(rows[r]) + 1
        kr, vr = (c[slots[r], :n].repeat_interleave(H // G, dim=1).float()
                  for c in (k_cache, v_cache))
        s = torch.einsum("hd,jhd->hj", q[r].float(), kr) * spec.scale
        out.append(torch.einsum("hj,jhd->hd", _softmax_sink(s, sink), vr).reshape(-1))
    return torch.stack(out).to(proj.dtype)
