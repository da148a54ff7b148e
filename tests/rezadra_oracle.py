"""Plain, slow implementation of the Rezadra design, one function per mechanism.

Independent of the product code: no import from ``automodel_amd``, no cache,
no batching, no fused weights. Everything is computed in the dtype of the
weights it is given (the tests pass float64 or float32). Weights are a flat
``{name: tensor}`` dict under the checkpoint's own names; the configuration is
the checkpoint's own config dict.

Planted mistakes (``fault=...``) let a test show that its inputs are able to
expose a given error; they exist only here.
"""

from __future__ import annotations

import math

import torch


def rms(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def relu_squared(z):
    return torch.where(z > 0, z * z, torch.zeros_like(z))


def rotate(x, positions, base):
    """x [T, ..., n]: pairs (i, i + n/2) turned by position * base^(-2i/n)."""
    n = x.shape[-1]
    out = x.clone()
    for i in range(n // 2):
        angle = positions.double() * base ** (-2.0 * i / n)
        c, s = torch.cos(angle).to(x.dtype), torch.sin(angle).to(x.dtype)
        while c.dim() < x.dim() - 1:
            c, s = c.unsqueeze(-1), s.unsqueeze(-1)
        u, v = x[..., i], x[..., i + n // 2]
        out[..., i] = u * c - v * s
        out[..., i + n // 2] = v * c + u * s
    return out


def latent_attention(h, w, p, mixer, eps, fault=None):
    """h [T, width] of ONE sequence from position 0 -> [T, width]."""
    T = h.shape[0]
    H, dn, dr = mixer["heads"], mixer["dim"], mixer["rot_dim"]
    dv, rank = mixer["vdim"], mixer["kv_rank"]
    base, scale = mixer["rot"]["base"], mixer["scale"]
    pos = torch.arange(T)
    q = (h @ w[p + "q"].T).view(T, H, dn + dr)
    down = h @ w[p + "dkv"].T
    c = rms(down[:, :rank], w[p + "dkv.norm"], eps)
    if fault == "latent_not_normed":
        c = down[:, :rank]
    kr = down[:, rank:] if fault == "key_not_rotated" else rotate(down[:, rank:], pos, base)
    qn, qr = q[..., :dn], rotate(q[..., dn:], pos, base)
    kn = (c @ w[p + "uk"].T).view(T, H, dn)
    v = (c @ w[p + "uv"].T).view(T, H, dv)
    out = torch.empty(T, H, dv, dtype=h.dtype)
    for i in range(T):
        seen = list(range(i + 1))
        if isinstance(fault, tuple) and i > 0:      # ("lost", key) or ("lost", "own")
            lost = i if fault[1] == "own" else fault[1]
            seen = [j for j in seen if j != lost]
        for a in range(H):
            s = (kn[seen, a] @ qn[i, a] + kr[seen] @ qr[i, a]) * scale
            e = torch.exp(s - s.max())
            out[i, a] = (e / e.sum()) @ v[seen, a]
    return out.reshape(T, H * dv) @ w[p + "o"].T


def dense_ff(h, w, p):
    return relu_squared(h @ w[p + "up"].T) @ w[p + "down"].T


def layer(x, w, i, spec, eps, m, fault=None):
    p = f"l{i}."
    y = latent_attention(rms(x, w[p + "norm1"], eps), w, p + "mix.", spec["mixer"], eps, fault)
    x = x + m * rms(y, w[p + "norm1b"], eps)
    if spec.get("mlp") is not None:
        y = dense_ff(rms(x, w[p + "norm2"], eps), w, p + "mlp.")
        x = x + m * rms(y, w[p + "norm2b"], eps)
    return x


def layer_order(cfg):
    """[(layer index, True where a pass of the loop begins)]"""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, False) for i in range(n)]
    a, b = loop["start"], loop["stop"]
    order = [(i, False) for i in range(a)]
    for _ in range(loop["times"]):
        order += [(i, i == a) for i in range(a, b)]
    return order + [(i, False) for i in range(b, n)]


def forward(tokens, w, cfg, trace=None, fault=None):
    """tokens: list of ids of one sequence -> logits [T, vocab]."""
    eps = cfg["norm"]["eps"]
    x0 = rms(w["embed"][torch.as_tensor(tokens)], w["embed.norm"], eps)
    x = x0
    for i, begins in layer_order(cfg):
        if begins:
            x = torch.cat([x, x0], -1) @ w["loop.in"].T
        x = layer(x, w, i, cfg["layers"][i], eps, cfg["residual_mult"], fault)
        if trace is not None:
            trace.append(x)
    return rms(x, w["final.norm"], eps) @ w["head"].T


def greedy(prompt, n, w, cfg):
    ids = list(prompt)
    for _ in range(n):
        ids.append(int(forward(ids, w, cfg)[-1].argmax()))
    return ids


def make_config(vocab=61, width=40, layers=None, loop=None, eps=1e-5, mult=0.7):
    cfg = {"architecture": "Rezadra", "layers": layers, "norm": {"eps": eps},
           "residual_mult": mult, "vocab": vocab, "width": width}
    if loop is not None:
        cfg["loop"] = loop
    return cfg


def make_layer(heads=3, dim=16, rot_dim=8, vdim=24, kv_rank=32, base=1000.0,
               ff=56, scale=None):
    return {"type": "latent_attention",
            "mixer": {"dim": dim, "heads": heads, "kv_rank": kv_rank,
                      "rot": {"base": base, "dims": rot_dim}, "rot_dim": rot_dim,
                      "scale": scale or 1.0 / math.sqrt(dim + rot_dim), "vdim": vdim},
            "mlp": None if ff is None else {"ff": ff, "kind": "dense"}}


def make_weights(cfg, seed=0):
    """bfloat16 tensors under the checkpoint's names."""
    g = torch.Generator().manual_seed(seed)
    W, V = cfg["width"], cfg["vocab"]

    def lin(o, i, gain=1.0):
        return (torch.randn(o, i, generator=g) * gain / math.sqrt(i)).bfloat16()

    def nrm(n):
        return (1.0 + 0.3 * torch.randn(n, generator=g)).bfloat16()

    w = {"embed": torch.randn(V, W, generator=g).bfloat16(), "embed.norm": nrm(W),
         "final.norm": nrm(W), "head": lin(V, W)}
    if cfg.get("loop"):
        w["loop.in"] = lin(W, 2 * W)
    for i, spec in enumerate(cfg["layers"]):
        mx, p = spec["mixer"], f"l{i}."
        H, r = mx["heads"], mx["kv_rank"]
        w[p + "norm1"], w[p + "norm1b"] = nrm(W), nrm(W)
        w[p + "mix.q"] = lin(H * (mx["dim"] + mx["rot_dim"]), W, 1.5)
        w[p + "mix.dkv"] = lin(r + mx["rot_dim"], W)
        w[p + "mix.dkv.norm"] = nrm(r)
        w[p + "mix.uk"] = lin(H * mx["dim"], r)
        w[p + "mix.uv"] = lin(H * mx["vdim"], r)
        w[p + "mix.o"] = lin(W, H * mx["vdim"])
        if spec.get("mlp") is not None:
            w[p + "norm2"], w[p + "norm2b"] = nrm(W), nrm(W)
            w[p + "mlp.up"] = lin(spec["mlp"]["ff"], W)
            w[p + "mlp.down"] = lin(W, spec["mlp"]["ff"])
    return w
