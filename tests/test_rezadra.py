"""Rezadra against a plain implementation (rezadra_oracle.py): weights, every
mechanism alone, prompts, decoding, batches, slots, generation.

Each case runs on the CPU (torch expressions) and, marked gpu, on the HIP
kernels in float32 and bfloat16."""

import io
import json
import os
import sys

import pytest
import torch

import rezadra_oracle as oracle
from rezadra_oracle import make_config, make_layer, make_weights

from automodel_amd.models.registry import load_pretrained
from automodel_amd.ops import latent_attention as la
from automodel_amd.ops import residual_norm as rn
from automodel_amd.utils.generation import DecodeSession

PLACES = [
    pytest.param("cpu", "float32", id="cpu-f32"),
    pytest.param("cuda", "float32", id="gpu-f32", marks=pytest.mark.gpu),
    pytest.param("cuda", "bfloat16", id="gpu-bf16", marks=pytest.mark.gpu),
]
on_each = pytest.mark.parametrize("dev,dt", PLACES)
TOL = {"float32": 3e-5, "bfloat16": 3e-2}

CONFIGS = {
    # four different layers, one without a feed-forward, the loop in the middle
    "mixed": make_config(
        layers=[make_layer(), make_layer(heads=2, dim=8, rot_dim=16, vdim=8, kv_rank=40, ff=None),
                make_layer(heads=5, dim=24, rot_dim=4, vdim=12, kv_rank=16, base=77.0, ff=24),
                make_layer(heads=1, dim=32, rot_dim=32, vdim=40, kv_rank=72)],
        loop={"start": 1, "stop": 3, "times": 3}, mult=0.4),
    # no loop; sizes that are no multiples of 4 or 8
    "odd": make_config(vocab=37, width=30, layers=[
        make_layer(heads=3, dim=10, rot_dim=6, vdim=7, kv_rank=22, ff=34),
        make_layer(heads=2, dim=5, rot_dim=2, vdim=9, kv_rank=13, ff=17)], eps=1e-3, mult=1.0),
    # one pass over everything; one head; factor 1
    "once": make_config(width=64, layers=[make_layer(heads=1, dim=16, rot_dim=16, vdim=16,
                                                     kv_rank=64, ff=64)] * 2,
                        loop={"start": 0, "stop": 2, "times": 1}, mult=1.0),
    # more heads than one MFMA tile, and than two
    "wide": make_config(vocab=80, width=96, layers=[
        make_layer(heads=19, dim=16, rot_dim=32, vdim=16, kv_rank=160, ff=128),
        make_layer(heads=37, dim=8, rot_dim=8, vdim=8, kv_rank=288, ff=64)],
        loop={"start": 1, "stop": 2, "times": 2}, mult=0.6),
}
BIG = {
    # the head sizes of large models; flash pair (192, 128), rank 512
    "large-heads": make_config(vocab=128, width=256, layers=[
        make_layer(heads=4, dim=128, rot_dim=64, vdim=128, kv_rank=512, ff=512)],
        loop={"start": 0, "stop": 1, "times": 2}, mult=0.5),
    # beyond the MFMA kernels: head dim over 256, rank over 512
    "row-kernel": make_config(vocab=64, width=64, layers=[
        make_layer(heads=2, dim=240, rot_dim=24, vdim=264, kv_rank=56, ff=64),
        make_layer(heads=2, dim=32, rot_dim=16, vdim=32, kv_rank=544, ff=64)], mult=0.5),
}
ALL = {**CONFIGS, **BIG}

_models: dict = {}


@pytest.fixture(scope="session")
def checkpoints(tmp_path_factory):
    from safetensors.torch import save_file

    root = tmp_path_factory.mktemp("rezadra")

    def get(name):
        path = root / name
        if not path.exists():
            path.mkdir()
            (path / "config.json").write_text(json.dumps(ALL[name]))
            save_file(make_weights(ALL[name], seed=len(name)), str(path / "model.safetensors"))
        return str(path)

    return get


@pytest.fixture
def model_of(checkpoints):
    def get(name, dev, dt):
        key = (name, dev, dt)
        if key not in _models:
            _models[key] = load_pretrained(checkpoints(name), dtype=dt, device=dev)
        return _models[key]

    return get


def weights(name, dtype=torch.float64):
    return {k: v.to(dtype) for k, v in make_weights(ALL[name], seed=len(name)).items()}


def ids_of(name, n, seed=1):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, ALL[name]["vocab"], (n,), generator=g).tolist()


_logits: dict = {}


def want_logits(name, ids):
    key = (name, tuple(ids))
    if key not in _logits:
        _logits[key] = oracle.forward(ids, weights(name), ALL[name])
    return _logits[key]


def rel(got, want):
    """Largest row error, relative to the rows' root mean square."""
    got, want = got.detach().double().cpu(), want.double()
    assert got.shape == want.shape, (got.shape, want.shape)
    e = (got - want).pow(2).mean(-1).sqrt()
    return float((e / want.pow(2).mean().sqrt()).max())


def close(got, want, dt, factor=1.0):
    e = rel(got, want)
    assert e < TOL[dt] * factor, e


def whole(model, prompts, want=None):
    s = DecodeSession(model, len(prompts), max(len(p) for p in prompts))
    want = [list(range(len(p))) for p in prompts] if want is None else want
    return s.prefill(prompts, want)[1]


def by_parts(model, ids, first, max_len=None):
    """Prompt of ``first`` tokens, the rest decoded; logits of every place."""
    s = DecodeSession(model, 1, max_len or len(ids))
    h, lg = s.prefill([ids[:first]], [list(range(first))])
    out = [lg]
    for t in ids[first:]:
        out.append(s.decode(h, torch.tensor([t], device=s.device)))
    return torch.cat(out)


# ---------------------------------------------------------------- mechanisms
@on_each
@pytest.mark.parametrize("width", [64, 30, 7, 4096])
@torch.no_grad()
def test_norms_and_residual(dev, dt, width):
    dtype = getattr(torch, dt)
    g = torch.Generator().manual_seed(width)
    T, eps, m = 5, 1e-2, 0.37
    table = torch.randn(11, width, generator=g).to(dtype)
    w1, w2, w3 = ((1 + torch.randn(width, generator=g)).to(dtype) for _ in range(3))
    ids = torch.tensor([3, 10, 0, 3, 7])
    y = (3 * torch.randn(T, width, generator=g)).to(dtype)
    d = [t.to(dev) for t in (table, w1, w2, w3, ids, y)]
    x = rn.embed_rms_norm(d[4], d[0], d[1], eps)
    assert x.dtype == torch.float32
    x_ref = oracle.rms(table.double()[ids], w1.double(), eps)
    assert rel(x, x_ref) < 1e-6
    h = rn.residual_rms_norm(x, d[2], eps)
    assert h.dtype == dtype
    close(h, oracle.rms(x_ref, w2.double(), eps), dt)
    x2, h2 = rn.residual_add_norm(x.clone(), d[5], d[1], m, eps, d[3])
    new = x_ref + m * oracle.rms(y.double(), w1.double(), eps)
    assert x2.dtype == torch.float32 and rel(x2, new) < 1e-6    # 32-bit sum
    close(h2, oracle.rms(new, w3.double(), eps), dt)
    x3, none = rn.residual_add_norm(x.clone(), d[5], d[1], m, eps)
    assert none is None and rel(x3, new) < 1e-6
    cat = rn.concat_cast(x, x2, dtype)
    assert cat.dtype == dtype
    close(cat, torch.cat([x_ref, new], -1), dt)


@on_each
@pytest.mark.parametrize("shape", [(3, 40), (5, 7), (64, 1024)])
@torch.no_grad()
def test_relu_squared(dev, dt, shape):
    x = torch.randn(*shape, generator=torch.Generator().manual_seed(0)).to(getattr(torch, dt))
    got = rn.relu2(x.clone().to(dev))
    close(got, oracle.relu_squared(x.double()), dt)
    assert bool((got.cpu()[x < 0] == 0).all())


def test_layer_schedule():
    from automodel_amd.models.common.blocks import layer_schedule

    for cfg in ALL.values():
        assert layer_schedule(len(cfg["layers"]), cfg.get("loop")) == oracle.layer_order(cfg)
    for loop in ({"start": 2, "stop": 2, "times": 1}, {"start": 0, "stop": 4, "times": 1},
                 {"start": 0, "stop": 1, "times": 0}):
        with pytest.raises(ValueError):
            layer_schedule(3, loop)


def attention_case(mixer, n, seed=0, scale_q=1.0):
    cfg = make_config(width=48, layers=[{"type": "latent_attention", "mixer": mixer, "mlp": None}])
    w = {k[len("l0.mix."):]: v for k, v in make_weights(cfg, seed).items()
         if k.startswith("l0.mix.")}
    w["q"] = (w["q"].float() * scale_q).bfloat16()
    h = torch.randn(n, 48, generator=torch.Generator().manual_seed(seed + 1)).bfloat16()
    return w, h


def run_attention(w, h, mixer, dev, dt, eps, prompt_len=None, slot=0, n_slots=2, max_len=None):
    """The module's two paths: the first ``prompt_len`` tokens as a prompt, the
    rest as one-token steps."""
    dtype = getattr(torch, dt)
    spec = la.LatentAttentionSpec(
        heads=mixer["heads"], dim=mixer["dim"], rot_dim=mixer["rot_dim"], vdim=mixer["vdim"],
        kv_rank=mixer["kv_rank"], scale=mixer["scale"], rope_base=mixer["rot"]["base"], eps=eps)
    n = h.shape[0]
    prompt_len = n if prompt_len is None else prompt_len
    max_len = max_len or n
    W = {k: v.to(dev, dtype) for k, v in w.items()}
    qkv = torch.nn.functional.linear(h.to(dev, dtype), torch.cat([W["q"], W["dkv"]]))
    kv_b = torch.cat([W["uk"], W["uv"]])
    rope = la.rope_half_tables(spec.rot_dim, max_len, spec.rope_base, dev)
    cache = torch.zeros(n_slots, max_len, spec.cache_width, device=dev, dtype=dtype)
    out = []
    if prompt_len:
        step = la.PackedStep.for_prompts([prompt_len], dev, [slot])
        out.append(la.latent_attention_prompt(qkv[:prompt_len], W["dkv.norm"], kv_b, spec, rope,
                                              step, cache))
    for i in range(prompt_len, n):
        step = la.PackedStep(positions=torch.tensor([i], dtype=torch.int32, device=dev),
                             slots=torch.tensor([slot], dtype=torch.int32, device=dev),
                             prompt=False)
        out.append(la.latent_attention_decode(qkv[i:i + 1], W["dkv.norm"], kv_b, spec, rope,
                                              step, cache))
    o = torch.nn.functional.linear(torch.cat(out), W["o"])
    assert not cache[[s for s in range(n_slots) if s != slot]].any()     # own slot only
    return o


MIXERS = {
    "plain": make_layer(heads=3, dim=16, rot_dim=8, vdim=24, kv_rank=32)["mixer"],
    "odd": make_layer(heads=2, dim=9, rot_dim=6, vdim=5, kv_rank=19, base=50.0)["mixer"],
    "large": make_layer(heads=17, dim=128, rot_dim=64, vdim=128, kv_rank=512)["mixer"],
    "rotation-wider": make_layer(heads=3, dim=16, rot_dim=160, vdim=16, kv_rank=512)["mixer"],
    "value-wider": make_layer(heads=2, dim=8, rot_dim=56, vdim=120, kv_rank=200)["mixer"],
}


@on_each
@pytest.mark.parametrize("name", sorted(MIXERS))
@pytest.mark.parametrize("prompt_len", [None, 0, 65])
@torch.no_grad()
def test_latent_attention_alone(dev, dt, name, prompt_len):
    mixer, n, eps = MIXERS[name], 70, 1e-4
    w, h = attention_case(mixer, n)
    want = oracle.latent_attention(h.double(), {k: v.double() for k, v in w.items()}, "", mixer, eps)
    close(run_attention(w, h, mixer, dev, dt, eps, prompt_len, slot=1, max_len=200), want, dt)


def far_key_case(target, query, n):
    """Token ``query`` scores one key, ``target``, far above all others."""
    mixer = make_layer(heads=2, dim=16, rot_dim=8, vdim=16, kv_rank=32)["mixer"]
    mixer["rot"] = {"base": 10.0, "dims": 8}
    w, h = attention_case(mixer, n, seed=5)
    h = h.float() * 0.5
    # make W_q h_query the (unrotated) key direction of `target`, per head
    W = {k: v.double() for k, v in w.items()}

    def key(x):
        c = oracle.rms((x.double() @ W["dkv"].T)[..., :32], W["dkv.norm"], 1e-4)
        return (c @ W["uk"].T).view(-1, 2, 16)

    if target == query:                     # queries that are parallel to their own keys
        w = {k: v.clone() for k, v in w.items()}
        w["uk"] = torch.eye(16, 32).repeat(2, 1).bfloat16()
        w["dkv.norm"][:] = 1.0
        q = torch.zeros(2, 24, 48)
        q[:, :16] = 8.0 * w["dkv"][:16].float()
        w["q"] = q.view(48, 48).bfloat16()
        return mixer, w, h.bfloat16()
    kn = key(h[target])[0]
    goal = torch.cat([kn, torch.zeros(2, 8, dtype=torch.float64)], -1).reshape(-1)
    h[query] = (torch.linalg.pinv(W["q"]) @ goal * 6.0).float()
    return mixer, w, h.bfloat16()


EDGES = [(0, 1), (0, 63), (0, 64), (0, 127), (0, 128), (63, 64), (64, 64), (62, 128), (127, 128),
         (128, 128), (1, 129), (64, 129), (31, 32), (32, 95)]


@on_each
@pytest.mark.parametrize("target,query", EDGES)
@torch.no_grad()
def test_one_key_stands_out(dev, dt, target, query):
    """At tile borders, at the first key, at the query's own key: the one key
    that matters is seen by prompts and by decoding, and a mistake would show."""
    n = query + 1
    mixer, w, h = far_key_case(target, query, n)
    W = {k: v.double() for k, v in w.items()}

    def ref(fault=None):
        return oracle.latent_attention(h.double(), W, "", mixer, 1e-4, fault)[query:]

    want = ref()
    assert rel(ref(("lost", target)), want) > 0.3
    for prompt_len in (n, query):
        got = run_attention(w, h, mixer, dev, dt, 1e-4, prompt_len, max_len=192)[query:]
        close(got, want, dt)


def test_faults_would_show():
    """The tolerance separates right from wrong for each planted mistake."""
    ids = ids_of("mixed", 20)
    for fault in (("lost", 0), ("lost", "own"), "latent_not_normed", "key_not_rotated"):
        bad = oracle.forward(ids, weights("mixed"), ALL["mixed"], fault=fault)
        assert rel(bad, want_logits("mixed", ids)) > 5 * TOL["bfloat16"], fault


@pytest.mark.gpu
@pytest.mark.parametrize("splits", [1, 2, 3, 7, 33, 64])
@pytest.mark.parametrize("heads,rank,rot", [(5, 64, 32), (16, 200, 6), (33, 512, 64), (70, 96, 96)])
@torch.no_grad()
def test_decode_attention_splits(splits, heads, rank, rot):
    """Any number of splits, many tiles per split, empty splits, rows of
    different lengths in scattered slots; rows beyond a length are poison."""
    from automodel_amd.ops._backend import hip_ops

    g = torch.Generator().manual_seed(splits)
    lens, slots, n_slots, max_len = [1, 63, 64, 65, 500, 640, 321], [6, 0, 3, 8, 2, 7, 1], 9, 640
    RP, C = la.pad32(rank), la.pad32(rank) + la.pad32(rot)
    cache = torch.full((n_slots, max_len, C), 1e4).bfloat16()
    q = torch.zeros(len(lens), heads, C).bfloat16()
    q[:, :, :rank] = torch.randn(len(lens), heads, rank, generator=g).bfloat16()
    q[:, :, RP:RP + rot] = torch.randn(len(lens), heads, rot, generator=g).bfloat16()
    for s, n in zip(slots, lens):
        cache[s, :n] = torch.randn(n, C, generator=g).bfloat16()
    scale = 1.5 * (rank + rot) ** -0.5
    w_uv = torch.randn(heads * 12, rank, generator=g).bfloat16() / rank ** 0.5
    pos = torch.tensor(lens, dtype=torch.int32, device="cuda") - 1
    slot = torch.tensor(slots, dtype=torch.int32, device="cuda")
    part, ml = hip_ops().latent_decode_attn(q.cuda(), cache.cuda(), slot, pos, rank, rot, scale,
                                            splits)
    got = hip_ops().latent_decode_combine(part, ml, w_uv.cuda(), 12)
    want = []
    for r, (s, n) in enumerate(zip(slots, lens)):
        k = cache[s, :n].double()
        p = torch.softmax(q[r].double() @ k.T * scale, -1)
        o = p @ k[:, :rank]
        want.append(torch.einsum("hr,hvr->hv", o, w_uv.double().view(heads, 12, rank)).reshape(-1))
    close(got, torch.stack(want), "bfloat16")


@pytest.mark.gpu
@pytest.mark.parametrize("rows", [1, 3, 4, 5, 16, 17, 32, 33, 64])
@pytest.mark.parametrize("n,k", [(16, 8), (50, 72), (1000, 192), (129, 2048), (257, 4168)])
@pytest.mark.parametrize("relu2,f32", [(False, False), (True, False), (False, True)])
@torch.no_grad()
def test_decode_projection(rows, n, k, relu2, f32):
    from automodel_amd.serving.decode_linear import project

    g = torch.Generator().manual_seed(rows + n)
    lin = torch.nn.Linear(k, n, bias=False)
    lin.weight.data = torch.randn(n, k, generator=g) / k ** 0.5
    lin = lin.bfloat16()
    x = torch.randn(rows, k, generator=g).bfloat16()
    want = x.double() @ lin.weight.double().T
    want = oracle.relu_squared(want) if relu2 else want
    got = project(lin.cuda(), x.cuda(), relu2, f32)
    assert got.dtype == (torch.float32 if f32 else torch.bfloat16)
    assert rel(got, want) < (1e-5 if f32 else 6e-3)


@on_each
@torch.no_grad()
def test_far_positions_rotate_exactly(dev, dt):
    """Angles at large positions: scores depend on position differences only."""
    cos, sin = la.rope_half_tables(8, 40000, 500.0, dev)
    p = torch.tensor([39999])
    x = torch.randn(1, 8, dtype=torch.float64, generator=torch.Generator().manual_seed(3))
    got = la._rotate(x.float().to(dev), cos[p.to(dev)], sin[p.to(dev)])
    assert rel(got, oracle.rotate(x, p, 500.0)) < 1e-6


# ---------------------------------------------------------------- whole model
@on_each
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_prompt(model_of, dev, dt, name):
    ids = ids_of(name, 33)
    close(whole(model_of(name, dev, dt), [ids]), want_logits(name, ids), dt)


@on_each
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_decode_from_the_first_token(model_of, dev, dt, name):
    ids = ids_of(name, 33)
    close(by_parts(model_of(name, dev, dt), ids, 1), want_logits(name, ids), dt)


@on_each
@pytest.mark.parametrize("first", [2, 3, 17, 63, 64, 65, 69])
def test_prompt_then_decode(model_of, dev, dt, first):
    ids = ids_of("mixed", 70, seed=2)
    close(by_parts(model_of("mixed", dev, dt), ids, first), want_logits("mixed", ids), dt)


@pytest.mark.gpu
@pytest.mark.parametrize("dt", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(BIG))
@pytest.mark.parametrize("first", [1, 40, 130])
def test_large_sizes(model_of, dt, name, first):
    ids = ids_of(name, 130, seed=4)
    close(by_parts(model_of(name, "cuda", dt), ids, first), want_logits(name, ids), dt)


@on_each
def test_first_tokens(model_of, dev, dt):
    m = model_of("mixed", dev, dt)
    for n in (1, 2):
        ids = ids_of("mixed", n, seed=n)
        close(whole(m, [ids]), want_logits("mixed", ids), dt)


@on_each
def test_long_decode(model_of, dev, dt):
    """Decoding far past the prompt, over several key tiles, equals the prompt
    path over the same tokens (and the oracle at the end)."""
    n = 90 if dev == "cpu" else 300
    ids = ids_of("once", n, seed=6)
    m = model_of("once", dev, dt)
    a, b = by_parts(m, ids, 4, max_len=512), whole(m, [ids])
    close(a, b.cpu(), dt)
    close(a[:90], want_logits("once", ids[:90]), dt)


@on_each
@pytest.mark.parametrize("name", ["mixed", "wide"])
def test_unequal_batch_equals_each_alone(model_of, dev, dt, name):
    m = model_of(name, dev, dt)
    lens = [1, 5, 33, 2, 64, 19]
    seqs = [ids_of(name, n + 6, seed=10 + i) for i, n in enumerate(lens)]
    s = DecodeSession(m, 8, 80)
    handles, lg = s.prefill([q[:n] for q, n in zip(seqs, lens)])
    got = [[lg[i]] for i in range(len(lens))]
    for j in range(6):
        lg = s.decode(handles, torch.tensor([q[n + j] for q, n in zip(seqs, lens)],
                                            device=s.device))
        for i in range(len(lens)):
            got[i].append(lg[i])
    for i, (q, n) in enumerate(zip(seqs, lens)):
        close(torch.stack(got[i]), want_logits(name, q)[n - 1:], dt)
        alone = by_parts(m, q, n)[n - 1:]
        close(torch.stack(got[i]), alone.cpu(), dt, 0.5)


@on_each
def test_wanted_places(model_of, dev, dt):
    m = model_of("mixed", dev, dt)
    a, b, c = ids_of("mixed", 9), ids_of("mixed", 4, seed=3), ids_of("mixed", 3, seed=4)
    lg = whole(m, [a, b, c], [[8, 0, 3], [], [1]])
    wa, wc = want_logits("mixed", a), want_logits("mixed", c)
    close(lg, torch.stack([wa[8], wa[0], wa[3], wc[1]]), dt)
    assert whole(m, [a], [[]]).shape == (0, ALL["mixed"]["vocab"])


@on_each
def test_slots_are_given_back_and_used_again(model_of, dev, dt):
    """Shorter sequences leave the batch; a later batch lands in used slots."""
    name, m = "mixed", model_of("mixed", dev, dt)
    s = DecodeSession(m, 3, 48)
    first = [ids_of(name, n, seed=20 + n) for n in (30, 11, 40)]
    h, _ = s.prefill([q[:-2] for q in first])
    lg = s.decode(h, torch.tensor([q[-2] for q in first], device=s.device))
    s.release([h[1]])
    left = [h[0], h[2]]
    lg = s.decode(left, torch.tensor([first[0][-1], first[2][-1]], device=s.device))
    close(lg, torch.stack([want_logits(name, first[0])[-1], want_logits(name, first[2])[-1]]), dt)
    again = ids_of(name, 13, seed=50)
    h2, lg = s.prefill([again[:5]])
    assert h2 == [h[1]]                                  # the slot that was given back
    rows = [lg]
    for t in again[5:]:
        rows.append(s.decode(h2, torch.tensor([t], device=s.device)))
    close(torch.cat(rows), want_logits(name, again)[4:], dt)
    s.release(left + h2)
    assert s.cache.lens == [0, 0, 0] and s.live == []
    h3, lg = s.prefill([ids_of(name, n, seed=60 + n) for n in (7, 2, 21)])
    assert sorted(h3) == sorted(h)
    close(lg, torch.stack([want_logits(name, ids_of(name, n, seed=60 + n))[-1]
                           for n in (7, 2, 21)]), dt)


def test_cache_limits(model_of):
    m = model_of("mixed", "cpu", "float32")
    s = DecodeSession(m, 1, 4)
    h, _ = s.prefill([[1, 2, 3]])
    with pytest.raises(RuntimeError):
        s.prefill([[1]])                                 # no slot left
    s.decode(h, torch.tensor([1]))
    with pytest.raises(RuntimeError, match="overflow"):
        s.decode(h, torch.tensor([1]))
    with pytest.raises(ValueError):
        DecodeSession(m, 1, 4).prefill([[1, 2, 3, 4, 5]])


def test_every_pass_has_its_own_cache(model_of):
    m = model_of("mixed", "cpu", "float32")
    cache = DecodeSession(m, 2, 8).cache
    order = oracle.layer_order(ALL["mixed"])
    assert len(cache.rows) == len(order) == 8
    for (i, _), rows in zip(order, cache.rows):
        mx = ALL["mixed"]["layers"][i]["mixer"]
        assert rows.shape == (2, 8, la.pad32(mx["kv_rank"]) + la.pad32(mx["rot_dim"]))


# ---------------------------------------------------------------- generation
def _decided(name, prompt, n):
    """Greedy continuation by the oracle (the configs leave no near-ties)."""
    return oracle.greedy(prompt, n, weights(name), ALL[name])[len(prompt):]


@pytest.mark.parametrize("dev", ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)])
def test_greedy_generation(model_of, dev):
    """Every entry point, float32, against the oracle's greedy tokens."""
    from automodel_amd.utils.generation import (
        generate,
        generate_batch,
        generate_cached,
        generate_graphed,
    )

    m = model_of("mixed", dev, "float32")
    prompts = [ids_of("mixed", n, seed=70 + n) for n in (6, 3, 11, 6, 1)]
    want = [_decided("mixed", p, 7) for p in prompts]
    assert generate_batch(m, prompts, 7, max_batch=2) == want
    assert generate_batch(m, prompts, 7) == want
    pair = torch.tensor([prompts[0], prompts[3]], device=dev)
    both = torch.tensor([prompts[0] + want[0], prompts[3] + want[3]])
    for f in (generate, generate_cached, generate_graphed):
        assert torch.equal(f(m, pair, 7).cpu(), both), f.__name__
    stop = want[0][2]
    ended = generate_batch(m, prompts, 7, eos_token_id=stop)
    for got, full in zip(ended, want):
        cut = full.index(stop) + 1 if stop in full else len(full)
        assert got == full[:cut]
    torch.manual_seed(0)
    sampled = generate_batch(m, prompts, 5, temperature=1.0)
    assert all(len(s) == 5 for s in sampled)


@pytest.mark.gpu
@pytest.mark.parametrize("dt", ["float32", "bfloat16"])
@pytest.mark.parametrize("batch", [1, 3, 6])
@torch.no_grad()
def test_captured_step_replays_like_eager(model_of, dt, batch):
    """Each replay of the captured step, with eager work in between, gives the
    eager step's tokens and cache rows."""
    from automodel_amd.utils.generation import _GraphStep
    from automodel_amd.utils.kv_cache import kv_cache_context

    m = model_of("wide", "cuda", dt)
    prompts = [ids_of("wide", 40, seed=80 + i) for i in range(batch)]
    runs = []
    for graphed in (False, True):
        s = DecodeSession(m, batch, 64)
        h, lg = s.prefill(prompts)
        toks = []
        with kv_cache_context(s.cache):
            step = fn = _GraphStep(s, h, lg.argmax(-1, keepdim=True))
            for i in range(8):
                if graphed and i == 2:
                    g = torch.cuda.CUDAGraph()
                    torch.cuda.synchronize()
                    with torch.cuda.graph(g):
                        step()
                    fn = g.replay
                fn()
                toks.append(step.ids.clone())
                torch.cuda.synchronize()
                float(torch.randn(64, 64, device="cuda").sum())
        runs.append((torch.stack(toks), [r.clone() for r in s.cache.rows]))
    assert torch.equal(runs[0][0], runs[1][0])
    for a, b in zip(runs[0][1], runs[1][1]):
        assert torch.equal(a, b)


def test_command_line_generate(checkpoints, model_of, capsys):
    from automodel_amd.cli.app import main

    prompts = [ids_of("mixed", n, seed=70 + n) for n in (6, 3)]
    argv = ["generate", "--model", checkpoints("mixed"), "--dtype", "float32",
            "--max-new-tokens", "4"]
    for p in prompts:
        argv += ["--prompt-ids", ",".join(map(str, p))]
    main(argv)
    recs = [json.loads(x) for x in capsys.readouterr().out.splitlines() if x.startswith("{")]
    assert [r["output_ids"] for r in recs] == [_decided("mixed", p, 4) for p in prompts]


def test_server_batch(model_of):
    fastapi = pytest.importorskip("fastapi.testclient")
    from automodel_amd.serving.server import build_app

    c = fastapi.TestClient(build_app(model_of("mixed", "cpu", "float32"), None))
    prompts = [ids_of("mixed", n, seed=70 + n) for n in (6, 3)]
    r = c.post("/generate", json={"batch_prompt_ids": prompts, "max_new_tokens": 4}).json()
    assert r["output_ids"] == [_decided("mixed", p, 4) for p in prompts]
    r = c.post("/generate", json={"prompt_ids": prompts[1], "max_new_tokens": 4}).json()
    assert r["output_ids"] == _decided("mixed", prompts[1], 4)


# ---------------------------------------------------------------- replay
def _trace(name):
    a, b, c = (ids_of(name, n, seed=90 + n) for n in (12, 4, 7))
    yield {"step": 0, "entries": [{"id": "a", "tokens": a[:9], "want": [0, 8]},
                                  {"id": "b", "tokens": b[:2], "want": []}], "end": []}, \
        [(a, 0), (a, 8)]
    yield {"step": 1, "entries": [{"id": "b", "tokens": [b[2]], "want": [0]},
                                  {"id": "a", "tokens": [a[9]], "want": []}], "end": ["b"]}, \
        [(b, 2)]
    yield {"step": 2, "entries": [{"id": "a", "tokens": [a[10]], "want": [0]}], "end": []}, \
        [(a, 10)]
    yield {"step": 3, "entries": [{"id": "a", "tokens": [a[11]], "want": []}], "end": ["a"]}, []
    yield {"step": 7, "entries": [{"id": i, "tokens": c[:n], "want": [n - 1]}
                                  for i, n in (("a", 7), ("x", 1), ("y", 3))],
           "end": ["a", "x", "y"]}, [(c, 6), (c, 0), (c, 2)]


def test_replay_steps(model_of):
    from automodel_amd.serving.trace import TraceReplay

    r = TraceReplay(model_of("mixed", "cpu", "float32"), 32)
    for req, places in _trace("mixed"):
        lg = r.step(req["entries"], req["end"])
        if places:
            close(lg, torch.stack([want_logits("mixed", s)[i] for s, i in places]), "float32")
    assert not r.handles
    r.step([{"id": "a", "tokens": [1], "want": []}], [])
    with pytest.raises(ValueError):
        r.step([{"id": "a", "tokens": [1], "want": []}, {"id": "b", "tokens": [1], "want": []}], [])


@pytest.mark.gpu
@pytest.mark.parametrize("dt", ["float32", "bfloat16"])
def test_replay_program(checkpoints, tmp_path, monkeypatch, capsys, dt):
    from automodel_amd.serving.trace import main

    reqs = list(_trace("mixed"))
    monkeypatch.setattr(sys, "stdin", io.StringIO("\n".join(json.dumps(r) for r, _ in reqs)))
    assert main(["--model", checkpoints("mixed"), "--dtype", dt, "--out", str(tmp_path),
                 "--max-tokens", "32"]) == 0
    done = [x for x in capsys.readouterr().out.splitlines() if x.startswith("done ")]
    assert done == [f"done {r['step']}" for r, _ in reqs]
    for r, places in reqs:
        f = tmp_path / f"{r['step']}.f32"
        assert f.exists() == bool(places)
        if places:
            lg = torch.frombuffer(bytearray(f.read_bytes()), dtype=torch.float32)
            close(lg.view(len(places), -1),
                  torch.stack([want_logits("mixed", s)[i] for s, i in places]), dt)


def test_replay_needs_a_gpu(checkpoints, tmp_path):
    if torch.cuda.is_available():
        pytest.skip("GPU present")
    from automodel_amd.serving.trace import main

    with pytest.raises(RuntimeError, match="GPU"):
        main(["--model", checkpoints("mixed"), "--out", str(tmp_path), "--max-tokens", "8"])
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    assert os.access(os.path.join(root, "bin", "trace_run"), os.X_OK)


# ---------------------------------------------------------------- integration
def test_checkpoint_names_round_trip(model_of):
    for name in CONFIGS:
        m = model_of(name, "cpu", "float32")
        raw = make_weights(ALL[name], seed=len(name))
        back = m.state_dict_adapter.to_hf(m.state_dict())
        assert set(back) == set(raw)
        for k in raw:
            assert torch.equal(back[k], raw[k].float()), k
        params = dict(m.named_parameters())
        for k in raw:
            assert all(t in params for t in m.state_dict_adapter.hf_key_targets(k)), k


def test_missing_weight_is_an_error(checkpoints, tmp_path):
    from safetensors.torch import save_file

    w = make_weights(ALL["mixed"])
    del w["l2.mix.uv"]
    (tmp_path / "config.json").write_text(json.dumps(ALL["mixed"]))
    save_file(w, str(tmp_path / "model.safetensors"))
    with pytest.raises(RuntimeError, match="mismatch"):
        load_pretrained(str(tmp_path), dtype="float32", device="cpu")


def test_unknown_parts_are_refused():
    from automodel_amd.models.rezadra.model import RezadraConfig

    for bad in ({"type": "other"}, {"mlp": {"kind": "moe", "ff": 8}},
                {"mixer": {**make_layer()["mixer"], "rot": {"base": 10.0, "dims": 4}}}):
        with pytest.raises(ValueError):
            RezadraConfig.from_hf_config(make_config(layers=[{**make_layer(), **bad}]))


@pytest.mark.parametrize("dev,dt", [("cpu", "float32"),
                                    pytest.param("cuda", "bfloat16", marks=pytest.mark.gpu)])
def test_training_forward_and_gradients(model_of, dev, dt):
    """The same module trains: its recorded forward equals the oracle, and on
    the CPU so do the gradients."""
    m = model_of("mixed", dev, dt)
    ids = torch.tensor([ids_of("mixed", 12), ids_of("mixed", 12, seed=5)], device=dev)
    with torch.enable_grad():
        logits = m(ids)
        for b in range(2):
            close(logits[b], want_logits("mixed", ids[b].tolist()), dt)
        m.zero_grad()
        torch.nn.functional.cross_entropy(logits[0, :-1].float(), ids[0, 1:]).backward()
    grads = m.state_dict_adapter.to_hf({k: p.grad for k, p in m.named_parameters()})
    m.zero_grad()
    assert all(torch.isfinite(g).all() for g in grads.values())
    w = {k: v.requires_grad_() for k, v in weights("mixed").items()}
    ref = oracle.forward(ids[0].tolist(), w, ALL["mixed"])
    torch.nn.functional.cross_entropy(ref[:-1], ids[0, 1:].cpu()).backward()
    for k in ("l1.mix.uk", "l2.mlp.down", "loop.in", "embed", "l0.mix.dkv.norm"):
        e = (grads[k].double().cpu() - w[k].grad).norm() / w[k].grad.norm()
        assert e < (1e-4 if dt == "float32" else 0.1), (k, float(e))
