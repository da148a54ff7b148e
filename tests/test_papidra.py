"""Papidra against a plain implementation (papidra_oracle.py): weights, every
mechanism alone, prompts, decoding, batches, slots, generation.

Each case runs on the CPU (torch expressions) and, marked gpu, on the HIP
kernels in float32 and bfloat16."""

import io
import json
import sys

import pytest
import torch

import papidra_oracle as oracle
from papidra_oracle import make_config, make_parallel, make_weights, make_wkv

from automodel_amd.models.registry import load_pretrained
from automodel_amd.ops import grouped_attention as ga
from automodel_amd.ops import hyper, linear_scan
from automodel_amd.ops.packed_step import PackedStep
from automodel_amd.utils.generation import DecodeSession

PLACES = [
    pytest.param("cpu", "float32", id="cpu-f32"),
    pytest.param("cuda", "float32", id="gpu-f32", marks=pytest.mark.gpu),
    pytest.param("cuda", "bfloat16", id="gpu-bf16", marks=pytest.mark.gpu),
]
on_each = pytest.mark.parametrize("dev,dt", PLACES)
TOL = {"float32": 3e-5, "bfloat16": 4e-2}

CONFIGS = {
    # both mixers, with and without feed-forward, every layer of other sizes
    "mixed": make_config(streams=2, layers=[
        make_parallel(), make_wkv(), make_wkv(heads=2, dim=24, ff=32),
        make_parallel(heads=3, kv_heads=3, dim=24, vdim=8, dims=8, size=7, scaling=None,
                      ssm_heads=2, ssm_vdim=20, state=9, groups=1, norm_groups=4, conv=2, ff=None),
        make_parallel(heads=8, kv_heads=1, dim=8, vdim=40, size=32, base=50.0, ssm_heads=6,
                      ssm_vdim=4, state=40, groups=3, norm_groups=1, conv=3, limit=0.4)]),
    # sizes that are no multiples of 4 or 8; one tap, one stream
    "odd": make_config(vocab=37, width=30, streams=1, eps=1e-3, layers=[
        make_wkv(heads=2, dim=7, ff=17),
        make_parallel(heads=6, kv_heads=2, dim=10, vdim=7, dims=6, size=5, ssm_heads=3,
                      ssm_vdim=5, state=3, groups=3, norm_groups=5, conv=1, ff=19),
        make_parallel(heads=2, kv_heads=2, dim=6, vdim=9, size=1, ssm_heads=1, ssm_vdim=21,
                      state=17, groups=1, norm_groups=3, conv=6, ff=18)]),
    # one layer of one kind; three streams
    "attention-last": make_config(width=64, streams=3, layers=[
        make_parallel(heads=16, kv_heads=4, dim=32, vdim=32, size=33, ssm_heads=4, ssm_vdim=16,
                      state=32, groups=2, norm_groups=2, conv=4, ff=None)]),
    "wkv-only": make_config(width=64, streams=5, layers=[make_wkv(heads=2, dim=32),
                                                         make_wkv(heads=4, dim=64, ff=64)]),
}
BIG = {
    # the head sizes of large models; more query heads per group than an MFMA tile
    "large-heads": make_config(vocab=128, width=256, streams=4, layers=[
        make_parallel(heads=20, kv_heads=1, dim=128, vdim=128, dims=64, size=64, ssm_heads=4,
                      ssm_vdim=64, state=128, groups=2, norm_groups=2, ff=512),
        make_wkv(heads=4, dim=64, ff=128)]),
    # beyond the MFMA attention kernels; large states; wide values, many streams
    "row-kernel": make_config(vocab=64, width=64, streams=9, layers=[
        make_parallel(heads=2, kv_heads=1, dim=264, vdim=40, dims=24, size=50, ssm_heads=2,
                      ssm_vdim=72, state=200, groups=1, norm_groups=1, conv=4, ff=64),
        make_wkv(heads=1, dim=144),
        make_parallel(heads=4, kv_heads=2, dim=72, vdim=200, size=90, ssm_heads=1, ssm_vdim=136,
                      state=72, groups=1, norm_groups=2, conv=5, ff=64)]),
}
ALL = {**CONFIGS, **BIG}

_models: dict = {}


@pytest.fixture(scope="session")
def checkpoints(tmp_path_factory):
    from safetensors.torch import save_file

    root = tmp_path_factory.mktemp("papidra")

    def get(name):
        path = root / name
        if not path.exists():
            path.mkdir()
            (path / "config.json").write_text(json.dumps(ALL[name]))
            save_file(raw_weights(name), str(path / "model.safetensors"))
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


def raw_weights(name):
    return make_weights(ALL[name], seed=len(name), rank=20 if name == "odd" else 12)


def weights(name, dtype=torch.float64):
    return {k: v.to(dtype) for k, v in raw_weights(name).items()}


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


def randn(*shape, seed=0, std=1.0):
    return std * torch.randn(*shape, generator=torch.Generator().manual_seed(seed))


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


def decode_step(pos, slots, dev):
    i32 = dict(dtype=torch.int32, device=dev)
    return PackedStep(torch.tensor(pos, **i32), torch.tensor(slots, **i32), prompt=False)


# ---------------------------------------------------------------- hyper-connections
@on_each
@pytest.mark.parametrize("streams", [1, 2, 3, 4, 7, 16])
@pytest.mark.parametrize("width", [64, 30, 7, 4096])
@torch.no_grad()
def test_hyper_connections(dev, dt, streams, width):
    dtype, eps, T = getattr(torch, dt), 1e-2, 5
    r = [randn(*s, seed=i).to(dtype) for i, s in enumerate(
        [(11, width), (streams,), (width,), (streams, streams), (streams,), (streams,), (width,),
         (T, width), (T, width), (width,), (width,)])]
    table, w_in, n1, mix, out, w_in2, n2, ya, yb, wa, wb = r
    ids = torch.tensor([3, 10, 0, 3, 7])
    d = [t.to(dev) for t in r]
    f = [t.double() for t in r]
    x, h = hyper.hyper_embed(ids.to(dev), d[0], 2.5, d[1], d[2], eps)
    assert x.dtype == torch.float32 and h.dtype == dtype and x.shape == (T, streams, width)
    xs = [f[0][ids] * 2.5] * streams
    assert rel(x, torch.stack(xs, 1)) < 1e-6
    close(h, oracle.rms(oracle.streams_in(xs, f[1]), f[2], eps), dt)
    x = x + randn(T, streams, width, seed=99).to(dev)          # streams that differ
    xs = list(x.double().cpu().unbind(1))
    # one output, then two branches
    for pair in (False, True):
        y = f[7]
        if pair:
            y = 0.5 * (oracle.rms(f[7], f[9], eps) + oracle.rms(f[8], f[10], eps))
        want = oracle.streams_out(xs, y, f[3], f[4])
        if streams > 1:
            assert rel(torch.stack(want, 1),
                       torch.stack(oracle.streams_out(xs, y, f[3], f[4], "mix_transposed"),
                                   1)) > 0.05
        given = hyper.NormedPair(d[7], d[8], d[9], d[10]) if pair else d[7]
        x2, h2 = hyper.hyper_step(x.clone(), given, d[3], d[4], d[5], d[6], eps)
        assert x2.dtype == torch.float32
        assert rel(x2, torch.stack(want, 1)) < 2e-6            # 32-bit sums
        close(h2, oracle.rms(oracle.streams_in(want, f[5]), f[6], eps), dt)
        _, h3 = hyper.hyper_step(x.clone(), given, d[3], d[4], None, d[6], eps, keep=False)
        close(h3, oracle.rms(sum(want), f[6], eps), dt)


@on_each
@pytest.mark.parametrize("rows,ff", [(3, 40), (5, 7), (70, 1024)])
@torch.no_grad()
def test_clamped_glu(dev, dt, rows, ff):
    gu = randn(rows, 2 * ff, std=2.0).to(getattr(torch, dt))
    limit = 1.25
    g, u = gu.double().split(ff, -1)
    assert (g > limit).any() and (u > limit).any() and (u < -limit).any()
    eye = {"gate": torch.eye(2 * ff)[:ff], "up": torch.eye(2 * ff)[ff:], "down": torch.eye(ff)}
    want = oracle.clamped_glu(gu.double(), {k: v.double() for k, v in eye.items()}, "", limit)
    close(hyper.clamped_glu(gu.to(dev), limit), want, dt)


# ---------------------------------------------------------------- attention
def spec_of(m):
    from automodel_amd.models.papidra.model import PapidraConfig

    cfg = make_config(layers=[{"type": "parallel", "mixer": {**make_parallel()["mixer"], "left": m},
                               "mlp": None}])
    return PapidraConfig.from_hf_config(cfg).attention_spec(0)


ROTATIONS = [dict(dims=16, scaling=None), dict(dims=8, scaling=(4.0, 32.0, 256, 1.0)),
             dict(dims=16, scaling=(1.0, 32.0, 256, 1.0)), dict(dims=16, scaling=(8., 2., 64, 2.)),
             dict(dims=64, base=500000.0, scaling=(2.5, 1000.0, 4096, 0.01))]


@pytest.mark.parametrize("kw", ROTATIONS)
def test_rotation_frequencies(kw):
    m = make_parallel(dim=64, **kw)["mixer"]["left"]
    cos, sin = spec_of(m).rope_tables(3000, "cpu")
    x = torch.zeros(1, 64, dtype=torch.float64)
    x[0, :kw["dims"] // 2] = 1.0
    for p in (0, 1, 77, 2999):
        y = oracle.rotate(x, torch.tensor([p]), m["rot"])[0]
        half = kw["dims"] // 2
        assert torch.allclose(cos[p].double(), y[:half], atol=1e-6)
        assert torch.allclose(sin[p].double(), y[half:2 * half], atol=1e-6)


def attention_case(m, n, seed=0):
    cfg = make_config(width=48, layers=[{"type": "parallel", "mlp": None,
                                         "mixer": {**make_parallel()["mixer"], "left": m}}])
    p = "l0.mix.left."
    w = {k[len(p):]: v for k, v in make_weights(cfg, seed).items() if k.startswith(p)}
    return w, randn(n, 48, seed=seed + 1).bfloat16()


def run_attention(w, h, m, dev, dt, prompt_len, slot=0, n_slots=2, max_len=None, extra=8):
    """The op's two paths: the first ``prompt_len`` tokens as a prompt, the
    rest as one-token steps. ``extra`` columns follow in the projection."""
    dtype, n, spec = getattr(torch, dt), h.shape[0], spec_of(m)
    W = {k: v.to(dev, dtype) for k, v in w.items()}
    max_len = max_len or n
    proj = torch.nn.functional.linear(h.to(dev, dtype), torch.cat([W["q"], W["k"], W["v"]]))
    proj = torch.nn.functional.pad(proj, (0, extra), value=9.0)
    rope = spec.rope_tables(max_len, dev)
    state = spec.make_state(n_slots, max_len, dev, dtype)
    out = []
    if prompt_len:
        step = PackedStep.for_prompts([prompt_len], dev, [slot])
        out.append(ga.grouped_attention_prompt(proj[:prompt_len], W["sink"], spec, rope, step,
                                               state))
    for i in range(prompt_len, n):
        out.append(ga.grouped_attention_decode(proj[i:i + 1], W["sink"], spec, rope,
                                               decode_step([i], [slot], dev), state))
    for t in state.values():
        assert not t[[s for s in range(n_slots) if s != slot]].any()     # own slot only
    return torch.nn.functional.linear(torch.cat(out), W["o"])


def left(**kw):
    return make_parallel(**kw)["mixer"]["left"]


ATTENTIONS = {
    "grouped": left(heads=6, kv_heads=2, dim=16, vdim=24, size=40),
    "one chunk": left(heads=4, kv_heads=4, dim=32, vdim=32, size=1000),
    "odd": left(heads=2, kv_heads=1, dim=9, vdim=5, dims=4, size=17, scaling=None),
    "large": left(heads=24, kv_heads=1, dim=128, vdim=128, dims=32, size=32),
    "values wider": left(heads=4, kv_heads=2, dim=24, vdim=160, size=64),
    "keys wider": left(heads=2, kv_heads=2, dim=256, vdim=16, size=33),
    "beyond": left(heads=2, kv_heads=1, dim=40, vdim=272, size=48),
}


@on_each
@pytest.mark.parametrize("name", sorted(ATTENTIONS))
@pytest.mark.parametrize("prompt_len", [70, 0, 65])
@torch.no_grad()
def test_attention_alone(dev, dt, name, prompt_len):
    m = ATTENTIONS[name]
    w, h = attention_case(m, 70)
    want = oracle.chunked_attention(h.double(), {k: v.double() for k, v in w.items()}, "", m)
    close(run_attention(w, h, m, dev, dt, prompt_len, slot=1, max_len=200), want, dt)


SIZE = 40
EDGES = [(0, 1), (0, 0), (0, 39), (39, 39), (40, 41), (40, 79), (79, 79), (80, 80), (80, 119),
         (31, 32), (72, 79), (120, 124)]
OUTSIDE = [(39, 40), (79, 80), (0, 40), (39, 79), (80, 120)]


def stand_out(target, query, n):
    """The query's score with one key is far above its others."""
    m = left(heads=2, kv_heads=1, dim=16, vdim=16, size=SIZE, base=10.0, dims=4)
    w, h = attention_case(m, n, seed=5)
    h = (h.float() * 0.5)
    W = {k: v.double() for k, v in w.items()}
    k = oracle.rotate((h[target].double() @ W["k"].T).view(1, 1, 16), torch.tensor([target]),
                      m["rot"])[0, 0]
    k[:4] = 0                                     # the unrotated part alone
    if target != query:
        goal = torch.cat([k * 6.0, k * 6.0, torch.zeros(16, dtype=k.dtype)])   # own key: none
        h[query] = (torch.linalg.pinv(torch.cat([W["q"], W["k"]])) @ goal).float()
    w["sink"][:] = 3.0
    return m, w, h.bfloat16()


@on_each
@pytest.mark.parametrize("target,query", EDGES + OUTSIDE)
@torch.no_grad()
def test_one_key_stands_out(dev, dt, target, query):
    """Just inside and just outside a chunk, at the first key, at the query's own
    key: prompts and decoding agree with the plain form, and a mistake would show."""
    n = query + 1
    m, w, h = stand_out(target, query, n)
    W = {k: v.double() for k, v in w.items()}

    def ref(fault=None):
        return oracle.chunked_attention(h.double(), W, "", m, fault)[query:]

    want = ref()
    if query == target:
        assert rel(ref("no_sink"), want) > 0.05 or n == 1
    elif (target, query) in EDGES:
        assert rel(ref(("lost", target)), want) > 0.3
        if target % SIZE == 0:
            assert rel(ref("edge_in"), want) > 0.3
    elif target % SIZE == SIZE - 1 and target + 1 == query // SIZE * SIZE:
        assert rel(ref("edge_out"), want) > 0.3
    for prompt_len in {n, query}:
        close(run_attention(w, h, m, dev, dt, prompt_len, max_len=192)[query:], want, dt)


@on_each
@pytest.mark.parametrize("sink", [-30.0, 0.0, 6.0, 60.0])
@torch.no_grad()
def test_sinks(dev, dt, sink):
    """One sink per head: absent, moderate, dominant, alone."""
    m = ATTENTIONS["grouped"]
    w, h = attention_case(m, 45, seed=3)
    w["sink"][:] = sink
    w["sink"][1] = -sink if abs(sink) < 50 else sink
    W = {k: v.double() for k, v in w.items()}
    want = oracle.chunked_attention(h.double(), W, "", m)
    if sink in (0.0, 6.0):
        assert rel(oracle.chunked_attention(h.double(), W, "", m, "no_sink"), want) > 0.2
    for prompt_len in (45, 20):
        got = run_attention(w, h, m, dev, dt, prompt_len)
        if sink == 60.0:
            assert float(got.abs().max()) < 1e-12          # nothing but the sink
        else:
            close(got, want, dt)


@pytest.mark.gpu
@pytest.mark.parametrize("splits", [1, 2, 3, 7, 33, 64])
@pytest.mark.parametrize("heads,groups,d,dv", [(5, 1, 64, 32), (16, 4, 40, 72), (34, 2, 128, 128),
                                               (8, 8, 256, 200)])
@torch.no_grad()
def test_decode_attention_splits(splits, heads, groups, d, dv):
    """Any number of splits, empty ones too; rows of different lengths in
    scattered slots; keys beyond a row's chunk position are poison."""
    from automodel_amd.ops._backend import hip_ops

    chunk, n_slots = 320, 9
    lens, slots = [1, 32, 33, 319, 320, 321, 1000], [6, 0, 3, 8, 2, 7, 1]
    spec = ga.GroupedAttentionSpec(heads, groups, d, dv, 1.5 * d ** -0.5, 0, chunk=chunk)
    state = spec.make_state(n_slots, chunk, "cuda", torch.bfloat16)
    state["k"].fill_(1e4), state["v"].fill_(1e4)
    state["k"][..., d:] = 0
    rope = spec.rope_tables(2000, "cuda")
    sink = randn(heads, seed=7).bfloat16()
    proj = randn(1000, spec.in_width, seed=splits).bfloat16()
    q, k, v = proj.double().split([heads * d, groups * d, groups * dv], -1)
    rows, want = [], []
    for s, n in zip(slots, lens):
        first = (n - 1) // chunk * chunk                  # earlier chunks leave no trace
        for p in range(first, n - 1):
            hip_ops().gqa_prep(proj[p:p + 1].cuda(), *rope, *_at(p, s), None, None, state["k"],
                               state["v"], chunk, heads, groups, d, dv, state["k"].shape[3], dv,
                               1, True)
        rows.append(proj[n - 1])
        kk, vv = k[first:n].view(-1, groups, d), v[first:n].view(-1, groups, dv)
        out = []
        for a in range(heads):
            sc = kk[:, a // (heads // groups)] @ q[n - 1].view(heads, d)[a] * spec.scale
            sc = torch.cat([sc, sink[a:a + 1].double()])
            out.append(torch.softmax(sc, -1)[:-1] @ vv[:, a // (heads // groups)])
        want.append(torch.cat(out))
    step = decode_step([n - 1 for n in lens], slots, "cuda")
    qs, _, _ = hip_ops().gqa_prep(torch.stack(rows).cuda(), *rope, step.positions, step.slots, None,
                                  None, state["k"], state["v"], chunk, heads, groups, d, dv,
                                  state["k"].shape[3], dv, len(lens), True)
    got = hip_ops().gqa_decode_attn(qs, state["k"], state["v"], step.slots, step.positions,
                                    sink.cuda(), chunk, dv, spec.scale, splits)
    close(got, torch.stack(want), "bfloat16")


def _at(p, s):
    step = decode_step([p], [s], "cuda")
    return step.positions, step.slots


# ---------------------------------------------------------------- recurrences
LENS = [1, 2, 15, 16, 17, 33, 50]


def in_parts(run, lens, cut, dev, slots=None):
    """``run(rows, step)`` over packed prompts cut short, then one token at a
    time for those that go on; -> outputs per sequence."""
    slots = slots or list(range(len(lens)))[::-1]
    starts = [sum(lens[:i]) for i in range(len(lens))]
    first = [min(n, cut) for n in lens]
    rows = torch.cat([torch.arange(s, s + f) for s, f in zip(starts, first)])
    out = run(rows, PackedStep.for_prompts(first, dev, slots))
    got = [[o] for o in out.split(first)]
    for p in range(cut, max(lens)):
        on = [i for i, n in enumerate(lens) if n > p]
        o = run(torch.tensor([starts[i] + p for i in on]),
                decode_step([p] * len(on), [slots[i] for i in on], dev))
        for j, i in enumerate(on):
            got[i].append(o[j:j + 1])
    return [torch.cat(g) for g in got]


@on_each
@pytest.mark.parametrize("taps", [1, 2, 3, 4, 7])
@pytest.mark.parametrize("cut", [1, 3, 50])
@torch.no_grad()
def test_short_convolution(dev, dt, taps, cut):
    dtype, C = getattr(torch, dt), 24
    x = randn(sum(LENS), C + 5, seed=1).to(dtype)
    w, b = randn(C, taps, seed=2).to(dtype), randn(C, seed=3).to(dtype)
    state = torch.full((len(LENS), taps - 1, C), 50.0, dtype=dtype, device=dev)   # stale
    wd, bd, xd = w.to(dev), b.to(dev), x.to(dev)
    got = in_parts(lambda rows, step: linear_scan.causal_conv_silu(
        xd[rows.to(dev)][:, 5:], wd, bd, step, state), LENS, cut, dev)
    for g, xs in zip(got, x.split(LENS)):
        close(g, oracle.causal_conv(xs[:, 5:].double(), w.double(), b.double()), dt)


@on_each
@pytest.mark.parametrize("width", [24, 7])
@pytest.mark.parametrize("cut", [1, 3, 50])
@torch.no_grad()
def test_token_shift(dev, dt, width, cut):
    dtype = getattr(torch, dt)
    h, mu = randn(sum(LENS), width).to(dtype), randn(5, width, seed=2).to(dtype)
    state = torch.full((len(LENS), width), 50.0, dtype=dtype, device=dev)
    got = in_parts(lambda rows, step: linear_scan.token_shift(
        h.to(dev)[rows.to(dev)], mu.to(dev), step, state).transpose(0, 1).flatten(1),
        LENS, cut, dev)
    for g, hs in zip(got, h.double().split(LENS)):
        want = torch.cat([oracle.token_mix(hs, m) for m in mu.double()], -1)
        close(g, want, dt)


@on_each
@pytest.mark.parametrize("groups,size,first", [(3, 8, True), (1, 700, True), (5, 7, False),
                                               (4, 64, False), (2, 1024, True)])
@torch.no_grad()
def test_gated_group_norm(dev, dt, groups, size, first):
    dtype, n = getattr(torch, dt), groups * size
    y, zz, w = randn(6, n).to(dtype), randn(6, n + 8, seed=1).to(dtype), randn(n, seed=2).to(dtype)
    got = linear_scan.gated_group_norm(y.to(dev), zz.to(dev)[:, 8:], w.to(dev), groups, 1e-2, first)
    yd, z, wd = y.double(), zz.double()[:, 8:], w.double()
    if first:
        want = oracle.gated_group_norm(yd, z, wd, groups, 1e-2)
    else:
        want = oracle.unit_rms(yd.view(6, groups, size), 1e-2).reshape(6, n) * wd * oracle.silu(z)
    close(got, want, dt)


@on_each
@pytest.mark.parametrize("H,P,N,G", [(4, 8, 16, 2), (3, 5, 7, 1), (2, 64, 128, 2), (1, 136, 200, 1),
                                     (6, 20, 40, 3)])
@pytest.mark.parametrize("cut", [1, 16, 50])
@torch.no_grad()
def test_state_space_recurrence(dev, dt, H, P, N, G, cut):
    """Heads that forget at once, slowly and hardly at all."""
    dtype, T = getattr(torch, dt), sum(LENS)
    xbc = randn(T, H * P + 2 * G * N, seed=H).to(dtype)
    dt_in, dt_bias = randn(T, H + 3, seed=2, std=2.0).to(dtype), randn(H, seed=3).to(dtype)
    a_log = torch.linspace(-6, 4, H).to(dtype)
    D = randn(H, seed=5).to(dtype)
    state = torch.full((len(LENS), H, N, P), 1e4, device=dev)
    args = [t.to(dev) for t in (dt_bias, a_log, D)]
    got = in_parts(lambda rows, step: linear_scan.ssd_scan(
        xbc.to(dev)[rows.to(dev)], dt_in.to(dev)[rows.to(dev)][:, 3:], *args, G, N, step, state),
        LENS, cut, dev)
    for g, xs, ds in zip(got, xbc.double().split(LENS), dt_in.double().split(LENS)):
        x, B, C = xs.split([H * P, G * N, G * N], -1)
        n = x.shape[0]
        want = oracle.ssd_recurrence(
            x.reshape(n, H, P), B.reshape(n, G, N), C.reshape(n, G, N),
            oracle.softplus(ds[:, 3:] + dt_bias.double()), a_log.double(), D.double())
        close(g, want.reshape(n, H * P), dt, 0.3)


@on_each
@pytest.mark.parametrize("H,n", [(3, 16), (2, 7), (2, 64), (1, 144), (4, 40)])
@pytest.mark.parametrize("cut", [1, 16, 50])
@torch.no_grad()
def test_wkv_recurrence(dev, dt, H, n, cut):
    """Channels that forget at once (log decay -1000), slowly and hardly at all,
    next to one another; norm and gate as decoding fuses them."""
    dtype, T, rank, eps = getattr(torch, dt), sum(LENS), 12, 1e-3
    proj = randn(T, 4 * H * n + rank, seed=n).to(dtype)
    w2 = randn(H * n, rank, seed=2, std=0.3).to(dtype)
    w0 = torch.linspace(-9, 6, H * n)[torch.randperm(
        H * n, generator=torch.Generator().manual_seed(1))].to(dtype)
    u, norm = randn(H, n, seed=3).to(dtype), randn(H * n, seed=4).to(dtype)
    state = torch.full((len(LENS), H, n, n), 1e4, device=dev)
    d = [t.to(dev) for t in (w2, w0, u, norm)]

    def run(rows, step):
        x = proj.to(dev)[rows.to(dev)]
        if not step.prompt:
            return linear_scan.wkv_decode(x, d[0], d[1], d[2], d[3], eps, step, state)
        r, k, v, g, low = x.split([H * n] * 4 + [rank], -1)
        low = torch.tanh(low.float()) @ d[0].float().T
        o = linear_scan.wkv_scan(r, k, v, low, d[1], d[2], step, state)
        return linear_scan.gated_group_norm(o, g, d[3], H, eps, False)

    got = in_parts(run, LENS, cut, dev)
    for gt, xs in zip(got, proj.double().split(LENS)):
        r, k, v, g, low = xs.split([H * n] * 4 + [rank], -1)
        m = r.shape[0]
        w = torch.exp(-torch.exp(torch.tanh(low) @ w2.double().T + w0.double()))
        o = oracle.wkv_recurrence(*(t.reshape(m, H, n) for t in (r, k, v, w)), u.double())
        want = oracle.unit_rms(o, eps).reshape(m, H * n) * norm.double() * oracle.silu(g)
        # a norm makes a small head's rounding as large as a large one's
        close(gt, want, dt, 3.0 if dt == "float32" else 1.0)


@on_each
@pytest.mark.parametrize("kind", ["ssd", "wkv"])
@torch.no_grad()
def test_long_prompts_of_few_heads(dev, dt, kind):
    """Lengths at which the GPU works on parts of a sequence at once; the state
    that is left behind continues the sequence."""
    dtype, lens, H, n, N = getattr(torch, dt), [390, 1, 257, 128], 2, 16, 24
    T = sum(lens)
    u, w0 = randn(H, n, seed=3).to(dtype), torch.linspace(-8, 1, H * n).to(dtype)
    x = randn(T, 3 * H * n + 2 * N + H, seed=5).to(dtype)
    norm, w2 = torch.ones(H * n).to(dtype), torch.zeros(H * n, 8).to(dtype)
    a_log, D = torch.tensor([-4.0, 0.5]).to(dtype), randn(H, seed=6).to(dtype)
    state = torch.full((4, H, n if kind == "wkv" else N, n), 1e4, device=dev)
    d = [t.to(dev) for t in (x, u, w0, norm, w2, a_log, D)]

    def run(rows, step):
        xs = d[0][rows.to(dev)]
        if kind == "ssd":
            return linear_scan.ssd_scan(xs[:, :H * n + 2 * N].contiguous(), xs[:, -H:], d[6], d[5],
                                        d[6], 1, N, step, state)
        r, k, v = xs[:, :3 * H * n].split(H * n, -1)
        if step.prompt:
            low = torch.zeros(xs.shape[0], H * n, device=dev)
            o = linear_scan.wkv_scan(r, k, v, low, d[2], d[1], step, state)
            return linear_scan.gated_group_norm(o, torch.ones_like(o), d[3], H, 1e-3, False)
        proj = torch.cat([r, k, v, torch.ones_like(r), torch.zeros_like(r[:, :8])], -1)
        return linear_scan.wkv_decode(proj, d[4], d[2], d[1], d[3], 1e-3, step, state)

    got = in_parts(run, lens, 386, dev)
    for g, xs in zip(got, x.double().split(lens)):
        m = xs.shape[0]
        if kind == "ssd":
            v, B, C = xs[:, :H * n + 2 * N].split([H * n, N, N], -1)
            want = oracle.ssd_recurrence(v.reshape(m, H, n), B.reshape(m, 1, N),
                                         C.reshape(m, 1, N),
                                         oracle.softplus(xs[:, -H:] + D.double()),
                                         a_log.double(), D.double()).reshape(m, -1)
        else:
            r, k, v = (t.reshape(m, H, n) for t in xs[:, :3 * H * n].split(H * n, -1))
            w = torch.exp(-torch.exp(w0.double())).view(1, H, n).expand(m, -1, -1)
            o = oracle.unit_rms(oracle.wkv_recurrence(r, k, v, w, u.double()), 1e-3)
            want = o.reshape(m, -1) * oracle.silu(torch.ones(1).double())
        close(g, want, dt, 1.0)


@on_each
@torch.no_grad()
def test_states_remember_for_long(dev, dt):
    """One early token is all there is; it is read back 300 tokens later."""
    T, H, n = 301, 2, 16
    dtype = getattr(torch, dt)
    r, k, v = torch.zeros(T, H * n), torch.zeros(T, H * n), torch.zeros(T, H * n)
    k[0], v[0], r[-1] = randn(H * n, seed=1), randn(H * n, seed=2), randn(H * n, seed=3)
    w0 = torch.full((H * n,), -7.0)
    w = torch.exp(-torch.exp(w0.double())).view(1, H, n).expand(T, -1, -1)
    r, k, v = (t.to(dtype) for t in (r, k, v))
    want = oracle.wkv_recurrence(*(t.double().view(T, H, n) for t in (r, k, v)), w,
                                 torch.zeros(H, n).double()).reshape(T, -1)
    assert float(want[-1].abs().max()) > 0.1
    step = PackedStep.for_prompts([T], dev)
    got = linear_scan.wkv_scan(r.to(dev), k.to(dev), v.to(dev), torch.zeros(T, H * n, device=dev),
                               w0.to(dev, dtype), torch.zeros(H, n, device=dev, dtype=dtype), step,
                               None)
    close(got[-1:], want[-1:], dt, 0.3)


@pytest.mark.gpu
@pytest.mark.parametrize("rows", [1, 3, 4, 5, 16, 33, 64, 65])
@pytest.mark.parametrize("group,rank,k", [(32, 16, 8), (48, 48, 72), (144, 5, 2048), (7, 3, 24),
                                          (16, 40, 64)])
@torch.no_grad()
def test_grouped_projection(rows, group, rank, k):
    from automodel_amd.serving.decode_linear import project_grouped

    lin = torch.nn.Linear(k, 4 * group + rank, bias=False).bfloat16()
    x = randn(5, rows, k).bfloat16()
    got = project_grouped(lin.cuda(), x.cuda(), [group] * 4 + [rank])
    parts = lin.weight.detach().double().cpu().split([group] * 4 + [rank])
    for y, xi, w in zip(got, x.double(), parts):
        assert rel(y, xi @ w.T) < 1e-2


# ---------------------------------------------------------------- whole model
@on_each
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_prompt(model_of, dev, dt, name):
    ids = ids_of(name, 45)
    close(whole(model_of(name, dev, dt), [ids]), want_logits(name, ids), dt)


@on_each
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_decode_from_the_first_token(model_of, dev, dt, name):
    ids = ids_of(name, 45)
    close(by_parts(model_of(name, dev, dt), ids, 1), want_logits(name, ids), dt)


@on_each
@pytest.mark.parametrize("first", [2, 3, 12, 15, 16, 17, 31, 32, 33, 63, 69])
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
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_first_tokens(model_of, dev, dt, name):
    m = model_of(name, dev, dt)
    for n in (1, 2, 3):
        ids = ids_of(name, n, seed=n)
        close(whole(m, [ids]), want_logits(name, ids), dt)


@on_each
def test_long_decode(model_of, dev, dt):
    """Decoding far past the prompt, over many chunks, equals the prompt path
    over the same tokens (and the oracle at the start)."""
    n = 100 if dev == "cpu" else 300
    ids = ids_of("mixed", n, seed=2)
    m = model_of("mixed", dev, dt)
    a, b = by_parts(m, ids, 4, max_len=512), whole(m, [ids])
    close(a, b.cpu(), dt, 2.0)                             # both are rounded
    close(a[:70], want_logits("mixed", ids[:70]), dt)


@pytest.mark.parametrize("fault", ["edge_in", "edge_out", "no_sink", "no_shift", "mix_transposed",
                                   ("lost", "own")])
def test_faults_would_show(fault):
    """The tolerance separates right from wrong for each planted mistake."""
    ids = ids_of("mixed", 30)
    bad = oracle.forward(ids, weights("mixed"), ALL["mixed"], fault=fault)
    assert rel(bad, want_logits("mixed", ids)) > 4 * TOL["bfloat16"]


@on_each
@pytest.mark.parametrize("name", ["mixed", "odd"])
def test_unequal_batch_equals_each_alone(model_of, dev, dt, name):
    m = model_of(name, dev, dt)
    lens = [1, 5, 33, 2, 48, 19]
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
    for name in ("mixed", "attention-last", "wkv-only"):
        m = model_of(name, dev, dt)
        a, b, c = ids_of(name, 9), ids_of(name, 4, seed=3), ids_of(name, 3, seed=4)
        lg = whole(m, [a, b, c], [[8, 0, 3], [], [1]])
        wa, wc = want_logits(name, a), want_logits(name, c)
        close(lg, torch.stack([wa[8], wa[0], wa[3], wc[1]]), dt)
        assert whole(m, [a], [[]]).shape == (0, ALL[name]["vocab"])


@on_each
def test_slots_are_given_back_and_used_again(model_of, dev, dt):
    """Shorter sequences leave the batch; a later batch lands in used slots."""
    name, m = "mixed", model_of("mixed", dev, dt)
    s = DecodeSession(m, 3, 48)
    first = [ids_of(name, n, seed=20 + n) for n in (30, 11, 40)]
    h, _ = s.prefill([q[:-2] for q in first])
    s.decode(h, torch.tensor([q[-2] for q in first], device=s.device))
    s.release([h[1]])
    left_ = [h[0], h[2]]
    lg = s.decode(left_, torch.tensor([first[0][-1], first[2][-1]], device=s.device))
    close(lg, torch.stack([want_logits(name, first[0])[-1], want_logits(name, first[2])[-1]]), dt)
    again = ids_of(name, 13, seed=50)
    h2, lg = s.prefill([again[:1]])
    assert h2 == [h[1]]                                  # the slot that was given back
    rows = [lg]
    for t in again[1:]:
        rows.append(s.decode(h2, torch.tensor([t], device=s.device)))
    close(torch.cat(rows), want_logits(name, again), dt)
    s.release(left_ + h2)
    assert s.cache.lens == [0, 0, 0] and s.live == []
    h3, lg = s.prefill([ids_of(name, n, seed=60 + n) for n in (7, 2, 21)])
    assert sorted(h3) == sorted(h)
    close(lg, torch.stack([want_logits(name, ids_of(name, n, seed=60 + n))[-1]
                           for n in (7, 2, 21)]), dt)


def test_cache_holds_a_chunk(model_of):
    cache = DecodeSession(model_of("mixed", "cpu", "float32"), 2, 100).cache
    assert len(cache.layers) == 5
    assert cache.layers[0]["k"].shape == (2, 12, 2, 16)
    assert cache.layers[3]["v"].shape == (2, 7, 3, 8)
    assert cache.layers[0]["conv"].shape == (2, 3, 96)
    assert cache.layers[0]["ssm"].shape == (2, 4, 16, 8)
    assert cache.layers[1]["wkv"].shape == (2, 3, 16, 16)
    assert all(t.dtype == torch.float32 for s in cache.layers for t in s.values())
    small = DecodeSession(model_of("mixed", "cpu", "float32"), 2, 9).cache
    assert small.layers[4]["k"].shape[1] == 9


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
    """Each replay of the captured step, with eager work in between and over a
    chunk's edge, gives the eager step's tokens and states."""
    from automodel_amd.utils.generation import _GraphStep
    from automodel_amd.utils.kv_cache import kv_cache_context

    m = model_of("large-heads", "cuda", dt)
    prompts = [ids_of("large-heads", 60, seed=80 + i) for i in range(batch)]
    runs = []
    for graphed in (False, True):
        s = DecodeSession(m, batch, 80)
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
        runs.append((torch.stack(toks), [t.clone() for st in s.cache.layers for t in st.values()]))
    assert torch.equal(runs[0][0], runs[1][0])
    for a, b in zip(runs[0][1], runs[1][1]):
        assert torch.equal(a, b)


def test_command_line_generate(checkpoints, capsys):
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


# ---------------------------------------------------------------- replay
def _trace(name):
    a, b, c = (ids_of(name, n, seed=90 + n) for n in (14, 4, 7))
    yield {"step": 0, "entries": [{"id": "a", "tokens": a[:11], "want": [0, 10]},
                                  {"id": "b", "tokens": b[:2], "want": []}], "end": []}, \
        [(a, 0), (a, 10)]
    yield {"step": 1, "entries": [{"id": "b", "tokens": [b[2]], "want": [0]},
                                  {"id": "a", "tokens": [a[11]], "want": []}], "end": ["b"]}, \
        [(b, 2)]
    yield {"step": 2, "entries": [{"id": "a", "tokens": [a[12]], "want": [0]}], "end": []}, \
        [(a, 12)]
    yield {"step": 3, "entries": [{"id": "a", "tokens": [a[13]], "want": []}], "end": ["a"]}, []
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


# ---------------------------------------------------------------- integration
def test_checkpoint_names_round_trip(model_of):
    for name in CONFIGS:
        m = model_of(name, "cpu", "float32")
        raw = raw_weights(name)
        back = m.state_dict_adapter.to_hf(m.state_dict())
        assert set(back) == set(raw)
        for k in raw:
            assert torch.equal(back[k], raw[k].float()), k
        params = dict(m.named_parameters())
        for k in raw:
            assert all(t in params for t in m.state_dict_adapter.hf_key_targets(k)), k
        assert m.lm_head.weight is m.model.embed_tokens.weight


@pytest.mark.parametrize("key", ["l0.mix.left.k", "l1.mix.mu.g", "l2.mlp.up", "l0.hc2.mix"])
def test_missing_weight_is_an_error(tmp_path, key):
    from safetensors.torch import save_file

    w = raw_weights("mixed")
    del w[key]
    (tmp_path / "config.json").write_text(json.dumps(ALL["mixed"]))
    save_file(w, str(tmp_path / "model.safetensors"))
    with pytest.raises(RuntimeError, match="mismatch"):
        load_pretrained(str(tmp_path), dtype="float32", device="cpu")


def test_unknown_parts_are_refused():
    from automodel_amd.models.papidra.model import PapidraConfig

    for bad in ({**make_wkv(), "type": "other"}, {**make_wkv(), "mlp": {"kind": "moe", "ff": 8}},
                make_parallel(heads=3, kv_heads=2), make_parallel(dim=16, dims=18),
                make_parallel(ssm_heads=4, groups=3), make_parallel(norm_groups=5)):
        with pytest.raises(ValueError):
            PapidraConfig.from_hf_config(make_config(layers=[bad]))


def test_uniform_configuration_builds():
    from automodel_amd.models.registry import build_model

    m = build_model(config=dict(vocab_size=50, hidden_size=32, num_attention_heads=2,
                                num_key_value_heads=1, head_dim=16, intermediate_size=24,
                                ssm_head_dim=16, ssm_state_size=8, ssm_groups=2, wkv_head_dim=16,
                                wkv_rank=8, chunk_size=6, num_hidden_layers=3, streams=3),
                    architecture="Papidra", dtype="float32", meta_init=False)
    assert m(torch.tensor([[1, 2, 3, 4, 5, 6, 7, 8]])).shape == (1, 8, 50)


@pytest.mark.parametrize("dev,dt", [("cpu", "float32"),
                                    pytest.param("cuda", "bfloat16", marks=pytest.mark.gpu)])
def test_training_forward_and_gradients(model_of, dev, dt):
    """The same module trains: its recorded forward equals the oracle, and on
    the CPU so do the gradients."""
    m = model_of("mixed", dev, dt)
    ids = torch.tensor([ids_of("mixed", 14), ids_of("mixed", 14, seed=5)], device=dev)
    with torch.enable_grad():
        logits = m(ids)
        for b in range(2):
            close(logits[b], want_logits("mixed", ids[b].tolist()), dt)
        m.zero_grad()
        torch.nn.functional.cross_entropy(logits[0, :-1].float(), ids[0, 1:]).backward()
    grads = m.state_dict_adapter.to_hf(
        {k: p.grad for k, p in m.named_parameters() if p.grad is not None})
    m.zero_grad()
    assert all(torch.isfinite(g).all() for g in grads.values())
    w = {k: v.requires_grad_() for k, v in weights("mixed").items()}
    ref = oracle.forward(ids[0].tolist(), w, ALL["mixed"])
    torch.nn.functional.cross_entropy(ref[:-1], ids[0, 1:].cpu()).backward()
    for k in ("l0.mix.left.sink", "l0.mix.right.A_log", "l1.mix.w0", "l1.mix.mu.w", "l2.hc2.mix",
              "l3.mix.right.conv", "l4.mlp.gate", "embed"):
        e = (grads[k].double().cpu() - w[k].grad).norm() / w[k].grad.norm()
        assert e < (1e-4 if dt == "float32" else 0.15), (k, float(e))


@torch.no_grad()
def test_adapters_on_the_stacked_projection(checkpoints):
    """A wrapped projection is used as a whole; what decoding reads as a raw
    weight refuses a wrapper."""
    class Wrapped(torch.nn.Module):
        def __init__(self, lin, extra):
            super().__init__()
            self.lin, self.extra = lin, extra

        def forward(self, x):
            return self.lin(x) + x @ self.extra.T

    m = load_pretrained(checkpoints("wkv-only"), dtype="float32", device="cpu")
    ids = ids_of("wkv-only", 20)
    mixer = m.model.layers[0].mixer
    extra = 0.05 * randn(*mixer.in_proj.weight.shape)
    mixer.in_proj = Wrapped(mixer.in_proj, extra)
    got = by_parts(m, ids, 9)
    mixer.in_proj = mixer.in_proj.lin
    assert rel(by_parts(m, ids, 9), got) > 1e-3
    mixer.in_proj.weight += extra
    assert rel(by_parts(m, ids, 9), got) < 1e-5
    mixer.decay_proj = Wrapped(mixer.decay_proj, torch.zeros_like(mixer.decay_proj.weight))
    with pytest.raises(RuntimeError, match="adapters"):
        by_parts(m, ids, 9)
