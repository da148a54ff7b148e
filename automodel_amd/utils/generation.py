"""Greedy/sampled decoding: serving, in-loop evaluation and smoke tests.

Reference behavior: the reference's eval path generates with the HF model
(KV-cached ``model.generate``). ``generate`` recomputes the prefix each
step (simple, always correct for any module); everything else goes through
``DecodeSession``, the step function over the native preallocated cache
(utils/kv_cache.py) — O(T) per new token instead of O(T^2):

* ``generate_cached``  prefill, then one-token steps;
* ``generate_graphed`` the one-token step captured in a hipGraph;
* ``generate_batch``   any number of prompts of any lengths, in batches.
"""

from __future__ import annotations

from collections.abc import Sequence

import numpy as np
import torch

from automodel_amd.utils.kv_cache import kv_cache_context, make_cache


def _pick_next(next_logits: torch.Tensor, temperature: float) -> torch.Tensor:
    if temperature > 0:
        probs = torch.softmax(next_logits / temperature, dim=-1)
        return torch.multinomial(probs, 1)
    return next_logits.argmax(-1, keepdim=True)


@torch.no_grad()
def generate(
    model,
    input_ids: torch.Tensor,
    max_new_tokens: int = 32,
    temperature: float = 0.0,
    eos_token_id: int | None = None,
) -> torch.Tensor:
    model.eval()
    ids = input_ids
    for _ in range(max_new_tokens):
        logits = model(ids)
        nxt = _pick_next(logits[:, -1].float(), temperature)
        ids = torch.cat([ids, nxt], dim=1)
        if eos_token_id is not None and bool((nxt == eos_token_id).all()):
            break
    model.train()
    return ids


class DecodeSession:
    """One batch of sequences stepped through a model's cache.

    ``prefill`` starts sequences from whole prompts, ``decode`` moves sequences
    on by one token, ``release`` ends some. Sequences are named by the handles
    that ``prefill`` returns. With a ragged cache (SlotCache) prompts may
    differ in length, tokens are packed without padding, and a batch shrinks as
    its sequences end; the dense K/V cache holds one rectangular batch that
    ends as a whole.
    """

    def __init__(self, model, max_batch: int, max_len: int, static: bool = False):
        self.model = model
        self.cache = make_cache(model, max_batch, max_len, static)
        self.device = next(model.parameters()).device
        self.live: list[int] = []

    @torch.no_grad()
    def prefill(self, prompts: Sequence[Sequence[int]],
                want: Sequence[Sequence[int]] | None = None) -> tuple[list[int], torch.Tensor]:
        """-> (handles, logits [n, vocab]) at the wanted places of each prompt
        (its last token by default), prompts in order."""
        lens = [len(p) for p in prompts]
        want = [[n - 1] for n in lens] if want is None else [list(w) for w in want]
        cache = self.cache
        with kv_cache_context(cache):
            cache.begin_forward()
            if cache.ragged:
                handles = cache.alloc(len(prompts))
                flat = np.concatenate([np.asarray(p, dtype=np.int64) for p in prompts])
                starts = [sum(lens[:i]) for i in range(len(lens))]
                rows = [s + j for s, w in zip(starts, want) for j in w]
                cache.plan_prompts(handles, lens, rows)
                logits = self.model(torch.from_numpy(flat).to(self.device).unsqueeze(0))
                cache.advance()
            else:
                if self.live or len(set(lens)) != 1:
                    raise ValueError("a dense K/V cache takes one batch of equal prompts")
                handles = list(range(len(prompts)))
                full = self.model(torch.tensor([list(p) for p in prompts], device=self.device))
                self._check_dense()
                cache.advance(lens[0])
                logits = torch.cat([full[i, w] for i, w in enumerate(want)])
        self.live += handles
        return handles, logits

    @torch.no_grad()
    def decode(self, handles: list[int], tokens: torch.Tensor) -> torch.Tensor:
        """tokens [n], the next one of each handle -> logits [n, vocab]."""
        cache = self.cache
        with kv_cache_context(cache):
            cache.begin_forward()
            if cache.ragged:
                cache.plan_decode(handles)
                logits = self.model(tokens.reshape(1, -1))
                cache.advance()
                return logits
            if handles != self.live:
                raise ValueError("a dense K/V cache moves its whole batch on")
            pos = torch.arange(cache.pos, cache.pos + 1, device=self.device).unsqueeze(0)
            logits = self.model(tokens.reshape(-1, 1), position_ids=pos)[:, -1]
            cache.advance(1)
            return logits

    def release(self, handles: list[int]) -> None:
        """Give back what finished sequences hold."""
        for h in handles:
            self.live.remove(h)
        if self.cache.ragged:
            self.cache.free(handles)
        elif not self.live:
            self.cache.pos = 0

    def _check_dense(self) -> None:
        assert self.cache._layer == self.model.config.num_hidden_layers, (
            "model did not consult the KV cache (attention lacks "
            "maybe_update_kv) — cached decode would be silently wrong")


class _GraphStep:
    """The greedy one-token step with static shapes and device-side positions:
    tokens in ``ids``, replaced by the next ones."""

    def __init__(self, session: DecodeSession, handles: list[int], first: torch.Tensor):
        self.session, self.ids = session, first.clone()
        if session.cache.ragged:
            session.cache.plan_decode(handles)
        else:
            session.cache.freeze_for_graph()

    def __call__(self) -> None:
        cache, model = self.session.cache, self.session.model
        cache.begin_forward()
        if cache.ragged:
            logits = model(self.ids)
        else:
            logits = model(self.ids, position_ids=cache.position_ids())[:, -1]
        self.ids.copy_(logits.argmax(-1, keepdim=True))
        cache.advance_device()


@torch.no_grad()
def generate_graphed(
    model,
    input_ids: torch.Tensor,
    max_new_tokens: int = 32,
    use_hip_graph: bool | None = None,
) -> torch.Tensor:
    """Greedy decode with STATIC shapes: every per-token forward is the same
    launch sequence, so on GPU the whole step (embed → layers → argmax →
    feedback into the input buffer → position increment) is captured in ONE
    hipGraph and each token costs a single hipGraphLaunch instead of
    hundreds of kernel launches. CPU falls back to eager static-cache math
    (same numerics — tested for parity with ``generate``)."""
    model.eval()
    B, T = input_ids.shape
    dev = input_ids.device
    use_hip_graph = (dev.type == "cuda") if use_hip_graph is None else use_hip_graph
    session = DecodeSession(model, B, T + max_new_tokens, static=True)
    handles, logits = session.prefill(input_ids.tolist())
    out = torch.empty(B, max_new_tokens, dtype=input_ids.dtype, device=dev)
    with kv_cache_context(session.cache):
        nxt = logits.argmax(-1, keepdim=True)          # [B, 1]
        out[:, 0] = nxt[:, 0]
        decode_step = _GraphStep(session, handles, nxt)
        ids_buf = decode_step.ids
        start = 1
        if use_hip_graph and max_new_tokens >= 3:
            # warmup on a side stream (allocator state), then capture
            s = torch.cuda.Stream()
            s.wait_stream(torch.cuda.current_stream())
            with torch.cuda.stream(s):
                decode_step()
            torch.cuda.current_stream().wait_stream(s)
            out[:, 1] = ids_buf[:, 0]  # warmup emitted token 1; capture token 2
            g = torch.cuda.CUDAGraph()
            with torch.cuda.graph(g):
                decode_step()
            decode_step, start = g.replay, 2
        for i in range(start, max_new_tokens):
            decode_step()
            out[:, i] = ids_buf[:, 0]
    model.train()
    return torch.cat([input_ids, out], dim=1)


@torch.no_grad()
def generate_cached(
    model,
    input_ids: torch.Tensor,
    max_new_tokens: int = 32,
    temperature: float = 0.0,
    eos_token_id: int | None = None,
) -> torch.Tensor:
    """KV-cached decode: one prefill forward over the prompt, then one
    single-token forward per generated token. Greedy output is identical to
    ``generate``. Requires a model whose attention consults the cache
    context (the in-tree model families do)."""
    model.eval()
    B, T = input_ids.shape
    session = DecodeSession(model, B, T + max_new_tokens)
    handles, logits = session.prefill(input_ids.tolist())
    nxt = _pick_next(logits.float(), temperature)
    ids = torch.cat([input_ids, nxt], dim=1)
    for _ in range(max_new_tokens - 1):
        if eos_token_id is not None and bool((nxt == eos_token_id).all()):
            break
        nxt = _pick_next(session.decode(handles, nxt).float(), temperature)
        ids = torch.cat([ids, nxt], dim=1)
    model.train()
    return ids


@torch.no_grad()
def generate_batch(
    model,
    prompts: Sequence[Sequence[int]],
    max_new_tokens: int = 32,
    temperature: float = 0.0,
    eos_token_id: int | None = None,
    max_batch: int = 16,
) -> list[list[int]]:
    """Generated tokens for any number of prompts of any lengths.

    Prompts run in batches of up to ``max_batch``; a sequence leaves its batch
    at its end token, and the next batch reuses the cache. Models whose cache
    is rectangular only batch prompts of equal length.
    """
    model.eval()
    if not prompts:
        return []
    max_len = max(len(p) for p in prompts) + max_new_tokens
    session = DecodeSession(model, min(max_batch, len(prompts)), max_len)
    ragged = session.cache.ragged
    # similar lengths together; the dense cache needs them equal
    todo = sorted(range(len(prompts)), key=lambda i: len(prompts[i]))
    out: list[list[int]] = [[] for _ in prompts]
    while todo:
        batch = todo[:max_batch]
        if not ragged:
            batch = [i for i in batch if len(prompts[i]) == len(prompts[batch[0]])]
            session = DecodeSession(model, len(batch), max_len)
        todo = todo[len(batch):]
        handles, logits = session.prefill([prompts[i] for i in batch])
        owner = dict(zip(handles, batch))
        live = list(handles)
        for step in range(max_new_tokens):
            nxt = _pick_next(logits.float(), temperature)
            for h, t in zip(live, nxt[:, 0].tolist()):
                if eos_token_id is None or out[owner[h]][-1:] != [eos_token_id]:
                    out[owner[h]].append(t)
            done = [h for h in live if eos_token_id is not None
                    and out[owner[h]][-1] == eos_token_id]
            if step + 1 == max_new_tokens or len(done) == len(live):
                break
            if done and ragged:
                keep = [i for i, h in enumerate(live) if h not in done]
                session.release(done)
                live, nxt = [live[i] for i in keep], nxt[keep]
            logits = session.decode(live, nxt)
        session.release(list(session.live))
    model.train()
    return out
