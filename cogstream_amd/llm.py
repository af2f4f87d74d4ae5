"""Language-model engines: prefill / decode steps over caller-owned caches, generation, and batches of live requests.

Qwen2Engine is the host mirror of the Qwen2 seams the reference calls (transformers, pinned 4.46.3):
self.get_model()(inputs_embeds=..., attention_mask=...) (model/cogreasoner_chat.py:312-316,322) and
super().generate(inputs_embeds=...) (:802-807), computing through cogs_llm_forward. DecoderEngine runs decoder-only models
described layer by layer (weights.DecoderConfig) through cogs_decoder_forward. Both share CausalEngine's generation loop,
PrefixKV, and the batch steps of Sequences."""
from __future__ import annotations

import ctypes as C
from typing import Dict, Hashable, List, Optional, Sequence, Tuple

import torch

from . import _lib as L
from . import ops
from .runtime import get_handle
from .weights import DecoderConfig, LlmConfig, PackedDecoder, PackedLlm


class KVCache:
    def __init__(self, cfg: LlmConfig, max_len: int, dtype, device):
        kvd = cfg.num_key_value_heads * cfg.head_dim
        self.k = torch.empty(cfg.num_hidden_layers, max_len, kvd, device=device, dtype=dtype)
        self.v = torch.empty_like(self.k)
        self.struct = L.KV(self.k.data_ptr(), self.v.data_ptr(), max_len, 0)

    @property
    def len(self) -> int:
        return self.struct.len

    @property
    def max_len(self) -> int:
        return self.struct.max_len

    def reset(self, length: int = 0):
        self.struct.len = length

    def _blocks(self) -> List[torch.Tensor]:
        """views [..., max_len, columns] that hold the cached rows"""
        return [self.k, self.v]

    state: Optional[torch.Tensor] = None       # what the length `len` has besides its rows (recurrent models)
    stale = False

    def restore(self, length: int, state: Optional[torch.Tensor]):
        """back to a length whose rows are in place and whose `state` was kept"""
        self.reset(length)

    def copy_rows_from(self, old: "KVCache", n: int):
        for dst, src in zip(self._blocks(), old._blocks()):
            dst[..., :n, :].copy_(src[..., :n, :])


class DecoderCache(KVCache):
    """one sequence of a decoder described layer by layer: the rows of every layer run that caches rows (latents, or keys and values
    per head; weights.PackedDecoder.cache_widths) and, fp32, the state of every recurrent one. A state belongs to exactly the
    length it was left at: reset() to any other but 0 leaves the cache unusable until restore() brings a state back."""

    def __init__(self, widths: Sequence[int], state_floats: int, max_len: int, dtype, device):
        self.widths = list(widths)
        self.k = torch.empty(sum(self.widths) * max_len, device=device, dtype=dtype)
        self.state = torch.empty(state_floats, device=device, dtype=torch.float32) if state_floats else None
        self.struct = L.KV(self.k.data_ptr(), L.ptr(self.state) or None, max_len, 0)
        self.stale = False

    def reset(self, length: int = 0):
        if self.state is not None and length != self.len:
            self.stale = length != 0
        self.struct.len = length

    def restore(self, length: int, state: Optional[torch.Tensor]):
        self.struct.len = length
        if self.state is not None and length:
            self.state.copy_(state)
        self.stale = False

    def _blocks(self) -> List[torch.Tensor]:
        out, at = [], 0
        for w in self.widths:
            out.append(self.k[at:at + w * self.max_len].view(self.max_len, w))
            at += w * self.max_len
        return out


class PrefixKV:
    """KV rows of the previous prompt, kept so that the next generate() only prefills what differs (SURVEY.md §8f
    rank 3; the reference rebuilds the whole conversation every turn, evaluate/answer_generate.py:130-148).
    The reusable prefix is found by comparing the new input embeddings with the previous ones bit for bit on the
    device: KV row i depends only on rows 0..i and the position i, so every invalidation rule (resized frames, a
    history turn dropped by the selection stage, another question) is covered by that comparison. Only rows that
    were PREFILLED are reused -- rows written by decode steps went through the GEMV kernels. Models with recurrent
    state keep a copy of the state behind the prompt, so they can reuse the whole previous prompt or nothing of it."""

    def __init__(self, engine: "CausalEngine"):
        self.engine = engine
        self.cache: Optional[KVCache] = None
        self.rows: Optional[torch.Tensor] = None   # [n, H] embeddings whose KV rows 0..n-1 are in `cache`
        self.state: Optional[torch.Tensor] = None  # recurrent state behind row n-1
        self.reused = 0    # rows taken from the cache, summed over calls
        self.seen = 0      # prompt rows, summed over calls

    def plan(self, embeds: torch.Tensor, need: int) -> int:
        """-> number of leading rows of `embeds` whose KV is already in self.cache (at most len(embeds) - 2)"""
        if self.cache is None or self.cache.max_len < need:
            old = self.cache
            self.cache = self.engine.new_cache(need + need // 2)   # sessions grow: leave room for the next turns
            if old is not None and self.rows is not None:
                self.cache.copy_rows_from(old, self.rows.shape[0])
            else:
                self.rows = None
        p = 0
        if self.rows is not None and self.rows.dtype == embeds.dtype:
            # at least 2 rows are always prefilled: a 1-row forward is the decode GEMV, whose rounding differs
            n = min(self.rows.shape[0], embeds.shape[0] - 2)
            if n > 0:
                bits = torch.int16 if embeds.element_size() == 2 else torch.int32
                neq = (self.rows[:n].view(bits) != embeds[:n].view(bits)).any(dim=1)
                idx = torch.arange(n, device=embeds.device)
                p = int(torch.where(neq, idx, torch.full_like(idx, n)).min().item())
                if self.cache.state is not None and p < self.rows.shape[0]:
                    p = 0
        self.seen += embeds.shape[0]
        self.reused += p
        return p

    def drop(self):
        self.rows = None


class CausalEngine:
    """what generation needs of a model: cfg.vocab_size, new_cache, embed_tokens, forward (one sequence) and forward_batch"""
    cfg = None
    dtype = None
    device = None

    def new_cache(self, max_len: int) -> KVCache:
        raise NotImplementedError

    def embed_tokens(self, ids: torch.Tensor) -> torch.Tensor:
        raise NotImplementedError

    def forward(self, embeds: torch.Tensor, cache: Optional[KVCache] = None, **want) -> Dict[str, torch.Tensor]:
        raise NotImplementedError

    def logits_of(self, hidden: torch.Tensor) -> torch.Tensor:
        """final hidden states [n, hidden] -> fp32 logits [n, vocab]"""
        raise NotImplementedError

    def forward_batch(self, embeds: torch.Tensor, lens: Sequence[int], caches: Sequence[KVCache],
                      want: Sequence[int]) -> Optional[torch.Tensor]:
        """one step of several sequences: sequence i brings lens[i] rows of `embeds` (back to back) behind caches[i].
        -> fp32 logits [len(want), vocab] of the rows `want` (None if empty). Here one sequence at a time; engines with a
        batched step override it."""
        rows: Dict[int, torch.Tensor] = {}
        r0 = 0
        for n, cache in zip(lens, caches):
            mine = [w for w in want if r0 <= w < r0 + n]
            if mine == [r0 + n - 1]:
                rows[mine[0]] = self.forward(embeds[r0:r0 + n], cache)["logits"]
            else:
                hidden = self.forward(embeds[r0:r0 + n], cache, want_logits=False, want_hidden=bool(mine)).get("hidden")
                for w in mine:
                    rows[w] = self.logits_of(hidden[w - r0:w - r0 + 1])[0]
            r0 += n
        return torch.stack([rows[w] for w in want]) if len(want) else None

    def generate(self, embeds: torch.Tensor, *, max_new_tokens: int, eos_token_id: Sequence[int] = (),
                 do_sample: bool = False, temperature: float = 1.0, top_k: int = 0, top_p: float = 1.0,
                 repetition_penalty: float = 1.0, allowed_ids: Optional[Sequence[int]] = None,
                 prompt_ids: Optional[torch.Tensor] = None, generator: Optional[torch.Generator] = None,
                 sampler: str = "device", seed: Optional[int] = None,
                 cache: Optional[KVCache] = None, ignore_eos: bool = False,
                 prefix: Optional[PrefixKV] = None, prefilled: Optional[dict] = None,
                 stage_times: Optional[dict] = None) -> List[int]:
        """GenerationMixin.generate with inputs_embeds: prefill, then one cogs_llm_forward per token.
        Returns the NEW token ids only. Logits processors run in HF order:
        repetition penalty -> custom (allowed-id mask) -> temperature -> top-k -> top-p.
        `prefix`: reuse the KV rows of the leading embeddings that are unchanged since the previous call.
        `prefilled`: the result of a forward(embeds, cache) the caller has already run into `cache` (bench.py times the
        prefill and the token loop separately this way); the prompt is then not prefilled again.
        Sampling (do_sample): cogs_sample on the device, tokens never visit the host. sampler="device": Philox draws
        keyed by `seed` (default: one draw of the CPU generator) and the step; sampler="host": the CPU generator
        (`generator`, default the global one) makes the [vocab] exponential draws of every step exactly as
        torch.multinomial does in the reference's CPU run, so the sampled ids are the reference's."""
        S = embeds.shape[0]
        if stage_times is not None:        # bench.py's pipeline split: the prompt pass and the token loop, drained on both sides
            import time
            torch.cuda.synchronize()
            t_start = time.perf_counter()
        if prefilled is not None:
            assert cache is not None and prefix is None and cache.len >= S and "logits" in prefilled
            pos_start = cache.len
            res = prefilled
        elif prefix is not None:
            assert cache is None
            embeds = embeds.contiguous()
            p = prefix.plan(embeds, S + max_new_tokens)
            cache = prefix.cache
            cache.restore(p, prefix.state)
            prefix.rows = None          # not valid while this call is rewriting the cache
            res = self.forward(embeds[p:], cache)
            prefix.state = None if cache.state is None else cache.state.clone()
            prefix.rows = embeds        # rows 0..S-1 are prefilled; decode rows behind them are never reused
            pos_start = S
        else:
            if cache is None:
                cache = self.new_cache(S + max_new_tokens)
            pos_start = cache.len + S
            res = self.forward(embeds, cache)
        if stage_times is not None:
            torch.cuda.synchronize()
            t_loop = time.perf_counter()
            stage_times["answer_prefill"] = stage_times.get("answer_prefill", 0.0) + t_loop - t_start
        allowed = (torch.tensor(list(allowed_ids), dtype=torch.int32, device=self.device) if allowed_ids is not None else None)
        eos = set(int(e) for e in eos_token_id)
        # token ids stay on the device: the greedy id feeds the next embedding gather and the repetition-penalty
        # history without a host round trip; the host only looks at them every `check_every` steps (EOS test).
        n_prompt = int(prompt_ids.numel()) if prompt_ids is not None else 0
        seen = torch.empty(n_prompt + max_new_tokens, dtype=torch.int64, device=self.device)
        if n_prompt:
            seen[:n_prompt] = prompt_ids.reshape(-1).to(self.device)
        toks = seen[n_prompt:]        # the generated ids ARE the tail of the penalty history: argmax / the sampler write them once
        n_seen, produced = n_prompt, 0
        # host-drawn sampling (parity mode) consumes one [vocab] draw of the CPU generator per step: steps issued past
        # the EOS would advance that generator beyond where GenerationMixin stops, so the stop test runs every step
        # (nor can a recurrent state step back over tokens behind the EOS)
        check_every = 1 if (do_sample and sampler == "host") or cache.state is not None else 8
        if do_sample and sampler == "device" and seed is None:
            seed = int(torch.randint(0, 2 ** 62, (1,), generator=generator).item())
        need_proc = repetition_penalty != 1.0 or allowed is not None     # the temperature is applied inside cogs_sample
        stop_at = None
        for step in range(max_new_tokens):
            logits = res["logits"]
            if need_proc:
                prev = seen[:n_seen] if (n_seen and repetition_penalty != 1.0) else None
                ops.logits_process(logits, prev, repetition_penalty, allowed, 1.0)
            if do_sample:
                tok_dev = ops.sample(logits, top_k or 0, 1.0 if top_p is None else top_p,
                                     draws=self._draws(generator) if sampler == "host" else None,
                                     seed=seed or 0, offset=step, temperature=temperature, out=toks[step:step + 1])
            else:
                tok_dev = ops.argmax(logits, out=toks[step:step + 1])      # straight into the generated-ids buffer
            n_seen += 1
            produced += 1
            last = step + 1 == max_new_tokens
            if eos and not ignore_eos and ((step + 1) % check_every == 0 or last):
                host = toks[:produced].tolist()
                hit = next((i for i, t in enumerate(host) if t in eos), None)
                if hit is not None:
                    stop_at = hit + 1
                    break
            if not last:
                res = self.forward(self.embed_tokens(tok_dev), cache)
        out = toks[:produced].tolist()
        if stage_times is not None:
            stage_times["decode"] = stage_times.get("decode", 0.0) + time.perf_counter() - t_loop
        if stop_at is not None:
            out = out[:stop_at]
            # forwards issued past the EOS only wrote KV rows that are dropped again here
            cache.reset(min(cache.len, pos_start + stop_at - 1))
        return out

    def generate_batch(self, prompts: Sequence[Sequence[int]], *, max_new_tokens: int, eos_token_id: Sequence[int] = (),
                       do_sample: bool = False, temperature: float = 1.0, top_k: int = 0, top_p: float = 1.0,
                       repetition_penalty: float = 1.0, seed: int = 0, max_batch: int = 64) -> List[List[int]]:
        """new token ids of every prompt. Up to `max_batch` requests run at once: a group's prompts are one step, then every
        step carries one token of each request that has not finished; a finished request leaves the batch and its cache with
        it. Logits processors and samplers are generate()'s, per request (Philox offset = step, seed + request index)."""
        out: List[List[int]] = [[] for _ in prompts]
        eos = set(int(e) for e in eos_token_id)
        for g0 in range(0, len(prompts), max_batch):
            live = [i for i in range(g0, min(g0 + max_batch, len(prompts)))]
            seqs = Sequences(self)
            feed = {i: [int(t) for t in prompts[i]] for i in live}
            if any(not f for f in feed.values()):
                raise ValueError("empty prompt")
            for step in range(max_new_tokens):
                logits = seqs.step([(i, feed[i], [len(feed[i]) - 1]) for i in live])
                picked = torch.empty(len(live), dtype=torch.int64, device=self.device)
                for r, i in enumerate(live):
                    if repetition_penalty != 1.0:
                        prev = torch.tensor(list(prompts[i]) + out[i], dtype=torch.int64, device=self.device)
                        ops.logits_process(logits[r], prev, repetition_penalty, None, 1.0)
                    if do_sample:
                        ops.sample(logits[r], top_k or 0, top_p, seed=seed + i, offset=step, temperature=temperature, out=picked[r:r + 1])
                    else:
                        ops.argmax(logits[r], out=picked[r:r + 1])
                toks = picked.tolist()
                for i, t in zip(live, toks):
                    out[i].append(t)
                    feed[i] = [t]
                for i in [i for i in live if out[i][-1] in eos]:
                    seqs.release(i)
                live = [i for i in live if out[i][-1] not in eos]
                if not live:
                    break
        return out

    def _draws(self, generator) -> torch.Tensor:
        """parity mode: the [vocab] Exponential(1) draws torch.multinomial(probs, 1) makes on the CPU generator
        (GenerationMixin._sample, transformers 4.46.3; the reference's CPU path draws from the global generator)"""
        q = torch.empty(self.cfg.vocab_size, dtype=torch.float32).exponential_(1, generator=generator)
        return q.to(self.device, non_blocking=True)


class Qwen2Engine(CausalEngine):
    def __init__(self, state: Dict[str, torch.Tensor], cfg: LlmConfig, dtype=torch.bfloat16, device="cuda"):
        self.cfg, self.dtype, self.device = cfg, dtype, torch.device(device)
        self.handle = get_handle(self.device)
        self.packed = PackedLlm(state, cfg, dtype, self.device)
        self._activate()

    def _activate(self):
        self.handle.activate("llm", self, lambda: L.check(
            L.lib.cogs_llm_load(self.handle.h, C.byref(self.packed.struct)), "cogs_llm_load"))

    def new_cache(self, max_len: int) -> KVCache:
        return KVCache(self.cfg, max_len, self.dtype, self.device)

    def embed_tokens(self, ids: torch.Tensor) -> torch.Tensor:
        return ops.gather_rows(self.packed.embed, None, ids.reshape(-1).to(self.device, torch.int64))

    def forward(self, embeds: torch.Tensor, cache: Optional[KVCache] = None, *, want_logits: bool = True,
                want_pooled: bool = False, want_hidden: bool = False):
        """returns dict(logits fp32 [vocab] | pooled fp32 [H] | hidden [S,H])"""
        self._activate()
        embeds = embeds.contiguous()
        S = embeds.shape[0]
        ctx = S + (cache.len if cache is not None else 0)
        nbytes = C.c_size_t()
        L.check(L.lib.cogs_llm_workspace_bytes(self.handle.h, S, ctx, C.byref(nbytes)), "cogs_llm_workspace_bytes")
        ws = self.handle.workspace("llm", nbytes.value)
        out = {}
        logits = torch.empty(self.cfg.vocab_size, device=self.device, dtype=torch.float32) if want_logits else None
        pooled = torch.empty(self.cfg.hidden_size, device=self.device, dtype=torch.float32) if want_pooled else None
        hidden = torch.empty(S, self.cfg.hidden_size, device=self.device, dtype=self.dtype) if want_hidden else None
        L.check(L.lib.cogs_llm_forward(self.handle.h, L.current_stream(), embeds.data_ptr(), S,
                                       C.byref(cache.struct) if cache is not None else None, L.ptr(logits),
                                       L.ptr(pooled), L.ptr(hidden), ws.data_ptr(), ws.numel()), "cogs_llm_forward")
        if want_logits:
            out["logits"] = logits
        if want_pooled:
            out["pooled"] = pooled
        if want_hidden:
            out["hidden"] = hidden
        return out

    def logits_of(self, hidden: torch.Tensor) -> torch.Tensor:
        return ops.gemm(hidden.contiguous(), self.packed.lm_head, out_f32=True)

    def forward_segments(self, embeds: torch.Tensor, seg_lens: Sequence[int]) -> torch.Tensor:
        """several independent sequences stored back to back -> mean of the final hidden states of each, fp32
        [nseg, H] (cogs_llm_forward_segments): one var-len prefill instead of one forward per sequence"""
        self._activate()
        embeds = embeds.contiguous()
        S = embeds.shape[0]
        cu = [0]
        for n in seg_lens:
            cu.append(cu[-1] + int(n))
        assert cu[-1] == S and all(int(n) > 0 for n in seg_lens)
        nbytes = C.c_size_t()
        L.check(L.lib.cogs_llm_workspace_bytes(self.handle.h, S, S, C.byref(nbytes)), "cogs_llm_workspace_bytes")
        ws = self.handle.workspace("llm", nbytes.value)
        out = torch.empty(len(seg_lens), self.cfg.hidden_size, device=self.device, dtype=torch.float32)
        cua = (C.c_int32 * len(cu))(*cu)
        L.check(L.lib.cogs_llm_forward_segments(self.handle.h, L.current_stream(), embeds.data_ptr(), S, cua, len(seg_lens),
                                                out.data_ptr(), ws.data_ptr(), ws.numel()), "cogs_llm_forward_segments")
        return out


class DecoderEngine(CausalEngine):
    """a decoder-only model described layer by layer (weights.DecoderConfig), batched steps through cogs_decoder_forward"""

    def __init__(self, state: Dict[str, torch.Tensor], cfg: DecoderConfig, dtype=torch.bfloat16, device="cuda"):
        self.cfg, self.dtype, self.device = cfg, dtype, torch.device(device)
        self.handle = get_handle(self.device)
        self.packed = PackedDecoder(state, cfg, dtype, self.device)
        self._activate()

    def _activate(self):
        self.handle.activate("decoder", self, lambda: L.check(
            L.lib.cogs_decoder_load(self.handle.h, C.byref(self.packed.struct)), "cogs_decoder_load"))

    def new_cache(self, max_len: int) -> DecoderCache:
        return DecoderCache(self.packed.cache_widths, self.packed.state_floats, max_len, self.dtype, self.device)

    def embed_tokens(self, ids: torch.Tensor) -> torch.Tensor:
        return ops.gather_rows(self.packed.embed, None, ids.reshape(-1).to(self.device, torch.int64))

    def forward_batch(self, embeds: torch.Tensor, lens: Sequence[int], caches: Sequence[KVCache], want: Sequence[int],
                      streams: Optional[torch.Tensor] = None) -> Optional[torch.Tensor]:
        """streams, when given: fp32 [layer runs, rows, padded width], receives the residual stream behind every layer run"""
        self._activate()
        embeds = embeds.contiguous()
        S, n, nw = embeds.shape[0], len(lens), len(want)
        if any(c.stale for c in caches):
            raise L.CogsError("a cache's recurrent state does not belong to its length")
        limit = self.cfg.max_positions
        if limit and any(c.len + k > limit for c, k in zip(caches, lens)):
            raise L.CogsError(f"a sequence would pass the model's {limit} positions")
        assert sum(lens) == S and len(caches) == n and embeds.shape[1] == self.packed.width_p and embeds.dtype == self.dtype
        ctx = S + sum(c.len for c in caches)
        nbytes = C.c_size_t()
        L.check(L.lib.cogs_decoder_workspace_bytes(self.handle.h, S, n, ctx, nw, C.byref(nbytes)), "cogs_decoder_workspace_bytes")
        ws = self.handle.workspace("decoder", nbytes.value)
        logits = torch.empty(nw, self.packed.vocab_p, device=self.device, dtype=torch.float32) if nw else None
        kv = (C.POINTER(L.KV) * n)(*[C.pointer(c.struct) for c in caches])
        L.check(L.lib.cogs_decoder_forward(self.handle.h, L.current_stream(), embeds.data_ptr(), kv, (C.c_int32 * n)(*lens), n,
                                           (C.c_int32 * max(nw, 1))(*want), nw, L.ptr(logits), L.ptr(streams), ws.data_ptr(),
                                           ws.numel()), "cogs_decoder_forward")
        return logits[:, :self.cfg.vocab_size] if nw else None

    def forward(self, embeds: torch.Tensor, cache: Optional[KVCache] = None, *, want_logits: bool = True) -> Dict[str, torch.Tensor]:
        """one sequence -> dict(logits fp32 [vocab]) of its last row"""
        S = embeds.shape[0]
        if cache is None:
            cache = self.new_cache(S)
        out = self.forward_batch(embeds, [S], [cache], [S - 1] if want_logits else [])
        return {"logits": out[0]} if want_logits else {}


class Sequences:
    """the live requests of an engine: a cache per request id, steps that carry new tokens of any of them as one batch"""

    def __init__(self, engine: CausalEngine, reserve: int = 64):
        self.engine, self.reserve = engine, reserve
        self.caches: Dict[Hashable, KVCache] = {}

    def _cache(self, rid: Hashable, new: int) -> KVCache:
        """the request's cache with room for `new` more rows; a full one moves to one of twice the size"""
        old = self.caches.get(rid)
        need = new + (old.len if old is not None else 0)
        if old is None or old.max_len < need:
            grown = self.engine.new_cache(max(-(-need // self.reserve) * self.reserve, 2 * old.max_len if old is not None else 0))
            if old is not None:
                grown.copy_rows_from(old, old.len)
                grown.restore(old.len, old.state)
            self.caches[rid] = grown
        return self.caches[rid]

    def step(self, entries: Sequence[Tuple[Hashable, Sequence[int], Sequence[int]]]) -> Optional[torch.Tensor]:
        """entries (request id, its next token ids, places among them whose logits are wanted) -> fp32 logits, one row per
        wanted place in order, or None"""
        ids: List[int] = []
        lens, caches, want = [], [], []
        vocab = self.engine.cfg.vocab_size
        if len({rid for rid, _, _ in entries}) != len(entries):
            raise ValueError("a request appears twice in one step")
        for rid, toks, places in entries:
            if not toks or any(not 0 <= t < vocab for t in toks) or any(not 0 <= w < len(toks) for w in places):
                raise ValueError(f"request {rid!r}: no tokens, a token outside the vocabulary, or a wanted place outside the step")
            want += [len(ids) + w for w in places]
            ids += toks
            lens.append(len(toks))
        for (rid, toks, _), n in zip(entries, lens):
            caches.append(self._cache(rid, n))
        embeds = self.engine.embed_tokens(torch.tensor(ids, dtype=torch.int64))
        return self.engine.forward_batch(embeds, lens, caches, want)

    def release(self, rid: Hashable) -> None:
        del self.caches[rid]
