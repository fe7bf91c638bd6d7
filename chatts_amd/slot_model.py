"""SlotModel - what every model the engine serves has in common, whatever its layers are: sequence slots, the block-paged cache's
bookkeeping, prefix reuse by token identity, per-slot sampling settings, the captured batched step and the generation loops over it.

A model class adds its layers through a few methods:
  admit_begin / admit_step     a request enters a slot (all of its prompt, or a portion per call) and gets its first token
  _admit_packed                several requests enter in one pass
  _run_segments                one ragged batch of tokens through the model, logits of chosen rows (step_tokens' device half)
  _batched_step_eager          one token for every slot; its state lives in buf (pos_all, token_all, out_tokens_all, ...)
  _prefill_request, decode_step   the single-sequence path
  request_tokens, _request_idents, _install_sampling
and the attributes config, device, lib, plan, comm, buf, max_batch, max_ctx, t_max, _kv, _kv_replaced, _kv_dynamic, _slot_idents,
enable_prefix_caching, prefix_stats, use_graph, _graph, _graph_batched, _tp.
"""
import ctypes as C

import torch

from . import _lib


class SlotModel:
    step_is_idempotent = True        # a decode step repeated from the same positions and tokens changes nothing (pure KV caches)

    def check_ids(self, ids):
        """raise ValueError for a prompt the model cannot take (before it shares a pass with others)"""

    # ---- one ragged batch: any number of new tokens per slot --------------------------------------------------------------
    def step_tokens(self, entries):
        """entries: list of (slot, new token ids, wanted places among them), slots distinct.  Runs all tokens as one batch on top of what
        the slots hold (position = tokens the slot has seen; a slot starts over after release_slot) and returns the logits of the wanted
        places, in order, as float32 [wanted, vocab] on the device.  Pages are reserved as the sequences grow.  A batch of more than t_max
        tokens runs in several passes."""
        seen = self._slot_seen
        for slot, ids, _ in entries:
            if seen[slot] + len(ids) > self.max_ctx:
                raise ValueError(f"slot {slot}: {seen[slot] + len(ids)} tokens exceed max_ctx={self.max_ctx}")
            self._slot_idents[slot] = []                 # its rows change: not a prefix source
            self.reserve_kv(slot, seen[slot] + len(ids), write_from=seen[slot])
        out, work = [], [(slot, list(ids), sorted(set(want)), 0) for slot, ids, want in entries if len(ids)]
        rows_of = {}                                     # (slot, place) -> row of `out`
        n_out = 0
        while work:
            segs, ids, index, rest, row = [], [], [], [], 0
            for slot, tok, want, done in work:
                n = min(len(tok) - done, self.t_max - row)
                if n <= 0:
                    rest.append((slot, tok, want, done))
                    continue
                segs.append((row, n, seen[slot], slot))
                ids += tok[done:done + n]
                for w in want:
                    if done <= w < done + n:
                        rows_of[(slot, w)] = n_out + len(index)
                        index.append(row + w - done)
                seen[slot] += n
                row += n
                if done + n < len(tok):
                    rest.append((slot, tok, want, done + n))
            lg = self._run_segments(ids, segs, index)
            if index:
                out.append(lg.clone())
                n_out += len(index)
            work = rest
        order = [rows_of[(slot, w)] for slot, _, want in entries for w in want]
        if not order:
            return torch.empty((0, self.config.vocab_size), dtype=torch.float32, device=self.device)
        return torch.cat(out, dim=0)[torch.tensor(order, device=self.device)]

    def release_slot(self, slot):
        """the sequence in `slot` is finished and nothing of it is kept: its pages return to the pool"""
        self._slot_seen[slot] = 0
        self._slot_idents[slot] = []
        if self._kv is not None:
            if self._kv_dynamic:
                self._kv.release(slot)
            else:
                self._kv.retire(slot)                    # a full pool: every slot keeps its own pages for good

    # ---- block-paged KV cache: host bookkeeping (chatts_amd/kv_blocks.py) ------------------------------------------------
    def _push_kv_row(self, slot):
        row = self._kv.rows[slot]
        if row:                                  # stream-ordered: kernels enqueued after this see the new row
            self.buf["kv_table"][slot, :len(row)] = torch.tensor(row, dtype=torch.int32)

    def _kv_evicted(self, victim):
        self._slot_idents[victim] = []           # nothing is resident there any more (its stale table row is never read: parked)

    def reserve_kv(self, slot, n_tokens, idents=None, protect=(), write_from=0):
        """Make cache slot `slot` able to hold n_tokens positions (no-op with a contiguous cache) and mark it active.  idents = the
        request's token identities: the slot whose resident prefix will be reused is protected from eviction (like `protect`), and
        every block the request is going to WRITE - everything past the reused prefix; `write_from` positions for direct callers -
        is made private first if another slot shares it.  Raises kv_blocks.KvPoolExhausted (nothing changed) when even evicting
        every finished sequence does not free enough blocks."""
        if self._kv is None:
            return
        if n_tokens > self.max_ctx:
            raise ValueError(f"{n_tokens} positions exceed max_ctx={self.max_ctx}")
        keep = set(protect)
        first = int(write_from) // self._kv.block_size
        if idents is not None and self.enable_prefix_caching:
            n, src = self._match_prefix(slot, idents)
            n = min(n, len(idents) - 1)
            if src >= 0 and n >= 16:
                keep.add(src)
                first = n // self._kv.block_size          # own slot: rows below stay; other slot: blocks below get adopted
        order = sorted(range(self.max_batch), key=lambda sl: len(self._slot_idents[sl]))       # least resident first
        changed = self._kv.reserve(slot, n_tokens, protect=keep, evict_order=order, on_evict=self._kv_evicted, private_from=first)
        self._kv_replaced[slot] = self._kv_replaced.get(slot, set()) | self._kv.last_replaced
        if changed:
            self._push_kv_row(slot)

    def kv_fits(self, token_counts):
        """could requests needing these many positions (prompt + new tokens each) be admitted into free slots now?"""
        return self._kv is None or self._kv.fits(token_counts)

    def kv_stats(self):
        if self._kv is None:
            return None
        return {"block_size": self._kv.block_size, "blocks": self._kv.n_blocks, "free": len(self._kv.free),
                "active_slots": len(self._kv.active), "evictions": self._kv.evictions, "dynamic": self._kv_dynamic,
                "shared_blocks": self._kv.shared_blocks()}

    # ---- sampling --------------------------------------------------------------------------------------------------------
    def set_sampling(self, temperature=0.0, top_k=0, top_p=1.0, seed=0):
        """Token selection of every following step: greedy (temperature 0 / None, the default) or temperature / top-k /
        top-p sampling on the GPU (chatts_sample_batched).  Same seed + same prompt => same tokens."""
        if not temperature:
            args = None
        else:
            if temperature < 0 or not (0.0 < top_p <= 1.0):
                raise ValueError(f"temperature={temperature} must be >= 0 and top_p={top_p} in (0, 1]")
            args = _lib.SamplingArgs(temperature=float(temperature), top_k=int(top_k or 0), top_p=float(top_p),
                                     seed=int(seed) & 0xFFFFFFFF, n_kept=None, kept_mass=None)
        key = None if args is None else (args.temperature, args.top_k, args.top_p, args.seed)
        if key == getattr(self, "_sampling_key", None):
            return
        self._install_sampling(args)
        self._sampling, self._sampling_key = args, key
        self._graph = None               # the captured steps have the old selection kernel baked in
        self._graph_batched = None

    def _sampling_arrays(self):
        if "samp_temp" not in self.buf:
            dev, n = self.device, max(1, self.max_batch)
            self.buf["samp_temp"] = torch.zeros(n, dtype=torch.float32, device=dev)     # 0 = the slot decodes greedily
            self.buf["samp_topk"] = torch.zeros(n, dtype=torch.int32, device=dev)
            self.buf["samp_topp"] = torch.ones(n, dtype=torch.float32, device=dev)
            self.buf["samp_seed"] = torch.zeros(n, dtype=torch.int32, device=dev)       # (bit pattern of the uint32 seed)
        return self.buf

    def _rows_args(self, slot):
        B = self._sampling_arrays()
        return _lib.SamplingArgs(temperature=1.0, top_k=0, top_p=1.0, seed=0, n_kept=None, kept_mass=None,
                                 temperature_rows=B["samp_temp"][slot:].data_ptr(), top_k_rows=B["samp_topk"][slot:].data_ptr(),
                                 top_p_rows=B["samp_topp"][slot:].data_ptr(), seed_rows=B["samp_seed"][slot:].data_ptr())

    def set_sampling_rows(self):
        """Per-slot sampling (ChattsSamplingArgs.*_rows): every cache slot draws with its own (temperature, top_k, top_p, seed), read on
        the device at run time from four small arrays - requests with different settings share one captured step, and
        set_slot_sampling() changes a slot without re-capturing.  Slots start greedy (temperature 0)."""
        if getattr(self, "_sampling_key", None) == "rows":
            return
        args = self._rows_args(0)
        self._install_sampling(args)
        self._sampling, self._sampling_key = args, "rows"
        self._graph = None
        self._graph_batched = None

    def set_slot_sampling(self, slot, temperature=0.0, top_k=0, top_p=1.0, seed=0):
        """Sampling settings of the sequence in cache slot `slot`: used by every step in per-slot mode (set_sampling_rows), inert in
        the other modes.  A plain device write - no re-capture."""
        temperature = 0.0 if temperature is None else float(temperature)
        if temperature < 0 or not (0.0 < top_p <= 1.0):
            raise ValueError(f"temperature={temperature} must be >= 0 and top_p={top_p} in (0, 1]")
        B = self._sampling_arrays()
        B["samp_temp"][slot] = temperature
        B["samp_topk"][slot] = max(int(top_k or 0), 0)
        B["samp_topp"][slot] = float(top_p)
        s32 = int(seed) & 0xFFFFFFFF
        B["samp_seed"][slot] = s32 - (1 << 32) if s32 >= (1 << 31) else s32

    # ---- batched decode / continuous batching ----------------------------------------------------------------------------
    def batched_step(self):
        """One greedy token for EVERY cache slot (idle slots compute harmlessly; their position saturates)."""
        if self.plan.world != 1 and self._tp is None:
            raise NotImplementedError("batched decode under tensor parallelism needs the peer-to-peer exchange (use_p2p=True)")
        if not self.use_graph:
            return self._batched_step_eager()
        if self._graph_batched is None:
            B = self.buf
            keys = ("pos_all", "step_all", "token_all", "token_logit_all", "out_tokens_all")
            saved = {k: B[k].clone() for k in keys}
            if not self.step_is_idempotent:              # warm up on parked slots: nothing a slot holds changes
                B["pos_all"].fill_(-1)
            torch.cuda.synchronize()
            side = torch.cuda.Stream()
            side.wait_stream(torch.cuda.current_stream())
            with torch.cuda.stream(side):
                self._batched_step_eager()
            torch.cuda.current_stream().wait_stream(side)
            torch.cuda.synchronize()
            for k in keys:
                B[k].copy_(saved[k])
            g = torch.cuda.CUDAGraph()
            with torch.cuda.graph(g):
                self._batched_step_eager()
            torch.cuda.synchronize()
            for k in keys:
                B[k].copy_(saved[k])
            self._graph_batched = g
        self._graph_batched.replay()

    def _match_prefix(self, slot, idents, exclude=()):
        """(n, src): the longest prefix of `idents` resident in some cache slot (ties prefer `slot` itself: zero copy)."""
        best, src = 0, -1
        for s, have in enumerate(self._slot_idents):
            if s in exclude:
                continue
            n = 0
            for a, b in zip(idents, have):
                if a != b:
                    break
                n += 1
            if n > best or (n == best and s == slot and n > 0):
                best, src = n, s
        return best, src

    def note_generated(self, slot, tokens):
        """After a request finished: its generated tokens (all but the last, which was never fed back) also have K/V rows in
        the slot - a follow-up turn that re-sends prompt + answer reuses them."""
        if self.enable_prefix_caching and tokens:
            self._slot_idents[slot] = self._slot_idents[slot] + [int(t) for t in tokens[:-1]]
        if self._kv is not None:
            self._kv.retire(slot)                # blocks stay resident for prefix reuse; evictable from now on

    def pick_slot(self, free_slots, idents=None):
        """Which free cache slot a new request should take: the one whose resident prefix matches best (zero copy), else the
        one whose resident tokens are least worth keeping (fewest)."""
        if not self.enable_prefix_caching or idents is None:
            return free_slots[0]
        def match(s):
            n = 0
            for a, b in zip(idents, self._slot_idents[s]):
                if a != b:
                    break
                n += 1
            return n
        best = max(free_slots, key=match)
        if match(best) >= 16:
            return best
        return min(free_slots, key=lambda s: len(self._slot_idents[s]))

    def _admit(self, slot, ids, series, lengths, max_new_tokens=1):
        """Prefill one request into cache slot `slot` and produce its first token (out_tokens_all[slot, 0])."""
        st = self.admit_begin(slot, ids, series, lengths, max_new_tokens)
        self.admit_step(st)
        return st["T"]

    def plan_pack(self, candidates, free_slots):
        """Which of the waiting requests should be prefilled TOGETHER (chatts_decoder_prefill_packed).  candidates: list of
        (ids, series, lengths, max_new_tokens) in arrival order.  Greedy: take requests while their not-yet-cached rows fit the
        prefill buffers and slots are free; a request that shares most of its prompt with one already in the pack is left for the
        next round (it will then reuse that request's K/V rows instead of computing them again).  -> indices into candidates."""
        if self.plan.world != 1 or len(free_slots) < 2 or len(candidates) < 2:
            return []
        pack, rows, pack_idents = [], 0, []
        for i, (ids, series, lengths, max_new) in enumerate(candidates):
            if len(pack) >= len(free_slots):
                break
            idents = self._request_idents(ids, series, lengths)
            if idents is None:          # lengths unknown / prefix caching off: size by the expanded prompt alone
                try:
                    T = self.request_tokens(ids, None, lengths)
                except ValueError:
                    continue
                need, idents = T, None
            else:
                T = len(idents)
                n, _ = self._match_prefix(-1, idents)
                n = min(n, T - 1)
                need = T - (n if n >= 16 else 0)
                dup = False
                for other in pack_idents:
                    if other is None:
                        continue
                    k = 0
                    for a, b in zip(idents, other):
                        if a != b:
                            break
                        k += 1
                    if k >= max(16, T // 2):
                        dup = True
                        break
                if dup:
                    continue
            if T + max_new > self.max_ctx or rows + need > self.t_max:
                continue
            pack.append(i)
            pack_idents.append(idents)
            rows += need
        return pack if len(pack) >= 2 else []

    @torch.no_grad()
    def generate_batch(self, requests, max_new_tokens=64, eos_token_id=None, sync_every=8):
        """Continuous batching over `max_batch` cache slots.  requests: list of (ids, series [n,2Lmax,1] | None,
        lengths | None).  A finished sequence frees its slot for the next waiting request at the next sync point.
        Returns the list of generated token lists, in request order."""
        if self.max_batch < 2:
            return [self.generate_one(i, s, l, max_new_tokens, eos_token_id) for (i, s, l) in requests]
        eos = set(eos_token_id if isinstance(eos_token_id, (list, tuple, set)) else
                  ([] if eos_token_id is None else [eos_token_id]))
        B = self.buf
        results = [None] * len(requests)
        waiting = list(range(len(requests)))[::-1]
        slots = [None] * self.max_batch              # request index per slot
        produced = [0] * self.max_batch
        B["pos_all"].fill_(-1); B["step_all"].zero_(); B["token_all"].zero_()
        steps_since_sync = 0

        def harvest(final=False):
            toks_all = B["out_tokens_all"].cpu()
            if self._tp is not None and self._tp.status():
                raise RuntimeError("tensor-parallel exchange timed out (a peer rank did not reach the collective): tokens are invalid")
            for s, r in enumerate(slots):
                if r is None:
                    continue
                toks = toks_all[s, :produced[s]].tolist()
                cut = next((i + 1 for i, t in enumerate(toks) if t in eos), None) if eos else None
                if cut is not None or produced[s] >= max_new_tokens or final:
                    results[r] = toks[:cut] if cut is not None else toks[:max_new_tokens]
                    slots[s] = None
                    B["pos_all"][s] = -1         # parked: the batched step neither attends nor writes this slot's cache
                    self.note_generated(s, results[r])

        while waiting or any(r is not None for r in slots):
            while waiting and any(v is None for v in slots):
                free = [i for i, v in enumerate(slots) if v is None]
                cands = waiting[::-1][:len(free)]            # the next requests in arrival order
                pack = self.plan_pack([requests[r] + (max_new_tokens,) for r in cands], free)
                if pack and self._kv_dynamic and not self.kv_fits(
                        [self.request_tokens(*requests[cands[j]]) + max_new_tokens for j in pack]):
                    pack = []                                # the block pool cannot take them all at once: one at a time
                if pack:                                     # several short prompts: one packed prefill pass
                    items, members = [], []
                    for j in pack:
                        r = cands[j]
                        ids, series, lengths = requests[r]
                        s = self.pick_slot(free, self._request_idents(ids, series, lengths))
                        free.remove(s)
                        items.append((s, ids, series, lengths, max_new_tokens))
                        members.append((s, r))
                    try:
                        self._admit_packed(items)
                    except RuntimeError as e:                # the pool could not cover the pack after all (a protected prefix
                        if type(e).__name__ != "KvPoolExhausted" or all(v is None for v in slots):     # source): the touched slots forgot their resident prefixes
                            raise
                        break
                    for s, r in members:
                        slots[s], produced[s] = r, 1
                        waiting.remove(r)
                    continue
                ids, series, lengths = requests[waiting[-1]]
                if self._kv_dynamic and not self.kv_fits([self.request_tokens(ids, series, lengths) + max_new_tokens]):
                    if all(v is None for v in slots):        # nothing left to finish and free blocks: it can never fit
                        from .kv_blocks import KvPoolExhausted
                        raise KvPoolExhausted(f"request {waiting[-1]} needs more KV blocks than the pool holds ({self.kv_stats()})")
                    break                                    # wait until a running sequence finishes and its blocks become evictable
                s = self.pick_slot(free, self._request_idents(ids, series, lengths))
                try:
                    self._admit(s, ids, series, lengths, max_new_tokens)
                except RuntimeError as e:                    # (the reservation is _admit's first change: nothing to undo)
                    if type(e).__name__ != "KvPoolExhausted" or all(v is None for v in slots):
                        raise
                    break
                r = waiting.pop()
                slots[s], produced[s] = r, 1
            if all(r is None or produced[s] >= max_new_tokens for s, r in enumerate(slots)):
                harvest()
                continue
            self.batched_step()
            for s, r in enumerate(slots):
                if r is not None and produced[s] < max_new_tokens:
                    produced[s] += 1
            steps_since_sync += 1
            if steps_since_sync >= sync_every or all(r is None or produced[s] >= max_new_tokens for s, r in enumerate(slots)):
                harvest()
                steps_since_sync = 0
        return results

    @torch.no_grad()
    def generate_one(self, ids, series=None, lengths=None, max_new_tokens=64, eos_token_id=None, sync_every=16,
                     return_logits=False):
        """ids: un-expanded prompt ids (host list); series: [n, 2*Lmax, 1] tensor of this prompt's series."""
        self._prefill_request(ids, series, lengths, max_new_tokens)
        logits0 = self.buf["logits"].clone() if return_logits else None
        eos = set(eos_token_id if isinstance(eos_token_id, (list, tuple, set)) else
                  ([] if eos_token_id is None else [eos_token_id]))
        produced = 1
        toks = None
        while produced < max_new_tokens:
            self.decode_step()
            produced += 1
            if eos and (produced % sync_every == 0):
                toks = self.buf["out_tokens"][:produced].tolist()
                if any(t in eos for t in toks):
                    break
        toks = self.buf["out_tokens"][:produced].tolist()
        if self._tp is not None and self._tp.status():
            raise RuntimeError("tensor-parallel exchange timed out (a peer rank did not reach the collective): tokens are invalid")
        if eos:
            for i, t in enumerate(toks):
                if t in eos:
                    toks = toks[:i + 1]
                    break
        self.note_generated(0, toks)
        return (toks, logits0) if return_logits else toks

    @torch.no_grad()
    def generate_stream(self, ids, series=None, lengths=None, max_new_tokens=64, eos_token_id=None, chunk=1):
        """Generator over the new tokens of ONE request: yields a list of token ids every `chunk` decode steps (chunk=1: token by
        token, what an SSE stream / HF TextStreamer consumes; each yield costs one device->host read of the tokens so far).
        Stops after an EOS token (which is yielded) or max_new_tokens.  Same kernels and tokens as generate_one."""
        eos = set(eos_token_id if isinstance(eos_token_id, (list, tuple, set)) else ([] if eos_token_id is None else [eos_token_id]))
        self._prefill_request(ids, series, lengths, max_new_tokens)
        produced, sent = 1, 0
        while True:
            if produced - sent >= chunk or produced >= max_new_tokens:
                toks = self.buf["out_tokens"][sent:produced].tolist()
                if self._tp is not None and self._tp.status():
                    raise RuntimeError("tensor-parallel exchange timed out (a peer rank did not reach the collective): tokens are invalid")
                hit = next((i for i, t in enumerate(toks) if t in eos), None)
                if hit is not None:
                    yield toks[:hit + 1]
                    return
                yield toks
                sent = produced
            if produced >= max_new_tokens:
                return
            self.decode_step()
            produced += 1

    def eval(self):
        return self

    def to(self, *a, **k):
        return self
