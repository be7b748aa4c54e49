"""ServingSession: the host loop of the serving mode (MPK in "online_notoken" mode).

The caller says, step by step, which requests bring which tokens; the session keeps every live request's pages, packs the
tokens of a step into passes of at most `max_num_batched_tokens` rows (single decoded tokens beside portions of prompts,
at most `max_tokens_per_request` rows of one request per pass), describes each pass in the meta tensors and launches the
megakernel once for it.  What a request has in the cache is its pages, its length and, where the model has recurrent layers,
its state slot, so a request may pause for any number of steps, and a portion may end anywhere.

`generate` is the greedy loop on top: continuous batching over a list of prompts with as many live requests as there are
batch slots and pages.
"""
from dataclasses import dataclass, field
from typing import Dict, List, Sequence, Tuple

import torch

from .mpk import MPK, MPKMetadata


class PagePool:
    """Free list of cache pages (or state slots).  What is given back is handed out again first."""

    def __init__(self, num_pages: int, what: str = "cache pages"):
        self.num_pages, self.what = num_pages, what
        self._free = list(range(num_pages - 1, -1, -1))

    def __len__(self):
        return len(self._free)

    def take(self, n: int) -> List[int]:
        if n > len(self._free):
            raise RuntimeError(f"out of {self.what}: {n} asked for, {len(self._free)} of {self.num_pages} free")
        return [self._free.pop() for _ in range(n)]

    def give(self, pages: List[int]):
        self._free.extend(reversed(pages))


@dataclass
class _Request:
    pages: List[int] = field(default_factory=list)
    length: int = 0  # positions whose keys and values are in the cache
    slot: int = -1   # recurrent-state slot (models with recurrent layers)


class ServingSession:
    # models with recurrent layers: the tensor that names every batch slot's state slot, and the pool of state slots
    state_slots = slots = None

    def __init__(self, mpk: MPK):
        if mpk.metadata.mode != "online_notoken":
            raise ValueError("a serving session drives an MPK in online_notoken mode")
        self.mpk = mpk
        pk = mpk.persistent_kernel
        self.page_size, self.max_rows, self.max_requests = pk.page_size, pk.max_num_batched_tokens, pk.max_num_batched_requests
        self.rows_per_request, self.max_seq = pk.max_tokens_per_request, min(pk.max_seq_length, mpk.model_builder.max_positions or pk.max_seq_length)
        self.pool = PagePool(pk.max_num_pages)
        # one state slot per batch slot: the kernel starts a request's state from zero where its position is zero
        self.state_slots = getattr(mpk.model_builder, "state_slots", None)
        if self.state_slots is not None:
            self.slots = PagePool(self.max_requests, "state slots")
        self.requests: Dict[object, _Request] = {}
        mpk._ensure_compiled()

    @staticmethod
    def open(model_path: str = None, model_config=None, model_name: str = None, dtype=torch.bfloat16, max_tokens: int = 4096, max_requests: int = 4,
             page_size: int = 64, max_rows: int = 64, max_seq_length: int = None, device: str = "cuda") -> "ServingSession":
        """Build and compile the model found at `model_path` (class chosen by its config.json) or given as `model_config`,
        with a cache of `max_tokens` positions."""
        pages = max(1, max_tokens // page_size)
        max_seq = max_seq_length or pages * page_size
        # the batch description of a pass travels in one copy: the five index tensors are slices of one buffer
        R = max_requests
        block = torch.zeros(4 * R + 2 + pages, dtype=torch.int32, device=device)
        qo, kv, last, slots, idx = block.split([R + 1, R + 1, R, R, pages])
        meta = MPKMetadata(mode="online_notoken", max_seq_length=max(2, max_seq), max_num_batched_requests=R, max_num_batched_tokens=max_rows, max_num_pages=pages,
                           page_size=page_size, device=device, weight_from_model=model_path is not None, model_path=model_path, model_name=model_name,
                           model_config=model_config, max_tokens_per_request=min(max_rows, 64), dtype=dtype, qo_indptr_buffer=qo, paged_kv_indptr_buffer=kv,
                           paged_kv_last_page_len_buffer=last, paged_kv_indices_buffer=idx, state_slots_buffer=slots)
        mpk = MPK(meta)
        mpk.build()
        session = ServingSession(mpk)
        session._block = block
        return session

    # ------------------------------------------------------------------ steps
    def logits(self) -> torch.Tensor:
        """Logits of the rows of the last pass (a view of the library's tensor)."""
        return self.mpk.model_builder.logits.to_torch()

    def step(self, entries: Sequence[Tuple[object, Sequence[int]]], want: Sequence[Sequence[int]] = None):
        """Run `entries` = (request, its next tokens) as one batch.  Returns (logits, next tokens): float32 rows for the
        wanted places (want[i] indexes entries[i]'s tokens) in order, or None, and the greedy token after each entry."""
        if len({rid for rid, _ in entries}) != len(entries):
            raise ValueError("a request may appear once in a step")
        want = want if want is not None else [[] for _ in entries]
        for rid, toks in entries:
            r = self.requests.get(rid)
            if (r.length if r else 0) + len(toks) > self.max_seq:
                raise ValueError(f"request {rid!r} would grow beyond max_seq_length={self.max_seq}")
        found = [dict.fromkeys(w) for w in want]
        greedy = [None] * len(entries)
        done = [0] * len(entries)
        # single tokens first, so that they share their pass with the head of the longer portions
        order = sorted(range(len(entries)), key=lambda i: len(entries[i][1]))
        while True:
            batch, room = [], self.max_rows
            for i in order:
                n = min(len(entries[i][1]) - done[i], self.rows_per_request, room)
                if n > 0 and len(batch) < self.max_requests:
                    batch.append((i, n))
                    room -= n
            if not batch:
                break
            self._pass([(entries[i][0], entries[i][1][done[i]:done[i] + n]) for i, n in batch])
            row, logits, sampled = 0, None, None
            for i, n in batch:
                lo, hi = done[i], done[i] + n
                places = [p for p in found[i] if lo <= p < hi]
                if places:
                    logits = self.logits() if logits is None else logits
                    for p in places:
                        found[i][p] = logits[row + p - lo].to(torch.float32, copy=True)
                if hi == len(entries[i][1]):
                    sampled = self.mpk.output_tokens.view(-1).tolist() if sampled is None else sampled
                    greedy[i] = sampled[row + n - 1]
                row, done[i] = row + n, hi
        rows = [found[i][p] for i in range(len(entries)) for p in want[i]]
        return (torch.stack(rows) if rows else None), greedy

    def _pass(self, batch):
        ps = self.page_size
        ids, qo, kv, last, slots, pages = [], [0], [0], [], [], []
        for rid, toks in batch:
            r = self.requests.get(rid)
            if r is None:
                r = _Request(slot=-1 if self.slots is None else self.slots.take(1)[0])
                self.requests[rid] = r
            r.length += len(toks)
            need = -(-r.length // ps) - len(r.pages)
            if need > 0:
                try:
                    r.pages += self.pool.take(need)
                except RuntimeError:
                    r.length -= len(toks)
                    raise
            ids += list(toks)
            pages += r.pages
            qo.append(len(ids))
            kv.append(len(pages))
            last.append(r.length - (len(r.pages) - 1) * ps)
            slots.append(max(r.slot, 0))
        R, m = self.max_requests, self.mpk
        pad = R - len(batch)
        desc = qo + [qo[-1]] * pad + kv + [kv[-1]] * pad + last + [0] * pad + slots + [0] * pad + pages
        if getattr(self, "_block", None) is not None:
            self._block[:len(desc)].copy_(torch.tensor(desc, dtype=torch.int32))
        else:
            t = torch.tensor(desc, dtype=torch.int32)
            for dst, lo, n in ((m.qo_indptr_buffer, 0, R + 1), (m.paged_kv_indptr_buffer, R + 1, R + 1), (m.paged_kv_last_page_len_buffer, 2 * R + 2, R),
                               (self.state_slots, 3 * R + 2, R), (m.paged_kv_indices_buffer, 4 * R + 2, len(pages))):
                if dst is not None:
                    dst[:n].copy_(t[lo:lo + n])
        m.input_tokens.view(-1)[:len(ids)].copy_(torch.tensor(ids, dtype=torch.int64))
        m()

    def end(self, rid):
        """The request is finished: its pages and its state slot go back to their pools."""
        r = self.requests.pop(rid, None)
        if r is not None:
            self.pool.give(r.pages)
            if self.slots is not None:
                self.slots.give([r.slot])

    # ------------------------------------------------------------------ greedy generation
    def generate(self, prompts: Sequence[Sequence[int]], max_new_tokens: int, eos_token_id: int = -1) -> List[List[int]]:
        """Greedy continuation of every prompt, continuously batched: a request is admitted when a batch slot and the pages
        for its whole length are free; prompts enter in portions beside the running requests' tokens."""
        out = [list(p) for p in prompts]
        need = [-(-(len(p) + max_new_tokens) // self.page_size) for p in prompts]
        for i, p in enumerate(prompts):
            if not p or need[i] > self.pool.num_pages or len(p) + max_new_tokens - 1 > self.max_seq:
                raise ValueError(f"prompt {i} is empty or its {len(p) + max_new_tokens} positions exceed the cache or max_seq_length={self.max_seq}")
        waiting, live, reserved = list(range(len(prompts))), {}, 0
        while waiting or live:
            while waiting and len(live) < self.max_requests and reserved + need[waiting[0]] <= self.pool.num_pages:
                i = waiting.pop(0)
                live[i] = 0  # tokens of out[i] already in the cache
                reserved += need[i]
            entries, room = [], self.max_rows
            for i in sorted(live, key=lambda i: len(out[i]) - live[i]):
                n = min(len(out[i]) - live[i], self.rows_per_request, room)
                if n > 0:
                    entries.append((i, n))
                    room -= n
            _, greedy = self.step([(("generate", i), out[i][live[i]:live[i] + n]) for i, n in entries])
            for (i, n), tok in zip(entries, greedy):
                live[i] += n
                if live[i] < len(out[i]):
                    continue
                out[i].append(tok)
                if len(out[i]) - len(prompts[i]) == max_new_tokens or tok == eos_token_id:
                    self.end(("generate", i))
                    reserved -= need[i]
                    del live[i]
        return out

    def finalize(self):
        self.mpk.finalize()
