"""Batched serving of any registered decoder: the step batch, the slot manager / lock-step scheduler, and generation on top of it.

A batch is a set of requests that start together (prompts of any lengths, packed without padding) and then advance by one token a step; a request
that ends leaves its cache slot to a later batch.  A model serves through three methods:

* ``setup_caches(slots, max_len)`` -- static caches for that many sequences;
* ``step(batch) -> float32 [wanted, vocab]`` -- run the batch's tokens from and into the caches, logits at the wanted rows;
* ``vocab``, ``device`` -- columns of the logits, where tensors live.

``duguzen.DuguzenForCausalLM`` and ``kozipel.KozipelForCausalLM`` run a batch as one; ``gptfast.Transformer`` (Aria) runs its sequences one after the other on the slots' caches.  The same ``step`` is what ``generate`` and the trace runner (bin/trace_run) drive."""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Dict, List, Optional, Sequence

import torch

from . import gptfast as G


@dataclass
class StepBatch:
    """Tokens of one step, packed sequence after sequence.  Device tensors are int32; ``lengths`` / ``starts`` / ``slots`` are the host's copy (one
    entry per sequence)."""

    ids: torch.Tensor            # [T]
    slot: torch.Tensor           # [T] cache slot of every token's sequence
    pos: torch.Tensor            # [T] position of every token in its sequence
    cu: torch.Tensor             # [sequences + 1] first row of every sequence
    wanted: Optional[torch.Tensor]   # rows whose logits are asked for (None: every row)
    lengths: List[int]
    starts: List[int]
    slots: List[int]
    rows: Optional[List[int]] = None   # the host's copy of ``wanted``
    seq: Optional[torch.Tensor] = None   # [T] which sequence every token belongs to
    made: Dict[object, object] = field(default_factory=dict)   # tables derived from the lengths, by what they are for

    def chunks(self, size: int):
        """The sequences cut at the multiples of ``size`` from their first token, for a batch of whole prompts: (first row of every piece and the end,
        int32 on the device; length of the longest piece)."""
        assert self.fresh
        if ("chunks", size) not in self.made:
            cu = [0]
            for n in self.lengths:
                cu += [cu[-1] + min(at + size, n) for at in range(0, n, size)]
            self.made["chunks", size] = (torch.tensor(cu, dtype=torch.int32).to(self.ids.device), min(size, self.longest))
        return self.made["chunks", size]

    def linear_tables(self, block: int, per_chunk: int):
        """The sequences cut into blocks of up to ``block`` rows, ``per_chunk`` of them (the last ones of a sequence: fewer) a chunk; int32 on the device:
        blocks (first row, rows), chunks (first block, blocks, first of its sequence, last of it), sequences (first chunk, chunks)."""
        if ("linear", block, per_chunk) not in self.made:
            blocks, chunks, seqs, row = [], [], [], 0
            for n in self.lengths:
                b0, c0 = len(blocks), len(chunks)
                blocks += [(row + at, min(block, n - at)) for at in range(0, n, block)]
                firsts = range(b0, len(blocks), per_chunk)
                chunks += [(b, min(per_chunk, len(blocks) - b), int(b == b0), int(b == firsts[-1])) for b in firsts]
                seqs.append((c0, len(chunks) - c0))
                row += n
            flat = torch.tensor([x for t in (blocks, chunks, seqs) for r in t for x in r], dtype=torch.int32).to(self.ids.device)
            nb, nc = 2 * len(blocks), 4 * len(chunks)
            self.made["linear", block, per_chunk] = (flat[:nb].view(-1, 2), flat[nb:nb + nc].view(-1, 4), flat[nb + nc:].view(-1, 2))
        return self.made["linear", block, per_chunk]

    def wanted_by_sequence(self) -> List[List[int]]:
        """per sequence: the wanted places among its own tokens, in order"""
        out, first = [], 0
        for n in self.lengths:
            out.append(list(range(n)) if self.rows is None else [r - first for r in self.rows if first <= r < first + n])
            first += n
        return out

    @property
    def fresh(self) -> bool:
        """every sequence starts at its first token"""
        return not any(self.starts)

    @property
    def longest(self) -> int:
        return max(self.lengths)

    @property
    def max_len(self) -> int:
        """cache rows the longest sequence holds after this step"""
        return max(s + n for s, n in zip(self.starts, self.lengths))

    @property
    def n_wanted(self) -> int:
        return self.ids.numel() if self.wanted is None else self.wanted.numel()

    @classmethod
    def build(cls, tokens: Sequence, slots: Sequence[int], starts: Sequence[int], wanted: Optional[Sequence[int]], device) -> "StepBatch":
        """tokens: one list of ids per sequence, or an int32 device tensor with one id per sequence (a decode step whose ids never visited the host)."""
        on_device = isinstance(tokens, torch.Tensor)
        lengths = [1] * len(slots) if on_device else [len(t) for t in tokens]
        cu, slot, pos, seq = [0], [], [], []
        for i, (n, s, p) in enumerate(zip(lengths, slots, starts)):
            cu.append(cu[-1] + n)
            slot += [s] * n
            pos += range(p, p + n)
            seq += [i] * n
        T = cu[-1]
        host = ([] if on_device else [i for t in tokens for i in t]) + slot + pos + seq + cu + (list(wanted) if wanted is not None else [])
        buf = torch.tensor(host, dtype=torch.int32).to(device)      # one copy to the device per step
        at = 0

        def take(n):
            nonlocal at
            at += n
            return buf[at - n:at]

        ids = tokens if on_device else take(T)
        slot, pos, seq, cu = take(T), take(T), take(T), take(len(slots) + 1)
        return cls(ids, slot, pos, cu, take(len(wanted)) if wanted is not None else None, lengths, list(starts), list(slots),
                   list(wanted) if wanted is not None else None, seq)


class Scheduler:
    """Slots and positions of the live requests of one model.  A batch claims the free slots it needs; when there are too few and nothing is running the
    caches are set up again for it (a larger batch), when something is running that is an error: batches do not grow."""

    def __init__(self, model, max_tokens: int):
        self.model, self.max_len = model, int(max_tokens)
        self.slots = 0                            # slots the caches have
        self.free: List[int] = []
        self.live: Dict[object, List[int]] = {}   # request -> [slot, tokens held]

    def _reserve(self, n: int) -> None:
        if len(self.free) >= n:
            return
        if self.live:
            raise RuntimeError(f"{n} requests start while {len(self.live)} are running and {len(self.free)} of {self.slots} slots are free")
        self.model.setup_caches(n, self.max_len)
        self.slots, self.free = n, list(range(n))

    def step(self, requests: Sequence, tokens, wanted: Optional[Sequence[Sequence[int]]] = None) -> Optional[torch.Tensor]:
        """Run ``tokens`` (per request: its next ids; or an int32 tensor, one id each) and return float32 logits [rows, vocab]: of the wanted places
        of each request in turn (``wanted[i]``: indices into tokens[i]), or of every request's last token when ``wanted`` is None.  No logits
        asked for: None."""
        new = [r for r in requests if r not in self.live]
        counts = [1] * len(requests) if isinstance(tokens, torch.Tensor) else [len(t) for t in tokens]
        if not requests or min(counts) < 1:
            raise ValueError("a step needs at least one token of every request in it")
        for r, n in zip(requests, counts):
            if (self.live[r][1] if r in self.live else 0) + n > self.max_len:
                raise ValueError(f"request {r!r} would hold more than {self.max_len} tokens")
        self._reserve(len(new))
        for r in new:
            self.live[r] = [self.free.pop(0), 0]
        starts, slots = [self.live[r][1] for r in requests], [self.live[r][0] for r in requests]
        rows, at = [], 0
        for i, n in enumerate(counts):
            rows += [at + j for j in (wanted[i] if wanted is not None else (n - 1,))]
            at += n
        batch = StepBatch.build(tokens, slots, starts, rows, self.model.device)
        logits = self.model.step(batch)
        for r, n in zip(requests, counts):
            self.live[r][1] += n
        return logits if rows else None

    def finish(self, request) -> None:
        """The request's slot is free for a later batch."""
        slot, _ = self.live.pop(request)
        self.free.append(slot)


@torch.no_grad()
def generate(model, prompts: Sequence[Sequence[int]], max_new_tokens: int, *, temperature: float = 0.8, top_k: Optional[int] = 200,
             stop_token: Optional[int] = None, max_batch: int = 16, scheduler: Optional[Scheduler] = None) -> List[List[int]]:
    """New tokens of every prompt.  Prompts run in lock-step batches of at most ``max_batch``; ``temperature`` 0 (or ``top_k`` 1) is greedy, anything
    else samples with gptfast's ``sample``."""
    if max_new_tokens < 1 or not prompts:
        return [[] for _ in prompts]
    sched = scheduler or Scheduler(model, max(len(p) for p in prompts) + max_new_tokens)
    greedy = temperature == 0 or top_k == 1

    def choose(logits):
        if greedy:
            return logits.argmax(-1).to(torch.int32)
        return torch.cat([G.sample(row.view(1, 1, -1), temperature, top_k)[0].view(1) for row in logits]).to(torch.int32)

    out: List[List[int]] = [[] for _ in prompts]
    order = sorted(range(len(prompts)), key=lambda i: -len(prompts[i]))   # batches of like lengths
    for first in range(0, len(order), max_batch):
        group = order[first:first + max_batch]
        nxt = choose(sched.step(group, [list(prompts[i]) for i in group]))
        made = [nxt]
        if stop_token is None:      # every request runs to the end: ids stay on the device until then
            for _ in range(max_new_tokens - 1):
                nxt = choose(sched.step(group, nxt))
                made.append(nxt)
            for i, ids in zip(group, torch.stack(made, 1).tolist()):
                out[i] = ids
                sched.finish(i)
            continue
        running, ids = list(group), nxt.tolist()
        while running:
            keep = []
            for i, t in zip(running, ids):
                out[i].append(t)
                if t == stop_token or len(out[i]) >= max_new_tokens:
                    sched.finish(i)
                else:
                    keep.append(i)
            running = keep
            if running:
                ids = choose(sched.step(running, [[out[i][-1]] for i in running])).tolist()
    return out
