"""Continuous batching for checkpoint-loaded models (models.ARCHITECTURES).

`Engine` owns the model and its caches and runs one step at a time: every entry of a step brings the next tokens of one
sequence -- a portion of a prompt or a single decoded token -- and all entries run as one batch.  `Scheduler` decides
what goes into each step (decoding sequences first, then prompt portions up to a token budget, new requests as long as
their whole length fits the pool), samples and ends requests.

A step's rows are ordered by the host: first the sequences that bring a single row, then the longer portions.  A step of
single rows only is replayed from a HIP graph captured per batch size: everything that changes from step to step is read
from one integer buffer at a fixed address.
"""
from __future__ import annotations

import dataclasses
from collections import deque
from typing import Dict, List, Optional, Sequence as Seq

import numpy as np
import torch

from . import ops
from .mem_cache.memory_pool import HybridCache
from .ops_hybrid import RowSeqs, assign_slots

SCAN_TILE = 64   # rows of a sequence the recurrence's tile kernel takes at a time


@dataclasses.dataclass
class Expansion:
    """Tokens the longer portions of a step can see under one window, sequence by sequence (device arrays)."""
    table_index: torch.Tensor   # per token: its place in the flattened request table
    row0: torch.Tensor          # per sequence: first row of its portion (of all rows), rows, first token, tokens in front
    rows: torch.Tensor
    tok0: torch.Tensor
    ahead: torch.Tensor
    max_rows: int


class StepBatch:
    """Rows of one step on the device.  All integers lie in one buffer, every array 16-byte aligned."""

    FIELDS = ("ids", "positions", "loc", "row_seq", "row_req", "row0", "rows", "start", "slot", "tile0", "tile_row", "tile_rows",
              "logit_rows")

    def __init__(self, host: Dict[str, np.ndarray], singles: int, req_to_token: torch.Tensor, max_context: int):
        self.host = host
        self.T = len(host["ids"])
        self.singles = singles
        self.wanted = len(host["logit_rows"])
        self.req_to_token = req_to_token
        self.max_context = max_context
        self._expansions: Dict[int, Expansion] = {}
        self._spans = {}
        n = 0
        for f in self.FIELDS:
            self._spans[f] = (n, len(host[f]))
            n += (len(host[f]) + 3) // 4 * 4
        self.ints = max(n, 4)

    def pack(self) -> torch.Tensor:
        buf = np.zeros(self.ints, dtype=np.int32)
        for f, (o, n) in self._spans.items():
            buf[o: o + n] = self.host[f]
        return torch.from_numpy(buf)

    def bind(self, dev: torch.Tensor):
        """Point the device arrays at `dev` (the packed integers)."""
        v = {f: dev[o: o + n] for f, (o, n) in self._spans.items()}
        self.ids, self.positions, self.loc = v["ids"], v["positions"], v["loc"]
        self.row_req, self.logit_rows = v["row_req"], v["logit_rows"]
        self.tile0, self.tile_row, self.tile_rows = v["tile0"], v["tile_row"], v["tile_rows"]
        self.seqs = RowSeqs(v["row_seq"], v["row0"], v["rows"], v["start"], v["slot"])
        return self

    def expansion(self, window: int) -> Expansion:
        e = self._expansions.get(window)
        if e is None:
            h, n1 = self.host, self.singles
            start, rows, row0, slot = (h[k][n1:].astype(np.int64) for k in ("start", "rows", "row0", "slot"))
            lo = np.maximum(start - window + 1, 0) if window else np.zeros_like(start)
            count = start + rows - lo
            tok0 = np.cumsum(count) - count
            table = np.repeat(slot * self.req_to_token.stride(0) + lo - tok0, count) + np.arange(int(count.sum()))
            pads = [np.asarray(a, dtype=np.int64) for a in (row0, rows, tok0, start - lo, table)]
            at, sizes = [], 0
            for a in pads:
                at.append(sizes)
                sizes += (len(a) + 3) // 4 * 4
            buf = np.zeros(sizes, dtype=np.int32)
            for o, a in zip(at, pads):
                buf[o: o + len(a)] = a
            d = torch.from_numpy(buf).to(self.req_to_token.device)
            r0, r, t0, ah, ti = (d[o: o + len(a)] for o, a in zip(at, pads))
            e = self._expansions[window] = Expansion(ti, r0, r, t0, ah, int(rows.max()))
        return e


@dataclasses.dataclass
class Sequence:
    """A live sequence: its row of the request table (and state slot), how many tokens are in the caches, their slots."""
    slot: int
    length: int = 0
    locs: List[torch.Tensor] = dataclasses.field(default_factory=list)


@dataclasses.dataclass
class Entry:
    """The next tokens of a sequence and the places among them whose logits are asked for."""
    seq: Sequence
    tokens: Seq[int]
    want: Seq[int] = ()


class _Graph:
    def __init__(self, ints, graph, logits):
        self.ints, self.graph, self.logits = ints, graph, logits


class Engine:
    def __init__(self, model, max_tokens: int, max_requests: int, max_context: Optional[int] = None, use_graph: bool = True):
        """max_tokens: slots of the pools (all live sequences together); max_requests: live sequences."""
        self.model, self.device = model, model.device
        self.max_context = min(max_context or model.max_context, model.max_context)
        self.cache = HybridCache(model.cache_layers(), max_tokens, max_requests, self.max_context, model.dtype, model.device)
        self.req_to_token = self.cache.req_pool.req_to_token
        if self.req_to_token.numel() >= 2 ** 31:
            raise ValueError("request table too large: fewer requests or a shorter context")
        # library products of the fp32 path may not be capturable; bf16 single-row steps are hand-written kernels only
        self.use_graph = use_graph and model.dtype == torch.bfloat16
        self.graphs: Dict[int, _Graph] = {}
        self._seen = set()

    # ---- sequences ---------------------------------------------------------------------------------------------------
    def open(self) -> Sequence:
        row = self.cache.req_pool.alloc(1)
        if row is None:
            raise RuntimeError("no free request slot")
        return Sequence(row[0])

    def close(self, seq: Sequence):
        """Give back what a sequence holds in the pools."""
        if seq.locs:
            self.cache.allocator.free(torch.cat(seq.locs))
        seq.locs = []
        seq.length = 0
        self.cache.req_pool.free(seq.slot)
        seq.slot = -1

    def free_tokens(self) -> int:
        return self.cache.allocator.available_size()

    # ---- one step ----------------------------------------------------------------------------------------------------
    def _check(self, entries):
        seen = set()
        total = 0
        for e in entries:
            if e.seq.slot < 0 or id(e.seq) in seen:
                raise ValueError("a step takes every open sequence at most once")
            seen.add(id(e.seq))
            n = len(e.tokens)
            if n == 0:
                raise ValueError("an entry brings no tokens")
            if e.seq.length + n > self.max_context:
                raise ValueError(f"a sequence of {e.seq.length + n} tokens, at most {self.max_context}")
            if min(e.tokens) < 0 or max(e.tokens) >= self.model.vocab:
                raise ValueError("token id outside the vocabulary")
            if any(not 0 <= w < n for w in e.want):
                raise ValueError("a wanted place lies outside the entry's tokens")
            total += n
        if total > self.free_tokens():
            raise RuntimeError(f"KV pool exhausted: {total} tokens, {self.free_tokens()} free")
        return total

    def _layout(self, entries, total, all_rows):
        """Host arrays of a step: the entries' order among the rows, and every entry's first row."""
        loc = self.cache.allocator.alloc(total)
        if total == len(entries):
            return self._layout_singles(entries, loc, all_rows)
        order = sorted(range(len(entries)), key=lambda i: len(entries[i].tokens) > 1)   # stable: single rows first
        ids, pos, row_seq, row_req, first = [], [], [], [], {}
        row0, rows, start, slot, tile0, tile_row, tile_rows = [], [], [], [], [], [], []
        r = singles = 0
        for s, i in enumerate(order):
            e = entries[i]
            n, at = len(e.tokens), e.seq.length
            e.seq.locs.append(loc[r: r + n])
            first[i] = r
            ids.append(np.asarray(e.tokens, dtype=np.int32))
            pos.append(np.arange(at, at + n))
            row_seq.append(np.full(n, s))
            row_req.append(np.full(n, e.seq.slot))
            row0.append(r)
            rows.append(n)
            start.append(at)
            slot.append(e.seq.slot)
            tile0.append(len(tile_row))
            if n == 1:
                singles += 1
            else:
                t = np.arange(0, n, SCAN_TILE)
                tile_row += list(r + t)
                tile_rows += list(np.minimum(SCAN_TILE, n - t))
            e.seq.length = at + n
            r += n
        want = list(range(total)) if all_rows else [first[i] + w for i, e in enumerate(entries) for w in e.want]
        cat = lambda a: np.concatenate(a).astype(np.int32)
        i32 = lambda a: np.asarray(a, dtype=np.int32)
        host = dict(ids=cat(ids), positions=cat(pos), loc=loc.numpy().astype(np.int32), row_seq=cat(row_seq), row_req=cat(row_req),
                    row0=i32(row0), rows=i32(rows), start=i32(start), slot=i32(slot), tile0=i32(tile0), tile_row=i32(tile_row),
                    tile_rows=i32(tile_rows), logit_rows=i32(want))
        return StepBatch(host, singles, self.req_to_token, self.max_context), first

    def _layout_singles(self, entries, loc, all_rows):
        """The same for a step of single rows (every decode step)."""
        n = len(entries)
        seqs = [e.seq for e in entries]
        at = np.asarray([s.length for s in seqs], dtype=np.int32)
        slot = np.asarray([s.slot for s in seqs], dtype=np.int32)
        rows, none = np.arange(n, dtype=np.int32), np.zeros(0, dtype=np.int32)
        for s, one in zip(seqs, loc.split(1)):
            s.locs.append(one)
            s.length += 1
        want = rows if all_rows else np.asarray([i for i, e in enumerate(entries) for _ in e.want], dtype=np.int32)
        host = dict(ids=np.asarray([e.tokens[0] for e in entries], dtype=np.int32), positions=at, loc=loc.numpy().astype(np.int32),
                    row_seq=rows, row_req=slot, row0=rows, rows=np.ones(n, dtype=np.int32), start=at, slot=slot,
                    tile0=np.zeros(n, dtype=np.int32), tile_row=none, tile_rows=none, logit_rows=want)
        return StepBatch(host, n, self.req_to_token, self.max_context), dict(enumerate(range(n)))

    def _forward(self, batch, collect=None):
        assign_slots(self.req_to_token, batch.seqs.row_seq, batch.seqs.slot, batch.positions, batch.loc)
        return self.model.forward(batch, self.cache, collect)

    def step(self, entries: List[Entry], collect: Optional[list] = None) -> Optional[torch.Tensor]:
        """Runs the entries as one batch; fp32 logits [wanted, vocab] in the order of the entries and their `want`.
        collect (debugging aid): receives the residual stream after every layer run, rows in the step's own order."""
        if not entries:
            return None
        total = self._check(entries)
        graphable = self.use_graph and total == len(entries) and collect is None
        batch, first = self._layout(entries, total, all_rows=graphable)
        if not graphable:
            return self._forward(batch.bind(batch.pack().to(self.device)), collect)
        logits = self._graph_step(batch)
        pick = [first[i] + w for i, e in enumerate(entries) for w in e.want]
        if not pick:
            return None
        if pick == list(range(total)):
            return logits.clone()
        return logits.index_select(0, torch.tensor(pick, device=self.device))

    def _graph_step(self, batch):
        B = batch.T
        g = self.graphs.get(B)
        if g is None and B not in self._seen:       # the first step of a size runs eagerly: lazy initialisations
            self._seen.add(B)
            return self._forward(batch.bind(batch.pack().to(self.device)))
        if g is None:
            ints = batch.pack().to(self.device)
            static = StepBatch(batch.host, batch.singles, self.req_to_token, self.max_context).bind(ints)
            torch.cuda.synchronize(self.device)
            graph = torch.cuda.CUDAGraph()
            with torch.cuda.graph(graph):
                logits = self._forward(static)
            g = self.graphs[B] = _Graph(ints, graph, logits)
        g.ints.copy_(batch.pack())
        g.graph.replay()
        return g.logits


# ---- sampling and scheduling ---------------------------------------------------------------------------------------------
@dataclasses.dataclass
class SamplingParams:
    max_new_tokens: int = 16
    temperature: float = 0.0          # 0: greedy
    top_k: int = 0                    # 0: no limit
    top_p: float = 1.0
    min_p: float = 0.0
    stop_token_ids: Seq[int] = ()


class Sampler:
    def __init__(self, device, seed: int = 0):
        self.gen = torch.Generator(device=device).manual_seed(seed)

    def __call__(self, logits: torch.Tensor, params: List[SamplingParams]) -> List[int]:
        out = torch.empty(logits.shape[0], dtype=torch.int64, device=logits.device)
        ops.argmax(logits, out)
        drawn = [i for i, p in enumerate(params) if p.temperature > 0]
        if drawn:
            at = torch.tensor(drawn, device=logits.device)
            ps = [params[i] for i in drawn]
            vec = lambda v, dt: torch.tensor(v, dtype=dt, device=logits.device)
            V = logits.shape[1]
            probs = torch.softmax(logits.index_select(0, at) / vec([p.temperature for p in ps], torch.float32)[:, None], -1)
            uniform = torch.rand(len(ps), device=logits.device, generator=self.gen)
            # two passes over the filters, as the sampling kernel offers them: min-p, or top-k and top-p together
            picks = torch.empty(len(ps), dtype=torch.int64, device=logits.device)
            for use_min_p in (False, True):
                rows = [j for j, p in enumerate(ps) if (p.min_p > 0) == use_min_p]
                if not rows:
                    continue
                r = torch.tensor(rows, device=logits.device)
                k = vec([ps[j].top_k if ps[j].top_k > 0 else V for j in rows], torch.int32)
                pp = vec([ps[j].top_p for j in rows], torch.float32)
                mp = vec([ps[j].min_p for j in rows], torch.float32)
                sub, un = probs.index_select(0, r).contiguous(), uniform.index_select(0, r)
                if use_min_p:
                    sub = ops.top_p_renorm_probs(ops.top_k_renorm_probs(sub, k), pp)
                    picks[r] = ops.sampling_from_probs(sub, un, min_p=mp).long()
                else:
                    picks[r] = ops.sampling_from_probs(sub, un, top_k=k, top_p=pp).long()
            out[at] = picks
        return out.tolist()


@dataclasses.dataclass
class Request:
    id: object
    prompt: List[int]
    params: SamplingParams
    seq: Optional[Sequence] = None
    output: List[int] = dataclasses.field(default_factory=list)
    finished: bool = False

    @property
    def reserve(self) -> int:
        """Tokens the request can come to hold."""
        return len(self.prompt) + max(self.params.max_new_tokens - 1, 0)


class Scheduler:
    def __init__(self, engine: Engine, prefill_budget: int = 2048, seed: int = 0):
        """prefill_budget: prompt tokens a step takes at most beside the decoding sequences."""
        if prefill_budget < 1:
            raise ValueError("prefill_budget must be positive")
        self.engine, self.budget = engine, prefill_budget
        self.sampler = Sampler(engine.device, seed)
        self.waiting: deque = deque()
        self.running: List[Request] = []

    def add(self, prompt: Seq[int], params: SamplingParams = SamplingParams(), id=None) -> Request:
        r = Request(id, [int(t) for t in prompt], params)
        if not r.prompt:
            raise ValueError("an empty prompt")
        if min(r.prompt) < 0 or max(r.prompt) >= self.engine.model.vocab:
            raise ValueError("token id outside the vocabulary")
        if r.reserve > min(self.engine.max_context, self.engine.cache.allocator.size):
            raise ValueError(f"the request can come to hold {r.reserve} tokens, more than the engine offers")
        if params.max_new_tokens < 1:
            raise ValueError("max_new_tokens must be positive")
        self.waiting.append(r)
        return r

    def _admit(self):
        """First come, first served; a request starts when its whole length fits beside what the running ones may need."""
        while self.waiting:
            need = sum(r.reserve - r.seq.length for r in self.running)
            r = self.waiting[0]
            if r.reserve + need > self.engine.free_tokens() or not self.engine.cache.req_pool.available_size():
                return
            self.waiting.popleft()
            r.seq = self.engine.open()
            self.running.append(r)

    def step(self) -> List[Request]:
        """One engine step; returns the requests that ended with it."""
        self._admit()
        entries, owners, left = [], [], self.budget
        for r in self.running:
            if r.output:
                entries.append(Entry(r.seq, [r.output[-1]], [0]))
                owners.append(r)
        for r in self.running:
            if not r.output and left > 0:
                n = min(len(r.prompt) - r.seq.length, left)
                part = r.prompt[r.seq.length: r.seq.length + n]
                last = r.seq.length + n == len(r.prompt)
                entries.append(Entry(r.seq, part, [n - 1] if last else []))
                if last:
                    owners.append(r)
                left -= n
        if not entries:
            return []
        logits = self.engine.step(entries)
        if logits is None:
            return []
        done = []
        for r, t in zip(owners, self.sampler(logits, [r.params for r in owners])):
            r.output.append(t)
            if len(r.output) >= r.params.max_new_tokens or t in r.params.stop_token_ids:
                r.finished = True
                self.engine.close(r.seq)
                done.append(r)
        self.running = [r for r in self.running if not r.finished]
        return done

    def run(self):
        """Steps until every request has ended."""
        while self.waiting or self.running:
            self.step()

    def generate(self, prompts: Seq[Seq[int]], params: SamplingParams = SamplingParams()) -> List[List[int]]:
        reqs = [self.add(p, params, i) for i, p in enumerate(prompts)]
        self.run()
        return [r.output for r in reqs]
