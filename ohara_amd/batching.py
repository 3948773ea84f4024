"""Continuous batching on the decode path: sequences of different lengths share one batch, join
when a slot is free and leave when they finish.

The reference drives `Llama.forward` with a single scalar position for the whole batch
(ohara/models/llama.py:287-299, ohara/chat_engine.py:395-405), so all sequences of a batch must
have the same length and start together.  Here every slot of the KV caches has its own length: a
prompt is prefilled into its slot alone, and one decode step advances every active slot at its own
position (`Llama.forward` with one position per sequence).  Selection is greedy or the fused
temperature / top-k / top-p sampler of ohara/chat_engine.py:51-82.
"""

from __future__ import annotations

import torch

from . import ops
from .llama import Llama


class ContinuousBatcher:
    def __init__(self, model: Llama, slots: int, sampling=None, valid_vocab: int = 0, generator=None, int8: bool = False):
        if slots < 1:
            raise ValueError("batch_size must be at least 1")
        self.model, self.slots = model, slots
        self.sampling = sampling if (sampling is not None and sampling.temperature > 0) else None
        self.valid_vocab = valid_vocab
        self.generator = generator
        self.cache = model.build_kv_cache(slots, int8=int8)  # int8: the caches of ohara/modules/kv_cache.py:15-32
        for c in self.cache:
            c._commit_ragged(slots, [0] * slots)
        self.active = [False] * slots
        self.lengths = [0] * slots
        self.last = torch.zeros(slots, dtype=torch.int64, device=model.device)
        self.seq_pos = torch.zeros(slots, dtype=torch.int32, device=model.device)
        self.active_dev = torch.zeros(slots, dtype=torch.uint8, device=model.device)
        self._toks = self._u = self._graph = None

    def free_slots(self) -> list[int]:
        return [b for b in range(self.slots) if not self.active[b]]

    def _select(self, logits: torch.Tensor) -> torch.Tensor:
        """logits (rows, V) -> ids (rows,) on the device."""
        vv = self.valid_vocab or None
        if self.sampling is None:
            return ops.argmax(logits, valid_vocab=vv)
        u = torch.rand(logits.shape[0], device=logits.device, dtype=torch.float32, generator=self.generator)
        return ops.sample_topk_topp(logits, self.sampling.temperature, self.sampling.top_k, self.sampling.top_p, u,
                                    valid_vocab=vv)

    def _padded_forward(self, slots: list[int], tokens: list, last_only: bool) -> torch.Tensor:
        """The given tokens of several slots in one call (models with ``supports_seq_lens``), each from its slot's own
        position -> logits (rows, S or 1, V); rows shorter than the longest are padded."""
        lens = [len(t) for t in tokens]
        ids = torch.zeros(len(slots), max(lens), dtype=torch.int64)
        for row, t in zip(ids, tokens):
            row[: len(t)] = t
        return self.model.forward(ids, self.cache, [self.lengths[b] for b in slots], last_only=last_only, seq_lens=lens,
                                  slots=slots)

    def _prefill(self, slots: list[int], prompts: list, last_only: bool = True) -> list[torch.Tensor]:
        """Run prompts (1-D ids, on the host) into free slots -> the logits (1 or len, V) of each: one call for all where the
        model takes prompts of different lengths, else one call per prompt over its slot's rows of the cache."""
        for b in slots:
            for c in self.cache:
                c.lengths[b] = 0
            self.lengths[b] = 0
        if getattr(self.model, "supports_seq_lens", False):
            logits = self._padded_forward(slots, prompts, last_only)
            out = [row[: 1 if last_only else len(p)] for row, p in zip(logits, prompts)]
        else:
            out = []
            for b, ids in zip(slots, prompts):
                views = [c._row_view(b) for c in self.cache]
                out.append(self.model.forward(ids.view(1, -1).to(self.model.device), views, 0, last_only=last_only)[0])
        for b, ids in zip(slots, prompts):
            self._book(b, len(ids))
        return out

    def _book(self, b: int, length: int) -> None:
        """Slot b holds ``length`` tokens from now on."""
        for c in self.cache:
            c.lengths[b] = length
            c.length = max(c.lengths)
        self.lengths[b] = length
        self.active[b] = True
        self.seq_pos[b] = length
        self.active_dev[b] = 1

    def _host_ids(self, tokens, start: int = 0) -> torch.Tensor:
        ids = torch.as_tensor(tokens, dtype=torch.int64).reshape(-1).cpu()
        if ids.numel() < 1:
            raise ValueError("input sequence cannot be empty")
        if start + ids.numel() > self.model.config.max_sequence_length:
            raise ValueError("input exceeds max_sequence_length")
        return ids

    @torch.no_grad()
    def add(self, prompt_ids) -> tuple[int, int]:
        """Prefill a prompt (1-D ids) into a free slot -> (slot, first generated id)."""
        return self.add_many([prompt_ids])[0]

    @torch.no_grad()
    def add_many(self, prompts) -> list[tuple[int, int]]:
        """Prefill several prompts into free slots -> [(slot, first generated id)]."""
        free = self.free_slots()
        if len(free) < len(prompts):
            raise RuntimeError("no free slot")
        prompts = [self._host_ids(p, start=1) for p in prompts]  # room for one generated token at least
        slots = free[: len(prompts)]
        out = []
        for b, logits in zip(slots, self._prefill(slots, prompts)):
            tok = self._select(logits.reshape(1, -1))
            self.last[b:b + 1] = tok
            out.append((b, int(tok.item())))
        return out

    @torch.no_grad()
    def feed(self, entries) -> list[tuple[int, torch.Tensor]]:
        """One step over GIVEN tokens instead of selected ones: ``entries`` holds (slot, ids), slot None for a sequence that
        starts -> [(slot, logits (len(ids), V))] in the same order.  One id for each active slot runs the decode step of
        ``step``; anything else runs the prompt path, all entries in one call where the model takes tokens of different
        slots and lengths.  The next ``step`` continues from the last of the ids fed and the token after it is the
        caller's to select."""
        entries = [(b, self._host_ids(ids, 0 if b is None else self.lengths[b])) for b, ids in entries]
        named = [b for b, _ in entries if b is not None]
        if any(not self.active[b] for b in named) or len(set(named)) != len(named):
            raise ValueError("entries must name distinct active slots")
        free = iter(self.free_slots())
        if len(entries) - len(named) > len(self.free_slots()):
            raise RuntimeError("no free slot")
        fresh = [b is None for b, _ in entries]
        slots = [next(free) if b is None else b for b, _ in entries]
        tokens = [ids for _, ids in entries]
        if all(fresh):
            out = self._prefill(slots, tokens, last_only=False)
        elif not any(fresh) and all(len(t) == 1 for t in tokens) and sorted(slots) == [b for b in range(self.slots) if self.active[b]]:
            for b, t in zip(slots, tokens):
                self.last[b] = int(t)
            logits = self._device_forward()
            out = [logits[b] for b in slots]
            for c in self.cache:
                c.lengths = list(self.lengths)
            for b in slots:
                self._book(b, self.lengths[b] + 1)
        elif getattr(self.model, "supports_seq_lens", False):
            for b, new in zip(slots, fresh):
                if new:
                    self._book(b, 0)
            logits = self._padded_forward(slots, tokens, False)
            out = [row[: len(t)] for row, t in zip(logits, tokens)]
            for b, t in zip(slots, tokens):
                self._book(b, self.lengths[b] + len(t))
        else:
            raise ValueError("this model cannot mix prompts and continued sequences in one step")
        return list(zip(slots, out))

    def remove(self, slot: int) -> None:
        self.active[slot] = False
        self.lengths[slot] = 0
        self.last[slot] = 0
        self.seq_pos[slot] = 0
        self.active_dev[slot] = 0
        for c in self.cache:
            c.lengths[slot] = 0

    def _device_forward(self) -> torch.Tensor:
        """Logits (slots, 1, V) of the fed ids at the slots' own positions."""
        return self.model.forward(self.last.view(self.slots, 1), self.cache, list(self.lengths), last_only=True,
                                  seq_pos=self.seq_pos)

    def _device_step(self) -> None:
        """Everything of a step that runs on the device, with no host synchronisation: forward at
        the slots' own positions, selection, position advance, next inputs.  Capturable."""
        logits = self._device_forward()
        vv = self.valid_vocab or None
        if self.sampling is None:
            ops.argmax(logits.view(self.slots, -1), valid_vocab=vv, next_ids=self._toks)
        else:
            ops.sample_topk_topp(logits.view(self.slots, -1), self.sampling.temperature, self.sampling.top_k,
                                 self.sampling.top_p, self._u, valid_vocab=vv, out=self._toks)
        # idle slots stay at position 0 and are fed id 0; active ones advance and are fed what they selected
        ops.advance_ragged(self.seq_pos, self.active_dev, self._toks, self.last, 1)

    def _enqueue_step(self, use_graph: bool) -> None:
        """One decode step of every active slot, enqueued; the host books advance, nothing is read back."""
        if max(n for n, a in zip(self.lengths, self.active) if a) + 1 > self.model.config.max_sequence_length:
            raise ValueError("input exceeds max_sequence_length")
        if self._toks is None:
            self._toks = torch.zeros(self.slots, dtype=torch.int64, device=self.model.device)
            self._u = torch.zeros(self.slots, dtype=torch.float32, device=self.model.device)
        if self.sampling is not None:
            self._u.copy_(torch.rand(self.slots, device=self.model.device, dtype=torch.float32, generator=self.generator))
        if use_graph and self._graph is None:
            # the capture itself executes nothing: the books it touches are restored, and the step
            # is then replayed like any other
            torch.cuda.synchronize()
            g = torch.cuda.CUDAGraph()
            with torch.cuda.graph(g):
                self._device_step()
            self._graph = g
        if use_graph:
            self._graph.replay()
        else:
            self._device_step()
        for b in range(self.slots):
            if self.active[b]:
                self.lengths[b] += 1
        for c in self.cache:
            c.lengths = list(self.lengths)
            c.length = max(self.lengths)

    @torch.no_grad()
    def step(self, use_graph: bool = True) -> dict[int, int]:
        """One decode step for every active slot -> {slot: new id}.  Idle slots ride along at
        position 0 of their own cache rows (overwritten when the slot is taken again).  The device
        work is captured once into a HIP graph (positions, inputs and the active mask live in
        device tensors, so joins and leaves need no re-capture) and replayed per step."""
        if not any(self.active):
            return {}
        self._enqueue_step(use_graph)
        host = self._toks.tolist()
        return {b: host[b] for b in range(self.slots) if self.active[b]}

    @torch.no_grad()
    def steps(self, n: int, use_graph: bool = True) -> dict[int, list[int]]:
        """``n`` decode steps of every active slot with ONE read-back at the end -> {slot: its n new ids}: the
        chunked read-back of the single-sequence engines (a stop id is looked for in the chunk afterwards; a
        slot that met one has run on to the end of the chunk and is trimmed and removed by the caller)."""
        if n < 1 or not any(self.active):
            return {}
        if max(m for m, a in zip(self.lengths, self.active) if a) + n > self.model.config.max_sequence_length:
            raise ValueError("input exceeds max_sequence_length")
        rows = torch.empty(n, self.slots, dtype=torch.int64, device=self.model.device)
        for i in range(n):
            self._enqueue_step(use_graph)
            rows[i].copy_(self._toks)
        host = rows.t().tolist()
        return {b: host[b] for b in range(self.slots) if self.active[b]}
