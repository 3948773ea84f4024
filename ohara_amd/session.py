"""Device-resident decode loop for models whose step is a chain of launches: the surface of
``ohara_amd.llama.DecodeSession`` for any model with ``forward``, ``build_kv_cache`` and
``decode_step(ids, kv_cache, pos_dev)``."""

from __future__ import annotations

import torch

from . import ops


class GraphDecodeSession:
    """One batch of equal-length sequences: the prompt goes through ``model.forward`` once, then every token is one replay
    of a captured graph (the step's launches and the selection that feeds the next one; position, fed ids and step
    index live on the device)."""

    GRAPH_STEPS = 8  # steps in the second captured graph: one host launch for eight tokens

    persistent = False

    def __init__(self, model, batch: int, max_new_tokens: int, valid_vocab: int = 0, kv_cache=None, sampling=None, u=None):
        """``sampling`` / ``u`` as in ``ohara_amd.llama.DecodeSession``."""
        self.model, self.batch, self.valid_vocab = model, batch, valid_vocab
        self.sampling = sampling if (sampling is not None and sampling.temperature > 0) else None
        rows, dev = max(max_new_tokens, 1), model.device
        self.u = None
        if self.sampling is not None:
            if u is None:
                u = torch.rand(rows, batch, device=dev, dtype=torch.float32)
            if u.shape != (rows, batch):
                raise ValueError("u must have shape (max_new_tokens, batch)")
            self.u = u.to(device=dev, dtype=torch.float32).contiguous()
            self._sample_ws = ops.sample_workspace(dev)  # this session's own: sessions may overlap
        self.cache = kv_cache if kv_cache is not None else model.build_kv_cache(batch)
        self.history = torch.zeros(rows, batch, dtype=torch.int64, device=dev)
        self.ids = torch.zeros(batch, dtype=torch.int64, device=dev)
        self.step_state = torch.zeros(4, dtype=torch.int32, device=dev)  # position, step, arrivals, unused
        self.logits = None  # (batch, vocab) of the last eager step or of the captured one
        self.pos = self.produced = 0
        self.graph = self.graph_multi = None

    def _select(self, logits) -> None:
        """The next ids, their history entry and the advance of position and step, all on the device."""
        vv = self.valid_vocab or None
        if self.sampling is None:
            ops.argmax(logits, vv, next_ids=self.ids, history=self.history, step_state=self.step_state)
        else:
            ops.sample_topk_topp(logits, self.sampling.temperature, self.sampling.top_k, self.sampling.top_p, self.u, vv,
                                 out=self.ids, history=self.history, step_state=self.step_state, u_per_step=True,
                                 workspace=self._sample_ws)

    @torch.no_grad()
    def prefill(self, prompt_ids: torch.Tensor) -> None:
        if prompt_ids.ndim != 2 or prompt_ids.shape[0] != self.batch:
            raise ValueError("input token IDs must have shape (batch, sequence)")
        logits = self.model.forward(prompt_ids, self.cache, 0, last_only=True)[:, 0]  # validates the rest
        P = prompt_ids.shape[1]
        # the selection advances the position by one: it starts one short of the first decoded token's
        self.step_state.copy_(torch.tensor([P - 1, 0, 0, 0], dtype=torch.int32))
        self._select(logits)
        self.logits = logits
        self.pos, self.produced = P, 1

    def restart(self, u: torch.Tensor | None = None) -> None:
        """Forget the sequences decoded so far; caches and captured graphs are kept."""
        for cc in self.cache:
            cc.length, cc.batch_size, cc.lengths = 0, None, None
        self.pos = self.produced = 0
        if u is not None:
            if self.u is None:
                raise ValueError("this session selects greedily: it takes no uniform draws")
            if u.ndim != 2 or u.shape[1] != self.batch or u.shape[0] > self.u.shape[0]:
                raise ValueError("u must have shape (rows <= max_new_tokens, batch)")
            self.u[: u.shape[0]].copy_(u)

    def feed(self, ids: torch.Tensor) -> None:
        """Replace the ids the next step consumes (teacher forcing); the history keeps what was selected."""
        if self.produced < 1:
            raise RuntimeError("prefill first")
        ids = ids.reshape(-1)
        if ids.numel() != self.batch:
            raise ValueError("one id per sequence is required")
        self.ids.copy_(ids.to(device=self.model.device, dtype=torch.int64))

    @torch.no_grad()
    def _launch_step(self) -> None:
        self.logits = self.model.decode_step(self.ids, self.cache, self.step_state)
        self._select(self.logits)

    def _room(self, n: int) -> None:
        if self.produced < 1:
            raise RuntimeError("prefill first")
        if self.pos + n > self.model.config.max_sequence_length:
            raise ValueError("input exceeds max_sequence_length")
        if self.produced + n > self.history.shape[0]:
            raise ValueError("max_new_tokens exceeded")

    def _advance(self, n: int) -> None:
        self.pos += n
        self.produced += n
        for cc in self.cache:
            cc._commit(self.batch, self.pos)

    def step(self) -> None:
        """One eager decode step (enqueue only)."""
        self._room(1)
        self._launch_step()
        self._advance(1)

    def capture(self) -> None:
        """One eager step (allocations, lazy loading), then one step into one HIP graph and GRAPH_STEPS into another."""
        if self.graph is not None:
            return
        self.step()
        torch.cuda.synchronize()
        graph = torch.cuda.CUDAGraph()
        with torch.cuda.graph(graph):
            self._launch_step()
        many = torch.cuda.CUDAGraph()
        with torch.cuda.graph(many):
            for _ in range(self.GRAPH_STEPS):
                self._launch_step()
        self.graph, self.graph_multi = graph, many

    def run(self, n: int, use_graph: bool = True) -> None:
        """Enqueue n more decode steps."""
        if n <= 0:
            return
        self._room(n)
        if not use_graph or (self.graph is None and n < 3):
            for _ in range(n):
                self.step()
            return
        if self.graph is None:
            self.capture()
            n -= 1
        many, rest = divmod(n, self.GRAPH_STEPS)
        for _ in range(many):
            self.graph_multi.replay()
        for _ in range(rest):
            self.graph.replay()
        self._advance(n)

    def error_word(self):
        """No barrier waits in a chain of launches: nothing to report (see ``DecodeSession.error_word``)."""
        return None

    def check_error(self) -> None:
        pass

    def tokens(self) -> torch.Tensor:
        """(B, produced) generated ids (synchronises)."""
        return self.history[: self.produced].t().contiguous()
