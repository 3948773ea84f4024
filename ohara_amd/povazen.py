"""Povazen: a decoder whose layers mix by attention with a distance bias or by a gated delta rule, in the
order its config lists them, with norms on the sublayer outputs and a causal convolution in front of
every mixer.

    x <- x + norm1(mixer(x + conv(x)));   x <- x + norm2(swiglu(x))     (layers without a feed-forward: the first only)

The call surface is the other models': ``forward(tokens, kv_cache, position)``, ``build_kv_cache``, ``session``,
``generate_greedy``; ``position`` may be one per sequence, prompts of one call may have different lengths
(``seq_lens``) and sit in chosen cache rows (``slots``).  ``dtype`` float32 serves the model in 32-bit throughout.

Decode steps run 4 launches per recurrent layer and 5 per attention layer (+ 3 with a feed-forward), all
capturable: residual update, norm, convolution and ring are one launch, and everything of the delta rule
between its two matrix products is another.
"""

from __future__ import annotations

from dataclasses import dataclass, field

import torch

from . import ops
from ._lib import lib
from .hybrid import BF16, F32, BiasedAttention, ChannelDelta, GroupNorm, InputConv, Linear, SwiGLU, distance_slopes
from .llama import _check_ids_on_host
from .session import GraphDecodeSession
from .state_cache import LayerState


@dataclass
class PovazenLayer:
    type: str               # "attention" or "channel_delta"
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float = 1.0      # attention: of the scores
    conv: int = 0           # channel_delta: taps of the short convolutions
    ff: int = 0             # hidden width of the feed-forward, 0: none


@dataclass
class PovazenConfig:
    vocab_size: int
    hidden_size: int
    layers: list = field(default_factory=list)
    conv_taps: int = 1
    norm_eps: float = 1e-6
    norm_groups: int = 1
    logit_softcap: float = 0.0      # 0: none
    max_sequence_length: int = 4096  # cache capacity per sequence: the design itself has no limit

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)

    @property
    def num_attention_heads(self) -> int:
        return max(layer.heads for layer in self.layers)

    @classmethod
    def from_dict(cls, payload: dict, max_sequence_length: int | None = None) -> "PovazenConfig":
        """The contents of a config.json whose "architecture" is "Povazen"."""
        layers = []
        for i, entry in enumerate(payload["layers"]):
            m, mlp = entry["mixer"], entry.get("mlp")
            kind = entry["type"]
            if kind not in ("attention", "channel_delta"):
                raise ValueError(f"layer {i}: unknown mixer {kind!r}")
            if mlp is not None and mlp.get("kind", "dense") != "dense":
                raise ValueError(f"layer {i}: unknown feed-forward {mlp['kind']!r}")
            layers.append(PovazenLayer(
                type=kind, heads=int(m["heads"]), kv_heads=int(m["kv_heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]),
                scale=float(m["scale"]) if kind == "attention" else 1.0, conv=int(m["conv"]) if kind == "channel_delta" else 0,
                ff=0 if mlp is None else int(mlp["ff"])))
        extra = {} if max_sequence_length is None else {"max_sequence_length": int(max_sequence_length)}
        return cls(vocab_size=int(payload["vocab"]), hidden_size=int(payload["width"]), layers=layers,
                   conv_taps=int(payload["canon"]["taps"]), norm_eps=float(payload["norm"]["eps"]),
                   norm_groups=int(payload["norm"]["groups"]), logit_softcap=float(payload.get("logit_softcap") or 0.0), **extra)


def _validate(c: PovazenConfig) -> None:
    if c.vocab_size < 2:
        raise ValueError("vocab_size must be at least 2")
    if c.hidden_size < 1 or not c.layers:
        raise ValueError("hidden_size and num_hidden_layers must be positive")
    if c.norm_groups < 1 or c.hidden_size % c.norm_groups:
        raise ValueError("norm groups must divide hidden_size")
    if c.conv_taps < 1 or c.max_sequence_length < 1:
        raise ValueError("conv_taps and max_sequence_length must be positive")
    if c.logit_softcap < 0:
        raise ValueError("logit_softcap cannot be negative")


class Povazen:
    supports_last_only = True   # forward(..., last_only=True) computes the last row of logits only
    supports_seq_lens = True    # forward(..., seq_lens=, slots=): prompts of different lengths, chosen cache rows

    def __init__(self, config: PovazenConfig, state: dict, device="cuda", dtype=BF16):
        _validate(config)
        if dtype not in (BF16, F32):
            raise ValueError("Povazen is served in bfloat16 or float32")
        lib()  # fail loudly now if the HIP library is missing
        self.config, self.device, self.dtype = config, torch.device(device), dtype
        c, kw = config, dict(dtype=dtype, device=self.device)

        def get(name, *shape):
            t = state[name]
            if tuple(t.shape) != shape:
                raise ValueError(f"{name} has shape {tuple(t.shape)}, the config says {shape}")
            return t

        d = c.hidden_size
        norm = lambda name: GroupNorm(get(name, d), c.norm_groups, c.norm_eps, self.device)  # noqa: E731
        self.embed = get("embed", c.vocab_size, d).detach().to(device=self.device, dtype=dtype).contiguous()
        self.final_norm = norm("final.norm")
        self.head = Linear(get("head", c.vocab_size, d), exact=True, cap=c.logit_softcap, **kw)
        self.layers = []
        for i, layer in enumerate(c.layers):
            p = f"l{i}."
            block = dict(conv=InputConv(get(p + "canon1", d, c.conv_taps), self.device), norm1=norm(p + "norm1"),
                         mixer=self._mixer(layer, {k[len(p) + 4:]: t for k, t in state.items() if k.startswith(p + "mix.")}, kw),
                         mlp=None)
            if layer.ff:
                block["norm2"] = norm(p + "norm2")
                block["mlp"] = SwiGLU(get(p + "mlp.gate", layer.ff, d), get(p + "mlp.up", layer.ff, d),
                                      get(p + "mlp.down", d, layer.ff), **kw)
            self.layers.append(block)
        self.trace = None  # a list: forward() appends the residual stream after every layer to it
        torch.cuda.synchronize(self.device)

    def _mixer(self, layer: PovazenLayer, w: dict, kw: dict):
        sizes = dict(heads=layer.heads, kv_heads=layer.kv_heads, dim=layer.dim, vdim=layer.vdim, eps=self.config.norm_eps)
        if layer.type == "attention":
            return BiasedAttention((w["q"], w["q.b"]), (w["k"], w["k.b"]), (w["v"], w["v.b"]), (w["g"], None), w["o"],
                                   w["q.norm"], w["k.norm"], scale=layer.scale, slopes=distance_slopes(layer.heads), **sizes, **kw)
        if w["q.conv"].shape[1] != layer.conv:
            raise ValueError(f"short convolution has {w['q.conv'].shape[1]} taps, the config says {layer.conv}")
        return ChannelDelta(w["q"], w["k"], w["v"], w["q.conv"], w["k.conv"], w["v.conv"], w["b"], w["A_log"], w["a1"], w["a2"],
                            w["dt_bias"], w["g1"], w["g2"], w["norm"], w["o"], **sizes, **kw)

    def eval(self):
        return self

    def to(self, *args, **kwargs):
        """A request for the device / dtype the model was built with is a no-op, anything else raises."""
        for a in (*args, kwargs.get("device"), kwargs.get("dtype")):
            if isinstance(a, torch.dtype):
                if a != self.dtype:
                    raise ValueError(f"ohara_amd: the model was built in {self.dtype}; build it in {a} instead of casting it")
            elif a is not None:
                want = torch.device(a)
                if want.type != self.device.type or (want.index is not None and want.index != (self.device.index or 0)):
                    raise ValueError(f"ohara_amd: the model lives on {self.device}; build it on {want} instead of moving it")
        return self

    def parameters(self):
        yield self.embed
        yield self.final_norm.w
        yield from self.head.tensors()
        for block in self.layers:
            yield block["conv"].w
            yield block["norm1"].w
            yield from block["mixer"].tensors()
            if block["mlp"] is not None:
                yield block["norm2"].w
                yield from block["mlp"].tensors()

    def build_kv_cache(self, batch_size: int = 1, int8: bool = False) -> list[LayerState]:
        """One ``LayerState`` per layer: keys and values or the recurrent state and its convolution's past inputs, and the
        past inputs of the convolution in front of the mixer."""
        if batch_size < 1:
            raise ValueError("batch_size must be at least 1")
        if int8:
            raise ValueError("Povazen keeps its caches in the model's dtype (no int8 mode)")
        t = self.config.max_sequence_length
        return [LayerState(t, {"conv": b["conv"].state(batch_size), **b["mixer"].state(batch_size, t)}, i)
                for i, b in enumerate(self.layers)]

    @torch.no_grad()
    def forward(self, x: torch.Tensor, kv_cache: list | None = None, position_ids=None, *, last_only: bool = False,
                seq_pos: torch.Tensor | None = None, seq_lens=None, slots=None) -> torch.Tensor:
        """Logits (B, S, vocab), or (B, 1, vocab) of every sequence's last token with ``last_only``.  ``position_ids``: one
        position, or a list with one per sequence (``seq_pos``: the same as an int32 device tensor the caller keeps up to
        date).  ``seq_lens``: tokens of each sequence in this call, the rest of its row is padding.  ``slots``: the cache row
        of each sequence (rows not named are left alone)."""
        c = self.config
        if x.ndim != 2:
            raise ValueError("input token IDs must have shape (batch, sequence)")
        B, S = x.shape
        if isinstance(position_ids, torch.Tensor):
            position_ids = [int(p) for p in position_ids.tolist()] if position_ids.numel() > 1 else int(position_ids.item())
        if S < 1:
            raise ValueError("input sequence cannot be empty")
        if kv_cache is None:
            if position_ids is not None or slots is not None:
                raise ValueError("position_ids is only valid when using a KV cache")
            if S > c.max_sequence_length:
                raise ValueError("input exceeds max_sequence_length")
            kv_cache, position_ids = self.build_kv_cache(B), 0
        if len(kv_cache) != c.num_hidden_layers:
            raise ValueError("KV cache must contain one entry per model layer")
        lens = [S] * B if seq_lens is None else [int(n) for n in seq_lens]
        if len(lens) != B or min(lens) < 1 or max(lens) > S:
            raise ValueError("seq_lens must hold one count in [1, sequence] per sequence")
        ragged = isinstance(position_ids, (list, tuple))
        starts = [int(p) for p in position_ids] if ragged else [position_ids] * B
        if len(starts) != B:
            raise ValueError("one position per sequence is required")
        if any(p is None or p < 0 for p in starts):
            raise ValueError("a non-negative position_ids is required with KV cache")
        if max(p + n for p, n in zip(starts, lens)) > c.max_sequence_length:
            raise ValueError("input exceeds max_sequence_length")
        if slots is not None:
            slots = [int(s) for s in slots]
            if len(slots) != B:
                raise ValueError("one slot per sequence is required")
            ends = [cc._reserve_rows(slots, lens, starts) for cc in kv_cache]
        elif ragged or len(set(lens)) > 1:
            ends = [cc._reserve_ragged(B, lens, starts) for cc in kv_cache]
        else:
            ends = [cc._reserve(B, lens[0], starts[0]) for cc in kv_cache]
        _check_ids_on_host(x, c.vocab_size)

        def dev32(values):
            return torch.tensor(values, dtype=torch.int32).to(self.device)

        per_sequence = seq_pos is not None or len(set(starts)) > 1
        if per_sequence and seq_pos is None:
            seq_pos = dev32(starts)
        seq = ops.Seq(B, S, starts[0], seq_pos, per_sequence, None if lens == [S] * B else dev32(lens),
                      None if slots is None else dev32(slots))
        logits = self._run(x.reshape(-1).to(device=self.device, dtype=torch.int64), kv_cache, seq, last_only)
        for cc, end in zip(kv_cache, ends):
            if slots is not None:
                cc._commit_rows(slots, end)
            elif isinstance(end, list):
                cc._commit_ragged(B, end)
            else:
                cc._commit(B, end)
        return logits.view(B, 1 if last_only else S, c.vocab_size)

    __call__ = forward

    def _run(self, ids: torch.Tensor, kv_cache: list, seq: ops.Seq, last_only: bool) -> torch.Tensor:
        """The launches of one call; no host-side state, so a one-token call can be captured in a graph."""
        dt, one = self.dtype, seq.seq_len == 1
        x = torch.empty(seq.rows, self.config.hidden_size, dtype=F32, device=self.device)
        source = dict(ids=ids.contiguous(), table=self.embed)  # what the next residual update adds

        def update(mode="none", **more):
            return ops.residual_norm(x, seq, dt, mode=mode, **{**source, **more})

        def pending(y, norm):
            # columns past the width are zeros, so only the row stride differs
            return dict(y=y, norm_w=norm.w, groups=norm.groups, eps=norm.eps)

        for block, state in zip(self.layers, kv_cache):
            conv = block["conv"]
            if one:
                h = update("conv", conv_w=conv.w, ring=state.conv)
            else:
                update()
                h = conv(x, state.conv, seq, dt)
            source = pending(block["mixer"](h, state, seq), block["norm1"])
            if block["mlp"] is not None:
                source = pending(block["mlp"](update("copy")), block["norm2"])
            if self.trace is not None:
                update()
                self.trace.append(x.clone())
                source = {}
        fin = self.final_norm
        h = update("norm", norm2_w=fin.w, groups=fin.groups, eps=fin.eps)
        if last_only and not one:
            last = torch.arange(seq.batch, device=self.device) * seq.seq_len - 1
            h = h[last + (seq.seq_len if seq.lens is None else seq.lens)]
        return self.head(h)

    # -- device-resident loop ------------------------------------------------------------------

    def supports_persistent(self, batch: int) -> bool:
        """There is no single-launch decode kernel for this model: sessions replay the captured chain."""
        return False

    def session(self, batch: int, max_new_tokens: int, valid_vocab: int = 0, kv_cache: list | None = None,
                persistent: bool | None = None, sampling=None, u=None) -> GraphDecodeSession:
        if persistent:
            raise ValueError("the persistent decode kernel does not cover this shape")
        return GraphDecodeSession(self, batch, max_new_tokens, valid_vocab, kv_cache, sampling, u)

    def decode_step(self, ids: torch.Tensor, kv_cache: list, pos_dev: torch.Tensor) -> torch.Tensor:
        """Logits (B, vocab) of one more token per sequence at the shared position ``pos_dev[0]`` (int32, on the device);
        touches no host-side bookkeeping."""
        return self._run(ids, kv_cache, ops.Seq(ids.numel(), 1, 0, pos_dev), False)

    @torch.no_grad()
    def generate_greedy(self, prompt_ids: torch.Tensor, steps: int, *, use_graph: bool = True, valid_vocab: int = 0,
                        kv_cache: list | None = None) -> torch.Tensor:
        """Prefill the prompts, then ``steps`` greedy tokens with no host round trip per token -> (B, steps) ids."""
        if steps < 1:
            return torch.zeros(prompt_ids.shape[0], 0, dtype=torch.int64, device=self.device)
        sess = self.session(prompt_ids.shape[0], steps, valid_vocab, kv_cache)
        sess.prefill(prompt_ids)
        sess.run(steps - 1, use_graph=use_graph)
        return sess.tokens()
