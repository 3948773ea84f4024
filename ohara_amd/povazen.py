"""Povazen: a decoder whose layers mix by attention with a distance bias or by a gated delta rule, in the
order its config lists them, with norms on the sublayer outputs and a causal convolution in front of
every mixer.

    x <- x + norm1(mixer(x + conv(x)));   x <- x + norm2(swiglu(x))     (layers without a feed-forward: the first only)

The call surface is the other models' (``ohara_amd.hybrid_model``).  ``dtype`` float32 serves the model in 32-bit throughout.

Decode steps run 4 launches per recurrent layer and 5 per attention layer (+ 3 with a feed-forward), all
capturable: residual update, norm, convolution and ring are one launch, and everything of the delta rule
between its two matrix products is another.
"""

from __future__ import annotations

from dataclasses import dataclass, field

import torch

from . import ops
from .hybrid import BF16, F32, BiasedAttention, ChannelDelta, GroupNorm, InputConv, Linear, SwiGLU, distance_slopes
from .hybrid_model import HybridDecoder


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


class Povazen(HybridDecoder):
    def __init__(self, config: PovazenConfig, state: dict, device="cuda", dtype=BF16):
        _validate(config)
        super().__init__(config, device, dtype)
        c, kw = config, dict(dtype=dtype, device=self.device)

        def get(name, *shape):
            return self._tensor(state, name, *shape)

        d = c.hidden_size
        norm = lambda name: GroupNorm(get(name, d), c.norm_groups, c.norm_eps, self.device)  # noqa: E731
        self.embed = get("embed", c.vocab_size, d).detach().to(device=self.device, dtype=dtype).contiguous()
        self.final_norm = norm("final.norm")
        self.head = Linear(get("head", c.vocab_size, d), exact=True, cap=c.logit_softcap, **kw)
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

    def _layer_state(self, block: dict, rows: int, max_seq_length: int) -> dict:
        return {"conv": block["conv"].state(rows), **super()._layer_state(block, rows, max_seq_length)}

    def _run(self, ids: torch.Tensor, kv_cache: list, seq: ops.Seq, last_only: bool) -> torch.Tensor:
        dt, one = self.dtype, seq.seq_len == 1
        x = torch.empty(seq.rows, self.config.hidden_size, dtype=F32, device=self.device)
        source = dict(ids=ids.contiguous(), table=self.embed)  # what the next residual update adds

        def update(mode="none", **more):
            return ops.residual_norm(x, seq, dt, mode=mode, **{**source, **more})

        for block, state in zip(self.layers, kv_cache):
            conv = block["conv"]
            if one:
                h = update("conv", conv_w=conv.w, ring=state.conv)
            else:
                update()
                h = conv(x, state.conv, seq, dt)
            source = block["norm1"].of(block["mixer"](h, state, seq))
            if block["mlp"] is not None:
                source = block["norm2"].of(block["mlp"](update("copy")))
            if self.trace is not None:
                update()
                self.trace.append(x.clone())
                source = {}
        h = update(**self.final_norm.out())
        if last_only and not one:
            h = self._last_rows(h, seq)
        return self.head(h)
