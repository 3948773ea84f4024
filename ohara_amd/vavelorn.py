"""Vavelorn: a decoder whose layers mix by latent attention, by a gated delta rule or by rotary attention inside chunks, in the order
its config lists them, with layer norms before and after every sublayer and an embedding of the token added per layer.

    x <- x + norm1b(mixer(norm1(x)));   x <- x + norm2b(swiglu(norm2(x)))     (layers without a feed-forward: the first only)
    x <- x + rms(proj(gelu(gate x) * e)) * w                                  e: the layer's part of the token's side embedding

The call surface is the other models' (``ohara_amd.hybrid_model``).  ``dtype`` float32 serves the model in 32-bit throughout.

Residual update and the norm of the next sublayer are one launch.  Decode steps run 3 launches per recurrent mixer, 4 per rotary
attention and 7 or 8 per latent attention, 3 per feed-forward and 1 (wide models: 4) per side embedding, all capturable.
"""

from __future__ import annotations

from dataclasses import dataclass, field

import torch

from . import ops
from .hybrid import BF16, F32, HeadDelta, LatentAttention, LayerNorm, Linear, RotaryAttention, SwiGLU, TokenSide
from .hybrid_model import HybridDecoder


@dataclass
class VavelornLayer:
    type: str               # "attention", "latent_attention" or "delta"
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float = 1.0      # of the attention scores
    rot_base: float = 1.0   # attention
    rot_dims: int = 0
    softcap: float = 0.0    # 0: none
    chunk: int = 0          # 0: the whole context
    q_rank: int = 0         # latent_attention
    kv_rank: int = 0
    conv: int = 0           # delta: taps of the short convolutions
    ff: int = 0             # hidden width of the feed-forward, 0: none


@dataclass
class VavelornConfig:
    vocab_size: int
    hidden_size: int
    layers: list = field(default_factory=list)
    side_dim: int = 1
    norm_eps: float = 1e-5
    max_sequence_length: int = 4096  # cache capacity per sequence: the design itself has no limit

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)

    @property
    def num_attention_heads(self) -> int:
        return max(layer.heads for layer in self.layers)

    @classmethod
    def from_dict(cls, payload: dict, max_sequence_length: int | None = None) -> "VavelornConfig":
        """The contents of a config.json whose "architecture" is "Vavelorn"."""
        layers = []
        for i, entry in enumerate(payload["layers"]):
            m, mlp, kind = entry["mixer"], entry.get("mlp"), entry["type"]
            if mlp is not None and mlp.get("kind", "dense") != "dense":
                raise ValueError(f"layer {i}: unknown feed-forward {mlp['kind']!r}")
            heads = int(m["heads"])
            more = dict(ff=0 if mlp is None else int(mlp["ff"]), kv_heads=int(m.get("kv_heads") or heads))
            if kind == "attention":
                rot, mask = m.get("rot") or {"base": 1.0, "dims": 0}, m.get("mask") or {"size": 0}
                more.update(scale=float(m["scale"]), rot_base=float(rot["base"]), rot_dims=int(rot["dims"]), chunk=int(mask["size"]),
                            softcap=float(m.get("softcap") or 0.0))
            elif kind == "latent_attention":
                more.update(scale=float(m["scale"]), q_rank=int(m["q_rank"]), kv_rank=int(m["kv_rank"]))
            elif kind == "delta":
                more.update(conv=int(m["conv"]))
            else:
                raise ValueError(f"layer {i}: unknown mixer {kind!r}")
            layers.append(VavelornLayer(type=kind, heads=heads, dim=int(m["dim"]), vdim=int(m["vdim"]), **more))
        extra = {} if max_sequence_length is None else {"max_sequence_length": int(max_sequence_length)}
        return cls(vocab_size=int(payload["vocab"]), hidden_size=int(payload["width"]), layers=layers,
                   side_dim=int(payload["token_side"]["dim"]), norm_eps=float(payload["norm"]["eps"]), **extra)


def _validate(c: VavelornConfig) -> None:
    if c.vocab_size < 2:
        raise ValueError("vocab_size must be at least 2")
    if c.hidden_size < 1 or not c.layers:
        raise ValueError("hidden_size and num_hidden_layers must be positive")
    if c.side_dim < 1 or c.max_sequence_length < 1:
        raise ValueError("side_dim and max_sequence_length must be positive")


class Vavelorn(HybridDecoder):
    def __init__(self, config: VavelornConfig, state: dict, device="cuda", dtype=BF16):
        _validate(config)
        super().__init__(config, device, dtype)
        c, kw = config, dict(dtype=dtype, device=self.device)
        d, n = c.hidden_size, c.num_hidden_layers

        def get(name, *shape):
            return self._tensor(state, name, *shape)

        norm = lambda name: LayerNorm(get(name, d), c.norm_eps, self.device)  # noqa: E731
        self.embed = get("embed", c.vocab_size, d).detach().to(device=self.device, dtype=dtype).contiguous()
        self.side_table = TokenSide.lay_out(get("side.embed", c.vocab_size, n * c.side_dim), n, **kw)
        self.final_norm = norm("final.norm")
        self.head = Linear(get("head", c.vocab_size, d), exact=True, **kw)
        for i, layer in enumerate(c.layers):
            p = f"l{i}."
            block = dict(norm1=norm(p + "norm1"), norm1b=norm(p + "norm1b"), mlp=None,
                         mixer=self._mixer(layer, {k[len(p) + 4:]: t for k, t in state.items() if k.startswith(p + "mix.")}, kw),
                         side=TokenSide(get(p + "side.gate", c.side_dim, d), get(p + "side.proj", d, c.side_dim),
                                        get(p + "side.norm", d), self.side_table, i * ops.round8(c.side_dim), eps=c.norm_eps, **kw))
            if layer.ff:
                block["norm2"], block["norm2b"] = norm(p + "norm2"), norm(p + "norm2b")
                block["mlp"] = SwiGLU(get(p + "mlp.gate", layer.ff, d), get(p + "mlp.up", layer.ff, d),
                                      get(p + "mlp.down", d, layer.ff), **kw)
            self.layers.append(block)
        torch.cuda.synchronize(self.device)

    def _mixer(self, layer: VavelornLayer, w: dict, kw: dict):
        sizes = dict(heads=layer.heads, dim=layer.dim, vdim=layer.vdim)
        if layer.type == "attention":
            return RotaryAttention(w["q"], w["k"], w["v"], w["o"], kv_heads=layer.kv_heads, scale=layer.scale, rot_base=layer.rot_base,
                                   rot_dims=layer.rot_dims, cap=layer.softcap, chunk=layer.chunk, **sizes, **kw)
        if layer.type == "latent_attention":
            if (w["dq"].shape[0], w["dkv"].shape[0]) != (layer.q_rank, layer.kv_rank):
                raise ValueError(f"latents have {w['dq'].shape[0]} and {w['dkv'].shape[0]} entries, the config says "
                                 f"{layer.q_rank} and {layer.kv_rank}")
            return LatentAttention(w["dq"], w["dq.norm"], w["uq"], w["dkv"], w["dkv.norm"], w["uk"], w["uv"], w["g"], w["o"],
                                   scale=layer.scale, eps=self.config.norm_eps, **sizes, **kw)
        if w["q.conv"].shape[1] != layer.conv:
            raise ValueError(f"short convolution has {w['q.conv'].shape[1]} taps, the config says {layer.conv}")
        return HeadDelta(w["q"], w["k"], w["v"], w["q.conv"], w["k.conv"], w["v.conv"], w["b"], w["A_log"], w["a"], w["dt_bias"], w["g"],
                         w["norm"], w["o"], kv_heads=layer.kv_heads, eps=self.config.norm_eps, **sizes, **kw)

    def parameters(self):
        yield self.embed
        yield self.side_table
        yield self.final_norm.w
        yield from self.head.tensors()
        for block in self.layers:
            for part in ("mixer", "side", "mlp"):
                if block[part] is not None:
                    yield from block[part].tensors()
            for name in ("norm1", "norm1b", "norm2", "norm2b"):
                if name in block:
                    yield block[name].w

    def _run(self, ids: torch.Tensor, kv_cache: list, seq: ops.Seq, last_only: bool) -> torch.Tensor:
        ids = ids.contiguous()
        x = torch.empty(seq.rows, self.config.hidden_size, dtype=F32, device=self.device)

        def update(source, want):  # add `source` to the residual, return what `want` makes of it
            return ops.residual_norm(x, seq, self.dtype, **{**source, **want})

        nexts = [block["norm1"] for block in self.layers[1:]] + [self.final_norm]
        h = update(dict(ids=ids, table=self.embed), self.layers[0]["norm1"].out())
        for block, state, after in zip(self.layers, kv_cache, nexts):
            y, norm = block["mixer"](h, state, seq), block["norm1b"]
            if block["mlp"] is not None:
                y, norm = block["mlp"](update(norm.of(y), block["norm2"].out())), block["norm2b"]
            h = block["side"].update(x, seq, ids, y, norm, after)
            if self.trace is not None:
                self.trace.append(x.clone())
        if last_only and seq.seq_len > 1:
            h = self._last_rows(h, seq)
        return self.head(h)
