"""Fibirax: a decoder whose mixers are windowed rotary attention and retention side by side, with norms on the sublayer outputs, a
scale per channel behind each of them, and routed experts as feed-forwards.

    x <- x + ls1 * norm1(mixer(x));   x <- x + ls2 * norm2(experts(x))     (layers without a feed-forward: the first only)

The call surface is the other models' (``ohara_amd.hybrid_model``).  ``dtype`` float32 serves the model in 32-bit throughout.

Decode steps run 6 launches per mixer (with the residual update in front of it) and 4 per feed-forward, all capturable: both mixers'
projections are one product, and the sum over a token's experts is part of the residual update that follows.
"""

from __future__ import annotations

from dataclasses import dataclass, field

import torch

from . import ops
from .hybrid import BF16, F32, GroupNorm, Linear, ParallelMixer, Retention, RotaryAttention, RoutedExperts
from .hybrid_model import HybridDecoder


@dataclass
class FibiraxAttention:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot_base: float = 1.0
    rot_dims: int = 0
    rot_scaling: tuple | None = None  # factor, low, high, original
    softcap: float = 0.0              # 0: none
    window: int = 0                   # 0: the whole context


@dataclass
class FibiraxRetention:
    heads: int
    dim: int
    vdim: int
    decay: tuple = ()


@dataclass
class FibiraxExperts:
    experts: int
    top: int
    ff: int
    limit: float
    identity: int = 0       # router outputs that return the input
    groups: int = 1
    keep: int = 1
    shared_ff: int = 0      # 0: no shared expert
    shared_limit: float = 0.0


@dataclass
class FibiraxLayer:
    left: FibiraxAttention
    right: FibiraxRetention
    left_scale: float = 1.0
    right_scale: float = 1.0
    mlp: FibiraxExperts | None = None


@dataclass
class FibiraxConfig:
    vocab_size: int
    hidden_size: int
    layers: list = field(default_factory=list)
    embedding_scale: float = 1.0
    norm_eps: float = 1e-6
    max_sequence_length: int = 4096  # cache capacity per sequence: the design itself has no limit

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)

    @property
    def num_attention_heads(self) -> int:
        return max(layer.left.heads for layer in self.layers)

    @classmethod
    def from_dict(cls, payload: dict, max_sequence_length: int | None = None) -> "FibiraxConfig":
        """The contents of a config.json whose "architecture" is "Fibirax"."""
        layers = []
        for i, entry in enumerate(payload["layers"]):
            if entry["type"] != "parallel":
                raise ValueError(f"layer {i}: unknown mixer {entry['type']!r}")
            m = entry["mixer"]
            layers.append(FibiraxLayer(left=_attention(m["left"]), right=_retention(m["right"]), left_scale=float(m["left_scale"]),
                                       right_scale=float(m["right_scale"]), mlp=_experts(entry.get("mlp"), i)))
        extra = {} if max_sequence_length is None else {"max_sequence_length": int(max_sequence_length)}
        return cls(vocab_size=int(payload["vocab"]), hidden_size=int(payload["width"]), layers=layers,
                   embedding_scale=float((payload.get("embedding") or {}).get("scale", 1.0)), norm_eps=float(payload["norm"]["eps"]), **extra)


def _attention(m: dict) -> FibiraxAttention:
    rot, mask = m.get("rot") or {"base": 1.0, "dims": 0}, m.get("mask") or {"size": 0}
    scaling = rot.get("scaling")
    return FibiraxAttention(heads=int(m["heads"]), kv_heads=int(m.get("kv_heads") or m["heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]),
                            scale=float(m["scale"]), rot_base=float(rot["base"]), rot_dims=int(rot["dims"]),
                            rot_scaling=tuple(float(scaling[k]) for k in ("factor", "low", "high", "original")) if scaling else None,
                            softcap=float(m.get("softcap") or 0.0), window=int(mask["size"]))


def _retention(m: dict) -> FibiraxRetention:
    return FibiraxRetention(heads=int(m["heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]), decay=tuple(float(g) for g in m["decay"]))


def _experts(mlp: dict | None, i: int) -> FibiraxExperts | None:
    if mlp is None:
        return None
    if mlp.get("kind", "moe") != "moe":
        raise ValueError(f"layer {i}: unknown feed-forward {mlp['kind']!r}")
    r, e, shared = mlp["router"], mlp["expert"], mlp.get("shared") or {"ff": 0, "limit": 0.0}
    groups = r.get("groups") or {"count": 1, "keep": 1}
    return FibiraxExperts(experts=int(r["experts"]), top=int(r["top"]), ff=int(e["ff"]), limit=float(e["limit"]),
                          identity=int(r.get("identity") or 0), groups=int(groups["count"]), keep=int(groups["keep"]),
                          shared_ff=int(shared["ff"]), shared_limit=float(shared["limit"]))


def _validate(c: FibiraxConfig) -> None:
    if c.vocab_size < 2:
        raise ValueError("vocab_size must be at least 2")
    if c.hidden_size < 1 or not c.layers:
        raise ValueError("hidden_size and num_hidden_layers must be positive")
    if c.max_sequence_length < 1:
        raise ValueError("max_sequence_length must be positive")


class Fibirax(HybridDecoder):
    def __init__(self, config: FibiraxConfig, state: dict, device="cuda", dtype=BF16):
        _validate(config)
        super().__init__(config, device, dtype)
        c, kw = config, dict(dtype=dtype, device=self.device)
        d = c.hidden_size

        def get(name, *shape):
            return self._tensor(state, name, *shape)

        self.embed = get("embed", c.vocab_size, d).detach().to(device=self.device, dtype=dtype).contiguous()
        self.final_norm = GroupNorm(get("final.norm", d), 1, c.norm_eps, self.device)
        self.head = Linear(get("head", c.vocab_size, d), exact=True, **kw)
        for i, layer in enumerate(c.layers):
            p = f"l{i}."
            norm = lambda n: GroupNorm(get(f"{p}norm{n}", d), 1, c.norm_eps, self.device, scale=get(f"{p}ls{n}", d))  # noqa: B023, E731
            block = dict(norm1=norm(1), mlp=None, mixer=self._mixer(layer, lambda name, *shape: get(f"{p}mix.{name}", *shape), kw))  # noqa: B023
            if layer.mlp is not None:
                block["norm2"] = norm(2)
                block["mlp"] = self._mlp(layer.mlp, lambda name, *shape: get(f"{p}mlp.{name}", *shape), kw)  # noqa: B023
            self.layers.append(block)
        torch.cuda.synchronize(self.device)

    def _mixer(self, layer: FibiraxLayer, get, kw: dict) -> ParallelMixer:
        d, eps = self.config.hidden_size, self.config.norm_eps
        a, H, G = layer.left, layer.left.heads, layer.left.kv_heads
        left = RotaryAttention(get("left.q", H * a.dim, d), get("left.k", G * a.dim, d), get("left.v", G * a.vdim, d),
                               get("left.o", d, H * a.vdim), heads=H, kv_heads=G, dim=a.dim, vdim=a.vdim, scale=a.scale, rot_base=a.rot_base,
                               rot_dims=a.rot_dims, rot_scaling=a.rot_scaling, cap=a.softcap, window=a.window,
                               q_norm=get("left.q.norm", a.dim), k_norm=get("left.k.norm", a.dim), eps=eps,
                               sinks=torch.zeros(H), bare=True, **kw)
        r = layer.right
        nk, nv = r.heads * r.dim, r.heads * r.vdim
        right = Retention(get("right.q", nk, d), get("right.k", nk, d), get("right.v", nv, d), get("right.g", nv, d), get("right.o", d, nv),
                          heads=r.heads, dim=r.dim, vdim=r.vdim, decay=r.decay, k_scale=r.dim ** -0.5, eps=eps, bare=True, **kw)
        return ParallelMixer(left, right, layer.left_scale, layer.right_scale, **kw)

    def _mlp(self, m: FibiraxExperts, get, kw: dict) -> RoutedExperts:
        d, n = self.config.hidden_size, m.experts + m.identity
        three = lambda name, ff: (get(name + ".gate", ff, d), get(name + ".up", ff, d), get(name + ".down", d, ff))  # noqa: E731
        shared = (*three("shared", m.shared_ff), m.shared_limit) if m.shared_ff else None
        return RoutedExperts([three(f"e{e}", m.ff) for e in range(m.experts)], get("router", n, d), get("correction", n), top=m.top,
                             limit=m.limit, groups=m.groups, keep=m.keep, identity=m.identity, shared=shared, **kw)

    def parameters(self):
        yield self.embed
        yield self.final_norm.w
        yield from self.head.tensors()
        for block in self.layers:
            yield block["norm1"].w
            yield from block["mixer"].tensors()
            if block["mlp"] is not None:
                yield block["norm2"].w
                yield from block["mlp"].tensors()

    def _run(self, ids: torch.Tensor, kv_cache: list, seq: ops.Seq, last_only: bool) -> torch.Tensor:
        x = torch.empty(seq.rows, self.config.hidden_size, dtype=F32, device=self.device)
        # what the next residual update adds
        source = dict(ids=ids.contiguous(), table=self.embed, table_scale=self.config.embedding_scale)

        def update(mode="none", **more):
            return ops.residual_norm(x, seq, self.dtype, mode=mode, **{**source, **more})

        for block, state in zip(self.layers, kv_cache):
            source = block["norm1"].of(block["mixer"](update("copy"), state, seq))
            if block["mlp"] is not None:
                source = block["norm2"].of(block["mlp"](update("copy")))
            if self.trace is not None:
                update()
                self.trace.append(x.clone())
                source = {}
        h = update(**self.final_norm.out())
        if last_only and seq.seq_len > 1:
            h = self._last_rows(h, seq)
        return self.head(h)
