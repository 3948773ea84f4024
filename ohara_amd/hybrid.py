"""Building blocks of hybrid decoders (attention layers beside recurrent ones) over the HIP kernels.

Every class is one mechanism with its sizes and constants as constructor arguments; none knows a model's
config keys or tensor names.  A mixer offers ``state(rows, max_seq_length)`` (the tensors it keeps per sequence) and
``__call__(h, state, seq)`` with h the (rows, width rounded up to 8) activations of the call and ``seq`` an
``ops.Seq``.  Activations, caches and matrices are bfloat16 or, for a model served in 32-bit, fp32; the residual
stream, norms, scores, decays and recurrent states are fp32 in both.
"""

from __future__ import annotations

import torch
import torch.nn.functional as F

from . import ops
from ._lib import OharaDelta

BF16, F32 = torch.bfloat16, torch.float32


def _pad(w: torch.Tensor, rows: int, cols: int | None = None) -> torch.Tensor:
    """Zero rows / columns up to the given sizes."""
    if w.ndim == 1:
        return F.pad(w, (0, rows - w.shape[0]))
    return F.pad(w, (0, (cols or w.shape[1]) - w.shape[1], 0, rows - w.shape[0]))


class Linear:
    """y = x W^T (+ bias).  Inputs and outputs are padded to multiples of 8 columns (the pad rows and columns of W are
    zero, so an output's pad columns are exact zeros); ``exact`` keeps W's own row count.  ``cap``: the result is
    soft-capped, cap * tanh(y / cap)."""

    def __init__(self, w: torch.Tensor, bias: torch.Tensor | None = None, *, dtype=BF16, device="cuda", exact: bool = False,
                 cap: float = 0.0):
        n, k = w.shape
        self.n, self.k, self.dtype, self.cap = (n if exact else ops.round8(n)), ops.round8(k), dtype, float(cap)
        w = _pad(w.detach().to(device=device, dtype=dtype), self.n, self.k).contiguous()
        self.bias = None if bias is None else _pad(bias.detach().to(device=device, dtype=dtype), self.n).contiguous()
        self.w = w if dtype == F32 else ops.pack_linear(w)

    def __call__(self, x: torch.Tensor) -> torch.Tensor:
        if self.dtype == F32:
            return ops.gemm_f32(x, self.w, self.bias, cap=self.cap)
        if self.cap:
            return ops.gemm_softcap(x, self.w, self.cap)
        if self.bias is not None:
            return ops.linear_bias(x, self.w, self.bias)
        if x.stride(0) != x.shape[1]:
            return ops.gemm(x, self.w)  # a column slice of a wider buffer
        return ops.gemm_skinny(x, self.w)

    def tensors(self):
        yield self.w if self.dtype == F32 else self.w.data
        if self.bias is not None:
            yield self.bias


class SwiGLU:
    """down(silu(gate x) * (up x)); gate and up are one launch."""

    def __init__(self, gate, up, down, *, dtype=BF16, device="cuda"):
        ff, k = gate.shape
        ffp, kp = ops.round8(ff), ops.round8(k)
        gate, up = (_pad(w.detach().to(device=device, dtype=dtype), ffp, kp).contiguous() for w in (gate, up))
        self.dtype = dtype
        self.gate_up = (gate, up) if dtype == F32 else ops.pack_gate_up(gate, up)
        self.down = Linear(_pad(down.detach(), down.shape[0], ffp), dtype=dtype, device=device)

    def __call__(self, x: torch.Tensor) -> torch.Tensor:
        if self.dtype == F32:
            act = ops.gemm_f32(x, self.gate_up[0], w_up=self.gate_up[1])
        else:
            act = ops.gemm_skinny(x, self.gate_up)
        return self.down(act)

    def tensors(self):
        yield from (self.gate_up if self.dtype == F32 else (self.gate_up.data,))
        yield from self.down.tensors()


class GroupNorm:
    """RMS norm in ``groups`` equal runs of the row, times w (applied inside ``ops.residual_norm``)."""

    def __init__(self, w, groups: int, eps: float, device="cuda"):
        if w.numel() % groups:
            raise ValueError("norm groups must divide the width")
        self.w = w.detach().to(device=device, dtype=F32).contiguous()
        self.groups, self.eps = groups, float(eps)


class InputConv:
    """h + causal depthwise convolution of h over time; w (width, taps), the last column is the current token's."""

    def __init__(self, w, device="cuda"):
        self.w = w.detach().to(device=device, dtype=F32).t().contiguous()  # (taps, width)
        self.device = device

    def state(self, rows: int) -> torch.Tensor:
        taps, width = self.w.shape
        return torch.zeros(rows, taps, width, dtype=F32, device=self.device)

    def __call__(self, x, ring, seq: ops.Seq, dtype):
        return ops.input_conv(x, self.w, ring, seq, dtype)


def distance_slopes(heads: int) -> torch.Tensor:
    """2^(-8 (h + 1) / heads) for head h: the slopes of a linear distance bias (ALiBi)."""
    return torch.tensor([2.0 ** (-8.0 * (h + 1) / heads) for h in range(heads)], dtype=F32)


class BiasedAttention:
    """Causal attention without rotation: q and k normed over the whole projection, values over each head without a
    weight, a linear distance bias on the scores, one sigmoid gate per head on the outputs.

    q, k, v, gate, out: (weight, bias or None) pairs of the projections off the same input."""

    WORKGROUPS = 1024   # decode: a context is cut into chunks until about this many workgroups run
    MIN_CHUNK = 128     # positions of a chunk at least (of the cache's capacity)

    def __init__(self, q, k, v, gate, out, q_norm, k_norm, *, heads: int, kv_heads: int, dim: int, vdim: int, scale: float,
                 eps: float, slopes: torch.Tensor, dtype=BF16, device="cuda"):
        if heads < 1 or kv_heads < 1 or heads % kv_heads:
            raise ValueError("kv_heads must divide heads")
        for name, (w, b), n in (("q", q, heads * dim), ("k", k, kv_heads * dim), ("v", v, kv_heads * vdim), ("gate", gate, heads)):
            if w.shape[0] != n or (b is not None and b.numel() != n):
                raise ValueError(f"attention {name} projection has {w.shape[0]} rows, {n} expected")
        if max(dim, vdim) > 256:
            raise ValueError("attention head sizes up to 256 are supported")
        self.heads, self.kv_heads, self.dim, self.vdim = heads, kv_heads, dim, vdim
        self.scale, self.eps, self.dtype, self.device = float(scale), float(eps), dtype, device
        pairs = (q, k, v, gate)
        biases = [b if b is not None else torch.zeros(w.shape[0], dtype=w.dtype, device=w.device) for w, b in pairs]
        has_bias = any(b is not None for _, b in pairs)
        self.proj = Linear(torch.cat([w for w, _ in pairs]), torch.cat(biases) if has_bias else None, dtype=dtype, device=device)
        self.out = Linear(out, dtype=dtype, device=device)
        dev = lambda t: t.detach().to(device=device, dtype=F32).contiguous()  # noqa: E731
        self.q_norm, self.k_norm, self.slopes = dev(q_norm), dev(k_norm), dev(slopes)
        self.gate_at = heads * dim + kv_heads * (dim + vdim)
        self._ws: dict = {}

    def state(self, rows: int, max_seq_length: int) -> dict:
        zeros = lambda n: torch.zeros(rows, max_seq_length, self.kv_heads, ops.round8(n), dtype=self.dtype, device=self.device)  # noqa: E731
        self._split(rows, max_seq_length)  # a step captured before any eager one finds its workspace initialised
        return {"key": zeros(self.dim), "value": zeros(self.vdim)}

    def n_split(self, batch: int, max_seq_length: int) -> int:
        rep = self.heads // self.kv_heads
        sets = self.kv_heads * -(-rep // (4 if rep >= 4 else (2 if rep >= 2 else 1)))
        return max(1, min(64, self.WORKGROUPS // (batch * sets), max_seq_length // self.MIN_CHUNK))

    def _split(self, batch: int, max_seq_length: int):
        """(chunks, workspace) of a decode step; steps of the same batch size share the workspace, so they must run on one
        stream or otherwise in turn."""
        ns = self.n_split(batch, max_seq_length)
        if ns == 1:
            return 1, None
        ws = self._ws.get((batch, ns))
        if ws is None:
            ws = self._ws[(batch, ns)] = ops.attn_bias_workspace(batch, self.heads, self.vdim, ns, self.device)
        return ns, ws

    def __call__(self, h, state, seq: ops.Seq):
        p = self.proj(h)
        q = ops.qkv_norm_append(p, self.heads, self.kv_heads, self.dim, self.vdim, self.q_norm, self.k_norm, self.eps,
                                state.key, state.value, seq)
        ns, ws = self._split(seq.batch, state.key.shape[1]) if seq.seq_len == 1 else (1, None)
        gate = p[:, self.gate_at:self.gate_at + self.heads]
        att = ops.attn_bias(q, state.key, state.value, self.heads, self.kv_heads, self.dim, self.vdim, self.scale, self.slopes,
                            gate, seq, ns, ws)
        return self.out(att)

    def tensors(self):
        yield from self.proj.tensors()
        yield from self.out.tensors()
        yield from (self.q_norm, self.k_norm)


class ChannelDelta:
    """Gated delta rule with one decay per head and key channel (see csrc/delta_rule.hip for the equations): short
    convolutions with silu on q, k and v, unit q and k, low-rank decay and output-gate projections, gated norm
    per head.  q, k: (kv_heads * dim, width); v: (heads * vdim, width); convs: (channels, taps) each."""

    WORKSPACE = 1 << 30  # bytes of per-chunk intermediates at most; longer prompts are walked in segments
    _workspaces: dict = {}  # device -> the workspace every layer on that device shares (prompts run on one stream)

    def __init__(self, q, k, v, q_conv, k_conv, v_conv, beta, a_log, a1, a2, dt_bias, g1, g2, norm_w, out, *, heads: int,
                 kv_heads: int, dim: int, vdim: int, eps: float, dtype=BF16, device="cuda"):
        if heads < 1 or kv_heads < 1 or heads % kv_heads:
            raise ValueError("kv_heads must divide heads")
        for name, w, n in (("q", q, kv_heads * dim), ("k", k, kv_heads * dim), ("v", v, heads * vdim), ("beta", beta, heads),
                           ("a2", a2, heads * dim), ("g2", g2, heads * vdim)):
            if w.shape[0] != n:
                raise ValueError(f"delta rule {name} projection has {w.shape[0]} rows, {n} expected")
        if max(dim, vdim) > 256:
            raise ValueError("delta rule head sizes up to 256 are supported")
        self.heads, self.kv_heads, self.dim, self.vdim = heads, kv_heads, dim, vdim
        self.dtype, self.device = dtype, torch.device(device)
        self.channels = 2 * kv_heads * dim + heads * vdim
        self.taps = q_conv.shape[1]
        ra, rg = ops.round8(a1.shape[0]), ops.round8(g1.shape[0])
        self.off_a = ops.round8(self.channels)
        self.off_g, self.off_b = self.off_a + ra, self.off_a + ra + rg
        qkv = _pad(torch.cat([q, k, v]), self.off_a)
        self.proj = Linear(torch.cat([qkv, _pad(a1, ra), _pad(g1, rg), beta]), dtype=dtype, device=device)
        a2, g2 = _pad(a2, a2.shape[0], ra), _pad(g2, g2.shape[0], rg)
        self.a2_proj, self.g2_proj = (Linear(w, dtype=dtype, device=device) for w in (a2, g2))
        self.out = Linear(out, dtype=dtype, device=device)
        dev = lambda t, dt=F32: t.detach().to(device=device, dtype=dt).contiguous()  # noqa: E731
        self.a2, self.g2 = dev(a2, dtype), dev(g2, dtype)
        self.conv_w = dev(torch.cat([q_conv, k_conv, v_conv]).t())
        self.neg_a = -torch.exp(dev(a_log))
        self.dt_bias, self.norm_w = dev(dt_bias), dev(norm_w)
        d = OharaDelta()
        d.heads, d.kv_heads, d.dim, d.vdim, d.taps = heads, kv_heads, dim, vdim, self.taps
        d.rank_a, d.rank_g, d.off_a, d.off_g, d.off_b, d.eps = ra, rg, self.off_a, self.off_g, self.off_b, float(eps)
        d.conv_w, d.a2, d.g2 = self.conv_w.data_ptr(), self.a2.data_ptr(), self.g2.data_ptr()
        d.neg_a, d.dt_bias, d.norm_w = self.neg_a.data_ptr(), self.dt_bias.data_ptr(), self.norm_w.data_ptr()
        self._c = d

    def state(self, rows: int, max_seq_length: int) -> dict:
        return {"delta": torch.zeros(rows, self.heads, self.dim, (self.vdim + 3) // 4 * 4, dtype=F32, device=self.device),
                "ring": torch.zeros(rows, self.taps, self.channels, dtype=self.dtype, device=self.device)}

    def _workspace(self, batch: int, tokens: int) -> torch.Tensor:
        need = ops.delta_workspace_bytes(self.heads, self.dim, self.vdim, batch, tokens)
        need = max(min(need, self.WORKSPACE), ops.delta_workspace_bytes(self.heads, self.dim, self.vdim, batch, 1))
        ws = ChannelDelta._workspaces.get(self.device)
        if ws is None or ws.numel() < need:
            ws = ChannelDelta._workspaces[self.device] = torch.empty(need, dtype=torch.uint8, device=self.device)
        return ws

    def __call__(self, h, state, seq: ops.Seq):
        p = self.proj(h)
        if seq.seq_len == 1:
            return self.out(ops.delta_step(self._c, p, state.delta, state.ring, seq))
        za = self.a2_proj(p[:, self.off_a:self.off_g])
        zg = self.g2_proj(p[:, self.off_g:self.off_b])
        o = ops.delta_prefill(self._c, p, za, zg, state.delta, state.ring, self._workspace(seq.batch, seq.seq_len), seq)
        return self.out(o)

    def tensors(self):
        for lin in (self.proj, self.a2_proj, self.g2_proj, self.out):
            yield from lin.tensors()
        yield from (self.conv_w, self.neg_a, self.dt_bias, self.norm_w)
