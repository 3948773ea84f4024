"""Plain CPU statement of the Povazen decoder, one function per mechanism, written from the
equations in the docstrings.

TEST INFRASTRUCTURE ONLY (see oracle/__init__.py): it shares no code with ``ohara_amd`` and is slow
on purpose - whole sequences at once, loops over tokens where the mechanism is a recurrence.

Everything is computed in the dtype of the weights handed in (the tests use float64 or float32).
A model is a config dict (the layout of its config.json) and a flat dict of tensors.

Pinning status: PARITY UNPINNED by an external implementation (none exists).  What holds each
function is tests/test_oracle_povazen.py: closed forms, brute-force loops and library routines.
"""

from __future__ import annotations

import torch
import torch.nn.functional as F


def rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    """x / sqrt(mean(x^2) + eps) over the last dimension."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def group_rms_norm(x: torch.Tensor, w: torch.Tensor, groups: int, eps: float) -> torch.Tensor:
    """The last dimension in ``groups`` equal runs, each over its own root mean square; then times w."""
    n = x.shape[-1]
    parts = [rms(x[..., i * (n // groups):(i + 1) * (n // groups)], eps) for i in range(groups)]
    return torch.cat(parts, dim=-1) * w


def causal_conv(x: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """x (T, C), w (C, taps): y_t = sum_j w[:, j] x_(t - taps + 1 + j), zeros before the start."""
    T, taps = x.shape[0], w.shape[1]
    padded = torch.cat([torch.zeros(taps - 1, x.shape[1], dtype=x.dtype), x])
    y = torch.zeros_like(x)
    for j in range(taps):
        y = y + padded[j:j + T] * w[:, j]
    return y


def input_conv(x: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """What a mixer reads: h + conv(h)."""
    return x + causal_conv(x, w)


def alibi_slopes(heads: int, dtype) -> torch.Tensor:
    return torch.tensor([2.0 ** (-8.0 * (h + 1) / heads) for h in range(heads)], dtype=dtype)


def attention_core(q, k, v, scale: float) -> torch.Tensor:
    """q (T, H, D), k (T, G, D), v (T, G, V) -> (T, H, V): causal softmax of
    (q_i . k_j) scale - slope_h (i - j); head h reads key/value head h // (H / G)."""
    T, H, _ = q.shape
    G = k.shape[1]
    slopes = alibi_slopes(H, q.dtype)
    i = torch.arange(T).unsqueeze(1)
    j = torch.arange(T).unsqueeze(0)
    dist = (i - j).to(q.dtype)
    out = []
    for h in range(H):
        g = h // (H // G)
        s = (q[:, h] @ k[:, g].t()) * scale - slopes[h] * dist
        s = s.masked_fill(j > i, float("-inf"))
        out.append(torch.softmax(s, dim=-1) @ v[:, g])
    return torch.stack(out, dim=1)


def attention_mixer(h: torch.Tensor, w: dict, p: str, m: dict, eps: float) -> torch.Tensor:
    """h (T, width): projections with bias, q / k normed over the whole projection, values over each
    head without a weight, attention, one sigmoid gate per head, output projection."""
    T = h.shape[0]
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (h @ w[p + n].t() + w[p + n + ".b"] for n in ("q", "k", "v"))
    q = rms(q, eps) * w[p + "q.norm"]
    k = rms(k, eps) * w[p + "k.norm"]
    v = rms(v.view(T, G, V), eps)
    o = attention_core(q.view(T, H, D), k.view(T, G, D), v, m["scale"])
    gate = torch.sigmoid(h @ w[p + "g"].t())
    return (o * gate.unsqueeze(-1)).reshape(T, H * V) @ w[p + "o"].t()


def unit(x: torch.Tensor) -> torch.Tensor:
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def delta_rule(q, k, v, beta, log_decay, state=None):
    """Token by token: q, k, log_decay (T, H, D), v (T, H, V), beta (T, H); S (H, D, V) from zero.
    S <- exp(log_decay) S (rows = key channels); u = beta (v - S^T k); S <- S + k u^T; o = S^T q."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[-1], dtype=q.dtype) if state is None else state.clone()
    out = []
    for t in range(T):
        S = torch.exp(log_decay[t]).unsqueeze(-1) * S
        u = beta[t].unsqueeze(-1) * (v[t] - torch.einsum("hdv,hd->hv", S, k[t]))
        S = S + k[t].unsqueeze(-1) * u.unsqueeze(1)
        out.append(torch.einsum("hdv,hd->hv", S, q[t]))
    return torch.stack(out), S


def delta_inputs(h: torch.Tensor, w: dict, p: str, m: dict):
    """-> q, k, log_decay (T, H, D), v (T, H, V), beta (T, H), all per value head."""
    T = h.shape[0]
    H, K, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (F.silu(causal_conv(h @ w[p + n].t(), w[p + n + ".conv"])) for n in ("q", "k", "v"))
    q = unit(q.view(T, K, D)) * D ** -0.5
    k = unit(k.view(T, K, D))
    rep = H // K
    q, k = (torch.stack([t[:, i // rep] for i in range(H)], dim=1) for t in (q, k))
    beta = torch.sigmoid(h @ w[p + "b"].t())
    z = (h @ w[p + "a1"].t()) @ w[p + "a2"].t() + w[p + "dt_bias"]
    log_decay = -torch.exp(w[p + "A_log"]).view(1, H, 1) * F.softplus(z, threshold=60.0).view(T, H, D)
    return q, k, log_decay, v.view(T, H, V), beta


def delta_mixer(h: torch.Tensor, w: dict, p: str, m: dict, eps: float) -> torch.Tensor:
    T = h.shape[0]
    q, k, log_decay, v, beta = delta_inputs(h, w, p, m)
    o, _ = delta_rule(q, k, v, beta, log_decay)
    gate = torch.sigmoid((h @ w[p + "g1"].t()) @ w[p + "g2"].t()).view(T, m["heads"], m["vdim"])
    return (rms(o, eps) * w[p + "norm"] * gate).reshape(T, -1) @ w[p + "o"].t()


def dense_mlp(x: torch.Tensor, w: dict, p: str) -> torch.Tensor:
    return (F.silu(x @ w[p + "gate"].t()) * (x @ w[p + "up"].t())) @ w[p + "down"].t()


MIXERS = {"attention": attention_mixer, "channel_delta": delta_mixer}


def forward(cfg: dict, w: dict, tokens, trace: list | None = None) -> torch.Tensor:
    """Logits (T, vocab) of one sequence from its start; ``trace`` collects the residual after every layer."""
    eps, groups = cfg["norm"]["eps"], cfg["norm"]["groups"]
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        h = input_conv(x, w[p + "canon1"])
        x = x + group_rms_norm(MIXERS[layer["type"]](h, w, p + "mix.", layer["mixer"], eps), w[p + "norm1"], groups, eps)
        if layer["mlp"] is not None:
            x = x + group_rms_norm(dense_mlp(x, w, p + "mlp."), w[p + "norm2"], groups, eps)
        if trace is not None:
            trace.append(x.clone())
    logits = group_rms_norm(x, w["final.norm"], groups, eps) @ w["head"].t()
    cap = cfg.get("logit_softcap")
    return cap * torch.tanh(logits / cap) if cap else logits


def greedy(cfg: dict, w: dict, tokens, steps: int) -> list[int]:
    """The whole sequence again for every token."""
    seq = list(tokens)
    for _ in range(steps):
        seq.append(int(forward(cfg, w, seq)[-1].argmax()))
    return seq[len(tokens):]


def random_weights(cfg: dict, seed: int = 0, decay_rank: int = 8, gate_rank: int = 8) -> dict:
    """bfloat16 weights of the config's shapes.  Scales are chosen so that every mechanism moves the
    logits: norm weights around one, decays spread between a few and a few hundred tokens."""
    g = torch.Generator().manual_seed(seed)
    d = cfg["width"]

    def n(*shape, s=1.0):
        return torch.randn(*shape, generator=g) * s

    def lin(o, i, s=1.0):
        return n(o, i, s=s / i ** 0.5)

    def norm(k):
        return 1 + n(k, s=0.2)

    w = {"embed": n(cfg["vocab"], d), "head": lin(cfg["vocab"], d, 4.0), "final.norm": norm(d)}
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        w[p + "norm1"] = norm(d)
        w[p + "canon1"] = n(d, cfg["canon"]["taps"], s=0.3)
        if layer["mlp"] is not None:
            ff = layer["mlp"]["ff"]
            w[p + "norm2"] = norm(d)
            w[p + "mlp.gate"], w[p + "mlp.up"], w[p + "mlp.down"] = lin(ff, d), lin(ff, d), lin(d, ff)
        H, K, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        p += "mix."
        w[p + "q"], w[p + "k"], w[p + "o"] = lin(H * D if layer["type"] == "attention" else K * D, d), lin(K * D, d), lin(d, H * V)
        if layer["type"] == "attention":
            w[p + "v"] = lin(K * V, d)
            for nm, k in (("q", H * D), ("k", K * D), ("v", K * V)):
                w[p + nm + ".b"] = n(k, s=0.3)
            w[p + "q.norm"], w[p + "k.norm"] = 1.5 * norm(H * D), 1.5 * norm(K * D)
            w[p + "g"] = lin(H, d)
        else:
            w[p + "v"] = lin(H * V, d)
            for nm, k in (("q", K * D), ("k", K * D), ("v", H * V)):
                w[p + nm + ".conv"] = n(k, m["conv"], s=0.6)
            w[p + "b"], w[p + "norm"] = lin(H, d), norm(V)
            w[p + "A_log"] = torch.linspace(-3.0, 1.0, H) if H > 1 else torch.zeros(1)
            w[p + "a1"], w[p + "a2"] = lin(decay_rank, d), lin(H * D, decay_rank)
            w[p + "dt_bias"] = n(H * D) - 2.0
            w[p + "g1"], w[p + "g2"] = lin(gate_rank, d), lin(H * V, gate_rank)
    return {k: v.to(torch.bfloat16) for k, v in w.items()}
