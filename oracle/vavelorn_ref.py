"""Plain CPU statement of the Vavelorn decoder, one function per mechanism, written from the
equations in the docstrings.

TEST INFRASTRUCTURE ONLY (see oracle/__init__.py): it shares no code with ``ohara_amd`` and is slow
on purpose - whole sequences at once, loops over heads and tokens.

Everything is computed in the dtype of the weights handed in (the tests use float64).  A model is a
config dict (the layout of its config.json) and a flat dict of tensors.

Pinning status: PARITY UNPINNED by an external implementation (none exists).  What holds each
function is tests/test_oracle_vavelorn.py: closed forms, brute-force loops and library routines.
"""

from __future__ import annotations

import math

import torch
import torch.nn.functional as F

from .povazen_ref import causal_conv, delta_rule, dense_mlp, rms, unit


def layer_norm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    """(x - mean) / sqrt(mean squared deviation + eps) * w over the last dimension."""
    c = x - x.mean(-1, keepdim=True)
    return rms(c, eps) * w


def gelu_tanh(z: torch.Tensor) -> torch.Tensor:
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))


def rotate_pairs(x: torch.Tensor, base: float, dims: int) -> torch.Tensor:
    """x (T, heads, D): dimensions (2i, 2i + 1) of the first ``dims`` turned by position * base^(-2i / dims)."""
    out = x.clone()
    p = torch.arange(x.shape[0], dtype=x.dtype)
    for i in range(dims // 2):
        a = (p * base ** (-2.0 * i / dims)).unsqueeze(1)
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * torch.cos(a) - v * torch.sin(a)
        out[..., 2 * i + 1] = v * torch.cos(a) + u * torch.sin(a)
    return out


def softmax_attention(q, k, v, scale: float, cap: float | None = None, chunk: int | None = None) -> torch.Tensor:
    """q (T, H, D), k (T, G, D), v (T, G, V) -> (T, H, V).  Scores (q . k) scale, then cap tanh(s / cap); j <= i, and with
    ``chunk`` only j of i's own chunk of that many positions; head h reads key/value head h // (H / G)."""
    T, H, _ = q.shape
    G = k.shape[1]
    i, j = torch.arange(T).unsqueeze(1), torch.arange(T).unsqueeze(0)
    hidden = j > i
    if chunk is not None:
        hidden = hidden | (i // chunk != j // chunk)
    out = []
    for h in range(H):
        g = h // (H // G)
        s = (q[:, h] @ k[:, g].t()) * scale
        if cap:
            s = cap * torch.tanh(s / cap)
        out.append(torch.softmax(s.masked_fill(hidden, float("-inf")), dim=-1) @ v[:, g])
    return torch.stack(out, dim=1)


def attention_mixer(h: torch.Tensor, w: dict, p: str, m: dict, eps: float) -> torch.Tensor:
    """h (T, width): q and k rotated, capped scores inside chunks, output projection."""
    T = h.shape[0]
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (h @ w[p + n].t() for n in "qkv")
    q, k = (rotate_pairs(t.view(T, -1, D), m["rot"]["base"], m["rot"]["dims"]) for t in (q, k))
    o = softmax_attention(q, k, v.view(T, G, V), m["scale"], m["softcap"], m["mask"]["size"])
    return o.reshape(T, H * V) @ w[p + "o"].t()


def latent_mixer(h: torch.Tensor, w: dict, p: str, m: dict, eps: float) -> torch.Tensor:
    """Queries through a normed latent, keys and values expanded per head from another; no positions; every element of the
    concatenated heads gated."""
    T, H, D, V = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = (rms(h @ w[p + "dq"].t(), eps) * w[p + "dq.norm"]) @ w[p + "uq"].t()
    c = rms(h @ w[p + "dkv"].t(), eps) * w[p + "dkv.norm"]
    k, v = c @ w[p + "uk"].t(), c @ w[p + "uv"].t()
    o = softmax_attention(q.view(T, H, D), k.view(T, H, D), v.view(T, H, V), m["scale"])
    return (o.reshape(T, H * V) * torch.sigmoid(h @ w[p + "g"].t())) @ w[p + "o"].t()


def delta_inputs(h: torch.Tensor, w: dict, p: str, m: dict):
    """-> q, k (T, H, D), v (T, H, V), beta and log decay (T, H), all per value head."""
    T = h.shape[0]
    H, K, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (F.silu(causal_conv(h @ w[p + n].t(), w[p + n + ".conv"])) for n in "qkv")
    q, k = unit(q.view(T, K, D)) * D ** -0.5, unit(k.view(T, K, D))
    q, k = (torch.stack([t[:, i // (H // K)] for i in range(H)], dim=1) for t in (q, k))
    beta = torch.sigmoid(h @ w[p + "b"].t())
    log_decay = -torch.exp(w[p + "A_log"]) * F.softplus(h @ w[p + "a"].t() + w[p + "dt_bias"], threshold=60.0)
    return q, k, v.view(T, H, V), beta, log_decay


def delta_mixer(h: torch.Tensor, w: dict, p: str, m: dict, eps: float) -> torch.Tensor:
    T, H, D, V = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q, k, v, beta, log_decay = delta_inputs(h, w, p, m)
    o, _ = delta_rule(q, k, v, beta, log_decay.unsqueeze(-1).expand(T, H, D))
    gate = F.silu(h @ w[p + "g"].t()).view(T, H, V)
    return (rms(o, eps) * w[p + "norm"] * gate).reshape(T, H * V) @ w[p + "o"].t()


def token_side(x: torch.Tensor, e: torch.Tensor, w: dict, p: str, eps: float) -> torch.Tensor:
    """What a layer's own token embedding e (T, dim) adds to the residual x."""
    y = (gelu_tanh(x @ w[p + "gate"].t()) * e) @ w[p + "proj"].t()
    return rms(y, eps) * w[p + "norm"]


MIXERS = {"attention": attention_mixer, "latent_attention": latent_mixer, "delta": delta_mixer}


def forward(cfg: dict, w: dict, tokens, trace: list | None = None) -> torch.Tensor:
    """Logits (T, vocab) of one sequence from its start; ``trace`` collects the residual after every layer."""
    eps, dim = cfg["norm"]["eps"], cfg["token_side"]["dim"]
    ids = torch.as_tensor(tokens, dtype=torch.long)
    x, side = w["embed"][ids], w["side.embed"][ids]
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        norm = lambda t, n: layer_norm(t, w[p + n], eps)  # noqa: B023, E731
        x = x + norm(MIXERS[layer["type"]](norm(x, "norm1"), w, p + "mix.", layer["mixer"], eps), "norm1b")
        if layer["mlp"] is not None:
            x = x + norm(dense_mlp(norm(x, "norm2"), w, p + "mlp."), "norm2b")
        x = x + token_side(x, side[:, i * dim:(i + 1) * dim], w, p + "side.", eps)
        if trace is not None:
            trace.append(x.clone())
    return layer_norm(x, w["final.norm"], eps) @ w["head"].t()


def greedy(cfg: dict, w: dict, tokens, steps: int) -> list[int]:
    """The whole sequence again for every token."""
    seq = list(tokens)
    for _ in range(steps):
        seq.append(int(forward(cfg, w, seq)[-1].argmax()))
    return seq[len(tokens):]


def random_weights(cfg: dict, seed: int = 0) -> dict:
    """bfloat16 weights of the config's shapes.  Scales are chosen so that every mechanism moves the logits: norm weights
    around one, decays spread between one and some hundred tokens, attention scores of a few units."""
    g = torch.Generator().manual_seed(seed)
    d, side = cfg["width"], cfg["token_side"]["dim"]

    def n(*shape, s=1.0):
        return torch.randn(*shape, generator=g) * s

    def lin(o, i, s=1.0):
        return n(o, i, s=s / i ** 0.5)

    def norm(k):
        return 1 + n(k, s=0.2)

    w = {"embed": n(cfg["vocab"], d), "side.embed": n(cfg["vocab"], side * len(cfg["layers"])), "head": lin(cfg["vocab"], d, 4.0),
         "final.norm": norm(d)}
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        w[p + "norm1"], w[p + "norm1b"] = norm(d), norm(d)
        if layer["mlp"] is not None:
            ff = layer["mlp"]["ff"]
            w[p + "norm2"], w[p + "norm2b"] = norm(d), norm(d)
            w[p + "mlp.gate"], w[p + "mlp.up"], w[p + "mlp.down"] = lin(ff, d), lin(ff, d), lin(d, ff)
        w[p + "side.gate"], w[p + "side.proj"], w[p + "side.norm"] = lin(side, d), lin(d, side), norm(d)
        H, D, V = m["heads"], m["dim"], m["vdim"]
        p += "mix."
        w[p + "o"] = lin(d, H * V)
        if layer["type"] == "attention":
            w[p + "q"], w[p + "k"], w[p + "v"] = lin(H * D, d, 1.5), lin(m["kv_heads"] * D, d, 1.5), lin(m["kv_heads"] * V, d)
        elif layer["type"] == "latent_attention":
            r, rq = m["kv_rank"], m["q_rank"]
            w[p + "dq"], w[p + "dq.norm"], w[p + "uq"] = lin(rq, d), norm(rq), lin(H * D, rq, 1.5)
            w[p + "dkv"], w[p + "dkv.norm"] = lin(r, d), norm(r)
            w[p + "uk"], w[p + "uv"], w[p + "g"] = lin(H * D, r, 1.5), lin(H * V, r), lin(H * V, d)
        else:
            K = m["kv_heads"]
            for nm, k in (("q", K * D), ("k", K * D), ("v", H * V)):
                w[p + nm], w[p + nm + ".conv"] = lin(k, d), n(k, m["conv"], s=0.6)
            for nm in ("k", "k.conv"):  # keys near the queries: a read-out of nearly nothing is all rounding after its norm
                w[p + nm] = 0.8 * w[p + nm.replace("k", "q", 1)] + 0.6 * w[p + nm]
            w[p + "b"], w[p + "a"], w[p + "g"], w[p + "norm"] = lin(H, d), lin(H, d), lin(H * V, d), norm(V)
            w[p + "A_log"] = torch.linspace(-3.0, 1.0, H) if H > 1 else torch.zeros(1)
            w[p + "dt_bias"] = n(H) - 1.5
    return {k: v.to(torch.bfloat16) for k, v in w.items()}
