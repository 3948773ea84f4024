"""Plain CPU statement of the Fibirax decoder, one function per mechanism, written from the equations in
the docstrings.

TEST INFRASTRUCTURE ONLY (see oracle/__init__.py): it shares no code with ``ohara_amd`` and is slow
on purpose - whole sequences at once, loops over heads, tokens and experts.

Everything is computed in the dtype of the weights handed in (the tests use float64).  A model is a
config dict (the layout of its config.json) and a flat dict of tensors.

Pinning status: PARITY UNPINNED by an external implementation (none exists).  What holds each
function is tests/test_oracle_fibirax.py: closed forms, brute-force loops and library routines.
"""

from __future__ import annotations

import math

import torch
import torch.nn.functional as F

from .povazen_ref import rms


def rotary_frequencies(base: float, dims: int, scaling: dict | None = None) -> list[float]:
    """f_i = base^(-2i / dims), i < dims / 2.  With ``scaling`` the wavelength l = 2 pi / f decides: below original / high f stays,
    above original / low it is divided by factor, in between it is mixed linearly in original / l."""
    out = []
    for i in range(dims // 2):
        f = base ** (-2.0 * i / dims)
        if scaling:
            turns = scaling["original"] * f / (2 * math.pi)  # original / l
            if turns < scaling["low"]:
                f = f / scaling["factor"]
            elif turns <= scaling["high"]:
                s = (turns - scaling["low"]) / (scaling["high"] - scaling["low"])
                f = (1 - s) * f / scaling["factor"] + s * f
        out.append(f)
    return out


def rotate(x: torch.Tensor, freqs: list[float]) -> torch.Tensor:
    """x (T, heads, D): the pairs (2i, 2i + 1), i < len(freqs), turned by position * freqs[i]."""
    out = x.clone()
    p = torch.arange(x.shape[0], dtype=x.dtype).unsqueeze(1)
    for i, f in enumerate(freqs):
        c, s = torch.cos(p * f), torch.sin(p * f)
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i], out[..., 2 * i + 1] = u * c - v * s, v * c + u * s
    return out


def window_attention(q, k, v, scale: float, cap: float | None = None, window: int | None = None, sink: bool = True) -> torch.Tensor:
    """q (T, H, D), k (T, G, D), v (T, G, V) -> (T, H, V).  s = (q . k) scale, then cap tanh(s / cap); position i sees the
    ``window`` positions up to and including itself; weights exp(s) over sum exp(s), the sum plus one with ``sink``."""
    T, H, _ = q.shape
    G = k.shape[1]
    out = []
    for h in range(H):
        g = h // (H // G)
        s = (q[:, h] @ k[:, g].t()) * scale
        if cap:
            s = cap * torch.tanh(s / cap)
        rows = []
        for i in range(T):
            lo = 0 if window is None else max(0, i - window + 1)
            e = s[i, lo:i + 1]
            m = e.max().clamp(min=0.0)
            p = torch.exp(e - m)
            rows.append((p / (p.sum() + (torch.exp(-m) if sink else 0.0))) @ v[lo:i + 1, g])
        out.append(torch.stack(rows))
    return torch.stack(out, dim=1)


def attention_heads(h: torch.Tensor, w: dict, p: str, m: dict, eps: float) -> torch.Tensor:
    """h (T, width) -> concatenated heads: q and k over their own size's root mean square times a shared weight, then rotated."""
    T, D = h.shape[0], m["dim"]
    q, k, v = (h @ w[p + n].t() for n in "qkv")
    freqs = rotary_frequencies(m["rot"]["base"], m["rot"]["dims"], m["rot"].get("scaling")) if m.get("rot") else []
    q, k = (rotate(rms(t.view(T, -1, D), eps) * w[p + n + ".norm"], freqs) for t, n in ((q, "q"), (k, "k")))
    size = m["mask"]["size"] if m.get("mask") else None
    return window_attention(q, k, v.view(T, m["kv_heads"], m["vdim"]), m["scale"], m.get("softcap"), size).reshape(T, -1)


def retention(q, k, v, decay, state: torch.Tensor | None = None):
    """q, k (T, H, D), v (T, H, V): S <- decay_h S + k v^T, o = S^T q, token by token -> o (T, H, V), S (H, D, V)."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[2], dtype=q.dtype) if state is None else state.clone()
    g = torch.as_tensor(decay, dtype=q.dtype).view(H, 1, 1)
    out = []
    for t in range(T):
        S = g * S + k[t].unsqueeze(2) * v[t].unsqueeze(1)
        out.append((q[t].unsqueeze(1) @ S).squeeze(1))
    return torch.stack(out), S


def retention_heads(h: torch.Tensor, w: dict, p: str, m: dict, eps: float) -> torch.Tensor:
    """h (T, width) -> heads over their own root mean square, concatenated, times silu of the gate."""
    T, H, D, V = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q, k, v = (h @ w[p + n].t() for n in "qkv")
    o, _ = retention(q.view(T, H, D), k.view(T, H, D) * D ** -0.5, v.view(T, H, V), m["decay"])
    return rms(o, eps).reshape(T, H * V) * F.silu(h @ w[p + "g"].t())


def parallel_mixer(h: torch.Tensor, w: dict, p: str, m: dict, eps: float) -> torch.Tensor:
    left = attention_heads(h, w, p + "left.", m["left"], eps) @ w[p + "left.o"].t()
    right = retention_heads(h, w, p + "right.", m["right"], eps) @ w[p + "right.o"].t()
    return m["left_scale"] * left + m["right_scale"] * right


def clamped_glu(h: torch.Tensor, w: dict, p: str, limit: float) -> torch.Tensor:
    """down(g sigmoid(1.702 g) (u + 1)) with g = gate h capped from above and u = up h from both sides."""
    g = torch.clamp(h @ w[p + "gate"].t(), max=limit)
    u = torch.clamp(h @ w[p + "up"].t(), min=-limit, max=limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1)) @ w[p + "down"].t()


def route(z: torch.Tensor, correction: torch.Tensor, top: int, groups: int = 1, keep: int = 1):
    """One token's router logits z (n,) -> chosen outputs, best first, and their weights.  Softmax over all; the choice looks at
    score + correction and only at the ``keep`` groups of neighbours with the largest entry; the weights do not."""
    s = torch.softmax(z, dim=-1)
    choice = [(s[e] + correction[e]).item() for e in range(len(z))]
    size = len(z) // groups
    best = sorted(range(groups), key=lambda g: -max(choice[g * size:(g + 1) * size]))[:keep]
    open_ = [e for e in range(len(z)) if e // size in best]
    chosen = sorted(open_, key=lambda e: -choice[e])[:top]
    return chosen, s[chosen] / (s[chosen].sum() + 1e-20)


def moe(h: torch.Tensor, w: dict, p: str, mlp: dict) -> torch.Tensor:
    """Routed experts, outputs past them that return the input itself, and a shared expert for every token."""
    r = mlp["router"]
    groups = r.get("groups") or {"count": 1, "keep": 1}
    z = h @ w[p + "router"].t()
    rows = []
    for t in range(h.shape[0]):
        y = torch.zeros_like(h[t])
        for e, weight in zip(*route(z[t], w[p + "correction"], r["top"], groups["count"], groups["keep"])):
            y = y + weight * (h[t] if e >= r["experts"] else clamped_glu(h[t], w, f"{p}e{e}.", mlp["expert"]["limit"]))
        rows.append(y)
    out = torch.stack(rows)
    return out if not mlp.get("shared") else out + clamped_glu(h, w, p + "shared.", mlp["shared"]["limit"])


def forward(cfg: dict, w: dict, tokens, trace: list | None = None) -> torch.Tensor:
    """Logits (T, vocab) of one sequence from its start; ``trace`` collects the residual after every layer."""
    eps = cfg["norm"]["eps"]
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)] * cfg["embedding"]["scale"]
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        x = x + rms(parallel_mixer(x, w, p + "mix.", layer["mixer"], eps), eps) * w[p + "norm1"] * w[p + "ls1"]
        if layer["mlp"] is not None:
            x = x + rms(moe(x, w, p + "mlp.", layer["mlp"]), eps) * w[p + "norm2"] * w[p + "ls2"]
        if trace is not None:
            trace.append(x.clone())
    return rms(x, eps) * w["final.norm"] @ w["head"].t()


def greedy(cfg: dict, w: dict, tokens, steps: int) -> list[int]:
    """The whole sequence again for every token."""
    seq = list(tokens)
    for _ in range(steps):
        seq.append(int(forward(cfg, w, seq)[-1].argmax()))
    return seq[len(tokens):]


def random_weights(cfg: dict, seed: int = 0) -> dict:
    """bfloat16 weights of the config's shapes.  Scales are chosen so that every mechanism moves the logits: norm weights
    around one, scores of a few units, routers that favour no expert, corrections that change the choice."""
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
        p = f"l{i}."
        w[p + "norm1"], w[p + "ls1"] = norm(d), 0.7 + n(d, s=0.2)
        m, q = layer["mixer"]["left"], p + "mix.left."
        H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        w[q + "q"], w[q + "k"], w[q + "v"], w[q + "o"] = lin(H * D, d), lin(G * D, d), lin(G * V, d, 1.5), lin(d, H * V)
        w[q + "q.norm"], w[q + "k.norm"] = 1.3 * norm(D), 1.3 * norm(D)
        m, q = layer["mixer"]["right"], p + "mix.right."
        H, D, V = m["heads"], m["dim"], m["vdim"]
        w[q + "q"], w[q + "v"], w[q + "g"], w[q + "o"] = lin(H * D, d), lin(H * V, d), lin(H * V, d), lin(d, H * V)
        w[q + "k"] = 0.8 * w[q + "q"] + 0.6 * lin(H * D, d)  # a read-out of nearly nothing is all rounding after its norm
        if layer["mlp"] is None:
            continue
        w[p + "norm2"], w[p + "ls2"] = norm(d), 0.7 + n(d, s=0.2)
        r, q = layer["mlp"]["router"], p + "mlp."
        total = r["experts"] + (r.get("identity") or 0)
        w[q + "router"], w[q + "correction"] = lin(total, d, 1.5), n(total, s=0.5 / total)
        parts = [(f"e{e}.", layer["mlp"]["expert"]["ff"]) for e in range(r["experts"])]
        if layer["mlp"].get("shared"):
            parts.append(("shared.", layer["mlp"]["shared"]["ff"]))
        for name, ff in parts:
            w[q + name + "gate"], w[q + name + "up"], w[q + name + "down"] = lin(ff, d), lin(ff, d), lin(d, ff)
    return {k: v.to(torch.bfloat16) for k, v in w.items()}
