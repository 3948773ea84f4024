"""The plain Povazen statement (oracle/povazen_ref.py) against closed forms, brute-force loops and library routines, and
its sensitivity: every mechanism moves the logits of the test configs by far more than the tolerances used."""

import math

import pytest
import torch
import torch.nn.functional as F

from _povazen import CONFIGS, doubled, error, tokens
from oracle import povazen_ref as R

D = torch.float64


def rnd(*shape, seed=0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=D)


def test_group_norm_is_a_norm_per_run():
    x, w = rnd(5, 12), rnd(12, seed=1)
    got = R.group_rms_norm(x, w, 3, 1e-5)
    for g in range(3):
        part = x[:, 4 * g:4 * g + 4]
        want = F.rms_norm(part, (4,), eps=1e-5) * w[4 * g:4 * g + 4]
        assert torch.allclose(got[:, 4 * g:4 * g + 4], want, atol=1e-12)
    # eps inside the root: a zero row stays finite and a tiny one is damped
    assert R.rms(torch.full((4,), 1e-9, dtype=D), 1e-6).abs().max() < 1e-5


def test_causal_conv_matches_the_library_and_starts_from_zeros():
    x, w = rnd(9, 4), rnd(4, 3, seed=1)
    want = F.conv1d(F.pad(x.t().unsqueeze(0), (2, 0)), w.unsqueeze(1), groups=4)[0].t()
    assert torch.allclose(R.causal_conv(x, w), want, atol=1e-12)
    assert torch.allclose(R.causal_conv(x, w)[0], x[0] * w[:, -1])  # the last column is the current token's
    assert torch.allclose(R.input_conv(x, torch.zeros_like(w)), x)


def test_attention_core_brute_force():
    T, H, G, dim, V, scale = 6, 4, 2, 5, 3, 0.7
    q, k, v = rnd(T, H, dim), rnd(T, G, dim, seed=1), rnd(T, G, V, seed=2)
    got = R.attention_core(q, k, v, scale)
    for h in range(H):
        slope = 2.0 ** (-8.0 * (h + 1) / H)
        for i in range(T):
            s = [float(q[i, h] @ k[j, h // 2]) * scale - slope * (i - j) for j in range(i + 1)]
            e = [math.exp(a - max(s)) for a in s]
            want = sum(w * v[j, h // 2] for j, w in enumerate(e)) / sum(e)
            assert torch.allclose(got[i, h], want, atol=1e-12)


def test_delta_rule_closed_forms():
    T, H, K, V = 7, 2, 4, 3
    q, k = R.unit(rnd(T, H, K)), R.unit(rnd(T, H, K, seed=1))
    v, beta = rnd(T, H, V, seed=2), torch.sigmoid(rnd(T, H, seed=3))
    # no memory between tokens (decay 0): o = beta (q . k) v
    o, _ = R.delta_rule(q, k, v, beta, torch.full((T, H, K), -1e4, dtype=D))
    assert torch.allclose(o, (beta * (q * k).sum(-1)).unsqueeze(-1) * v, atol=1e-12)
    # no decay, beta 1, orthonormal keys: the state stores every value, reading a key returns it
    eye = torch.eye(K, dtype=D).unsqueeze(1).expand(K, H, K)
    o, S = R.delta_rule(eye, eye, v[:K], torch.ones(K, H, dtype=D), torch.zeros(K, H, K, dtype=D))
    assert torch.allclose(torch.einsum("hkv,thk->thv", S, eye), v[:K], atol=1e-12)
    # a repeated key overwrites its value; a carried state equals one pass
    lg = -torch.rand(T, H, K, generator=torch.Generator().manual_seed(4), dtype=D)
    whole, S = R.delta_rule(q, k, v, beta, lg)
    a, s = R.delta_rule(q[:3], k[:3], v[:3], beta[:3], lg[:3])
    b, s = R.delta_rule(q[3:], k[3:], v[3:], beta[3:], lg[3:], s)
    assert torch.allclose(torch.cat([a, b]), whole, atol=1e-12) and torch.allclose(s, S, atol=1e-12)
    # the recurrence as a matrix per token: S_t = (I - beta k k^T) diag(g) S_(t-1) + beta k v^T
    St = torch.zeros(K, V, dtype=D)
    for t in range(T):
        St = (torch.eye(K, dtype=D) - beta[t, 0] * torch.outer(k[t, 0], k[t, 0])) @ (torch.exp(lg[t, 0]).unsqueeze(1) * St)
        St = St + beta[t, 0] * torch.outer(k[t, 0], v[t, 0])
        assert torch.allclose(whole[t, 0], St.t() @ q[t, 0], atol=1e-12)


def test_forward_is_causal_and_capped():
    cfg = CONFIGS["odd"]
    w = doubled(R.random_weights(cfg))
    toks = tokens(cfg, 20)
    full = R.forward(cfg, w, toks)
    assert torch.allclose(R.forward(cfg, w, toks[:11]), full[:11], atol=1e-10)
    assert full.abs().max() < cfg["logit_softcap"]


BROKEN = {
    "no input convolution": ("input_conv", lambda x, w: x),
    "convolution one token late": ("causal_conv", lambda x, w: torch.cat([torch.zeros_like(x[:1]), _conv(x, w)[:-1]])),
    "one norm group": ("group_rms_norm", lambda x, w, g, eps: R.rms(x, eps) * w),
    "no distance bias": ("alibi_slopes", lambda h, dt: torch.zeros(h, dtype=dt)),
    "slopes one head off": ("alibi_slopes", lambda h, dt: torch.tensor([2.0 ** (-8.0 * i / h) for i in range(h)], dtype=dt)),
    "no unit norm": ("unit", lambda x: x),
    "keys not removed before the write": ("delta_rule", lambda q, k, v, b, lg: _no_delta(q, k, v, b, lg)),
    "read before the write": ("delta_rule", lambda q, k, v, b, lg: _late(q, k, v, b, lg)),
    "no decay": ("delta_rule", lambda q, k, v, b, lg: _rule(q, k, v, b, torch.zeros_like(lg))),
    "one decay per head": ("delta_rule", lambda q, k, v, b, lg: _rule(q, k, v, b, lg.mean(-1, keepdim=True).expand_as(lg))),
}
_conv, _rule = R.causal_conv, R.delta_rule


def _no_delta(q, k, v, b, lg):
    S, out = torch.zeros(q.shape[1], q.shape[2], v.shape[2], dtype=q.dtype), []
    for t in range(q.shape[0]):
        S = torch.exp(lg[t]).unsqueeze(-1) * S + k[t].unsqueeze(-1) * (b[t].unsqueeze(-1) * v[t]).unsqueeze(1)
        out.append(torch.einsum("hdv,hd->hv", S, q[t]))
    return torch.stack(out), S


def _late(q, k, v, b, lg):
    out, S = [], None
    for t in range(q.shape[0]):
        prev = torch.zeros(q.shape[1], q.shape[2], v.shape[2], dtype=q.dtype) if S is None else S
        out.append(torch.einsum("hdv,hd->hv", torch.exp(lg[t]).unsqueeze(-1) * prev, q[t]))
        _, S = _rule(q[t:t + 1], k[t:t + 1], v[t:t + 1], b[t:t + 1], lg[t:t + 1], S)
    return torch.stack(out), S


@pytest.mark.parametrize("name", BROKEN)
def test_every_mechanism_shows_in_the_logits(monkeypatch, name):
    cfg = CONFIGS["odd"]
    w, toks = doubled(R.random_weights(cfg, seed=3)), tokens(cfg, 40, seed=3)
    good = R.forward(cfg, w, toks)
    target, fn = BROKEN[name]
    monkeypatch.setattr(R, target, fn)
    assert error(R.forward(cfg, w, toks), good) > 0.05
