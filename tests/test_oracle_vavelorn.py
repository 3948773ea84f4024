"""The plain Vavelorn statement (oracle/vavelorn_ref.py) against closed forms, brute-force loops and library routines, and
its sensitivity: every mechanism moves the logits of the test configs by far more than the tolerances used."""

import math

import pytest
import torch
import torch.nn.functional as F

from _hybrid import doubled, error, tokens
from _vavelorn import CONFIGS
from oracle import vavelorn_ref as R

D = torch.float64


def rnd(*shape, seed=0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=D)


def test_layer_norm_and_gelu_are_the_library_ones():
    x, w = rnd(5, 12) + 3.0, rnd(12, seed=1)
    assert torch.allclose(R.layer_norm(x, w, 1e-3), F.layer_norm(x, (12,), w, eps=1e-3), atol=1e-12)
    z = torch.linspace(-6, 6, 101, dtype=D)
    assert torch.allclose(R.gelu_tanh(z), F.gelu(z, approximate="tanh"), atol=1e-12)


def test_rotation_is_a_complex_product_on_neighbouring_pairs():
    x, base, dims = rnd(9, 2, 10), 70.0, 6
    got = R.rotate_pairs(x, base, dims)
    f = base ** (-torch.arange(0, dims, 2, dtype=D) / dims)
    turn = torch.polar(torch.ones(9, 3, dtype=D), torch.arange(9, dtype=D).unsqueeze(1) * f)
    want = torch.view_as_real(torch.view_as_complex(x[..., :dims].reshape(9, 2, 3, 2)) * turn.unsqueeze(1)).flatten(2)
    assert torch.allclose(got[..., :dims], want, atol=1e-12) and torch.equal(got[..., dims:], x[..., dims:])
    # a product of two rotated vectors depends on the distance only
    q, k = rnd(1, 1, 6, seed=1).expand(9, 1, 6), rnd(1, 1, 6, seed=2).expand(9, 1, 6)
    s = (R.rotate_pairs(q, base, 6)[:, 0] @ R.rotate_pairs(k, base, 6)[:, 0].t())
    assert torch.allclose(s[3, 1], s[8, 6], atol=1e-12) and torch.allclose(s[7, 2], s[5, 0], atol=1e-12)


def test_attention_brute_force():
    T, H, G, dim, V, scale, cap, chunk = 9, 4, 2, 5, 3, 1.7, 2.0, 4
    q, k, v = rnd(T, H, dim), rnd(T, G, dim, seed=1), rnd(T, G, V, seed=2)
    for c, size in ((cap, chunk), (None, None)):
        got = R.softmax_attention(q, k, v, scale, c, size)
        for h in range(H):
            for i in range(T):
                seen = [j for j in range(i + 1) if size is None or i // size == j // size]
                s = [float(q[i, h] @ k[j, h // 2]) * scale for j in seen]
                s = [c * math.tanh(a / c) for a in s] if c else s
                e = [math.exp(a - max(s)) for a in s]
                want = sum(w * v[j, h // 2] for j, w in zip(seen, e)) / sum(e)
                assert torch.allclose(got[i, h], want, atol=1e-12)


def test_latent_mixer_equals_its_absorbed_form():
    """Keys and values as projections of the latent against projections moved to the query and to the weighted sum."""
    m = dict(heads=3, dim=6, vdim=4, scale=0.6, kv_rank=5, q_rank=7)
    w = {k: t.double() for k, t in R.random_weights(
        {"width": 8, "vocab": 4, "token_side": {"dim": 1}, "layers": [{"type": "latent_attention", "mixer": m, "mlp": None}]}).items()}
    h, p, eps = rnd(6, 8), "l0.mix.", 1e-3
    got = R.latent_mixer(h, w, p, m, eps)
    cq = F.rms_norm(h @ w[p + "dq"].t(), (7,), w[p + "dq.norm"], eps=eps)
    c = F.rms_norm(h @ w[p + "dkv"].t(), (5,), w[p + "dkv.norm"], eps=eps)
    q = torch.einsum("thd,hdr->thr", (cq @ w[p + "uq"].t()).view(6, 3, 6), w[p + "uk"].view(3, 6, 5))
    a = torch.softmax((torch.einsum("thr,jr->htj", q, c) * 0.6).masked_fill(torch.ones(6, 6).triu(1).bool(), -math.inf), -1)
    o = torch.einsum("htj,jr,hvr->thv", a, c, w[p + "uv"].view(3, 4, 5)).reshape(6, 12)
    want = (o * torch.sigmoid(h @ w[p + "g"].t())) @ w[p + "o"].t()
    assert torch.allclose(got, want, atol=1e-12)


def test_decay_of_one_head_brute_force():
    cfg = {"width": 6, "vocab": 4, "token_side": {"dim": 1},
           "layers": [{"type": "delta", "mixer": dict(heads=2, kv_heads=1, dim=4, vdim=3, conv=2), "mlp": None}]}
    w, m, p, h = {k: t.double() for k, t in R.random_weights(cfg).items()}, cfg["layers"][0]["mixer"], "l0.mix.", rnd(5, 6)
    got = R.delta_mixer(h, w, p, m, 1e-4)
    act = {}
    for n in "qkv":
        x = F.pad(h @ w[p + n].t(), (0, 0, 1, 0))
        act[n] = F.silu(x[:-1] * w[p + n + ".conv"][:, 0] + x[1:] * w[p + n + ".conv"][:, 1])
    out = torch.zeros(5, 6, dtype=D)
    for head in range(2):
        S = torch.zeros(4, 3, dtype=D)
        for t in range(5):
            q, k = (act[n][t] / math.sqrt(float((act[n][t] ** 2).sum()) + 1e-6) for n in "qk")
            beta = 1 / (1 + math.exp(-float(h[t] @ w[p + "b"][head])))
            z = float(h[t] @ w[p + "a"][head] + w[p + "dt_bias"][head])
            S = S * math.exp(-math.exp(float(w[p + "A_log"][head])) * math.log1p(math.exp(z)))
            S = S + torch.outer(k, beta * (act["v"][t, 3 * head:3 * head + 3] - S.t() @ k))
            o = S.t() @ (q / 2)
            out[t, 3 * head:3 * head + 3] = o / torch.sqrt((o ** 2).mean() + 1e-4) * w[p + "norm"]
    want = (out * F.silu(h @ w[p + "g"].t())) @ w[p + "o"].t()
    assert torch.allclose(got, want, atol=1e-10)


def test_forward_is_causal_and_chunks_count_from_the_start():
    cfg = CONFIGS["odd"]
    w = doubled(R.random_weights(cfg))
    toks = tokens(cfg, 20)
    full = R.forward(cfg, w, toks)
    assert torch.allclose(R.forward(cfg, w, toks[:11]), full[:11], atol=1e-10)
    # with chunks of one position the attention is v itself
    q, k, v = rnd(5, 2, 4), rnd(5, 1, 4, seed=1), rnd(5, 1, 3, seed=2)
    assert torch.allclose(R.softmax_attention(q, k, v, 0.5, 3.0, 1), v.expand(5, 2, 3))


_attn, _rule, _rot, _ln, _conv = R.softmax_attention, R.delta_rule, R.rotate_pairs, R.layer_norm, R.causal_conv


def _rms_only(x, w, eps):
    return R.rms(x, eps) * w


def _half_split(x, base, dims):
    order = [i for pair in zip(range(dims // 2), range(dims // 2, dims)) for i in pair] + list(range(dims, x.shape[-1]))
    return _rot(x[..., order], base, dims)[..., [order.index(i) for i in range(x.shape[-1])]]


def _window(q, k, v, scale, cap=None, chunk=None):
    """The last ``chunk`` keys instead of the chunk's."""
    if chunk is None:
        return _attn(q, k, v, scale, cap)
    T, rep = q.shape[0], q.shape[1] // k.shape[1]
    k, v = k.repeat_interleave(rep, 1), v.repeat_interleave(rep, 1)
    s = cap * torch.tanh(torch.einsum("ihd,jhd->hij", q, k) * scale / cap)
    d = torch.arange(T).unsqueeze(1) - torch.arange(T)
    return torch.einsum("hij,jhv->ihv", torch.softmax(s.masked_fill((d < 0) | (d >= chunk), -math.inf), -1), v)


def _no_delta(q, k, v, b, lg):
    S, out = torch.zeros(q.shape[1], q.shape[2], v.shape[2], dtype=q.dtype), []
    for t in range(q.shape[0]):
        S = torch.exp(lg[t]).unsqueeze(-1) * S + k[t].unsqueeze(-1) * (b[t].unsqueeze(-1) * v[t]).unsqueeze(1)
        out.append(torch.einsum("hdv,hd->hv", S, q[t]))
    return torch.stack(out), S


BROKEN = {
    "means not taken off": ("layer_norm", _rms_only),
    "no rotation": ("rotate_pairs", lambda x, base, dims: x),
    "halves instead of neighbours": ("rotate_pairs", _half_split),
    "everything rotated": ("rotate_pairs", lambda x, base, dims: _rot(x, base, x.shape[-1])),
    "no soft cap": ("softmax_attention", lambda q, k, v, s, c=None, n=None: _attn(q, k, v, s, None, n)),
    "no chunks": ("softmax_attention", lambda q, k, v, s, c=None, n=None: _attn(q, k, v, s, c)),
    "chunks one longer": ("softmax_attention", lambda q, k, v, s, c=None, n=None: _attn(q, k, v, s, c, n and n + 1)),
    "a window instead of chunks": ("softmax_attention", _window),
    "convolution one token late": ("causal_conv", lambda x, w: torch.cat([torch.zeros_like(x[:1]), _conv(x, w)[:-1]])),
    "no unit norm": ("unit", lambda x: x),
    "keys not removed before the write": ("delta_rule", _no_delta),
    "no decay": ("delta_rule", lambda q, k, v, b, lg: _rule(q, k, v, b, torch.zeros_like(lg))),
    "no side embedding": ("token_side", lambda x, e, w, p, eps: torch.zeros_like(x)),
    "side embedding ungated": ("gelu_tanh", torch.ones_like),
}


@pytest.mark.parametrize("name", BROKEN)
def test_every_mechanism_shows_in_the_logits(monkeypatch, name):
    cfg = CONFIGS["odd"]
    w, toks = doubled(R.random_weights(cfg, seed=3)), tokens(cfg, 60, seed=3)
    good = R.forward(cfg, w, toks)
    target, fn = BROKEN[name]
    monkeypatch.setattr(R, target, fn)
    assert error(R.forward(cfg, w, toks), good) > 0.05
