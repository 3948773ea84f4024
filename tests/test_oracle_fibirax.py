"""The plain Fibirax statement (oracle/fibirax_ref.py) against closed forms, brute-force loops and library routines, and
its sensitivity: every mechanism moves the logits of the test configs by far more than the tolerances used."""

import math

import pytest
import torch
import torch.nn.functional as F

from _fibirax import CONFIGS, experts
from _hybrid import doubled, error, tokens
from oracle import fibirax_ref as R

D = torch.float64


def rnd(*shape, seed=0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=D)


def test_frequencies_at_the_ends_and_in_between():
    f = R.rotary_frequencies(1e4, 64)
    assert len(f) == 32 and f[0] == 1.0 and math.isclose(f[16], 1e-2) and R.rotary_frequencies(5.0, 0) == []
    got = R.rotary_frequencies(1e4, 64, dict(factor=8.0, low=1.0, high=4.0, original=2048))
    kinds = set()
    for a, b in zip(f, got):
        wave = 2 * math.pi / a
        if wave < 2048 / 4:
            want, kind = a, "kept"
        elif wave > 2048:
            want, kind = a / 8, "divided"
        else:
            s = (2048 / wave - 1) / 3
            want, kind = a / 8 + s * (a - a / 8), "mixed"
        kinds.add(kind)
        assert math.isclose(b, want, rel_tol=1e-12)
    assert kinds == {"kept", "divided", "mixed"}


def test_rotation_is_a_complex_product_on_neighbouring_pairs():
    x, f = rnd(9, 2, 10), R.rotary_frequencies(70.0, 6)
    got = R.rotate(x, f)
    turn = torch.polar(torch.ones(9, 3, dtype=D), torch.arange(9, dtype=D).unsqueeze(1) * torch.tensor(f, dtype=D))
    want = torch.view_as_real(torch.view_as_complex(x[..., :6].reshape(9, 2, 3, 2)) * turn.unsqueeze(1)).flatten(2)
    assert torch.allclose(got[..., :6], want, atol=1e-12) and torch.equal(got[..., 6:], x[..., 6:])


def test_attention_brute_force():
    T, H, G, dim, V, scale, cap, window = 9, 4, 2, 5, 3, 1.7, 2.0, 4
    q, k, v = rnd(T, H, dim), rnd(T, G, dim, seed=1), rnd(T, G, V, seed=2)
    for c, size, sink in ((cap, window, True), (None, None, True), (cap, 1, False)):
        got = R.window_attention(q, k, v, scale, c, size, sink)
        for h in range(H):
            for i in range(T):
                seen = [j for j in range(i + 1) if size is None or i - j < size]
                s = [float(q[i, h] @ k[j, h // 2]) * scale for j in seen]
                s = [c * math.tanh(a / c) for a in s] if c else s
                e = [math.exp(a) for a in s]
                want = sum(w * v[j, h // 2] for j, w in zip(seen, e)) / (sum(e) + sink)
                assert torch.allclose(got[i, h], want, atol=1e-12)
    # without a window the sink is one more key of score 0 with a value of zero
    kk, vv = torch.cat([torch.zeros(1, 1, dim, dtype=D), k[:, :1]]), torch.cat([torch.zeros(1, 1, V, dtype=D), v[:, :1]])
    want = F.scaled_dot_product_attention(q[:, 0].unsqueeze(0), kk[:, 0].unsqueeze(0), vv[:, 0].unsqueeze(0), scale=scale,
                                          attn_mask=torch.ones(T, T + 1).tril(1).bool())[0]
    assert torch.allclose(R.window_attention(q, k, v, scale)[:, 0], want, atol=1e-12)


def test_retention_is_a_decayed_sum():
    T, H, dim, V, decay = 8, 3, 4, 5, [0.9, 1.0, 0.0]
    q, k, v = rnd(T, H, dim), rnd(T, H, dim, seed=1), rnd(T, H, V, seed=2)
    o, S = R.retention(q, k, v, decay)
    for h in range(H):
        s = q[:, h] @ k[:, h].t()
        back = torch.arange(T).unsqueeze(1) - torch.arange(T)
        w = torch.where(back >= 0, decay[h] ** back.clamp(min=0).to(D), torch.zeros(1, dtype=D))
        assert torch.allclose(o[:, h], (s * w) @ v[:, h], atol=1e-12)
    first, mid = R.retention(q[:3], k[:3], v[:3], decay)
    rest, end = R.retention(q[3:], k[3:], v[3:], decay, mid)
    assert torch.allclose(torch.cat([first, rest]), o) and torch.allclose(end, S)


def test_choice_of_experts_by_hand():
    z = torch.log(torch.tensor([4.0, 1.0, 3.0, 2.0, 6.0, 0.5], dtype=D))
    s = z.exp() / 16.5
    none = torch.zeros(6, dtype=D)
    assert R.route(z, none, 2)[0] == [4, 0]
    assert torch.allclose(R.route(z, none, 2)[1], torch.tensor([0.6, 0.4], dtype=D))
    assert R.route(z, none, 3, groups=3, keep=2)[0] == [4, 0, 1]      # groups (0 1) (2 3) (4 5): the second is shut
    assert R.route(z, none, 2, groups=2, keep=1)[0] == [4, 3]
    c = torch.tensor([-1.0, -1.0, -1.0, -1.0, -2.0, -1.5], dtype=D)   # every choice score is negative
    chosen, w = R.route(z, c, 3, groups=3, keep=2)
    assert chosen == [0, 2, 3] and torch.allclose(w, s[[0, 2, 3]] / s[[0, 2, 3]].sum())


def test_experts_brute_force():
    mlp, d = experts(4, 2, 6, 0.5, identity=2, groups=(2, 1), shared=(5, 0.3)), 8
    g = torch.Generator().manual_seed(3)
    n = lambda *s: torch.randn(*s, generator=g, dtype=D)  # noqa: E731
    w = {"router": n(6, d), "correction": 0.1 * n(6)}
    for name, ff in [(f"e{e}.", 6) for e in range(4)] + [("shared.", 5)]:
        w[name + "gate"], w[name + "up"], w[name + "down"] = n(ff, d), n(ff, d), n(d, ff)
    h = n(40, d)
    got, used = R.moe(h, w, "", mlp), set()

    def unit(x, p, limit):
        a, b = w[p + "gate"] @ x, w[p + "up"] @ x
        y = [min(float(u), limit) for u in a]
        y = [u / (1 + math.exp(-1.702 * u)) * (max(min(float(t), limit), -limit) + 1) for u, t in zip(y, b)]
        return w[p + "down"] @ torch.tensor(y, dtype=D)

    for t in range(40):
        s = torch.softmax(w["router"] @ h[t], 0)
        c = s + w["correction"]
        lo = 0 if c[:3].max() > c[3:].max() else 3
        best = (lo + torch.topk(c[lo:lo + 3], 2).indices).tolist()
        used |= set(best)
        want = unit(h[t], "shared.", 0.3)
        for e in best:
            want = want + s[e] / s[best].sum() * (h[t] if e >= 4 else unit(h[t], f"e{e}.", 0.5))
        assert torch.allclose(got[t], want, atol=1e-10)
    assert used == set(range(6))


def test_forward_is_causal():
    cfg = CONFIGS["odd"]
    w = doubled(R.random_weights(cfg))
    toks = tokens(cfg, 20)
    full = R.forward(cfg, w, toks)
    assert torch.allclose(R.forward(cfg, w, toks[:11]), full[:11], atol=1e-10)


_attn, _ret, _route, _freq, _rot, _glu, _rms = (R.window_attention, R.retention, R.route, R.rotary_frequencies, R.rotate, R.clamped_glu,
                                                R.rms)


def _half_split(x, freqs):
    n = 2 * len(freqs)
    order = [i for pair in zip(range(n // 2), range(n // 2, n)) for i in pair] + list(range(n, x.shape[-1]))
    return _rot(x[..., order], freqs)[..., [order.index(i) for i in range(x.shape[-1])]]


def _swiglu(h, w, p, limit):
    return (F.silu(h @ w[p + "gate"].t()) * (h @ w[p + "up"].t())) @ w[p + "down"].t()


def _weights_with_correction(z, correction, top, groups=1, keep=1):
    chosen, _ = _route(z, correction, top, groups, keep)
    c = torch.softmax(z, -1) + correction
    return chosen, c[chosen] / (c[chosen].sum() + 1e-20)


def _softmax_of_the_chosen(z, correction, top, groups=1, keep=1):
    """Scores over the experts alone, not the identity outputs: the weights stay, the choice does not."""
    return _route(torch.cat([z[:-1], z[-1:] - 30]), correction, top, groups, keep)


MUTANTS = {
    "window one longer": ("window_attention", lambda q, k, v, s, c=None, n=None, sink=True: _attn(q, k, v, s, c, n + 1, sink)),
    "window one shorter": ("window_attention", lambda q, k, v, s, c=None, n=None, sink=True: _attn(q, k, v, s, c, max(1, n - 1), sink)),
    "no sink": ("window_attention", lambda q, k, v, s, c=None, n=None, sink=True: _attn(q, k, v, s, c, n, False)),
    "no cap": ("window_attention", lambda q, k, v, s, c=None, n=None, sink=True: _attn(q, k, v, s, None, n, sink)),
    "rotated halves": ("rotate", _half_split),
    "no rotation": ("rotate", lambda x, f: x),
    "frequencies as they are": ("rotary_frequencies", lambda base, dims, scaling=None: _freq(base, dims)),
    "all frequencies divided": ("rotary_frequencies", lambda base, dims, scaling=None: [f / (scaling or {"factor": 1})["factor"]
                                                                                      for f in _freq(base, dims)]),
    "no decay": ("retention", lambda q, k, v, decay, state=None: _ret(q, k, v, [1.0] * len(decay), state)),
    "decay a token late": ("retention", lambda q, k, v, decay, state=None: _ret(
        q, k / torch.tensor(decay, dtype=D).clamp(min=1e-3).view(-1, 1), v, decay, state)),
    "plain gated unit": ("clamped_glu", _swiglu),
    "no limit": ("clamped_glu", lambda h, w, p, limit: _glu(h, w, p, 1e9)),
    "no correction": ("route", lambda z, c, top, groups=1, keep=1: _route(z, 0 * c, top, groups, keep)),
    "correction in the weights": ("route", _weights_with_correction),
    "no groups": ("route", lambda z, c, top, groups=1, keep=1: _route(z, c, top)),
    "last output never chosen": ("route", _softmax_of_the_chosen),
    "second best": ("route", lambda z, c, top, groups=1, keep=1: tuple(t[1:] for t in _route(z, c, top + 1, groups, keep))),
    "eps outside the root": ("rms", lambda x, eps: x / ((x * x).mean(-1, keepdim=True).sqrt() + eps)),
}


@pytest.mark.parametrize("name", MUTANTS)
def test_every_mechanism_shows_in_the_logits(monkeypatch, name):
    cfg = CONFIGS["odd"]
    w = doubled(R.random_weights(cfg, seed=1))
    toks = tokens(cfg, 90, seed=3)
    want = R.forward(cfg, w, toks)
    attr, fn = MUTANTS[name]
    monkeypatch.setattr(R, attr, fn)
    assert error(R.forward(cfg, w, toks), want) > 1e-3


@pytest.mark.parametrize("change", ["scale", "left_scale", "right_scale", "ls1", "ls2", "q.norm", "shared", "final.norm", "head"])
def test_every_constant_shows_in_the_logits(change):
    import copy

    cfg = copy.deepcopy(CONFIGS["odd"])
    w = doubled(R.random_weights(cfg, seed=1))
    toks = tokens(cfg, 30, seed=3)
    want = R.forward(cfg, w, toks)
    if change == "scale":
        cfg["embedding"]["scale"] *= 1.01
    elif change.endswith("_scale"):
        cfg["layers"][0]["mixer"][change] *= 1.02
    elif change == "shared":
        del cfg["layers"][0]["mlp"]["shared"]
    else:
        for k in [k for k in w if k.endswith(change)]:
            w[k] = w[k] * (1 + 0.1 * rnd(*w[k].shape, seed=9))
    assert error(R.forward(cfg, w, toks), want) > 1e-3
