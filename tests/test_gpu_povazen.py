"""Povazen on the GPU against the plain CPU statement (oracle/povazen_ref.py): each mechanism alone, whole prompts, decoding
through the caches, prompts in portions, batches of unequal sequences, reused cache rows, long decoding and the generation
entry points.  The 32-bit build is the sharp comparison, bfloat16 the served one."""

import io
import json
import sys

import pytest
import torch
import torch.nn.functional as F

from _hybrid import Tok, agrees, close, dev, poisoned, rnd, tokens
from _povazen import CONFIGS, attention, build, config, delta, reference
from oracle import povazen_ref as R

pytestmark = pytest.mark.gpu
BF, F32, D = torch.bfloat16, torch.float32, torch.float64


# ---- mechanisms -------------------------------------------------------------------------------


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("d, groups", [(60, 3), (40, 1), (64, 8), (35, 5), (2048, 2), (3000, 3), (4096, 1), (5000, 5)])
def test_residual_norm(cuda, dtype, d, groups):
    from ohara_amd import ops

    rows, eps = 5, 1e-4
    seq = ops.Seq(rows, 1)
    x, y, w, w2 = rnd(rows, d), rnd(rows, ops.round8(d), seed=1, s=3.0).to(dtype), rnd(d, seed=2), rnd(d, seed=3)
    xd = dev(x)
    out = ops.residual_norm(xd, seq, dtype, y=dev(y), norm_w=dev(w), groups=groups, eps=eps, mode="norm", norm2_w=dev(w2))
    want = x.double() + R.group_rms_norm(y[:, :d].double(), w.double(), groups, eps)
    close(xd, want, F32)
    close(out[:, :d], R.group_rms_norm(want, w2.double(), groups, eps), dtype)
    assert not out[:, d:].any()
    out = ops.residual_norm(xd, seq, dtype, mode="copy")
    close(xd, want, F32)
    assert torch.equal(out[:, :d], xd.to(dtype)) and not out[:, d:].any()
    table = dev(rnd(7, d, seed=4), dtype)
    ids = torch.tensor([6, 0, 3, 3, 1], device=cuda)
    ops.residual_norm(xd, seq, dtype, ids=ids, table=table)
    assert torch.equal(xd, table[ids].float())


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("taps", [1, 2, 3, 6])
def test_input_conv_in_any_portions(cuda, dtype, taps):
    from ohara_amd import ops

    for d in (20, 35):
        T, x, w = 23, rnd(23, d), rnd(d, taps, seed=1)
        want = R.input_conv(x.double(), w.double())
        wd = dev(w.t())
        for cuts in ([23], [1] * 23, [2] * 11 + [1], [5, 1, 2, 9, 1, 5]):
            ring = torch.full((3, taps, d), float("nan"), device=cuda)  # an earlier owner's leftovers
            slots = torch.tensor([2], dtype=torch.int32, device=cuda)
            at = 0
            for n in cuts:
                seq = ops.Seq(1, n, at, slots=slots)
                part = dev(x[at:at + n])
                if n == 1:
                    h = ops.residual_norm(part, seq, dtype, mode="conv", conv_w=wd, ring=ring)
                else:
                    h = ops.input_conv(part, wd, ring, seq, dtype)
                close(h[:, :d], want[at:at + n], dtype, scale=want.abs().max().item())
                assert not h[:, d:].any()
                at += n
            assert torch.isnan(ring[:2]).all()


@pytest.mark.parametrize("n, k, rows", [(50, 24, 3), (64, 200, 70), (130, 64, 129)])
def test_gemm_f32_and_softcap(cuda, n, k, rows):
    from ohara_amd import ops

    x, w, up, b = rnd(rows, k), rnd(n, k, seed=1), rnd(n, k, seed=2), rnd(n, seed=3)
    lin = x.double() @ w.double().t()
    tol = 3e-6 * k ** 0.5
    close(ops.gemm_f32(dev(x), dev(w)), lin, F32, tol=tol)
    close(ops.gemm_f32(dev(x), dev(w), dev(b)), lin + b.double(), F32, tol=tol)
    close(ops.gemm_f32(dev(x), dev(w), cap=3.0), 3.0 * torch.tanh(lin / 3.0), F32, tol=tol)
    close(ops.gemm_f32(dev(x), dev(w), w_up=dev(up)), F.silu(lin) * (x.double() @ up.double().t()), F32, tol=tol)
    xb, wb = x.to(BF), w.to(BF)
    lin = xb.double() @ wb.double().t()
    got = ops.gemm_softcap(dev(xb), ops.pack_linear(dev(wb)), 5.0)
    close(got, 5.0 * torch.tanh(lin / 5.0), BF, tol=1e-5)


def test_softcap_of_a_large_vocabulary(cuda):
    from ohara_amd import ops

    for rows in (1, 20, 64, 80):
        x, w = rnd(rows, 64).to(BF), rnd(16500, 64, seed=1).to(BF)
        lin = x.double() @ w.double().t()
        close(ops.gemm_softcap(dev(x), ops.pack_linear(dev(w)), 7.5), 7.5 * torch.tanh(lin / 7.5), BF, tol=1e-5)


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("H, G, dim, vdim", [(6, 2, 20, 12), (3, 3, 12, 28), (8, 1, 64, 96), (4, 4, 130, 200)])
def test_qkv_norm_append(cuda, dtype, H, G, dim, vdim):
    from ohara_amd import ops

    B, S, T, eps = 3, 4, 9, 1e-4
    n = H * dim + G * (dim + vdim)
    p = (rnd(B * S, ops.round8(n + H)) * torch.logspace(-2, 1, B * S).unsqueeze(1)).to(dtype)
    qn, kn = rnd(H * dim, seed=1), rnd(G * dim, seed=2)
    kc = torch.full((4, T, G, ops.round8(dim)), 7.0, dtype=dtype, device=cuda)
    vc = torch.full((4, T, G, ops.round8(vdim)), 7.0, dtype=dtype, device=cuda)
    starts, lens, slots = [0, 5, 2], [4, 1, 3], [3, 0, 1]
    i32 = lambda v: torch.tensor(v, dtype=torch.int32, device=cuda)  # noqa: E731
    seq = ops.Seq(B, S, 0, i32(starts), True, i32(lens), i32(slots))
    q = ops.qkv_norm_append(dev(p), H, G, dim, vdim, dev(qn), dev(kn), eps, kc, vc, seq).view(B, S, H, -1)
    pd = p.double().view(B, S, -1)
    for b in range(B):
        s, at = slice(0, lens[b]), starts[b]
        wq = (R.rms(pd[b, s, :H * dim], eps) * qn.double()).view(lens[b], H, dim)
        wk = (R.rms(pd[b, s, H * dim:(H + G) * dim], eps) * kn.double()).view(lens[b], G, dim)
        wv = R.rms(pd[b, s, (H + G) * dim:n].reshape(lens[b], G, vdim), eps)
        close(q[b, s, :, :dim], wq, dtype)
        close(kc[slots[b], at:at + lens[b], :, :dim], wk, dtype)
        close(vc[slots[b], at:at + lens[b], :, :vdim], wv, dtype)
        assert not q[b, s, :, dim:].any() and not kc[slots[b], at:at + lens[b], :, dim:].any()
        kc[slots[b], at:at + lens[b]], vc[slots[b], at:at + lens[b]] = 7.0, 7.0
    assert (kc == 7.0).all() and (vc == 7.0).all()  # nothing else was written


def _attention_case(cuda, dtype, H, G, dim, vdim, T, L, seed=0):
    from ohara_amd import ops

    q, k, v = rnd(L, H, dim, seed=seed), rnd(L, G, dim, seed=seed + 1), rnd(L, G, vdim, seed=seed + 2)
    q, k, v = (t.to(dtype) for t in (q, k, v))
    kc = torch.full((2, T, G, ops.round8(dim)), float("nan"), dtype=dtype)
    vc = torch.full((2, T, G, ops.round8(vdim)), float("nan"), dtype=dtype)
    kc[1, :L], vc[1, :L] = 0, 0
    kc[1, :L, :, :dim], vc[1, :L, :, :vdim] = k, v
    return q, k, v, dev(kc), dev(vc)


def _run_attention(q, kc, vc, H, G, dim, vdim, scale, gate, start, n, ns=1):
    from ohara_amd import ops
    from ohara_amd.hybrid import distance_slopes

    qp = F.pad(q[start:start + n], (0, ops.round8(dim) - dim)).reshape(n, -1)
    seq = ops.Seq(1, n, start, slots=torch.tensor([1], dtype=torch.int32, device="cuda"))
    ws = ops.attn_bias_workspace(1, H, vdim, ns, "cuda") if ns > 1 else None
    g = None if gate is None else dev(gate[start:start + n].to(q.dtype))
    out = ops.attn_bias(dev(qp), kc, vc, H, G, dim, vdim, scale, dev(distance_slopes(H)), g, seq, ns, ws)
    assert not out[:, H * vdim:].any()
    return out[:, :H * vdim].view(n, H, vdim)


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("H, G, dim, vdim", [(6, 2, 20, 12), (5, 5, 72, 40), (8, 1, 64, 128), (7, 1, 128, 96), (2, 1, 200, 256),
                                             (4, 2, 256, 130), (1, 1, 8, 8)])
def test_attention_prompt_and_decode(cuda, dtype, H, G, dim, vdim):
    L, scale = 200, 2.0 / dim ** 0.5
    q, k, v, kc, vc = _attention_case(cuda, dtype, H, G, dim, vdim, 256, L)
    gate = rnd(L, H, seed=9).to(dtype)
    want = R.attention_core(q.double(), k.double(), v.double(), scale) * torch.sigmoid(gate.double()).unsqueeze(-1)
    for start, n in ((0, L), (0, 16), (0, 64), (0, 65), (3, 61), (63, 17), (64, 64), (130, 70), (0, 2), (77, 5), (198, 2)):
        got = _run_attention(q, kc, vc, H, G, dim, vdim, scale, gate, start, n)
        close(got, want[start:start + n], dtype, scale=1.0)
    for t in (0, 1, 15, 16, 31, 63, 64, 127, 128, 199):
        for ns in (1, 2, 5, 64):
            close(_run_attention(q, kc, vc, H, G, dim, vdim, scale, gate, t, 1, ns), want[t:t + 1], dtype, scale=1.0)


@pytest.mark.parametrize("dtype", [F32, BF])
def test_attention_finds_one_far_key_and_the_first_token(cuda, dtype):
    H, G, dim, vdim, L, scale = 4, 2, 32, 16, 700, 1.0
    q, k, v, kc, vc = _attention_case(cuda, dtype, H, G, dim, vdim, 1024, L, seed=5)
    for far in (0, 1, 63, 64, 300, 511, 512, 698, 699):
        k2, q2 = k.clone(), q.clone()
        q2[-1] = 5.0 * torch.sign(q[-1, :1])
        k2[:, :] *= 0.05
        k2[far] = 5.0 * torch.sign(q[-1, 0])   # a score of 800 against distance biases of at most 175
        kc[1, :L, :, :dim] = dev(k2)
        want = R.attention_core(q2.double(), k2.double(), v.double(), scale)[-1:]
        assert (want[0] - v[far].double().repeat_interleave(2, 0)).abs().max() < 1e-6
        for ns in (1, 7, 64):
            close(_run_attention(q2, kc, vc, H, G, dim, vdim, scale, None, L - 1, 1, ns), want, dtype, scale=1.0)
        close(_run_attention(q2, kc, vc, H, G, dim, vdim, scale, None, L - 40, 40)[-1:], want, dtype, scale=1.0)


def test_softmax_weights_are_not_rounded(cuda):
    """Values of +-1024 that cancel under exact weights: bf16 weights would leave errors of about 0.1 to 1."""
    H, G, dim, vdim, L = 2, 1, 32, 32, 256
    q, k, v, kc, vc = _attention_case(cuda, BF, H, G, dim, vdim, 256, L, seed=7)
    sign = torch.ones(L)
    sign[1::2] = -1
    v2 = (1024.0 * sign).view(L, 1, 1).expand(L, G, vdim).to(BF)
    vc[1, :L] = dev(v2)
    want = R.attention_core(q.double(), k.double(), v2.double(), 0.05)
    got = _run_attention(q, kc, vc, H, G, dim, vdim, 0.05, None, 0, L)
    bound = 2.0 ** -8 * want.abs() + 5e-3
    assert ((got.double().cpu() - want).abs() <= bound).all()


def _delta_weights(H, K, dim, vdim, conv, width=24, ranks=(5, 12), seed=0, strong=False):
    m = {"heads": H, "kv_heads": K, "dim": dim, "vdim": vdim, "conv": conv}
    cfg = config(width, 16, 1, 1, None, [{"type": "channel_delta", "mixer": m, "mlp": None}])
    w = R.random_weights(cfg, seed, decay_rank=ranks[0], gate_rank=ranks[1])
    w = {k[len("l0.mix."):]: t for k, t in w.items() if k.startswith("l0.mix.")}
    if strong:  # decays from nothing to exp(-200) per token, channel by channel
        w["dt_bias"] = torch.linspace(-30.0, 40.0, H * dim).to(BF)
        w["A_log"] = torch.linspace(-6.0, 1.6, H).to(BF)
    return m, w


def _delta_mixer(m, w, dtype, eps=1e-5):
    from ohara_amd.hybrid import ChannelDelta

    return ChannelDelta(w["q"], w["k"], w["v"], w["q.conv"], w["k.conv"], w["v.conv"], w["b"], w["A_log"], w["a1"], w["a2"],
                        w["dt_bias"], w["g1"], w["g2"], w["norm"], w["o"], heads=m["heads"], kv_heads=m["kv_heads"],
                        dim=m["dim"], vdim=m["vdim"], eps=eps, dtype=dtype)


DELTAS = [(4, 2, 24, 20, 2), (3, 1, 16, 37, 5), (1, 1, 8, 4, 1), (2, 2, 128, 128, 4), (2, 1, 100, 256, 3), (2, 1, 256, 48, 2),
          (1, 1, 256, 256, 4), (6, 3, 64, 64, 4)]


@pytest.mark.parametrize("strong", [False, True])
@pytest.mark.parametrize("shape", DELTAS)
def test_delta_rule_portions(cuda, shape, strong):
    from ohara_amd import ops
    from ohara_amd.state_cache import LayerState

    m, w = _delta_weights(*shape, strong=strong)
    T = 101
    h = rnd(T, 24, seed=4)
    want = R.delta_mixer(h.double(), {"" + k: t.double() for k, t in w.items()}, "", m, 1e-5)
    mixer = _delta_mixer(m, w, F32)
    slots = torch.tensor([1], dtype=torch.int32, device=cuda)
    # cuts around the kernels' 32-token chunks, down to two tokens and one
    for cuts in ([T], [1] * T, [2] * 50 + [1], [31, 32, 33, 5], [1, 63, 1, 36], [64, 2, 35], [32, 32, 32, 5]):
        st = LayerState(256, {k: torch.full_like(t, float("nan")) for k, t in mixer.state(3, 256).items()})
        at, got = 0, []
        for n in cuts:
            got.append(mixer(dev(h[at:at + n]), st, ops.Seq(1, n, at, slots=slots))[:, :24])
            at += n
        close(torch.cat(got), want, F32, tol=2e-5)


def test_delta_rule_segments_and_bf16(cuda, monkeypatch):
    """A workspace for a few chunks only: the prompt is walked in segments; and the bf16 build against the same
    projections (bf16 inputs and weights, fp32 recurrence)."""
    from ohara_amd import ops
    from ohara_amd.hybrid import ChannelDelta
    from ohara_amd.state_cache import LayerState

    m, w = _delta_weights(4, 2, 40, 24, 3)
    h = rnd(300, 24, seed=4).to(BF)
    want = R.delta_mixer(h.double(), {k: t.double() for k, t in w.items()}, "", m, 1e-5)
    for dtype, tol in ((F32, 2e-5), (BF, 3e-2)):
        mixer = _delta_mixer(m, w, dtype)
        monkeypatch.setattr(ChannelDelta, "_workspaces", {})
        monkeypatch.setattr(ChannelDelta, "WORKSPACE", 1 << 30)
        st = [LayerState(512, mixer.state(1, 512)) for _ in range(2)]
        a = mixer(dev(h, dtype), st[0], ops.Seq(1, 300))
        monkeypatch.setattr(ChannelDelta, "_workspaces", {})
        monkeypatch.setattr(ChannelDelta, "WORKSPACE", ops.delta_workspace_bytes(4, 40, 24, 1, 96))
        b = mixer(dev(h, dtype), st[1], ops.Seq(1, 300))
        assert torch.equal(a, b) and torch.equal(st[0].delta, st[1].delta)
        close(a[:, :24], want, dtype, tol=tol)


def test_delta_rule_remembers_a_far_token(cuda):
    """Without decay a key written once is read hundreds of tokens later; orthogonal keys in between leave it alone."""
    from ohara_amd import _lib, ops

    dim, vdim, T = 64, 16, 400
    off = 2 * dim + vdim
    d = _lib.OharaDelta()
    keep = dict(conv_w=torch.ones(1, off), a2=torch.zeros(dim, 8), g2=torch.zeros(vdim, 8), neg_a=-torch.exp(torch.tensor([-60.0])),
                dt_bias=torch.zeros(dim), norm_w=torch.ones(vdim))
    keep = {k: dev(t) for k, t in keep.items()}
    d.heads = d.kv_heads = d.taps = 1
    d.dim, d.vdim, d.rank_a, d.rank_g, d.off_a, d.off_g, d.off_b, d.eps = dim, vdim, 8, 8, off, off + 8, off + 16, 0.0
    for k, t in keep.items():
        setattr(d, k, t.data_ptr())
    big = 50.0
    p = torch.zeros(T, off + 24)
    k = torch.zeros(T, dim)
    k[:, 1:] = big * (torch.arange(1, dim) == (1 + torch.arange(T) % (dim - 1)).unsqueeze(1))
    k[3] = big * F.one_hot(torch.tensor(0), dim)
    p[:, :dim] = -40.0  # silu of it is nothing
    p[T - 1, 0] = big   # the last token asks for token 3's key
    p[:, dim:2 * dim] = torch.where(k > 0, k, torch.tensor(-40.0))
    v = rnd(T, vdim, seed=1, s=2.0)
    p[:, 2 * dim:off] = v
    p[:, off + 16] = 30.0  # step size 1
    want = R.rms(F.silu(v[3].double()), 0.0) * 0.5
    for cuts in ([T], [T - 1, 1], [200, 199, 1]):
        state, ring = torch.zeros(1, 1, dim, vdim, device=cuda), torch.zeros(1, 1, off, device=cuda)
        at = 0
        for n in cuts:
            seq, part = ops.Seq(1, n, at), dev(p[at:at + n])
            if n == 1:
                out = ops.delta_step(d, part, state, ring, seq)
            else:
                za, zg = torch.zeros(n, dim, device=cuda), torch.zeros(n, vdim, device=cuda)
                ws = torch.empty(ops.delta_workspace_bytes(1, dim, vdim, 1, n), dtype=torch.uint8, device=cuda)
                out = ops.delta_prefill(d, part, za, zg, state, ring, ws, seq)
            at += n
        close(out[-1], want, F32, tol=1e-4)


# ---- the model ------------------------------------------------------------------------------------


@pytest.fixture(scope="module")
def models():
    cache = {}

    def get(name, dtype):
        if (name, dtype) not in cache:
            cfg = CONFIGS[name]
            w = R.random_weights(cfg, seed=11)
            cache[name, dtype] = cfg, w, build(cfg, w, dtype)
        return cache[name, dtype]

    return get


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("name", CONFIGS)
def test_prompts_and_decoding_match_the_oracle(cuda, models, name, dtype):
    cfg, w, m = models(name, dtype)
    toks = tokens(cfg, 150)
    want = reference(cfg, w, toks)
    for n in (1, 2, 15, 16, 33, 64, 65, 150):
        got = m(torch.tensor([toks[:n]]), poisoned(m, 1), 0)
        assert got.shape == (1, n, cfg["vocab"]) and got.dtype == dtype
        assert agrees(got[0], want[:n], dtype), n
        last = m(torch.tensor([toks[:n]]), m.build_kv_cache(1), 0, last_only=True)
        assert agrees(last[0], want[n - 1:n], dtype)
    assert agrees(m(torch.tensor([toks]))[0], want, dtype)  # without a cache
    cache, got = poisoned(m, 1), []
    for t, tok in enumerate(toks):
        got.append(m(torch.tensor([[tok]]), cache, t)[0])
    assert agrees(torch.cat(got), want, dtype)


@pytest.mark.parametrize("name", CONFIGS)
def test_residual_after_every_layer(cuda, models, name):
    cfg, w, m = models(name, F32)
    toks, want = tokens(cfg, 40), []
    R.forward(cfg, {k: v.double() for k, v in w.items()}, toks, want)
    m.trace = []
    try:
        m(torch.tensor([toks]), m.build_kv_cache(1), 0)
        for got, ref in zip(m.trace, want):
            close(got, ref, F32, tol=2e-5)
        assert len(m.trace) == len(want)
    finally:
        m.trace = None


@pytest.mark.parametrize("dtype", [F32, BF])
def test_portions_of_prompts(cuda, models, dtype):
    cfg, w, m = models("odd", dtype)
    toks = tokens(cfg, 140, seed=2)
    want = reference(cfg, w, toks)
    for cuts in ([2] * 70, [1, 2, 3, 15, 16, 17, 31, 32, 23], [64, 64, 12], [65, 2, 63, 10], [33, 1, 1, 105], [7] * 20):
        cache, at, got = poisoned(m, 1), 0, []
        for n in cuts:
            got.append(m(torch.tensor([toks[at:at + n]]), cache, at)[0])
            at += n
        assert at == 140 and agrees(torch.cat(got), want, dtype), cuts


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("name", ["odd", "wide"])
def test_unequal_sequences_in_one_batch(cuda, models, name, dtype):
    """Prompts of different lengths in one call, in chosen cache rows; portions at different positions; decoding at
    different positions with rows that sit out."""
    cfg, w, m = models(name, dtype)
    lens = [1, 70, 33, 5]
    seqs = [tokens(cfg, n + 12, seed=20 + n) for n in lens]
    want = [reference(cfg, w, s) for s in seqs]
    cache, slots = poisoned(m, 6), [4, 0, 5, 2]
    pad = lambda rows: torch.tensor([r + [0] * (max(map(len, rows)) - len(r)) for r in rows])  # noqa: E731
    got = m(pad([s[:n] for s, n in zip(seqs, lens)]), cache, [0] * 4, seq_lens=lens, slots=slots)
    last = m(pad([s[:n] for s, n in zip(seqs, lens)]), m.build_kv_cache(4), [0] * 4, seq_lens=lens, last_only=True)
    for b, n in enumerate(lens):
        assert agrees(got[b, :n], want[b][:n], dtype)
        assert agrees(last[b], want[b][n - 1:n], dtype)
    more = [3, 1, 4, 2]  # one call, every sequence at its own position with its own count
    got = m(pad([s[n:n + k] for s, n, k in zip(seqs, lens, more)]), cache, lens, seq_lens=more, slots=slots)
    for b, (n, k) in enumerate(zip(lens, more)):
        assert agrees(got[b, :k], want[b][n:n + k], dtype)
    at = [n + k for n, k in zip(lens, more)]
    for step in range(4):  # sequence 1 sits out now and then
        rows = [b for b in range(4) if not (b == 1 and step % 2)]
        got = m(torch.tensor([[seqs[b][at[b]]] for b in rows]), cache, [at[b] for b in rows], slots=[slots[b] for b in rows])
        for i, b in enumerate(rows):
            assert agrees(got[i], want[b][at[b]:at[b] + 1], dtype)
            at[b] += 1
    assert cache[0].lengths[1] == 0 and torch.isnan(cache[0].tensors["conv"][[1, 3]]).all()


def test_long_decoding(cuda, models):
    cfg, w, m = models("odd", F32)
    toks = tokens(cfg, 500, seed=5)
    want = reference(cfg, w, toks)
    cache = m.build_kv_cache(1)
    assert agrees(m(torch.tensor([toks[:60]]), cache, 0)[0], want[:60], F32)
    got = [m(torch.tensor([[toks[t]]]), cache, t)[0] for t in range(60, 500)]
    assert agrees(torch.cat(got), want[60:], F32)


def test_errors(cuda, models):
    cfg, _, m = models("ones", F32)
    one = torch.tensor([[1]])
    cache = m.build_kv_cache(1)
    for args, kw, message in (
        ((torch.tensor([1]),), {}, "shape"), ((one, cache), {}, "non-negative"), ((one, cache[:1], 0), {}, "one entry per"),
        ((one, cache, 3), {}, "sequential"), ((torch.zeros(1, 513, dtype=torch.long), cache, 0), {}, "exceeds"),
        ((torch.zeros(1, 0, dtype=torch.long), cache, 0), {}, "empty"), ((one, cache, 0), {"slots": [1]}, "slots"),
        ((one, cache, 0), {"seq_lens": [2]}, "seq_lens"), ((one, cache, [0, 0]), {}, "one position"),
    ):
        with pytest.raises(ValueError, match=message):
            m(*args, **kw)
    with pytest.raises(IndexError):
        m(torch.tensor([[cfg["vocab"]]]), cache, 0)
    with pytest.raises(ValueError, match="int8"):
        m.build_kv_cache(1, int8=True)
    with pytest.raises(ValueError, match="built in"):
        m.to(torch.bfloat16)
    bad = R.random_weights(cfg)
    bad["l0.mix.q"] = bad["l0.mix.q"][:-1]
    with pytest.raises(ValueError, match="rows"):
        build(cfg, bad, F32)
    bad = R.random_weights(cfg)
    bad["head"] = bad["head"][:-1]
    with pytest.raises(ValueError, match="head"):
        build(cfg, bad, F32)


# ---- generation -------------------------------------------------------------------------------------


@pytest.mark.parametrize("name", ["odd", "ones"])
def test_greedy_sessions(cuda, models, name):
    cfg, w, m = models(name, F32)
    prompts = [tokens(cfg, 21, seed=s) for s in (1, 2, 3)]
    wd = {k: v.double() for k, v in w.items()}
    want = [R.greedy(cfg, wd, p, 30) for p in prompts]
    for use_graph in (True, False):
        assert m.generate_greedy(torch.tensor(prompts), 30, use_graph=use_graph).tolist() == want
    sess = m.session(1, 40)
    for p, ref in zip(prompts, want):  # the captured graph serves one sequence after another
        sess.prefill(torch.tensor([p]))
        sess.run(12)
        sess.run(17)
        torch.cuda.synchronize()
        assert sess.tokens()[0].tolist() == ref
        sess.restart()


def test_captured_steps_equal_eager_ones(cuda, models):
    """bf16, every replay compared: the same launches, so the same bits."""
    cfg, w, m = models("wide", BF)
    prompt = torch.tensor([tokens(cfg, 40, seed=s) for s in (4, 5)])
    a, b = m.session(2, 64), m.session(2, 64)
    a.prefill(prompt)
    b.prefill(prompt)
    a.capture()
    b.step()
    for n in (1, 3, 8, 9, 2):
        a.run(n)
        for _ in range(n):
            b.step()
        torch.cuda.synchronize()
        assert torch.equal(a.tokens(), b.tokens())
        for x, y in zip(a.cache, b.cache):
            assert all(torch.equal(x.tensors[k], y.tensors[k]) for k in x.tensors)


def test_sampled_sessions_follow_the_draws(cuda, models):
    from ohara_amd import ops
    from ohara_amd.sampling import SamplingConfig

    cfg, w, m = models("odd", BF)
    sc = SamplingConfig(temperature=0.9, top_k=20, top_p=0.9)
    u = torch.rand(24, 2, generator=torch.Generator().manual_seed(0))
    prompt = torch.tensor([tokens(cfg, 9, seed=s) for s in (6, 7)])
    sess = m.session(2, 24, sampling=sc, u=u)
    sess.prefill(prompt)
    sess.run(23)
    got = sess.tokens().tolist()
    cache, feed, at, want = m.build_kv_cache(2), prompt, 0, [[], []]
    for t in range(24):
        logits = m(feed, cache, at, last_only=True)[:, 0]
        ids = ops.sample_topk_topp(logits, 0.9, 20, 0.9, u[t].to(cuda))
        at += feed.shape[1]
        feed = ids.view(2, 1)
        for b in range(2):
            want[b].append(int(ids[b]))
    assert got == want


def test_inference_and_chat_engine(cuda, models, tmp_path):
    from ohara_amd.chat_engine import ChatEngine
    from ohara_amd.inference import Inference
    from ohara_amd.sampling import SamplingConfig
    from safetensors.torch import save_file

    cfg, w, m = models("odd", F32)
    prompt = tokens(cfg, 17, seed=8)
    want = R.greedy(cfg, {k: v.double() for k, v in w.items()}, prompt, 20)
    inf = Inference(m, Tok(cfg["vocab"]), temperature=0.0)
    text = inf.generate(" ".join(map(str, prompt)), max_new_tokens=20, stream=False)
    assert [int(t) for t in text.split()] == prompt + want
    save_file(w, str(tmp_path / "model.safetensors"))
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    eng = ChatEngine.from_checkpoint(tmp_path, Tok(cfg["vocab"]), dtype=F32, stop_ids=(),
                                     renderer=lambda tok, turns, max_tokens: prompt)
    reply = eng.generate([{"role": "user", "content": "x"}], SamplingConfig(temperature=0.0, max_new_tokens=20))
    assert [int(t) for t in reply.split()] == want
    meta = eng.metadata()
    assert meta["layers"] == 4 and meta["vocab_size"] == cfg["vocab"] and meta["dtype"] == "float32"


@pytest.mark.parametrize("use_graph", [True, False])
def test_continuous_batching_joins_leaves_and_reuses_rows(cuda, models, use_graph):
    from ohara_amd.batching import ContinuousBatcher

    cfg, w, m = models("odd", F32)
    wd = {k: v.double() for k, v in w.items()}
    prompts = [tokens(cfg, n, seed=30 + n) for n in (3, 40, 1, 18, 66)]
    want = [R.greedy(cfg, wd, p, 16) for p in prompts]
    bat = ContinuousBatcher(m, 3)
    bat.cache = poisoned(m, 3)
    for c in bat.cache:
        c._commit_ragged(3, [0] * 3)
    got, owner = {i: [] for i in range(5)}, {}

    def join(*idx):
        for i, (b, first) in zip(idx, bat.add_many([prompts[i] for i in idx])):
            got[i].append(first)
            owner[b] = i

    def run(n):
        for b, ids in bat.steps(n, use_graph=use_graph).items():
            got[owner[b]].extend(ids)

    join(0, 1)
    run(5)
    join(2)
    run(4)
    for b in [b for b, i in owner.items() if i == 1]:
        bat.remove(b)
        del owner[b]
    run(2)       # the freed row rides along
    join(3)      # and is taken again
    run(3)
    for b in [b for b, i in owner.items() if i == 0]:
        bat.remove(b)
        del owner[b]
    join(4)
    run(6)
    for i in range(5):
        n = min(len(got[i]), 16)
        assert n >= 7 and got[i][:n] == want[i][:n], i


def test_fed_tokens_through_the_batcher(cuda, models):
    from ohara_amd.batching import ContinuousBatcher

    cfg, w, m = models("wide", F32)
    seqs = [tokens(cfg, 50, seed=s) for s in (50, 51)]
    want = [reference(cfg, w, s) for s in seqs]
    bat = ContinuousBatcher(m, 3)
    (a, la), (b, lb) = bat.feed([(None, seqs[0][:33]), (None, seqs[1][:2])])
    assert agrees(la, want[0][:33], F32) and agrees(lb, want[1][:2], F32)
    (_, lb), (_, la) = bat.feed([(b, seqs[1][2:3]), (a, seqs[0][33:34])])        # a decode step
    assert agrees(la, want[0][33:34], F32) and agrees(lb, want[1][2:3], F32)
    (_, la), (c, lc), (_, lb) = bat.feed([(a, seqs[0][34:36]), (None, seqs[1][:5]), (b, seqs[1][3:20])])  # mixed
    assert agrees(la, want[0][34:36], F32) and agrees(lb, want[1][3:20], F32) and agrees(lc, want[1][:5], F32)
    bat.remove(a)
    for t in range(20, 24):
        (_, lb), (_, lc) = bat.feed([(b, [seqs[1][t]]), (c, [seqs[1][t - 15]])])
        assert agrees(lb, want[1][t:t + 1], F32) and agrees(lc, want[1][t - 15:t - 14], F32)
    with pytest.raises(ValueError, match="active"):
        bat.feed([(a, [1])])


def test_replayed_trace(cuda, tmp_path, monkeypatch, capsys):
    from safetensors.torch import save_file

    from ohara_amd import trace

    cfg = config(48, 75, 3, 2, 9.0, [delta(3, 3, 12, 20, 4), attention(2, 1, 28, 36, 0.25, 40)])
    w = R.random_weights(cfg, seed=6)
    save_file(w, str(tmp_path / "model.safetensors"))
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    a, b = tokens(cfg, 30, seed=1), tokens(cfg, 12, seed=2)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:28], "want": [0, 27, 5]}, {"id": "b", "tokens": b[:11], "want": []}],
              "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": b[11:], "want": [0]}, {"id": "a", "tokens": a[28:29], "want": [0]}],
              "end": ["b"]},
             {"step": 2, "entries": [{"id": "a", "tokens": a[29:], "want": []}], "end": ["a"]},
             {"step": 3, "entries": [{"id": "c", "tokens": b, "want": [11]}], "end": ["c"]}]
    wa, wb = reference(cfg, w, a), reference(cfg, w, b)
    want = {0: wa[[0, 27, 5]], 1: torch.stack([wb[11], wa[28]]), 3: wb[11:]}
    for dtype in ("float32", "bfloat16"):
        out = tmp_path / dtype
        out.mkdir()
        monkeypatch.setattr(sys, "stdin", io.StringIO("".join(json.dumps(s) + "\n" for s in steps)))
        assert trace.main(["--model", str(tmp_path), "--dtype", dtype, "--out", str(out), "--max-tokens", "42"]) == 0
        assert [l for l in capsys.readouterr().out.splitlines() if l.startswith("done")] == [f"done {i}" for i in range(4)]
        assert sorted(p.name for p in out.iterdir()) == ["0.f32", "1.f32", "3.f32"]
        for i, ref in want.items():
            got = torch.frombuffer(bytearray((out / f"{i}.f32").read_bytes()), dtype=torch.float32).view(ref.shape)
            assert agrees(got, ref, getattr(torch, dtype))
