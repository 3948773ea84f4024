"""Vavelorn on the GPU against the plain CPU statement (oracle/vavelorn_ref.py): each mechanism alone, whole prompts, decoding
through the caches, prompts in portions, batches of unequal sequences, reused cache rows, long decoding and the generation
entry points.  The 32-bit build is the sharp comparison, bfloat16 the served one."""

import io
import json
import sys

import pytest
import torch
import torch.nn.functional as F

from _hybrid import Tok, close, dev, i32, in_portions, poisoned, rnd, tokens
from _vavelorn import CONFIGS, agrees, attention, build, config, delta, latent, reference
from oracle import vavelorn_ref as R

pytestmark = pytest.mark.gpu
BF, F32, D = torch.bfloat16, torch.float32, torch.float64


def mixer_weights(layer, width, seed=0):
    """The tensors of one layer's mixer by their names inside the mixer."""
    w = R.random_weights({"width": width, "vocab": 4, "token_side": {"dim": 1}, "layers": [layer]}, seed)
    return {k[len("l0.mix."):]: t for k, t in w.items() if k.startswith("l0.mix.")}


# ---- mechanisms -------------------------------------------------------------------------------


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("d", [60, 35, 64, 1, 2048, 3000, 4096, 5000])
def test_layer_norms_of_the_residual_update(cuda, dtype, d):
    from ohara_amd import ops
    from ohara_amd.hybrid import GroupNorm, LayerNorm

    rows, eps = 5, 1e-4
    seq = ops.Seq(rows, 1)
    x, y = rnd(rows, d) - 7.0, (rnd(rows, ops.round8(d), seed=1, s=3.0) + 20.0).to(dtype)
    w, w2 = rnd(d, seed=2), rnd(d, seed=3)
    a, b, rms = LayerNorm(w, eps), LayerNorm(w2, eps), GroupNorm(w, 1, eps)
    yd = y[:, :d].double()
    for source, add in ((a.of(dev(y)), R.layer_norm(yd, w.double(), eps)), (rms.of(dev(y)), R.rms(yd, eps) * w.double())):
        want = x.double() + add
        xd = dev(x)
        out = ops.residual_norm(xd, seq, dtype, **{**source, **b.out()})
        close(xd, want, F32)
        close(out[:, :d], R.layer_norm(want, w2.double(), eps), dtype, tol=1e-4 if d == 1 else None)
        assert not out[:, d:].any()
        out = ops.residual_norm(xd.copy_(x), seq, dtype, **{**source, "mode": "copy"})
        close(xd, want, F32)
        assert torch.equal(out[:, :d], xd.to(dtype)) and not out[:, d:].any()


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("n, k", [(8, 64), (24, 200), (136, 72)])
def test_gelu_lookup(cuda, dtype, n, k):
    from ohara_amd import ops

    vocab, column = 11, 16
    table = rnd(vocab, column + n + 8, seed=3).to(dtype)
    w = rnd(n, k, seed=1, s=3 / k ** 0.5).to(dtype)
    for rows in (1, 3, 20, 64, 65, 130):
        x, ids = rnd(rows, k, seed=rows).to(dtype), torch.randint(0, vocab, (rows,), generator=torch.Generator().manual_seed(rows))
        packed = dev(w) if dtype == F32 else ops.pack_linear(dev(w))
        got = ops.gemm_gelu_lookup(dev(x), packed, dev(table), column, ids.cuda())
        close(got, R.gelu_tanh(x.double() @ w.double().t()) * table[ids, column:column + n].double(), dtype)


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("H, G, dim, vdim, rot", [(6, 2, 20, 12, 12), (3, 3, 14, 30, 6), (8, 1, 64, 96, 64), (4, 4, 130, 200, 0),
                                                  (2, 1, 24, 8, 2), (5, 1, 9, 7, 8)])
def test_rotation_and_append(cuda, dtype, H, G, dim, vdim, rot):
    from ohara_amd import ops
    from ohara_amd.hybrid import rotary_tables

    B, S, T, base = 3, 4, 200, 900.0
    n = H * dim + G * (dim + vdim)
    p = rnd(B * S, ops.round8(n)).to(dtype)
    cos, sin = rotary_tables(base, rot, T, "cuda")
    kc = torch.full((4, T, G, ops.round8(dim)), 7.0, dtype=dtype, device=cuda)
    vc = torch.full((4, T, G, ops.round8(vdim)), 7.0, dtype=dtype, device=cuda)
    starts, lens, slots = [0, 195, 2], [4, 1, 3], [3, 0, 1]
    seq = ops.Seq(B, S, 0, i32(starts), True, i32(lens), i32(slots))
    q = ops.qkv_rotate_append(dev(p), H, G, dim, vdim, cos, sin, rot, kc, vc, seq).view(B, S, H, -1)
    pd = p.double().view(B, S, -1)
    for b in range(B):
        m, at = lens[b], starts[b]
        x = pd[b, :m, :(H + G) * dim].reshape(m, H + G, dim)
        want = R.rotate_pairs(torch.cat([torch.zeros(at, H + G, dim, dtype=D), x]), base, rot)[at:]
        close(q[b, :m, :, :dim], want[:, :H], dtype)
        close(kc[slots[b], at:at + m, :, :dim], want[:, H:], dtype)
        assert torch.equal(vc[slots[b], at:at + m, :, :vdim].double().cpu(), pd[b, :m, (H + G) * dim:n].reshape(m, G, vdim))
        for t in (q[b, :m, :, dim:], kc[slots[b], at:at + m, :, dim:], vc[slots[b], at:at + m, :, vdim:]):
            assert not t.any()
        kc[slots[b], at:at + m], vc[slots[b], at:at + m] = 7.0, 7.0
    assert (kc == 7.0).all() and (vc == 7.0).all()  # nothing else was written


def scored_case(dtype, H, G, dim, vdim, T, L, seed=0):
    from ohara_amd import ops

    q, k, v = (rnd(L, n, w, seed=seed + i).to(dtype) for i, (n, w) in enumerate(((H, dim), (G, dim), (G, vdim))))
    kc = torch.full((2, T, G, ops.round8(dim)), float("nan"), dtype=dtype)
    vc = torch.full((2, T, G, ops.round8(vdim)), float("nan"), dtype=dtype)
    kc[1, :L], vc[1, :L] = 0, 0
    kc[1, :L, :, :dim], vc[1, :L, :, :vdim] = k, v
    return q, k, v, dev(kc), dev(vc)


def run_scored(q, kc, vc, dim, vdim, start, n, ns=1, gate=None, **kw):
    from ohara_amd import ops

    H, G = q.shape[1], kc.shape[2]
    qp = F.pad(q[start:start + n], (0, ops.round8(dim) - dim)).reshape(n, -1)
    seq = ops.Seq(1, n, start, slots=i32([1]))
    ws = ops.attn_bias_workspace(1, H, vdim, ns, "cuda") if ns > 1 else None
    g = None if gate is None else dev(gate[start:start + n])
    out = ops.attn_scored(dev(qp), kc, vc, H, G, dim, vdim, kc.shape[1], seq=seq, n_split=ns, workspace=ws, gate=g, **kw)
    assert not out[:, H * vdim:].any()
    return out[:, :H * vdim].view(n, H, vdim)


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("H, G, dim, vdim, cap, chunk", [
    (6, 2, 20, 12, 4.0, 24), (5, 5, 72, 40, 0.0, 64), (8, 1, 64, 128, 9.0, 65), (7, 1, 128, 96, 2.5, 1), (2, 1, 200, 256, 6.0, 63),
    (4, 2, 256, 130, 0.0, 7), (1, 1, 8, 8, 30.0, 0), (3, 1, 33, 17, 5.0, 1000), (8, 4, 96, 96, 30.0, 100)])
def test_capped_chunked_attention(cuda, dtype, H, G, dim, vdim, cap, chunk):
    L, scale = 200, 2.0 / dim ** 0.5
    q, k, v, kc, vc = scored_case(dtype, H, G, dim, vdim, 256, L)
    gate = rnd(L, H * vdim, seed=9).to(dtype)
    plain = R.softmax_attention(q.double(), k.double(), v.double(), scale, cap, chunk or None)
    for g in (None, gate):
        want = plain if g is None else plain * torch.sigmoid(g.double()).view(L, H, vdim)
        run = lambda start, n, ns=1: run_scored(q, kc, vc, dim, vdim, start, n, ns, g, scale=scale, cap=cap, chunk=chunk,  # noqa: E731, B023
                                                gate_elements=g is not None)  # noqa: B023
        for start, n in ((0, L), (0, 16), (0, 65), (3, 61), (63, 17), (64, 64), (130, 70), (0, 2), (77, 5), (198, 2)):
            close(run(start, n), want[start:start + n], dtype, scale=1.0)
    for t in (0, 1, 6, 7, 23, 24, 62, 63, 64, 65, 99, 100, 127, 128, 199):
        for ns in (1, 2, 5, 64):
            close(run(t, 1, ns), want[t:t + 1], dtype, scale=1.0)


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("chunk", [50, 64, 96])
def test_keys_at_the_edges_of_a_chunk(cuda, dtype, chunk):
    """One key with a score of 30 among keys of nearly none: seen from everywhere in its chunk and from nowhere else."""
    H, G, dim, vdim, L, T, cap = 4, 2, 32, 16, 400, 512, 30.0
    q, k, v, kc, vc = scored_case(dtype, H, G, dim, vdim, T, L, seed=5)
    run = lambda q, start, n, ns=1: run_scored(q, kc, vc, dim, vdim, start, n, ns, scale=1.0, cap=cap, chunk=chunk)  # noqa: E731
    q2 = (5.0 * torch.sign(q[:1, :1])).expand_as(q).contiguous()
    for far in (0, chunk - 1, chunk, 2 * chunk - 1, 2 * chunk):
        k2 = 0.01 * k
        k2[far] = 5.0 * torch.sign(q[0, 0])  # 800, capped to 30
        kc[1, :L, :, :dim] = dev(k2)
        want = R.softmax_attention(q2.double(), k2.double(), v.double(), 1.0, cap, chunk)
        end = (far // chunk + 1) * chunk
        one = v[far].double().repeat_interleave(2, 0)
        assert (want[far:end] - one).abs().max() < 1e-6
        assert end == L or (want[end] - one).abs().max() > 0.1
        close(run(q2, 0, L), want, dtype, scale=1.0)
        for t in (far, end - 1, end, end + 1):
            for ns in (1, 3, 64):
                close(run(q2, t, 1, ns), want[t:t + 1], dtype, scale=1.0)
        close(run(q2, end - 9, 20), want[end - 9:end + 11], dtype, scale=1.0)
        close(run(q2, end - 2, 4), want[end - 2:end + 2], dtype, scale=1.0)


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("layer", [attention(6, 2, 20, 12, 0.3, 300.0, 12, 8.0, 45), attention(3, 3, 14, 30, 0.2, 1e4, 6, 20.0, 7),
                                   attention(8, 1, 64, 128, 0.125, 5e5, 64, 30.0, 64)])
def test_rotary_attention_mixer_in_portions(cuda, dtype, layer):
    from ohara_amd.hybrid import RotaryAttention

    m, w = layer["mixer"], mixer_weights(layer, 24)
    h = rnd(150, 24, seed=4).to(dtype)
    want = R.attention_mixer(h.double(), {k: t.double() for k, t in w.items()}, "", m, 0.0)
    mixer = RotaryAttention(w["q"], w["k"], w["v"], w["o"], heads=m["heads"], kv_heads=m["kv_heads"], dim=m["dim"], vdim=m["vdim"],
                            scale=m["scale"], rot_base=m["rot"]["base"], rot_dims=m["rot"]["dims"], cap=m["softcap"],
                            chunk=m["mask"]["size"], dtype=dtype)
    for cuts in ([150], [1] * 150, [2] * 75, [44, 1, 1, 62, 42], [63, 2, 85]):
        close(in_portions(mixer, h, cuts, dtype), want, dtype, tol=2e-2 if dtype == BF else 1e-5)


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("q_rank, rank", [(20, 40), (9, 17), (96, 512), (1, 3), (1536, 128)])
def test_latent_front(cuda, dtype, q_rank, rank):
    from ohara_amd import ops

    B, S, T, eps = 3, 4, 12, 1e-4
    off = ops.round8(q_rank) + 8
    p = (rnd(B * S, ops.round8(off + rank)) * torch.logspace(-2, 1, B * S).unsqueeze(1)).to(dtype)
    qn, cn = rnd(q_rank, seed=1), rnd(rank, seed=2)
    cache = torch.full((4, T, ops.round8(rank)), 7.0, dtype=dtype, device=cuda)
    starts, lens, slots = [0, 5, 2], [4, 1, 3], [3, 0, 1]
    seq = ops.Seq(B, S, 0, i32(starts), True, i32(lens), i32(slots))
    q, c = ops.latent_front(dev(p), q_rank, off, rank, dev(qn), dev(cn), eps, cache, seq, True)
    q, c, pd = q.view(B, S, -1), c.view(B, S, -1), p.double().view(B, S, -1)
    for b in range(B):
        n, at = lens[b], starts[b]
        close(q[b, :n, :q_rank], R.rms(pd[b, :n, :q_rank], eps) * qn.double(), dtype)
        close(c[b, :n, :rank], R.rms(pd[b, :n, off:off + rank], eps) * cn.double(), dtype)
        assert torch.equal(c[b, :n], cache[slots[b], at:at + n])
        assert not q[b, :n, q_rank:].any() and not c[b, :n, rank:].any()
        cache[slots[b], at:at + n] = 7.0
    assert (cache == 7.0).all()


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("H, n, k, n_out", [(3, 16, 24, 13), (8, 128, 512, 128), (2, 264, 8, 264), (20, 72, 96, 65), (1, 8, 40, 1)])
def test_one_matrix_per_head(cuda, dtype, H, n, k, n_out):
    from ohara_amd import ops

    w = rnd(H, n, k, seed=1, s=k ** -0.5).to(dtype)
    for rows in (1, 5, 16, 17, 40):
        x, gate = rnd(rows, H * k + 8, seed=rows).to(dtype), rnd(rows, H * n_out + 3, seed=2).to(dtype)
        want = torch.stack([x[:, h * k:(h + 1) * k].double() @ w[h, :n_out].double().t() for h in range(H)], 1).flatten(1)
        for g in (None, dev(gate)[:, 3:]):
            got = ops.head_linear(dev(x), dev(w), n_out, g)
            close(got[:, :H * n_out], want if g is None else want * torch.sigmoid(gate[:, 3:].double()), dtype)
            assert not got[:, H * n_out:].any()


def latent_core(q, c, scale, first):
    """q (n, H, r) at positions first .. against latents c (L, r), keys and values at once."""
    s = torch.einsum("ihr,jr->hij", q, c) * scale
    i, j = torch.arange(len(q)).unsqueeze(1) + first, torch.arange(len(c)).unsqueeze(0)
    return torch.einsum("hij,jr->ihr", torch.softmax(s.masked_fill(j > i, float("-inf")), -1), c)


def run_latent(q, cache, H, rank, scale, start, n, ns):
    from ohara_amd import ops

    r8 = ops.round8(rank)
    qp = F.pad(q[start:start + n], (0, r8 - rank)).reshape(n, -1)
    ws = ops.attn_latent_workspace(n, H, rank, ns, "cuda") if ns > 1 else None
    out = ops.attn_latent(dev(qp), cache, H, rank, scale, ops.Seq(1, n, start, slots=i32([1])), ns, ws).view(n, H, r8)
    assert not out[..., rank:].any()
    return out[..., :rank]


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("H, rank", [(3, 40), (1, 3), (16, 128), (20, 200), (33, 256), (8, 512), (5, 300)])
def test_attention_over_latents(cuda, dtype, H, rank):
    from ohara_amd import ops

    L, T, scale = 300, 320, 1.5 / rank ** 0.5
    q, c = rnd(L, H, rank).to(dtype), rnd(L, rank, seed=1).to(dtype)
    cache = torch.full((2, T, ops.round8(rank)), float("nan"), dtype=dtype)
    cache[1, :L] = F.pad(c, (0, ops.round8(rank) - rank))
    cache = dev(cache)
    want = latent_core(q.double(), c.double(), scale, 0)
    for ns in (1, 2, 5, 64):
        for start, n in ((0, 1), (1, 1), (63, 1), (64, 1), (127, 3), (299, 1), (0, 15), (250, 9), (126, 2)):
            close(run_latent(q, cache, H, rank, scale, start, n, ns), want[start:start + n], dtype, scale=1.0)
    # one far latent stands out, also the first one
    for far in (0, 63, 64, 200, 298, 299):
        c2 = 0.02 * c
        c2[far] = c[far]
        cache[1, :L, :rank] = dev(c2)
        q2 = (c[far].double() * (60.0 / c[far].double().pow(2).sum())).to(dtype).expand(L, H, rank)
        want2 = latent_core(q2[-1:].double(), c2.double(), 1.0, L - 1)
        assert (want2 - c[far].double()).abs().max() < 1e-2
        for ns in (1, 7, 64):
            close(run_latent(q2, cache, H, rank, 1.0, L - 1, 1, ns), want2, dtype, scale=1.0)


def test_latent_weights_are_not_rounded(cuda):
    """Latents of +-1024 that cancel under exact weights: bf16 weights would leave errors of about 0.1 to 1."""
    from ohara_amd import ops

    L, H, rank = 256, 2, 32
    c = 1024.0 * torch.ones(L, rank)
    c[1::2] *= -1
    q = 1e-5 * rnd(L, H, rank)
    c, q = c.to(BF), q.to(BF)
    cache = dev(c.unsqueeze(0).expand(2, L, rank))
    want = latent_core(q.double(), c.double(), 1.0, 0)
    got = torch.cat([run_latent(q, cache, H, rank, 1.0, t, 8, ns) for t, ns in zip(range(0, L, 8), [1, 3] * 16)])
    assert ((got.double().cpu() - want).abs() <= 2.0 ** -8 * want.abs() + 5e-3).all()


LATENTS = [latent(3, 12, 28, 40, 20, 0.4), latent(2, 21, 11, 17, 9, 0.3), latent(20, 64, 96, 512, 96, 0.125), latent(1, 8, 4, 3, 1, 0.5),
           latent(4, 128, 128, 200, 144, 0.1)]


def latent_mixer(layer, w, dtype, eps=1e-5):
    from ohara_amd.hybrid import LatentAttention

    m = layer["mixer"]
    return LatentAttention(w["dq"], w["dq.norm"], w["uq"], w["dkv"], w["dkv.norm"], w["uk"], w["uv"], w["g"], w["o"], heads=m["heads"],
                           dim=m["dim"], vdim=m["vdim"], scale=m["scale"], eps=eps, dtype=dtype)


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("layer", LATENTS)
def test_latent_mixer_in_portions(cuda, dtype, layer):
    """Portions that form keys and values and shorter ones that do not, one after the other."""
    w = mixer_weights(layer, 24)
    h = rnd(150, 24, seed=4).to(dtype)
    want = R.latent_mixer(h.double(), {k: t.double() for k, t in w.items()}, "", layer["mixer"], 1e-5)
    mixer = latent_mixer(layer, w, dtype)
    for cuts in ([150], [1] * 150, [2] * 75, [15, 16, 17, 102], [64, 1, 63, 22], [3, 147]):
        close(in_portions(mixer, h, cuts, dtype), want, dtype, tol=2e-2 if dtype == BF else 1e-5)


def test_latent_mixer_of_unequal_sequences(cuda):
    from ohara_amd import ops
    from ohara_amd.state_cache import LayerState

    layer = LATENTS[0]
    w = mixer_weights(layer, 24)
    mixer = latent_mixer(layer, w, F32)
    hs = [rnd(90, 24, seed=s) for s in (1, 2, 3)]
    want = [R.latent_mixer(h.double(), {k: t.double() for k, t in w.items()}, "", layer["mixer"], 1e-5) for h in hs]
    st = LayerState(128, {k: torch.full_like(t, float("nan")) for k, t in mixer.state(5, 128).items()})
    slots, at = [4, 0, 2], [0, 0, 0]
    for lens in ([1, 40, 17], [30, 2, 20], [1, 1, 1], [5, 3, 15], [20, 20, 20]):
        S = max(lens)
        x = torch.full((3, S, 24), float("nan"))
        for b, n in enumerate(lens):
            x[b, :n] = hs[b][at[b]:at[b] + n]
        seq = ops.Seq(3, S, 0, i32(at), True, i32(lens), i32(slots), (list(at), lens, slots))
        got = mixer(dev(x.view(3 * S, 24)), st, seq)[:, :24].view(3, S, 24)
        for b, n in enumerate(lens):
            close(got[b, :n], want[b][at[b]:at[b] + n], F32, scale=want[b].abs().max().item())
            at[b] += n


def delta_case(H, K, dim, vdim, conv, strong=False):
    layer = delta(H, K, dim, vdim, conv)
    w = mixer_weights(layer, 24)
    if strong:  # from no decay to exp(-200) per token, head by head
        w["dt_bias"] = torch.linspace(-30.0, 40.0, H).to(BF) if H > 1 else torch.full((1,), 40.0).to(BF)
        w["A_log"] = torch.linspace(-6.0, 1.6, H).to(BF) if H > 1 else torch.full((1,), 1.6).to(BF)
    return layer["mixer"], w


def delta_mixer(m, w, dtype, eps=1e-5):
    from ohara_amd.hybrid import HeadDelta

    return HeadDelta(w["q"], w["k"], w["v"], w["q.conv"], w["k.conv"], w["v.conv"], w["b"], w["A_log"], w["a"], w["dt_bias"], w["g"],
                     w["norm"], w["o"], heads=m["heads"], kv_heads=m["kv_heads"], dim=m["dim"], vdim=m["vdim"], eps=eps, dtype=dtype)


DELTAS = [(4, 2, 24, 20, 2), (3, 1, 16, 37, 5), (1, 1, 8, 4, 1), (2, 2, 128, 128, 4), (2, 1, 100, 256, 3), (2, 1, 256, 48, 2),
          (6, 3, 64, 64, 4), (5, 5, 7, 9, 6)]


@pytest.mark.parametrize("strong", [False, True])
@pytest.mark.parametrize("shape", DELTAS)
def test_delta_rule_in_portions(cuda, shape, strong):
    m, w = delta_case(*shape, strong=strong)
    h = rnd(101, 24, seed=4)
    want = R.delta_mixer(h.double(), {k: t.double() for k, t in w.items()}, "", m, 1e-5)
    mixer = delta_mixer(m, w, F32)
    for cuts in ([101], [1] * 101, [2] * 50 + [1], [31, 32, 33, 5], [1, 63, 1, 36], [64, 2, 35]):
        close(in_portions(mixer, h, cuts, F32), want, F32, tol=2e-5)
    if not strong:
        for cuts in ([101], [40] + [1] * 61):
            close(in_portions(delta_mixer(m, w, BF), h.to(BF), cuts, BF),
                  R.delta_mixer(h.to(BF).double(), {k: t.double() for k, t in w.items()}, "", m, 1e-5), BF, tol=4e-2)


def test_delta_rule_remembers_a_far_token(cuda):
    """Without decay a key written once is read hundreds of tokens later; orthogonal keys in between leave it alone."""
    from ohara_amd import _lib, ops

    dim, vdim, T = 64, 16, 400
    off = 2 * dim + vdim
    keep = dict(conv_w=torch.ones(1, off), neg_a=-torch.exp(torch.tensor([-60.0])), dt_bias=torch.zeros(1), norm_w=torch.ones(vdim))
    keep = {k: dev(t) for k, t in keep.items()}
    d = _lib.OharaDelta()
    d.heads = d.kv_heads = d.taps = 1
    d.dim, d.vdim, d.off_g, d.off_a, d.off_b, d.eps, d.flags = dim, vdim, off, off + vdim, off + vdim + 1, 0.0, _lib.DELTA_SILU_GATE
    for k, t in keep.items():
        setattr(d, k, t.data_ptr())
    big = 50.0
    p = torch.zeros(T, off + vdim + 8)
    k = big * F.one_hot(1 + torch.arange(T) % (dim - 1), dim)
    k[3] = big * F.one_hot(torch.tensor(0), dim)
    p[:, :dim] = -40.0  # silu of it is nothing
    p[T - 1, 0] = big   # the last token asks for token 3's key
    p[:, dim:2 * dim] = torch.where(k > 0, k, -40.0 * torch.ones(1)).float()
    v, gate = rnd(T, vdim, seed=1, s=2.0), rnd(T, vdim, seed=2)
    p[:, 2 * dim:off], p[:, off:off + vdim], p[:, off + vdim + 1] = v, gate, 30.0  # step size 1
    want = R.rms(F.silu(v[3].double()), 0.0) * F.silu(gate[-1].double())
    for cuts in ([T], [T - 1, 1], [200, 199, 1]):
        state, ring, at = torch.zeros(1, 1, dim, vdim, device=cuda), torch.zeros(1, 1, off, device=cuda), 0
        for n in cuts:
            seq, part = ops.Seq(1, n, at), dev(p[at:at + n])
            if n == 1:
                out = ops.delta_step(d, part, state, ring, seq)
            else:
                ws = torch.empty(ops.delta_workspace_bytes(1, dim, vdim, 1, n), dtype=torch.uint8, device=cuda)
                out = ops.delta_prefill(d, part, None, None, state, ring, ws, seq)
            at += n
        close(out[-1], want, F32, tol=1e-4)


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("dim", [1, 5, 16, 256])
def test_token_side(cuda, dtype, dim):
    from ohara_amd import ops
    from ohara_amd.hybrid import TokenSide

    d, vocab, layers, eps = 36, 13, 3, 1e-4
    table, gate, proj, nw = rnd(vocab, layers * dim).to(BF), rnd(dim, d, seed=1, s=0.3).to(BF), rnd(d, dim, seed=2).to(BF), rnd(d, seed=3).to(BF)
    laid = TokenSide.lay_out(table, layers, dtype=dtype)
    for rows in (1, 7, 70):
        x, ids = rnd(rows, d, seed=rows), torch.randint(0, vocab, (rows,), generator=torch.Generator().manual_seed(rows))
        for i in (0, 2):
            side = TokenSide(gate, proj, nw, laid, i * ops.round8(dim), eps=eps, dtype=dtype)
            seq, xd = ops.Seq(rows, 1), dev(x)
            read = ops.residual_norm(xd, seq, dtype, mode="copy")
            ops.residual_norm(xd, seq, dtype, **side.norm.of(side(read, ids.cuda())))
            w = {"gate": gate.double(), "proj": proj.double(), "norm": nw.double()}
            want = R.token_side(x.double(), table[ids, i * dim:(i + 1) * dim].double(), w, "", eps)
            diff = (xd.double().cpu() - x.double() - want).pow(2).mean().sqrt() / want.pow(2).mean().sqrt()
            assert diff < (1e-5 if dtype == F32 else 2e-2), (rows, i, diff)


@pytest.mark.parametrize("d, dim", [(36, 5), (60, 16), (4, 1), (1000, 40), (1024, 64), (2048, 100), (5000, 256), (35, 7)])
def test_token_side_and_updates_in_one_launch(cuda, d, dim):
    """Against float64 with the launch's roundings (residual, gated embedding and projection to bf16), and against the
    separate launches of the 32-bit build."""
    from ohara_amd import ops
    from ohara_amd.hybrid import GroupNorm, LayerNorm, TokenSide

    vocab, layers, eps = 13, 2, 1e-4
    table, gate, proj = rnd(vocab, layers * dim).to(BF), rnd(dim, d, seed=1, s=2 / d ** 0.5).to(BF), rnd(d, dim, seed=2).to(BF)
    w1, w2, w3 = (rnd(d, seed=s) for s in (3, 4, 5))
    rounded = lambda t: t.to(BF).double()  # noqa: E731
    for rows in (1, 7, 70):
        x, y = rnd(rows, d, seed=rows), (rnd(rows, ops.round8(d), seed=rows + 1) + 0.5).to(BF)
        y[:, d:] = 0
        ids = torch.randint(0, vocab, (rows,), generator=torch.Generator().manual_seed(rows))
        yd, e = y[:, :d].double(), table[ids, dim:].double()
        for center in (True, False):
            kind = (lambda w: LayerNorm(w, eps)) if center else (lambda w: GroupNorm(w, 1, eps))
            norm = (lambda t, w: R.layer_norm(t, w.double(), eps)) if center else (lambda t, w: R.rms(t, eps) * w.double())  # noqa: E731
            mid = x.double() + norm(yd, w1)
            z = rounded(R.gelu_tanh(rounded(mid) @ gate.double().t()) * e)
            want = mid + R.rms(rounded(z @ proj.double().t()), eps) * w2.double()
            for groups in (None, 1, 2, 4, 8, 16):
                if groups and (groups * d > ops.TOKEN_SIDE_ELEMENTS or d % 4):
                    continue
                side = TokenSide(gate, proj, w2, TokenSide.lay_out(table, layers), ops.round8(dim), eps=eps)
                xd = dev(x)
                if groups is None:
                    out = side.update(xd, ops.Seq(rows, 1), ids.cuda(), dev(y), kind(w1), kind(w3))
                else:
                    out = ops.token_side(xd, dev(y), dev(w1), side.gate.w, side.proj.w, side.table, side.column, ids.cuda(), dev(w2), eps,
                                         dev(w3), center_y=center, center_out=center, rows_per_group=groups)
                # a rounding that falls the other way moves z, and with it everything after, by a bf16 step of one entry
                assert ((xd.double().cpu() - want).abs() <= 0.02 + 2.0 ** -6 * (want - mid).abs()).all(), (rows, groups)
                close(out[:, :d], norm(xd.double().cpu(), w3), BF)
                assert not out[:, d:].any()
            side = TokenSide(gate, proj, w2, TokenSide.lay_out(table, layers, dtype=F32), ops.round8(dim), eps=eps, dtype=F32)
            xd = dev(x)
            out = side.update(xd, ops.Seq(rows, 1), ids.cuda(), dev(y, F32), kind(w1), kind(w3))
            want = mid + R.rms((R.gelu_tanh(mid @ gate.double().t()) * e) @ proj.double().t(), eps) * w2.double()
            close(xd, want, F32, tol=3e-5)
            close(out[:, :d], norm(want, w3), F32, tol=1e-4)


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
@pytest.mark.parametrize("name", ["odd", "wide"])
def test_portions_of_prompts(cuda, models, name, dtype):
    cfg, w, m = models(name, dtype)
    toks = tokens(cfg, 140, seed=2)
    want = reference(cfg, w, toks)
    for cuts in ([2] * 70, [1, 2, 3, 15, 16, 17, 31, 32, 23], [64, 64, 12], [65, 2, 63, 10], [44, 1, 1, 94], [7] * 20):
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
    seqs = [tokens(cfg, n + 35, seed=20 + n) for n in lens]
    want = [reference(cfg, w, s) for s in seqs]
    cache, slots = poisoned(m, 6), [4, 0, 5, 2]
    pad = lambda rows: torch.tensor([r + [0] * (max(map(len, rows)) - len(r)) for r in rows])  # noqa: E731
    got = m(pad([s[:n] for s, n in zip(seqs, lens)]), cache, [0] * 4, seq_lens=lens, slots=slots)
    last = m(pad([s[:n] for s, n in zip(seqs, lens)]), m.build_kv_cache(4), [0] * 4, seq_lens=lens, last_only=True)
    for b, n in enumerate(lens):
        assert agrees(got[b, :n], want[b][:n], dtype)
        assert agrees(last[b], want[b][n - 1:n], dtype)
    at = list(lens)
    for more in ([3, 1, 4, 2], [20, 2, 17, 5]):  # one call, every sequence at its own position with its own count
        got = m(pad([s[n:n + k] for s, n, k in zip(seqs, at, more)]), cache, at, seq_lens=more, slots=slots)
        for b, (n, k) in enumerate(zip(at, more)):
            assert agrees(got[b, :k], want[b][n:n + k], dtype)
        at = [n + k for n, k in zip(at, more)]
    for step in range(4):  # sequence 1 sits out now and then
        rows = [b for b in range(4) if not (b == 1 and step % 2)]
        got = m(torch.tensor([[seqs[b][at[b]]] for b in rows]), cache, [at[b] for b in rows], slots=[slots[b] for b in rows])
        for i, b in enumerate(rows):
            assert agrees(got[i], want[b][at[b]:at[b] + 1], dtype)
            at[b] += 1
    assert cache[0].lengths[1] == 0
    assert all(torch.isnan(t[[1, 3]]).all() for c in cache for t in c.tensors.values())


@pytest.mark.parametrize("name, dtype", [("odd", F32), ("wide", BF)])
def test_long_decoding(cuda, models, name, dtype):
    cfg, w, m = models(name, dtype)
    toks = tokens(cfg, 500, seed=5)
    want = reference(cfg, w, toks)
    cache = m.build_kv_cache(1)
    assert agrees(m(torch.tensor([toks[:60]]), cache, 0)[0], want[:60], dtype)
    got = [m(torch.tensor([[toks[t]]]), cache, t)[0] for t in range(60, 500)]
    assert agrees(torch.cat(got), want[60:], dtype)


def test_a_far_token_shows_in_the_logits(cuda):
    """The first layer's latent attention, its queries and keys scaled up: changing a token hundreds of positions back moves
    the last logits as much as the oracle says."""
    cfg = config(48, 60, 4, [latent(4, 16, 12, 24, 20, 3.0), attention(2, 1, 16, 16, 1.0, 100.0, 8, 10.0, 50)])
    w = R.random_weights(cfg, seed=2)
    m = build(cfg, w, F32)
    toks = tokens(cfg, 450, seed=1)
    base = reference(cfg, w, toks)[-1]
    moved = 0.0
    for far in (0, 1, 130, 399, 400):
        other = list(toks)
        other[far] = (toks[far] + 7) % cfg["vocab"]
        want = reference(cfg, w, other)
        moved = max(moved, (want[-1] - base).abs().max().item())
        cache = m.build_kv_cache(1)
        assert agrees(m(torch.tensor([other[:-20]]), cache, 0)[0], want[:-20], F32)
        got = [m(torch.tensor([[other[t]]]), cache, t)[0] for t in range(430, 450)]
        assert agrees(torch.cat(got), want[-20:], F32)
    assert moved > 0.05


def test_errors(cuda, models):
    cfg, _, m = models("ones", F32)
    one = torch.tensor([[1]])
    cache = m.build_kv_cache(1)
    for args, kw, message in (
        ((torch.tensor([1]),), {}, "shape"), ((one, cache), {}, "non-negative"), ((one, cache[:1], 0), {}, "one entry per"),
        ((one, cache, 3), {}, "sequential"), ((torch.zeros(1, 513, dtype=torch.long), cache, 0), {}, "exceeds"),
        ((one, cache, 0), {"slots": [1]}, "slots"), ((one, cache, 0), {"seq_lens": [2]}, "seq_lens"),
    ):
        with pytest.raises(ValueError, match=message):
            m(*args, **kw)
    with pytest.raises(IndexError):
        m(torch.tensor([[cfg["vocab"]]]), cache, 0)
    for name, message in (("head", "head"), ("side.embed", "side.embed"), ("l0.mix.q", "rows"), ("l1.mix.dkv", "entries"),
                          ("l1.mix.uv", "rows"), ("l2.mix.a", "rows")):
        bad = R.random_weights(cfg)
        bad[name] = torch.cat([bad[name]] * 2)
        with pytest.raises(ValueError, match=message):
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
    sampled = eng.generate([{"role": "user", "content": "x"}], SamplingConfig(temperature=0.9, top_k=5, max_new_tokens=6))
    assert len(sampled.split()) == 6
    meta = eng.metadata()
    assert meta["layers"] == 6 and meta["vocab_size"] == cfg["vocab"] and meta["dtype"] == "float32"


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

    def leave(i):
        for b in [b for b, o in owner.items() if o == i]:
            bat.remove(b)
            del owner[b]

    join(0, 1)
    run(5)
    join(2)
    run(4)
    leave(1)
    run(2)       # the freed row rides along
    join(3)      # and is taken again
    run(3)
    leave(0)
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


def test_replayed_trace(cuda, tmp_path, monkeypatch, capsys):
    from safetensors.torch import save_file

    from ohara_amd import trace

    cfg = config(48, 75, 3, [delta(3, 3, 12, 20, 4), latent(2, 20, 12, 24, 28, 0.3, 40), attention(2, 1, 28, 36, 0.25, 80.0, 10, 7.0, 13)])
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
