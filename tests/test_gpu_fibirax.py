"""Fibirax on the GPU against the plain CPU statement (oracle/fibirax_ref.py): each mechanism alone, whole prompts, decoding
through the caches, prompts in portions, batches of unequal sequences, reused cache rows, long decoding and the generation
entry points.  The 32-bit build is the sharp comparison, bfloat16 the served one."""

import io
import json
import sys

import pytest
import torch
import torch.nn.functional as F

from _fibirax import CONFIGS, agrees, attention, build, config, experts, layer, reference, retention
from _hybrid import Tok, close, dev, doubled, i32, in_portions, poisoned, rnd, tokens
from oracle import fibirax_ref as R

pytestmark = pytest.mark.gpu
BF, F32, D = torch.bfloat16, torch.float32, torch.float64


def mixer_weights(left, right, width, seed=0):
    """The tensors of one layer's mixer by their names inside the mixer."""
    w = R.random_weights({"width": width, "vocab": 4, "layers": [layer(left, right)]}, seed)
    return {k[len("l0.mix."):]: t for k, t in w.items() if k.startswith("l0.mix.")}


# ---- mechanisms -------------------------------------------------------------------------------


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("d", [60, 35, 1024, 1500, 3000, 5000])
@pytest.mark.parametrize("top, share", [(1, False), (2, True), (7, True)])
def test_residual_update_with_scaled_embedding_and_mixture(cuda, dtype, d, top, share):
    from ohara_amd import ops
    from ohara_amd.hybrid import GroupNorm, LayerNorm

    rows, vocab, n, eps = 5, 11, 3, 1e-4
    d8, seq = ops.round8(d), ops.Seq(rows, 1)
    table, ids = rnd(vocab, d).to(dtype), torch.tensor([3, 10, 0, 3, 7])
    x = torch.empty(rows, d, device=cuda)
    out = ops.residual_norm(x, seq, dtype, ids=ids.cuda(), table=dev(table), table_scale=0.3, mode="copy")
    close(x, 0.3 * table[ids].double(), F32)
    assert torch.equal(out[:, :d], x.to(dtype)) and not out[:, d:].any()
    g = torch.Generator().manual_seed(1)
    idx = torch.stack([torch.randperm(n + top, generator=g)[:top] for _ in range(rows)]).int()  # ids from n on: the input itself
    wgt, pos = torch.rand(rows, top, generator=g), torch.randperm(rows * top, generator=g).view(rows, top).int()
    y, h, sh = (rnd(k, d8, seed=s, s=3.0).to(dtype) for k, s in ((rows * top, 2), (rows, 3), (rows, 4)))
    y[pos[idx >= n].long()] = float("nan")  # rows nobody wrote
    term = torch.where((idx < n).unsqueeze(-1), y[pos.long()].double(), h.double().unsqueeze(1))[..., :d]
    want_y = (wgt.double().unsqueeze(-1) * term).sum(1) + (sh.double()[:, :d] if share else 0)
    mix = ops.Mixture(dev(idx), dev(wgt), dev(pos), dev(y), dev(h), dev(sh) if share else None, n)
    x0, w, w2, ls = rnd(rows, d, seed=5), rnd(d, seed=6), rnd(d, seed=7), rnd(d, seed=8)
    for norm, ref in ((GroupNorm(w, 1, eps, scale=ls), R.rms(want_y, eps) * w.double() * ls.double()),
                      (LayerNorm(w, eps), R.rms(want_y - want_y.mean(-1, keepdim=True), eps) * w.double())):
        xd = dev(x0)
        out = ops.residual_norm(xd, seq, dtype, **{**norm.of(mix), **GroupNorm(w2, 1, eps).out()})
        want = x0.double() + ref
        close(xd, want, F32)
        close(out[:, :d], R.rms(want, eps) * w2.double(), dtype)
        assert not out[:, d:].any()


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("H, G, dim, vdim, rot", [(6, 2, 20, 12, 12), (3, 3, 14, 30, 6), (8, 1, 64, 96, 64), (4, 4, 130, 200, 0),
                                                  (2, 1, 24, 8, 2), (5, 1, 9, 7, 8), (40, 8, 128, 64, 128), (1, 1, 1, 1, 0), (2, 2, 256, 33, 256)])
def test_head_norms_rotation_and_append(cuda, dtype, H, G, dim, vdim, rot):
    from ohara_amd import ops
    from ohara_amd.hybrid import rotary_tables

    B, S, T, base, eps = 3, 4, 200, 900.0, 1e-3
    n = H * dim + G * (dim + vdim)
    p = (rnd(B * S, ops.round8(n)) * torch.logspace(-1, 1, B * S).unsqueeze(1)).to(dtype)
    qn, kn = rnd(dim, seed=1), rnd(dim, seed=2)
    cos, sin = rotary_tables(base, rot, T, "cuda")
    kc = torch.full((4, T, G, ops.round8(dim)), 7.0, dtype=dtype, device=cuda)
    vc = torch.full((4, T, G, ops.round8(vdim)), 7.0, dtype=dtype, device=cuda)
    starts, lens, slots = [0, 195, 2], [4, 1, 3], [3, 0, 1]
    seq = ops.Seq(B, S, 0, i32(starts), True, i32(lens), i32(slots))
    q = ops.qkv_headnorm_rotate_append(dev(p), H, G, dim, vdim, dev(qn), dev(kn), eps, cos, sin, rot, kc, vc, seq).view(B, S, H, -1)
    pd, freqs = p.double().view(B, S, -1), R.rotary_frequencies(base, rot)
    for b in range(B):
        m, at = lens[b], starts[b]
        x = R.rms(pd[b, :m, :(H + G) * dim].reshape(m, H + G, dim), eps)
        x = x * torch.cat([qn.double().expand(H, dim), kn.double().expand(G, dim)])
        want = R.rotate(torch.cat([torch.zeros(at, H + G, dim, dtype=D), x]), freqs)[at:]
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


def run_scored(q, kc, vc, dim, vdim, start, n, ns=1, **kw):
    """In the middle columns of a wider buffer, whose other columns stay as they are."""
    from ohara_amd import ops

    H, G, w = q.shape[1], kc.shape[2], ops.round8(q.shape[1] * vdim)
    qp = F.pad(q[start:start + n], (0, ops.round8(dim) - dim)).reshape(n, -1)
    seq = ops.Seq(1, n, start, slots=i32([1]))
    ws = ops.attn_bias_workspace(1, H, vdim, ns, "cuda") if ns > 1 else None
    wide = torch.full((n, w + 16), 9.0, dtype=q.dtype, device="cuda")
    out = ops.attn_scored(dev(qp), kc, vc, H, G, dim, vdim, kc.shape[1], seq=seq, n_split=ns, workspace=ws, out=wide[:, 8:8 + w], **kw)
    assert not out[:, H * vdim:].any() and (wide[:, :8] == 9.0).all() and (wide[:, 8 + w:] == 9.0).all()
    return out[:, :H * vdim].view(n, H, vdim)


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("H, G, dim, vdim, cap, window", [
    (6, 2, 20, 12, 4.0, 24), (5, 5, 72, 40, 0.0, 64), (8, 1, 64, 128, 9.0, 65), (7, 1, 128, 96, 2.5, 1), (2, 1, 200, 256, 6.0, 63),
    (4, 2, 256, 130, 0.0, 7), (1, 1, 8, 8, 30.0, 0), (3, 1, 33, 17, 5.0, 1000), (8, 4, 96, 96, 30.0, 100), (2, 2, 48, 24, 5.0, 2),
    (4, 4, 128, 128, 20.0, 128)])
def test_capped_attention_in_a_window_with_a_sink(cuda, dtype, H, G, dim, vdim, cap, window):
    L, scale = 200, 2.0 / dim ** 0.5
    q, k, v, kc, vc = scored_case(dtype, H, G, dim, vdim, 256, L)
    for sink in (True, False):
        want = 1.7 * R.window_attention(q.double(), k.double(), v.double(), scale, cap or None, window or None, sink)
        run = lambda start, n, ns=1: run_scored(q, kc, vc, dim, vdim, start, n, ns, scale=scale, cap=cap, window=window, out_scale=1.7,  # noqa: E731, B023
                                                sinks=torch.zeros(H, device="cuda") if sink else None)  # noqa: B023
        for start, n in ((0, L), (0, 16), (0, 65), (3, 61), (63, 17), (64, 64), (130, 70), (0, 2), (77, 5), (198, 2)):
            close(run(start, n), want[start:start + n], dtype, scale=1.0)
        for t in (0, 1, 6, 7, 23, 24, 62, 63, 64, 65, 99, 100, 127, 128, 199):
            for ns in (1, 2, 5, 64):
                close(run(t, 1, ns), want[t:t + 1], dtype, scale=1.0)


@pytest.mark.parametrize("dtype", [F32, BF])
def test_sinks_of_other_scores_chunks_in_windows(cuda, dtype):
    """A sink per head as one more key without a value, also far above and far below the scores; a window inside chunks."""
    H, G, dim, vdim, L = 4, 2, 24, 16, 150
    q, k, v, kc, vc = scored_case(dtype, H, G, dim, vdim, 256, L)
    sinks = torch.tensor([-40.0, 0.7, 3.0, 25.0])
    s = torch.einsum("ihd,jhd->hij", q.double(), k.double().repeat_interleave(2, 1)) * 0.3
    i, j = torch.arange(L).unsqueeze(1), torch.arange(L)
    hidden = (j > i) | (i - j >= 40) | (i // 50 != j // 50)
    s = torch.cat([s.masked_fill(hidden, float("-inf")), sinks.double().view(H, 1, 1).expand(H, L, 1)], -1)
    want = torch.einsum("hij,jhv->ihv", torch.softmax(s, -1)[..., :-1], v.double().repeat_interleave(2, 1))
    run = lambda start, n, ns=1: run_scored(q, kc, vc, dim, vdim, start, n, ns, scale=0.3, window=40, chunk=50, sinks=dev(sinks))  # noqa: E731
    for start, n in ((0, L), (45, 20), (99, 3)):
        close(run(start, n), want[start:start + n], dtype, scale=1.0)
    for t in (0, 39, 40, 49, 50, 89, 90, 100, 149):
        for ns in (1, 3, 64):
            close(run(t, 1, ns), want[t:t + 1], dtype, scale=1.0)


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("window", [50, 64, 129])
def test_keys_at_the_edges_of_a_window(cuda, dtype, window):
    """One key with a score of 30 among keys of nearly none: seen by the queries whose window holds it, by no other."""
    H, G, dim, vdim, L, T, cap = 4, 2, 32, 16, 400, 512, 30.0
    q, k, v, kc, vc = scored_case(dtype, H, G, dim, vdim, T, L, seed=5)
    q2 = (5.0 * torch.sign(q[:1, :1])).expand_as(q).contiguous()
    run = lambda start, n, ns=1: run_scored(q2, kc, vc, dim, vdim, start, n, ns, scale=1.0, cap=cap, window=window,  # noqa: E731
                                            sinks=torch.zeros(H, device="cuda"))
    for far in (0, 1, 63, 64, 200):
        k2 = 0.01 * k
        k2[far] = 5.0 * torch.sign(q[0, 0])  # 800, capped to 30
        kc[1, :L, :, :dim] = dev(k2)
        want = R.window_attention(q2.double(), k2.double(), v.double(), 1.0, cap, window)
        end = far + window  # the first query that does not see it
        one = v[far].double().repeat_interleave(2, 0)
        assert (want[far:end] - one).abs().max() < 1e-6 and (want[end] - one).abs().max() > 0.1
        close(run(0, L), want, dtype, scale=1.0)
        for t in (far, end - 1, end, end + 1):
            for ns in (1, 3, 64):
                close(run(t, 1, ns), want[t:t + 1], dtype, scale=1.0)
        close(run(end - 9, 20), want[end - 9:end + 11], dtype, scale=1.0)
        close(run(end - 2, 4), want[end - 2:end + 2], dtype, scale=1.0)


@pytest.mark.parametrize("dtype", [F32, BF])
def test_the_sink_takes_its_share(cuda, dtype):
    """Scores far below zero: without the sink the weights would add up to one, with it to nearly nothing."""
    H, dim, vdim, L = 2, 16, 8, 100
    q, k, v, kc, vc = scored_case(dtype, H, H, dim, vdim, 128, L)
    k2 = -torch.sign(q[0]).expand_as(k).contiguous()
    q2 = (0.5 * torch.sign(q[:1])).expand_as(q).contiguous()
    kc[1, :L, :, :dim] = dev(k2)
    v2 = v.abs() + 1
    vc[1, :L, :, :vdim] = dev(v2)
    want = R.window_attention(q2.double(), k2.double(), v2.double(), 1.0, None, 60)
    assert 0 < want.max() < 0.1
    for start, n in ((0, L), (0, 1), (59, 1), (60, 1), (99, 1), (90, 4)):
        got = run_scored(q2, kc, vc, dim, vdim, start, n, scale=1.0, window=60, sinks=torch.zeros(H, device="cuda"))
        close(got, want[start:start + n], dtype, scale=want.max().item())


ATTENTIONS = [attention(6, 2, 20, 12, 0.3, 45, dims=12, scaling=(4.0, 1.0, 4.0, 64)), attention(3, 3, 14, 30, 0.2, 7, base=1e4, dims=6, cap=20.0),
              attention(8, 1, 64, 128, 0.125, 64, base=5e5, cap=30.0)]


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("m", ATTENTIONS)
def test_attention_mixer_in_portions(cuda, dtype, m):
    from ohara_amd.hybrid import RotaryAttention

    w = {k[len("left."):]: t for k, t in mixer_weights(m, retention((0.5,), 8, 8), 24).items() if k.startswith("left.")}
    h = rnd(150, 24, seed=4).to(dtype)
    want = R.attention_heads(h.double(), doubled(w), "", m, 1e-4) @ w["o"].double().t()
    sc = m["rot"].get("scaling")
    mixer = RotaryAttention(w["q"], w["k"], w["v"], w["o"], heads=m["heads"], kv_heads=m["kv_heads"], dim=m["dim"], vdim=m["vdim"],
                            scale=m["scale"], rot_base=m["rot"]["base"], rot_dims=m["rot"]["dims"], cap=m["softcap"], window=m["mask"]["size"],
                            rot_scaling=tuple(sc[k] for k in ("factor", "low", "high", "original")) if sc else None, q_norm=w["q.norm"],
                            k_norm=w["k.norm"], eps=1e-4, sinks=torch.zeros(m["heads"]), dtype=dtype)
    for cuts in ([150], [1] * 150, [2] * 75, [44, 1, 1, 62, 42], [63, 2, 85]):
        close(in_portions(mixer, h, cuts, dtype), want, dtype, tol=2e-2 if dtype == BF else 1e-5)


RETENTIONS = [retention((0.9, 0.99, 0.5), 12, 20), retention((0.97, 1.0), 9, 7), retention((0.0, 0.999, 0.8), 16, 11), retention((0.6,), 1, 1),
              retention((0.97, 0.996), 128, 160), retention((0.99, 0.3), 256, 256), retention((0.9, 0.98, 0.999, 1.0, 0.0), 64, 64),
              retention((0.95, 0.999), 40, 96)]


def retention_mixer(m, w, dtype, eps=1e-5):
    from ohara_amd.hybrid import Retention

    return Retention(w["q"], w["k"], w["v"], w["g"], w["o"], heads=m["heads"], dim=m["dim"], vdim=m["vdim"], decay=m["decay"],
                     k_scale=m["dim"] ** -0.5, eps=eps, dtype=dtype)


def retention_weights(m, width=24):
    w = mixer_weights(attention(1, 1, 8, 8, 1.0, 1), m, width)
    return {k[len("right."):]: t for k, t in w.items() if k.startswith("right.")}


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("m", RETENTIONS)
def test_retention_in_portions(cuda, dtype, m):
    w, n = retention_weights(m), 300
    h = rnd(n, 24, seed=4).to(dtype)
    want = R.retention_heads(h.double(), doubled(w), "", m, 1e-5) @ w["o"].double().t()
    mixer = retention_mixer(m, w, dtype)
    for cuts in ([n], [1] * n, [2] * 150, [127, 128, 45], [129, 1, 63, 65, 42], [64, 2, 234], [1, 299], [255, 45]):
        close(in_portions(mixer, h, cuts, dtype), want, dtype, tol=4e-2 if dtype == BF else 2e-5)


@pytest.mark.parametrize("dtype", [F32, BF])
def test_retention_states_are_exact_sums(cuda, dtype):
    """The state after a prompt against the sum over its tokens: nothing but fp32 rounding, also where q, k and v are bf16."""
    from ohara_amd import _lib, ops

    heads, dim, vdim, T, decay = 3, 40, 24, 333, (0.99, 1.0, 0.9)
    n = 2 * heads * (dim + vdim)
    p = rnd(2 * T, n).to(dtype)
    powers = (torch.tensor(decay, dtype=D).unsqueeze(1) ** torch.arange(_lib.RETENTION_CHUNK + 1)).float().cuda()
    r = _lib.OharaRetention(heads, dim, vdim, vdim, 0, heads * dim, 2 * heads * dim, heads * (2 * dim + vdim), 1e-5, 0.5, 1.0, 0, powers.data_ptr())
    state = torch.full((3, heads, dim, vdim), float("nan"), device=cuda)
    lens, slots = [T, 70], [2, 0]
    seq = ops.Seq(2, T, 0, None, False, i32(lens), i32(slots))
    chunk = ops.retention_workspace_bytes(heads, dim, vdim, 2, 1)
    pd = p.double().view(2, T, n)
    for chunks in (1, 2, 3):  # also in segments that fit a small workspace
        state.fill_(float("nan"))
        ops.retention(r, dev(p), state, torch.empty(chunk * chunks, dtype=torch.uint8, device=cuda), seq)
        for b, (t, slot) in enumerate(zip(lens, slots)):
            k = pd[b, :t, heads * dim:2 * heads * dim].view(t, heads, dim) * 0.5
            v = pd[b, :t, 2 * heads * dim:heads * (2 * dim + vdim)].view(t, heads, vdim)
            want = R.retention(k, k, v, decay)[1]
            close(state[slot], want, F32, tol=3e-6)
        assert torch.isnan(state[1]).all()


def test_retention_remembers_a_far_token(cuda):
    """Without decay a key written once is read hundreds of tokens later; orthogonal keys in between leave it alone."""
    from ohara_amd import _lib, ops

    dim, vdim, T = 64, 16, 700
    powers = torch.ones(1, _lib.RETENTION_CHUNK + 1, device=cuda)
    r = _lib.OharaRetention(1, dim, vdim, vdim, 0, dim, 2 * dim, 2 * dim + vdim, 0.0, 1.0, 1.0, 0, powers.data_ptr())
    p = torch.zeros(T, 2 * dim + 2 * vdim)
    p[T - 1, 0] = 1.0
    p[:, dim:2 * dim] = F.one_hot(1 + torch.arange(T) % (dim - 1), dim)
    v, gate = rnd(T, vdim, seed=1), rnd(T, vdim, seed=2)
    p[:, 2 * dim:2 * dim + vdim], p[:, 2 * dim + vdim:] = v, gate
    for far in (0, 3, 127, 128, 400):
        p2 = p.clone()
        p2[far, dim:2 * dim] = F.one_hot(torch.tensor(0), dim)
        want = R.rms(v[far].double(), 0.0) * F.silu(gate[-1].double())
        for cuts in ([T], [T - 1, 1], [350, 348, 2]):
            state, at = torch.full((1, 1, dim, vdim), float("nan"), device=cuda), 0
            for n in cuts:
                ws = torch.empty(ops.retention_workspace_bytes(1, dim, vdim, 1, n), dtype=torch.uint8, device=cuda)
                out = ops.retention(r, dev(p2[at:at + n]), state, ws, ops.Seq(1, n, at))
                at += n
            close(out[-1], want, F32, tol=1e-5)


@pytest.mark.parametrize("m", [RETENTIONS[0], RETENTIONS[6]])
def test_retention_of_unequal_sequences(cuda, m):
    from ohara_amd import ops
    from ohara_amd.state_cache import LayerState

    w = retention_weights(m)
    mixer = retention_mixer(m, w, F32)
    hs = [rnd(400, 24, seed=s) for s in (1, 2, 3)]
    want = [R.retention_heads(h.double(), doubled(w), "", m, 1e-5) @ w["o"].double().t() for h in hs]
    st = LayerState(512, {k: torch.full_like(t, float("nan")) for k, t in mixer.state(5, 512).items()})
    slots, at = [4, 0, 2], [0, 0, 0]
    for lens in ([1, 200, 17], [130, 2, 128], [1, 1, 1], [5, 3, 129], [20, 20, 20]):
        S = max(lens)
        x = torch.full((3, S, 24), float("nan"))
        for b, n in enumerate(lens):
            x[b, :n] = hs[b][at[b]:at[b] + n]
        seq = ops.Seq(3, S, 0, i32(at), True, i32(lens), i32(slots), (list(at), lens, slots))
        got = mixer(dev(x.view(3 * S, 24)), st, seq)[:, :24].view(3, S, 24)
        for b, n in enumerate(lens):
            close(got[b, :n], want[b][at[b]:at[b] + n], F32, scale=want[b].abs().max().item(), tol=2e-5)
            at[b] += n
    assert torch.isnan(st.retention[[1, 3]]).all()


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("left, right", [(ATTENTIONS[0], RETENTIONS[1]), (ATTENTIONS[1], RETENTIONS[4])])
def test_parallel_mixer_in_portions(cuda, dtype, left, right):
    from ohara_amd.fibirax import Fibirax, FibiraxConfig

    w, eps = mixer_weights(left, right, 24), 1e-4
    one = layer(left, right, None, 1.3, 0.6)
    cfg = FibiraxConfig.from_dict(config(24, 8, [one], eps=eps))
    host = Fibirax.__new__(Fibirax)
    host.config = cfg
    mixer = host._mixer(cfg.layers[0], lambda name, *shape: w[name], dict(dtype=dtype, device="cuda"))
    h = rnd(150, 24, seed=4).to(dtype)
    want = R.parallel_mixer(h.double(), doubled(w), "", one["mixer"], eps)
    for cuts in ([150], [1] * 150, [2] * 75, [44, 1, 1, 62, 42], [127, 2, 21]):
        close(in_portions(mixer, h, cuts, dtype), want, dtype, tol=4e-2 if dtype == BF else 2e-5)


# ---- experts ------------------------------------------------------------------------------------------


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("ff, k", [(8, 64), (36, 200), (136, 72), (1, 8)])
def test_clamped_unit(cuda, dtype, ff, k):
    from ohara_amd.hybrid import ClampedGLU

    gate, up, down = (rnd(*s, seed=i).to(BF) * f for i, (s, f) in enumerate((((ff, k), 0.3), ((ff, k), 0.3), ((20, ff), 1.0))))
    w = {"gate": gate.double(), "up": up.double(), "down": down.double()}
    unit = ClampedGLU(gate, up, down, limit=0.8, dtype=dtype)
    for rows in (1, 3, 20, 64, 65, 130):
        x = rnd(rows, k, seed=rows).to(dtype)
        want = R.clamped_glu(x.double(), w, "", 0.8)
        close(unit(dev(x))[:, :20], want, dtype, tol=1.5e-2 if dtype == BF else 1e-5)
    h = torch.stack([x.double() @ w["gate"].t(), x.double() @ w["up"].t()])
    assert k < 16 or ((h[0] > 0.8).any() and (h[1] > 0.8).any() and (h[1] < -0.8).any())


def run_router(z_rows, correction, top, groups, keep, dtype, x=None):
    """The router over logits that are the weights' rows themselves (one-hot inputs) or products with x."""
    from ohara_amd import ops

    counter = torch.zeros(1, dtype=torch.int32, device="cuda")
    out = ops.moe_router(dev(x, dtype), dev(z_rows, dtype), None if correction is None else dev(correction), x.shape[1], top, groups, keep, counter)
    assert counter.item() == 0
    return [t.cpu() for t in out]


def check_sorted(idx, offs, pair_of, pos_of):
    """Pairs by expert, in token order inside one."""
    flat = idx.flatten().long()
    order = torch.argsort(flat, stable=True)
    assert torch.equal(pair_of.long(), order) and torch.equal(pos_of.long()[order], torch.arange(len(flat)))
    assert torch.equal(offs.long(), torch.cat([torch.zeros(1, dtype=torch.long), torch.bincount(flat, minlength=len(offs) - 1).cumsum(0)]))


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("n, top, groups, keep, k", [(12, 3, 4, 2, 64), (7, 2, 1, 1, 40), (1, 1, 1, 1, 8), (64, 8, 8, 4, 200), (66, 6, 1, 1, 72),
                                                     (160, 12, 16, 3, 136), (1000, 16, 50, 7, 64), (3, 1, 3, 1, 2048), (300, 64, 3, 1, 16)])
def test_router_and_sort(cuda, dtype, n, top, groups, keep, k):
    w = rnd(n, k, seed=1, s=2 / k ** 0.5).to(dtype)
    corr = rnd(n, seed=2, s=0.7 / n)
    if n == 12:
        corr = corr - 5.0  # every choice score is negative
    for rows in (1, 2, 16, 17, 130, 700):
        x = rnd(rows, k, seed=rows).to(dtype)
        z = x.double() @ w.double().t()
        idx, wgt, offs, pair_of, pos_of = run_router(w, corr, top, groups, keep, dtype, x)
        check_sorted(idx, offs, pair_of, pos_of)
        s = torch.softmax(z, -1)
        choice = s + corr.double()
        sure = 0
        for t in range(rows):
            chosen, want = R.route(z[t], corr.double(), top, groups, keep)
            assert len(set(idx[t].tolist())) == top
            got = s[t][idx[t].long()]
            close(wgt[t], got / got.sum(), F32, scale=1.0, tol=1e-5)
            if idx[t].tolist() != chosen:  # only among choices closer together than fp32 tells apart
                a, b = choice[t][idx[t].long()], choice[t][chosen]
                best = lambda c: torch.stack([c[g * (n // groups):(g + 1) * (n // groups)].max() for g in range(groups)]).sort().values  # noqa: E731
                assert (a - b).abs().max() < 1e-5 or (groups > 1 and best(choice[t]).diff().min() < 1e-5)
            else:
                sure += 1
                close(wgt[t], want, F32, scale=1.0, tol=1e-5)
        assert sure >= 0.98 * rows


def test_router_ties_and_rows_of_nothing(cuda):
    """Equal scores take the lowest outputs and groups; rows that are not numbers still take distinct outputs."""
    x = torch.zeros(5, 8)
    x[1], x[3] = float("nan"), float("inf")
    w = rnd(12, 8)
    idx, wgt, offs, pair_of, pos_of = run_router(w, None, 4, 3, 2, F32, x)
    assert idx[0].tolist() == idx[2].tolist() == idx[4].tolist() == [0, 1, 2, 3] and torch.allclose(wgt[[0, 2, 4]], torch.full((3, 4), 0.25))
    check_sorted(idx, offs, pair_of, pos_of)
    assert all(len(set(r)) == 4 and 0 <= min(r) and max(r) < 12 for r in idx.tolist())


EXPERTS = [(60, experts(10, 3, 36, 0.9, identity=2, groups=(4, 2), shared=(20, 1.7))), (35, experts(7, 2, 21, 1.4, identity=1)),
           (40, experts(1, 1, 16, 0.5, identity=1, groups=(1, 1), shared=(8, 0.4))), (160, experts(30, 4, 72, 1.0, identity=2, groups=(4, 2), shared=(136, 2.0))),
           (72, experts(66, 6, 40, 0.7, shared=(64, 0.5))), (600, experts(4, 2, 520, 1.1, identity=4, shared=(264, 0.8))), (24, experts(1, 1, 8, 1.0))]


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("width, mlp", EXPERTS)
def test_routed_experts(cuda, dtype, width, mlp):
    """Few pairs (weights streamed) and many (tiles), against the oracle with the router's own choice."""
    from ohara_amd import ops
    from ohara_amd.fibirax import Fibirax, FibiraxConfig
    from ohara_amd.hybrid import GroupNorm

    w = R.random_weights({"width": width, "vocab": 4, "layers": [layer(attention(1, 1, 8, 8, 1.0, 1), retention((0.5,), 8, 8), mlp)]}, 3)
    w = {k[len("l0.mlp."):]: t for k, t in w.items() if k.startswith("l0.mlp.")}
    cfg = FibiraxConfig.from_dict(config(width, 8, [layer(attention(1, 1, 8, 8, 1.0, 1), retention((0.5,), 8, 8), mlp)]))
    host = Fibirax.__new__(Fibirax)
    host.config = cfg
    block = host._mlp(cfg.layers[0].mlp, lambda name, *shape: w[name], dict(dtype=dtype, device="cuda"))
    wd, r = doubled(w), mlp["router"]
    for rows in (1, 5, 40, 300, 700):
        h = rnd(rows, width, seed=rows).to(dtype)
        hp = dev(F.pad(h, (0, ops.round8(width) - width)))
        block.trace = []
        mix = block(hp)
        idx, wgt = (t.cpu() for t in block.trace[0])
        x = torch.zeros(rows, width, device=cuda)
        norm = GroupNorm(torch.ones(width), 1, 1e-6)
        ops.residual_norm(x, ops.Seq(rows, 1), dtype, **norm.of(mix))
        hd = h.double()
        outs = torch.stack([R.clamped_glu(hd, wd, f"e{e}.", mlp["expert"]["limit"]) for e in range(r["experts"])] + [hd] * (r.get("identity") or 0))
        y = (wgt.double().unsqueeze(-1) * outs[idx.long(), torch.arange(rows).unsqueeze(1)]).sum(1)
        if mlp.get("shared"):
            y = y + R.clamped_glu(hd, wd, "shared.", mlp["shared"]["limit"])
        close(x, R.rms(y, 1e-6), F32, tol=2e-2 if dtype == BF else 3e-5)
        groups = r.get("groups") or {"count": 1, "keep": 1}
        same = sum(idx[t].tolist() == R.route(hd[t] @ wd["router"].t(), wd["correction"], r["top"], groups["count"], groups["keep"])[0]
                   for t in range(rows))
        assert same >= 0.98 * rows
        assert rows < 300 or len(set(idx.flatten().tolist())) == r["experts"] + (r.get("identity") or 0)


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
    for n in (1, 2, 15, 16, 33, 64, 65, 129, 150):
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
    R.forward(cfg, doubled(w), toks, want)
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
    toks = tokens(cfg, 300, seed=2)
    want = reference(cfg, w, toks)
    for cuts in ([2] * 150, [1, 2, 3, 15, 16, 17, 31, 32, 183], [64, 64, 172], [129, 2, 63, 106], [44, 1, 1, 254], [7] * 42 + [6], [128, 128, 44]):
        cache, at, got = poisoned(m, 1), 0, []
        for n in cuts:
            got.append(m(torch.tensor([toks[at:at + n]]), cache, at)[0])
            at += n
        assert at == 300 and agrees(torch.cat(got), want, dtype), cuts


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("name", ["odd", "wide"])
def test_unequal_sequences_in_one_batch(cuda, models, name, dtype):
    """Prompts of different lengths in one call, in chosen cache rows; portions at different positions; decoding at
    different positions with rows that sit out.  Every sequence is compared as a whole, as if it had been alone."""
    cfg, w, m = models(name, dtype)
    lens = [1, 70, 133, 5]
    seqs = [tokens(cfg, n + 35, seed=20 + n) for n in lens]
    want = [reference(cfg, w, s) for s in seqs]
    cache, slots = poisoned(m, 6), [4, 0, 5, 2]
    pad = lambda rows: torch.tensor([r + [0] * (max(map(len, rows)) - len(r)) for r in rows])  # noqa: E731
    got = m(pad([s[:n] for s, n in zip(seqs, lens)]), cache, [0] * 4, seq_lens=lens, slots=slots)
    last = m(pad([s[:n] for s, n in zip(seqs, lens)]), m.build_kv_cache(4), [0] * 4, seq_lens=lens, last_only=True)
    parts = [[got[b, :n]] for b, n in enumerate(lens)]
    for b, n in enumerate(lens):
        assert agrees(last[b], want[b][n - 1:n], dtype)
    at = list(lens)
    for more in ([3, 1, 4, 2], [20, 2, 17, 5]):  # one call, every sequence at its own position with its own count
        got = m(pad([s[n:n + k] for s, n, k in zip(seqs, at, more)]), cache, at, seq_lens=more, slots=slots)
        for b, k in enumerate(more):
            parts[b].append(got[b, :k])
        at = [n + k for n, k in zip(at, more)]
    for step in range(4):  # sequence 1 sits out now and then
        rows = [b for b in range(4) if not (b == 1 and step % 2)]
        got = m(torch.tensor([[seqs[b][at[b]]] for b in rows]), cache, [at[b] for b in rows], slots=[slots[b] for b in rows])
        for i, b in enumerate(rows):
            parts[b].append(got[i])
            at[b] += 1
    for b in range(4):
        assert agrees(torch.cat(parts[b]), want[b][:at[b]], dtype)
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
    """Retention without decay and scores that stand out: changing a token hundreds of positions back moves the last logits as much as
    the oracle says, through the state alone (the window is short)."""
    cfg = config(48, 60, [layer(attention(2, 1, 12, 20, 3.0, 30), retention((1.0, 0.9999), 8, 24), experts(3, 1, 16, 1.0)),
                          layer(attention(2, 1, 16, 16, 1.0, 20), retention((0.9995,), 12, 16))])
    w = R.random_weights(cfg, seed=2)
    m = build(cfg, w, F32)
    toks = tokens(cfg, 450, seed=1)
    base = reference(cfg, w, toks)[-1]
    moved = 0.0
    for far in (0, 1, 130, 399):
        other = list(toks)
        other[far] = (toks[far] + 7) % cfg["vocab"]
        want = reference(cfg, w, other)
        moved = max(moved, (want[-1] - base).abs().max().item())
        cache = m.build_kv_cache(1)
        assert agrees(m(torch.tensor([other[:-20]]), cache, 0)[0], want[:-20], F32)
        got = [m(torch.tensor([[other[t]]]), cache, t)[0] for t in range(430, 450)]
        assert agrees(torch.cat(got), want[-20:], F32)
    assert moved > 0.01


def test_errors(cuda, models):
    cfg, _, m = models("odd", F32)
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
    for name in ("head", "l0.mix.left.q", "l0.mix.right.g", "l0.mlp.e3.up", "l0.mlp.router", "l2.ls2", "l1.mix.left.k.norm"):
        bad = R.random_weights(cfg)
        bad[name] = torch.cat([bad[name]] * 2)
        with pytest.raises(ValueError, match=name):
            build(cfg, bad, F32)
    import copy

    for change, message in ((lambda c: c["layers"][0]["mixer"]["right"].update(decay=[0.5, 0.5]), "decay"),
                            (lambda c: c["layers"][0]["mixer"]["right"].update(decay=[0.5, 1.5, 0.5]), "decay"),
                            (lambda c: c["layers"][0]["mlp"]["router"].update(groups={"count": 5, "keep": 1}), "groups"),
                            (lambda c: c["layers"][0]["mlp"]["router"].update(groups={"count": 6, "keep": 1}), "kept groups"),
                            (lambda c: c["layers"][0]["mixer"]["left"]["rot"].update(dims=13), "rotated")):
        bad = copy.deepcopy(cfg)
        change(bad)
        with pytest.raises(ValueError, match=message):
            build(bad, R.random_weights(cfg), F32)


# ---- generation -------------------------------------------------------------------------------------


@pytest.mark.parametrize("name", ["odd", "ones"])
def test_greedy_sessions(cuda, models, name):
    cfg, w, m = models(name, F32)
    prompts = [tokens(cfg, 21, seed=s) for s in (1, 2, 3)]
    wd = doubled(w)
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
    want = R.greedy(cfg, doubled(w), prompt, 20)
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
    assert meta["layers"] == 3 and meta["vocab_size"] == cfg["vocab"] and meta["dtype"] == "float32"


@pytest.mark.parametrize("use_graph", [True, False])
def test_continuous_batching_joins_leaves_and_reuses_rows(cuda, models, use_graph):
    from ohara_amd.batching import ContinuousBatcher

    cfg, w, m = models("odd", F32)
    wd = doubled(w)
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

    cfg = config(48, 75, [layer(attention(3, 3, 12, 20, 0.4, 9), retention((0.9, 0.99), 20, 12), experts(5, 2, 24, 0.8, identity=1)),
                          layer(attention(2, 1, 28, 36, 0.25, 13, base=80.0, dims=10, cap=7.0), retention((0.8,), 12, 28), None, 0.5, 1.5)])
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
