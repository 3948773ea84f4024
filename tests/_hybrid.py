"""Helpers of the hybrid decoders' tests: random inputs, comparisons with float64, caches full of an earlier owner's leftovers."""

import torch
import torch.nn.functional as F

BF, F32 = torch.bfloat16, torch.float32


def tokens(cfg, n, seed=0):
    return torch.randint(0, cfg["vocab"], (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def doubled(weights):
    return {k: v.double() for k, v in weights.items()}


def row_errors(got, want):
    """Root mean square of the logits' difference, row by row, over that of the logits."""
    want = want.double()
    d = got.double().cpu() - want
    return d.pow(2).mean(-1).sqrt() / want.pow(2).mean().sqrt()


def error(got, want):
    return row_errors(got, want).max().item()


def agrees(got, want, dtype, f32=(2e-5, 2e-5), bf16=(0.12, 0.025)):
    """Logits row by row against float64, as a share of their root mean square: (largest, median) row.  The defaults are for
    norms on the sublayer outputs only, where the CPU statement with its activations rounded to bf16 lies 0.5 - 1 % away on
    average on random models and 6 % at single ill-conditioned positions (a norm over small values)."""
    rows, (largest, median) = row_errors(got, want), f32 if dtype == F32 else bf16
    return rows.max() < largest and (len(rows) < 8 or rows.median() < median)


def rnd(*shape, seed=0, s=1.0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed)) * s


def dev(t, dtype=None):
    return t.to("cuda", dtype if dtype is not None else t.dtype).contiguous()


def close(got, want, dtype, scale=None, tol=None):
    """bf16: one rounding of the result (2^-9 of it) plus fp32 noise; fp32: noise."""
    got, want = got.double().cpu(), want.double()
    scale = want.abs().max().item() if scale is None else scale
    bound = (2.0 ** -8 * want.abs() if dtype == BF else 0.0) + (tol or 1e-5) * scale
    bad = (got - want).abs() > bound
    assert not bad.any(), ((got - want).abs().max().item(), int(bad.sum()), scale)


def poisoned(model, rows):
    cache = model.build_kv_cache(rows)
    for c in cache:
        for t in c.tensors.values():
            t.fill_(float("nan"))
    return cache


def i32(values):
    return torch.tensor(values, dtype=torch.int32, device="cuda")


def in_portions(mixer, h, cuts, dtype, start=0):
    """The rows of h through a mixer in portions, in row 1 of a state full of an earlier owner's leftovers."""
    from ohara_amd import ops
    from ohara_amd.state_cache import LayerState

    st = LayerState(512, {k: torch.full_like(t, float("nan")) for k, t in mixer.state(3, 512).items()})
    at, got, slots = 0, [], i32([1])
    for n in cuts:
        seq = ops.Seq(1, n, at, slots=slots, host=([at], [n], [1]))
        x = F.pad(h[at:at + n], (0, ops.round8(h.shape[1]) - h.shape[1]))
        got.append(mixer(dev(x, dtype), st, seq)[:, :h.shape[1]])
        at += n
    assert at == len(h) and all(torch.isnan(t[[0, 2]]).all() for t in st.tensors.values())
    return torch.cat(got)


class Tok:
    eos_token_id = bos_token_id = None

    def __init__(self, vocab):
        self.vocab = vocab

    def __len__(self):
        return self.vocab

    def get_vocab(self):
        return {}

    def encode(self, text, add_special_tokens=False):
        return [int(t) for t in text.split()]

    def decode(self, ids, skip_special_tokens=True):
        return "".join(f"{i} " for i in ids)
