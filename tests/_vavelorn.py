"""Small Vavelorn configs with random weights for the tests (every size differs between layers; none is a multiple of
everything), and helpers to run the product and the oracle on them."""

import _hybrid
from _hybrid import doubled
from oracle import vavelorn_ref as R


def _layer(kind, ff, **mixer):
    return {"type": kind, "mixer": mixer, "mlp": {"kind": "dense", "ff": ff} if ff else None}


def attention(heads, kv, dim, vdim, scale, base, dims, cap, chunk, ff=0):
    return _layer("attention", ff, heads=heads, kv_heads=kv, dim=dim, vdim=vdim, scale=scale, rot={"base": base, "dims": dims},
                  softcap=cap, mask={"size": chunk})


def latent(heads, dim, vdim, kv_rank, q_rank, scale, ff=0):
    return _layer("latent_attention", ff, heads=heads, dim=dim, vdim=vdim, kv_rank=kv_rank, q_rank=q_rank, scale=scale)


def delta(heads, kv, dim, vdim, conv, ff=0):
    return _layer("delta", ff, heads=heads, kv_heads=kv, dim=dim, vdim=vdim, conv=conv)


def config(width, vocab, side, layers, eps=1e-5):
    return {"architecture": "Vavelorn", "width": width, "vocab": vocab, "token_side": {"dim": side}, "norm": {"eps": eps},
            "layers": layers}


CONFIGS = {
    # shared key heads, sizes that need padding, chunks that are no multiple of a tile, feed-forwards on some layers
    "odd": config(60, 97, 5, [delta(4, 2, 24, 20, 2, 44), attention(6, 2, 20, 12, 0.3, 300.0, 12, 8.0, 45),
                              latent(3, 12, 28, 40, 20, 0.4, 100), attention(3, 3, 14, 30, 0.2, 1e4, 6, 20.0, 7, 36),
                              latent(2, 21, 11, 17, 9, 0.3), delta(2, 1, 16, 36, 5)], eps=2e-3),
    # everything that can be 1 is 1, attention first (a side embedding of one entry over its own size is a sign: eps keeps it tame)
    "ones": config(40, 66, 1, [attention(1, 1, 8, 16, 0.5, 50.0, 2, 5.0, 1, 24), latent(1, 8, 4, 3, 1, 0.5), delta(1, 1, 8, 4, 1),
                               attention(1, 1, 16, 8, 0.4, 100.0, 16, 6.0, 10 ** 6)], eps=1e-2),
    # head sizes of real models
    "wide": config(160, 320, 32, [latent(20, 64, 96, 512, 96, 0.125, 72), delta(2, 2, 128, 128, 4, 136),
                                  attention(8, 1, 128, 64, 128 ** -0.5, 5e5, 64, 30.0, 64), delta(3, 1, 96, 160, 3),
                                  latent(4, 128, 128, 200, 144, 128 ** -0.5, 40)], eps=1e-6),
}


def build(cfg, weights, dtype, max_len=512):
    from ohara_amd.vavelorn import Vavelorn, VavelornConfig

    return Vavelorn(VavelornConfig.from_dict(cfg, max_len), weights, dtype=dtype)


def reference(cfg, weights, toks):
    return R.forward(cfg, doubled(weights), toks)


def agrees(got, want, dtype):
    """Two norms around every sublayer and one in the side embedding: more places where small values are blown up.  The CPU
    statement in fp32 lies up to 3e-5 away at single positions of these models, 2e-6 at most of them."""
    return _hybrid.agrees(got, want, dtype, f32=(1e-4, 6e-6), bf16=(0.3, 0.05))
