"""Small Povazen configs with random weights for the tests (every size differs between layers; none is a multiple of
everything), and helpers to run the product and the oracle on them."""

from _hybrid import doubled, error, row_errors, tokens  # noqa: F401
from oracle import povazen_ref as R


def attention(heads, kv, dim, vdim, scale, ff=0):
    return {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def delta(heads, kv, dim, vdim, conv, ff=0):
    return {"type": "channel_delta", "mixer": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "conv": conv},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def config(width, vocab, taps, groups, cap, layers, eps=1e-5):
    c = {"architecture": "Povazen", "width": width, "vocab": vocab, "canon": {"taps": taps},
         "norm": {"eps": eps, "groups": groups}, "layers": layers}
    if cap is not None:
        c["logit_softcap"] = cap
    return c


CONFIGS = {
    # shared key heads, sizes that need padding, feed-forwards on either kind of layer
    "odd": config(60, 97, 4, 3, 12.0, [delta(4, 2, 24, 20, 2, 44), attention(6, 2, 20, 12, 0.3),
                                       delta(2, 1, 16, 36, 5), attention(3, 3, 12, 28, 0.2, 100)]),
    # everything that can be 1 is 1, attention first, no cap
    "ones": config(40, 66, 1, 1, None, [attention(1, 1, 8, 16, 0.5, 24), delta(1, 1, 8, 4, 1)]),
    # head sizes of real models
    "wide": config(160, 320, 2, 5, 20.0, [delta(2, 2, 128, 128, 4, 72), attention(4, 1, 128, 64, 128 ** -0.5, 136),
                                          delta(3, 1, 96, 160, 3), attention(8, 1, 64, 128, 0.1)], eps=1e-6),
}


def build(cfg, weights, dtype, max_len=512):
    from ohara_amd.povazen import Povazen, PovazenConfig

    return Povazen(PovazenConfig.from_dict(cfg, max_len), weights, dtype=dtype)


def reference(cfg, weights, toks):
    return R.forward(cfg, doubled(weights), toks)
