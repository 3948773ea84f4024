"""Small Fibirax configs with random weights for the tests (every size differs between layers; none is a multiple of
everything), and helpers to run the product and the oracle on them."""

from _hybrid import F32, doubled, row_errors
from oracle import fibirax_ref as R


def attention(heads, kv, dim, vdim, scale, window, base=300.0, dims=None, scaling=None, cap=8.0):
    rot = {"base": base, "dims": dim // 2 * 2 if dims is None else dims}
    if scaling:
        rot["scaling"] = dict(zip(("factor", "low", "high", "original"), scaling))
    return {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale, "softcap": cap, "mask": {"size": window}, "rot": rot}


def retention(decay, dim, vdim):
    return {"heads": len(decay), "dim": dim, "vdim": vdim, "decay": list(decay)}


def experts(n, top, ff, limit, identity=0, groups=None, shared=None):
    router = {"experts": n, "top": top, "identity": identity}
    if groups:
        router["groups"] = {"count": groups[0], "keep": groups[1]}
    mlp = {"kind": "moe", "router": router, "expert": {"ff": ff, "limit": limit}}
    if shared:
        mlp["shared"] = {"ff": shared[0], "limit": shared[1]}
    return mlp


def layer(left, right, mlp=None, left_scale=1.0, right_scale=1.0):
    return {"type": "parallel", "mixer": {"left": left, "right": right, "left_scale": left_scale, "right_scale": right_scale}, "mlp": mlp}


def config(width, vocab, layers, scale=0.7, eps=1e-5):
    return {"architecture": "Fibirax", "width": width, "vocab": vocab, "embedding": {"scale": scale}, "norm": {"eps": eps}, "layers": layers}


CONFIGS = {
    # shared key heads, sizes that need padding, windows that are no multiple of a tile, feed-forwards on some layers
    "odd": config(60, 97, [
        layer(attention(6, 2, 20, 12, 0.3, 45, dims=12, scaling=(4.0, 1.0, 4.0, 64)), retention((0.9, 0.99, 0.5), 12, 20),
              experts(10, 3, 36, 0.9, identity=2, groups=(4, 2), shared=(20, 1.7)), 1.3, 0.8),
        layer(attention(3, 3, 14, 30, 0.2, 7, base=1e4, dims=6, cap=20.0), retention((0.97, 1.0), 9, 7), None, 0.6, 1.1),
        layer(attention(4, 1, 11, 17, 0.25, 64, dims=10), retention((0.0, 0.999, 0.8, 0.95, 0.7), 16, 11),
              experts(7, 2, 21, 1.4, identity=1), 1.0, 0.5)], scale=0.37, eps=2e-3),
    # everything that can be 1 is 1
    "ones": config(40, 66, [
        layer(attention(1, 1, 8, 16, 0.5, 1, dims=2), retention((0.9,), 8, 8), experts(1, 1, 8, 1.0)),
        layer(attention(1, 1, 16, 8, 0.4, 10 ** 6, base=100.0, cap=5.0), retention((1.0,), 16, 8),
              experts(1, 1, 16, 0.5, identity=1, groups=(1, 1), shared=(8, 0.4))),
        layer(attention(2, 1, 2, 1, 0.7, 3), retention((0.6,), 1, 1), experts(3, 1, 1, 2.0, groups=(3, 1)), 1.5, 0.5)], scale=1.0, eps=1e-2),
    # head sizes of real models, many experts
    "wide": config(160, 320, [
        layer(attention(8, 2, 128, 64, 128 ** -0.5, 100, base=5e5, scaling=(8.0, 1.0, 4.0, 8192), cap=30.0),
              retention((0.97, 0.996), 128, 160), experts(30, 4, 72, 1.0, identity=2, groups=(4, 2), shared=(136, 2.0)), 1.2, 0.9),
        layer(attention(5, 5, 96, 128, 0.1, 65, base=5e5, dims=64, cap=15.0), retention((0.9, 0.98, 0.999), 96, 256),
              experts(66, 6, 40, 0.7, shared=(64, 0.5)), 0.8, 1.4),
        layer(attention(2, 1, 256, 200, 0.06, 130), retention((0.99, 0.93), 256, 64), None, 1.1, 0.7)], scale=0.8, eps=1e-6),
}


def build(cfg, weights, dtype, max_len=512):
    from ohara_amd.fibirax import Fibirax, FibiraxConfig

    return Fibirax(FibiraxConfig.from_dict(cfg, max_len), weights, dtype=dtype)


def reference(cfg, weights, toks):
    return R.forward(cfg, doubled(weights), toks)


def agrees(got, want, dtype):
    """Logits row by row against float64.  In bf16 a token whose best experts score alike may take another one than the oracle,
    which moves that row (and a little those that read it) by more than rounding: the bounds are on the median and on the
    share of such rows.  The 32-bit build is the sharp comparison."""
    rows = row_errors(got, want)
    if dtype == F32:
        return rows.max() < 1e-4 and (len(rows) < 8 or rows.median() < 6e-6)
    if len(rows) < 8:
        return rows.max() < 1.0
    return rows.median() < 0.08 and rows.quantile(0.8) < 0.25
