"""Small Banazen configurations for the tests, and model folders made from them (never the product's own)."""
from __future__ import annotations

import atexit
import functools
import os
import shutil
import tempfile

import numpy as np

import plain_banazen as P
from lusalix_models import near, row_errors, write_model  # noqa: F401  (the same measures of a difference)


def moe(experts, top, ff, limit, scale=1.0, groups=None, shared=None):
    """``groups``: (count, keep) or None; ``shared``: (ff, limit) or None."""
    return {"kind": "moe", "router": {"experts": experts, "top": top, "scale": scale,
                                      "groups": None if groups is None else {"count": groups[0], "keep": groups[1]}},
            "expert": {"ff": ff, "limit": limit}, "shared": None if shared is None else {"ff": shared[0], "limit": shared[1]}}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def latent(heads, dim, vdim, rank, scale, size, mlp, kv_from=None):
    m = {"heads": heads, "dim": dim, "vdim": vdim, "kv_rank": rank, "scale": scale}
    if size is not None:
        m["mask"] = {"size": size}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m, "mlp": mlp}


def sides(left, right, mlp):
    """``left``: (heads, kv_heads, dim, vdim, conv, (base, dims) or None, scale); ``right``: (heads, kv_heads, dim, vdim, conv)."""
    H, G, D, Dv, taps, rot, scale = left
    a = {"heads": H, "kv_heads": G, "dim": D, "vdim": Dv, "conv": taps, "scale": scale}
    if rot is not None:
        a["rot"] = {"base": rot[0], "dims": rot[1]}
    b = dict(zip(("heads", "kv_heads", "dim", "vdim", "conv"), right))
    return {"type": "parallel", "mixer": {"left": a, "right": b}, "mlp": mlp}


def decoder(vocab, width, eps, embed, logit, side, layers):
    d = {"architecture": "Banazen", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": embed},
         "logit_scale": logit, "layers": layers}
    if side:
        d["token_side"] = {"dim": side}
    return d


# sizes that no tile divides; a reader whose window is wider than its source's, one that reads a source without a window, and
# one whose heads differ from the source's; more heads than kv heads on both sides; a rotation of a part of the head; a
# convolution of one tap; layers without a feed-forward; shared experts of the experts' form and of another
MIXED = decoder(300, 96, 1e-5, 2.5, 0.7, 10, [
    latent(3, 24, 40, 40, 0.2, 37, moe(6, 2, 40, 0.7, 2.5, (3, 2), (24, 1.3))),
    sides((4, 2, 24, 40, 4, (900.0, 12), 0.25), (4, 2, 24, 40, 2), dense(72)),
    latent(2, 16, 24, 40, 0.3, 64, None, kv_from=0),
    latent(4, 20, 12, 24, 0.25, None, moe(4, 1, 24, 2.0, 0.5, (2, 1), (24, 2.0))),
    latent(5, 8, 16, 24, 0.35, 21, moe(3, 3, 33, 1.0), kv_from=3),
    sides((6, 1, 40, 24, 1, None, 0.2), (3, 3, 20, 12, 5), None),
])
# no side table; one head; windows of 1, of 2 and of exactly a page; long convolutions; values larger than keys; one expert; as
# many groups as experts
REORDERED = decoder(211, 80, 1e-6, 0.5, 3.0, 0, [
    sides((1, 1, 16, 24, 7, (50.0, 16), 0.3), (6, 2, 8, 40, 3), moe(8, 3, 24, 0.4, 1.5, (8, 5))),
    latent(1, 32, 16, 48, 0.2, 64, moe(1, 1, 16, 1.0, 2.0, None, (40, 0.5))),
    latent(2, 8, 8, 48, 0.4, 1, dense(40), kv_from=1),
    latent(4, 12, 32, 16, 0.3, 2, None),
    sides((3, 3, 34, 10, 2, (10000.0, 6), 0.25), (1, 1, 40, 16, 8), moe(9, 4, 40, 3.0, 1.0, (3, 2), (40, 3.0))),
    latent(4, 12, 32, 48, 0.3, 100, dense(56), kv_from=1),
])
# head sizes, latents and widths that the matrix-core kernels are built for
TILED = decoder(704, 128, 1e-5, 1.5, 1.0, 32, [
    sides((4, 2, 64, 64, 4, (5000.0, 64), 0.15), (4, 4, 64, 64, 4), moe(8, 2, 64, 2.0, 2.0, (4, 2), (64, 2.0))),
    latent(8, 32, 64, 96, 0.2, 100, moe(16, 4, 32, 1.5, 1.0, (4, 3), (64, 1.0))),
    latent(4, 64, 32, 96, 0.15, 130, dense(192), kv_from=1),
    sides((8, 2, 32, 80, 3, (300.0, 16), 0.3), (4, 2, 128, 32, 3), dense(128)),
    latent(16, 16, 32, 128, 0.25, None, moe(8, 2, 64, 2.0, 1.0, None, None)),
])
BARE = decoder(150, 64, 1e-5, 1.0, 1.0, 0, [
    latent(2, 16, 16, 32, 0.25, None, dense(48)),
    sides((2, 1, 16, 16, 2, None, 0.25), (2, 1, 16, 16, 2), dense(32)),
])
CONFIGS = {"mixed": MIXED, "reordered": REORDERED, "tiled": TILED, "bare": BARE}


def ranks(i):
    """The inner sizes of layer i's two-step projections (of the decay, of the gate): the stored shapes alone say them."""
    return (8 + 5 * i, 40 - 6 * i)


_root = tempfile.mkdtemp(prefix="banazen-tests-")
atexit.register(shutil.rmtree, _root, ignore_errors=True)


@functools.lru_cache(maxsize=None)
def model(name, seed=3):
    """(folder, config dict, float32 numpy weights as the folder stores them in bfloat16)."""
    cfg = CONFIGS[name]
    W = P.make_weights(cfg, seed, ranks)
    folder = os.path.join(_root, f"{name}-{seed}")
    write_model(folder, cfg, W)
    return folder, cfg, W


@functools.lru_cache(maxsize=None)
def tokens(name, seed, n):
    """Token ids at which no router of the model makes a close call (``plain_banazen.tokens_with_clear_choices``)."""
    _, cfg, W = model(name)
    return P.tokens_with_clear_choices(cfg, W, seed, n)


def rounding(cfg, W, toks, ref):
    """Per row of the plain logits ``ref`` the error that rounding the activations to 16 bits makes by itself, at least
    that of all but a tenth of the model's rows."""
    e = row_errors(P.Sequence(cfg, W, r=P.to_16_bits).feed(toks), ref)
    return np.maximum(e, np.quantile(e, 0.9))


# Largest allowed difference of a row of logits (its mean taken off, root mean square over the vocabulary) as a
# fraction of the root mean square of the plain logits. float32: sums in another order. bfloat16: activations between
# the parts are rounded to 8 bits of mantissa; a wrong key, state or expert moves a row by tens of times the bound.
TOL = {"float32": 5e-5, "bfloat16": 3e-2}


def close(got, ref, dtype, what="", alone=None):
    """float32: every row within the bound. bfloat16: rounding has a tail, so one row in twenty-five may lie over the
    bound, and none over two and a half times it. ``alone``: each row's error by rounding alone, three times which is then
    a row's bound in bfloat16."""
    e = row_errors(got, ref)
    tol = TOL[dtype] if alone is None or dtype == "float32" else 3.0 * alone
    bad = np.flatnonzero(e > tol)
    allowed = 0 if dtype == "float32" else max(2, len(e) // 25)
    worst = np.flatnonzero(e > (tol if dtype == "float32" else 2.5 * tol))
    assert len(bad) <= allowed and not len(worst), \
        f"{what}: row {int(bad[0])} is the first of {len(bad)} over {np.max(tol):.1e}: {e[bad[0]]:.3e}; the worst has {e.max():.3e}"
    return float(e.max())
