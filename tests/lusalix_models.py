"""Small Lusalix configurations for the tests, and model folders made from them (never the product's own)."""
from __future__ import annotations

import atexit
import functools
import json
import os
import shutil
import tempfile

import numpy as np

import plain_lusalix as P


def _moe(experts, top, ff, shared=None):
    return {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff},
            "shared": None if shared is None else {"ff": shared}}


def _attn(heads, kv, dim, vdim, scale, cap, temp, size, mix, mlp):
    """``cap``, ``temp`` (coef, every) and ``size`` may be None: none."""
    m = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale, "v_mix": mix}
    if cap is not None:
        m["softcap"] = cap
    if temp is not None:
        m["q_temp"] = {"coef": temp[0], "every": temp[1]}
    if size is not None:
        m["mask"] = {"size": size}
    return {"type": "attention", "mixer": m, "mlp": mlp}


def _model(vocab, width, eps, scale, layers):
    return {"architecture": "Lusalix", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": scale},
            "layers": layers}


# sizes that no tile divides (heads of 24 and 40, values of 40, a width of 96), caps that bend most scores, temperatures
# that step inside a page, a layer in between that blends nothing, one without a feed-forward, shared experts of
# another size and of the experts' size, all experts chosen
MIXED = _model(300, 96, 1e-5, 2.5, [
    _attn(4, 2, 24, 40, 0.2, 6.0, (0.4, 33), 37, True, _moe(5, 3, 40, 24)),
    _attn(3, 1, 40, 16, 0.15, 3.0, (0.25, 10), None, False, _moe(4, 1, 32, 32)),
    _attn(6, 2, 16, 40, 0.25, None, None, 64, True, None),
    _attn(2, 2, 24, 40, 0.2, 8.0, (0.6, 100), 90, True, _moe(3, 3, 24)),
])
# a layer that blends nothing first; one head; as many kv heads as heads; a window of 1 and one of exactly a page; a
# temperature that changes with every position; an embedding made smaller; one expert; experts of an odd size; the first
# blending layer without a window
REORDERED = _model(211, 80, 1e-6, 0.5, [
    _attn(1, 1, 16, 24, 0.3, 2.0, (0.2, 1), 64, False, _moe(1, 1, 24, 40)),
    _attn(2, 2, 40, 16, 0.15, 5.0, None, None, True, _moe(6, 2, 33, 33)),
    _attn(5, 1, 8, 8, 0.35, None, (0.5, 64), 1, False, None),
    _attn(4, 2, 16, 16, 0.25, 4.0, (0.3, 7), 20, True, _moe(7, 2, 16)),
])
# head sizes that the matrix cores' kernels are built for, or that are padded to one (values larger and smaller than
# the keys); widths in whole tiles; shared experts inside the experts' launches and beside them
TILED = _model(704, 128, 1e-5, 1.5, [
    _attn(4, 2, 64, 64, 0.125, 10.0, (0.3, 50), 100, True, _moe(8, 2, 64, 64)),
    _attn(6, 2, 32, 80, 0.18, 20.0, (0.2, 128), None, False, _moe(4, 1, 64, 128)),
    _attn(8, 2, 128, 64, 0.09, 30.0, (0.5, 32), 130, True, _moe(6, 3, 32, 32)),
    _attn(16, 1, 96, 32, 0.1, 5.0, None, 33, False, None),
])
# nothing optional at all
BARE = _model(150, 64, 1e-5, 1.0, [
    _attn(2, 1, 32, 32, 0.18, None, None, None, False, _moe(3, 1, 24)),
    _attn(4, 4, 16, 24, 0.25, None, None, 21, False, None),
])
CONFIGS = {"mixed": MIXED, "reordered": REORDERED, "tiled": TILED, "bare": BARE}

_root = tempfile.mkdtemp(prefix="lusalix-tests-")
atexit.register(shutil.rmtree, _root, ignore_errors=True)


def write_model(folder, cfg, W):
    import torch
    from safetensors.torch import save_file
    os.makedirs(folder, exist_ok=True)
    save_file({k: torch.tensor(v).to(torch.bfloat16).contiguous() for k, v in W.items()},
              os.path.join(folder, "model.safetensors"))
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)


@functools.lru_cache(maxsize=None)
def model(name, seed=3):
    """(folder, config dict, float32 numpy weights as the folder stores them in bfloat16)."""
    cfg = CONFIGS[name]
    W = P.make_weights(cfg, seed)
    folder = os.path.join(_root, f"{name}-{seed}")
    write_model(folder, cfg, W)
    return folder, cfg, W


@functools.lru_cache(maxsize=None)
def tokens(name, seed, n):
    """Token ids at which no router of the model makes a close call (``plain_lusalix.tokens_with_clear_choices``)."""
    _, cfg, W = model(name)
    return P.tokens_with_clear_choices(cfg, W, seed, n)


# Largest allowed difference of a row of logits (its mean taken off, root mean square over the vocabulary) as a
# fraction of the root mean square of the plain logits. float32: sums in another order. bfloat16: activations between
# the parts are rounded to 8 bits of mantissa.
TOL = {"float32": 5e-5, "bfloat16": 3e-2}
# (narrow models average a row's rounding over the fewest elements; "tiled" has scores that are steep in front of their caps:
# its rows' rounding has a median of 1.6e-2 on every path alike, eager or captured, folded or not, prompt or decoded)
LOOSER = {"reordered": 1.5, "tiled": 1.25}


def row_errors(got, ref):
    got, ref = np.asarray(got, np.float64), np.asarray(ref, np.float64)
    assert got.shape == ref.shape, (got.shape, ref.shape)
    assert np.isfinite(got).all()
    d = got - ref
    d = d - d.mean(-1, keepdims=True)
    return np.sqrt((d * d).mean(-1)) / np.sqrt(((ref - ref.mean(-1, keepdims=True)) ** 2).mean())


def rounding(cfg, W, toks, ref):
    """Per row of the plain logits ``ref`` the error that rounding the activations to 16 bits makes by itself, at least
    that of all but a tenth of the model's rows."""
    e = row_errors(P.Sequence(cfg, W, r=P.to_16_bits).feed(toks), ref)
    return np.maximum(e, np.quantile(e, 0.9))


def close(got, ref, dtype, what="", alone=None):
    """float32: every row within the bound. bfloat16: rounding has a tail, so one row in twenty-five may lie over the
    bound, and none over two and a half times it; a wrong key, blend or expert moves a row by tens of times the bound.
    ``alone`` (models drawn from seeds, some of which amplify rounding far more than others): each row's error by
    rounding alone, three times which is then a row's bound in bfloat16."""
    e = row_errors(got, ref)
    tol = TOL[dtype] * (LOOSER.get(what.split()[0] if what else "", 1.0) if dtype == "bfloat16" else 1.0)
    if alone is not None and dtype == "bfloat16":
        tol = 3.0 * alone
    bad = np.flatnonzero(e > tol)
    allowed = 0 if dtype == "float32" else max(2, len(e) // 25)
    worst = np.flatnonzero(e > (tol if dtype == "float32" else 2.5 * tol))
    assert len(bad) <= allowed and not len(worst), \
        f"{what}: row {int(bad[0])} is the first of {len(bad)} over {np.max(tol):.1e}: {e[bad[0]]:.3e}; the worst has {e.max():.3e}"
    return float(e.max())


def near(got, ref, dtype, what=""):
    """Elements of residual rows against the plain ones, on the scale of the largest: float32 2e-5, bfloat16 2e-2 with
    one element in fifty up to five times that."""
    got, ref = np.asarray(got, np.float64), np.asarray(ref, np.float64)
    assert got.shape == ref.shape and np.isfinite(got).all(), what
    d = np.abs(got - ref) / max(np.abs(ref).max(), 1e-3)
    if dtype == "float32":
        assert d.max() < 2e-5, f"{what}: {d.max():.3e}"
    else:
        assert (d > 2e-2).mean() <= 2e-2 and d.max() < 0.1, f"{what}: {(d > 2e-2).mean():.2e} of the elements over, the worst {d.max():.3e}"
