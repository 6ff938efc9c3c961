"""The Lusalix decoder on the GPU against the plain implementation (``plain_lusalix.py``): each mechanism's kernels
alone, with inputs made so that a fault shows, then whole models through the engine's step function, its cache, its
batching and its generation loop."""
import numpy as np
import pytest
import torch

import plain_lusalix as P
from cache_order import tile_keys, tile_values, untile_keys, untile_values
from lusalix_models import CONFIGS, close, model, near, row_errors, tokens

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
DTYPES = ["float32", "bfloat16"]
TD = {"float32": torch.float32, "bfloat16": torch.bfloat16}


def dev(a, dtype=torch.float32):
    return torch.as_tensor(np.ascontiguousarray(a)).to(dtype).to(DEV)


def i32(a):
    return torch.as_tensor(np.asarray(a, np.int32)).to(DEV)


def host(t):
    return t.float().cpu().numpy().astype(np.float64)


def bf16_exact(a):
    return torch.tensor(np.asarray(a), dtype=torch.float32).to(torch.bfloat16).float().numpy()


def engine(name, dtype, **kw):
    from gpullama3_java_amd.engine import Engine
    folder, cfg, W = model(name)
    kw.setdefault("max_tokens", 2048)
    kw.setdefault("n_slots", 6)
    return Engine.from_folder(folder, dtype=dtype, **kw), cfg, W


# ----------------------------------------------------------------- attention: cap, temperature, distances, window, gate
def paged(k, v, page, dtype):
    """One sequence's keys [S, G, D] and values [S, G, Dv] as a paged cache in the kernels' order; its pages lie in
    another order than its positions. Returns (k_cache, v_cache, block table [1, pages])."""
    S, G, D = k.shape
    n = -(-S // page)
    table = 1 + (np.arange(n) * 3 + 1) % n if n % 3 else 1 + np.arange(n)[::-1]
    kc, vc = np.zeros((n + 1, G, page, D), np.float32), np.zeros((n + 1, G, v.shape[2], page), np.float32)
    for j in range(S):
        kc[table[j // page], :, j % page] = k[j]
        vc[table[j // page], :, :, j % page] = v[j]
    return dev(tile_keys(kc), TD[dtype]), dev(tile_values(vc), TD[dtype]), i32(table[None])


def plain_attention(q, k, v, positions, m, z):
    """q [T, H, D] without the temperature, k [S, G, D], v [S, G, Dv], z [T, H, Dv] the gate in front of its sigmoid."""
    H, G = m["heads"], m["kv_heads"]
    if m.get("q_temp"):
        q = q * P.temperature(positions, m["q_temp"]["coef"], m["q_temp"]["every"])[:, None, None]
    out = np.zeros((len(positions), H, v.shape[2]))
    for t, p in enumerate(positions):
        lo = P.visible(p, (m.get("mask") or {}).get("size"))
        j = np.arange(lo, p + 1)
        for h in range(H):
            g = h // (H // G)
            s = P.score(q[t, h].astype(np.float64), k[lo:p + 1, g].astype(np.float64), p, j, m, h)
            e = np.exp(s - s.max())
            out[t, h] = (e / e.sum()) @ v[lo:p + 1, g]
    return out if z is None else out * P.sigmoid(z)


def marked(rng, S, G, D, Dv, at, by):
    """Keys and values of which key ``at`` stands out: every query finds it if it may see it."""
    k, v = bf16_exact(rng.standard_normal((S, G, D)) * 0.3), bf16_exact(rng.standard_normal((S, G, Dv)))
    k[at] = bf16_exact(by * np.ones((G, D)) / np.sqrt(D))
    v[at] = 7.0
    return k, v


RULES = {"all": (20.0, (0.3, 50), True), "cap": (3.0, None, False), "temperature": (None, (0.7, 64), False),
         "gate": (None, None, True), "each position": (9.0, (0.15, 1), True)}


def attention_case(H, G, D, Dv, window, rule, decode=True):
    """Inputs around a marked key: positions at both its window's edges, at the temperature's steps, at page borders."""
    cap, temp, gate = RULES[rule]
    m = {"heads": H, "kv_heads": G, "scale": 0.5, "softcap": cap, "mask": {"size": window} if window else None,
         "q_temp": {"coef": temp[0], "every": temp[1]} if temp else None}
    rng = np.random.default_rng([H, D, Dv])
    S, at = 330, 150
    k, v = marked(rng, S, G, D, Dv, at, 26.0)
    w = window or 10 ** 6
    if decode:
        positions = [0, 1, 48, 49, 50, 63, 64, 98, 99, at - 1, at, at + 1, at + w - 2, at + w - 1, at + w, at + w + 1, 255, 256, S - 1]
        positions = [p for p in positions if p < S]
    else:
        first = max(0, at + w - 40) if window is not None and at + w + 20 < S else at - 30       # a portion that passes the edge
        positions = list(range(first, min(S, first + 90)))
    T = len(positions)
    q = bf16_exact(rng.standard_normal((T, H, D)) * 0.3 + 1.0 / np.sqrt(D))
    z = bf16_exact(rng.standard_normal((T, H, Dv)) * 2) if gate else None
    ref = plain_attention(q, k, v, positions, m, z)
    bare = plain_attention(q, k, v, positions, m, None)
    if decode and window is not None and at + w < S:           # the last head has the smallest slope: it shows the key
        seen, gone = bare[positions.index(at + w - 1), H - 1], bare[positions.index(at + w), H - 1]
        assert abs(seen).max() > (1.0 if cap == 3.0 else 2.0) * abs(gone).max() or cap == 3.0
    return m, k, v, positions, q, z, ref


def rule_of(K, m, z, dtype):
    t = m["q_temp"]
    gate = None
    if z is not None:       # (the gate's columns stand behind others in wider rows, as the stacked product leaves them)
        T, n = z.shape[0], z.shape[1] * z.shape[2]
        wide = torch.zeros(T, n + 16, dtype=TD[dtype], device=DEV)
        wide[:, 8:8 + n] = dev(z.reshape(T, -1), TD[dtype])
        gate = wide[:, 8:8 + n]
    return K.ScoreRule(m["softcap"], (t["coef"], t["every"]) if t else None, gate)


@pytest.mark.parametrize("rule", sorted(RULES))
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H, G, D, Dv, window", [(4, 2, 32, 48, 37), (3, 3, 16, 16, 64), (2, 1, 48, 32, 9), (4, 2, 64, 80, 100),
                                                 (4, 1, 80, 64, None), (2, 2, 160, 208, 1)])
def test_score_rules_in_the_kernel_for_any_sizes(H, G, D, Dv, window, dtype, rule):
    from gpullama3_java_amd.csrc import lib as K
    m, k, v, positions, q, z, ref = attention_case(H, G, D, Dv, window, rule)
    T = len(positions)
    kc, vc, table = paged(k, v, 64, dtype)
    out = torch.zeros(T, H * Dv, dtype=TD[dtype], device=DEV)
    K.attention_generic(dev(q.reshape(T, H * D), TD[dtype]), kc, vc, i32(positions), i32([0] * T), table, out, H, G, D, 64,
                        window, 0.5, v_head_dim=Dv, slopes=dev(P.slopes(H)), rule=rule_of(K, m, z, dtype))
    np.testing.assert_allclose(host(out).reshape(T, H, Dv), ref, atol=3e-5 if dtype == "float32" else 0.03)


@pytest.mark.parametrize("rule", sorted(RULES))
@pytest.mark.parametrize("kernel", [("decode", 1), ("decode", 3), ("prompt", 1), ("prompt", 10 ** 6)])
@pytest.mark.parametrize("H, G, D, window", [(8, 1, 64, 37), (4, 2, 32, 64), (2, 2, 96, 9), (3, 1, 128, 100), (4, 4, 64, None), (20, 1, 32, 33)])
def test_score_rules_on_the_matrix_cores(H, G, D, window, kernel, rule):
    from gpullama3_java_amd.csrc import lib as K
    m, k, v, positions, q, z, ref = attention_case(H, G, D, D, window, rule, decode=kernel[0] == "decode")
    T = len(positions)
    kc, vc, table = paged(k, v, 64, "bfloat16")
    qd, out = dev(q.reshape(T, H * D), torch.bfloat16), torch.zeros(T, H * D, dtype=torch.bfloat16, device=DEV)
    extras = dict(slopes=dev(P.slopes(H)), rule=rule_of(K, m, z, "bfloat16"))
    if kernel[0] == "decode":
        n = kernel[1]
        part_o = torch.zeros((T, H, n, D), dtype=torch.float32, device=DEV) if n > 1 else None
        part_ml = torch.zeros((T, H, n, 2), dtype=torch.float32, device=DEV) if n > 1 else None
        K.attention_decode(qd, kc, vc, i32(positions), i32([0] * T), table, out, H, G, D, 64, window, 0.5, n, part_o, part_ml, **extras)
    else:
        K.attention_prefill(qd, kc, vc, i32([0, T]), i32([positions[0]]), table, out, T, H, G, D, 64, window, 0.5,
                            wide_from=kernel[1], **extras)
    np.testing.assert_allclose(host(out).reshape(T, H, D), ref, atol=0.05)


def test_a_cap_far_away_changes_nothing_and_a_rule_needs_its_numbers():
    """A cap a million times the scores gives the plain scores (to the rounding of numbers near one times the cap in the
    kernel for any sizes, whose tanh is exact); senseless rules are refused on the host."""
    from gpullama3_java_amd.csrc import lib as K
    m, k, v, positions, q, _, _ = attention_case(4, 2, 32, 32, 37, "cap")
    ref = plain_attention(q, k, v, positions, dict(m, softcap=None), None)
    T = len(positions)
    kc, vc, table = paged(k, v, 64, "float32")
    out = torch.zeros(T, 4 * 32, device=DEV)
    args = (dev(q.reshape(T, -1)), kc, vc, i32(positions), i32([0] * T), table, out, 4, 2, 32, 64, 37, 0.5)
    K.attention_generic(*args, slopes=dev(P.slopes(4)), rule=K.ScoreRule(softcap=1e6))
    np.testing.assert_allclose(host(out).reshape(T, 4, 32), ref, atol=5e-5)
    for bad in (K.ScoreRule(softcap=0.0), K.ScoreRule(softcap=-2.0), K.ScoreRule(temperature=(0.1, 0)),
                K.ScoreRule(gate=torch.zeros(T, 64, device=DEV)), K.ScoreRule(gate=torch.zeros(T, 128, dtype=torch.bfloat16, device=DEV))):
        with pytest.raises(K.KernelError):
            K.attention_generic(*args, rule=bad)


# ----------------------------------------------------------------- keys and blended values into the cache
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("G, D, Dv, first_dim, off", [(2, 32, 48, 48, 8), (3, 16, 32, 16, 0), (1, 64, 64, 80, 16), (2, 48, 16, 16, 3)])
def test_values_blended_on_their_way_into_the_cache(G, D, Dv, first_dim, off, dtype):
    """Two sequences' tokens in one step (one from its start, one from inside a group of eight positions across a page
    border), other values with smaller and larger heads, columns at odd places (the kernel without 16-byte units)."""
    from gpullama3_java_amd.csrc import lib as K
    rng = np.random.default_rng([G, D, Dv])
    page = 32
    starts, lens = [0, 27], [19, 30]
    T = sum(lens)
    positions = np.concatenate([np.arange(s, s + n) for s, n in zip(starts, lens)])
    seqs = np.repeat([0, 1], lens)
    table = np.array([[3, 1], [2, 4]])
    rows = bf16_exact(rng.standard_normal((T, off + G * (D + Dv) + 8)))
    other = bf16_exact(rng.standard_normal((T, G * first_dim + 8)))
    k, v = rows[:, off:off + G * D].reshape(T, G, D), rows[:, off + G * D:off + G * (D + Dv)].reshape(T, G, Dv)
    f = np.zeros((T, G, Dv))
    n = min(first_dim, Dv)
    f[..., :n] = other[:, 8:].reshape(T, G, first_dim)[..., :n]
    for blend in (None, 0.3, 1.0):
        kc, vc = torch.zeros(5, G, page, D, dtype=TD[dtype], device=DEV), torch.zeros(5, G, Dv, page, dtype=TD[dtype], device=DEV)
        K.kv_write(dev(rows, TD[dtype]), off, off + G * D, i32(positions), i32(seqs), i32(table), kc, vc, G, D, Dv, page,
                   blend=None if blend is None else (dev(other, TD[dtype])[:, 8:], first_dim, blend))
        gk, gv = untile_keys(host(kc)), untile_values(host(vc))
        ref = v if blend is None else P.blend(v.astype(np.float64), f, blend)
        used = np.zeros((5, page), bool)
        for t in range(T):
            pg, at = table[seqs[t], positions[t] // page], positions[t] % page
            used[pg, at] = True
            np.testing.assert_array_equal(gk[pg, :, at], k[t])
            np.testing.assert_allclose(gv[pg, :, :, at], ref[t], atol=2e-6 if dtype == "float32" else 0.02)
        assert not gk.transpose(0, 2, 1, 3)[~used].any() and not gv.transpose(0, 3, 1, 2)[~used].any()


# ----------------------------------------------------------------- the mixture of experts
def routed(K, logits, top, E, always, gate_col=None, norm=None, apart=False):
    T, more = logits.shape[0], 1 if always else 0
    per = top + more
    o = dict(idx=torch.zeros(T, per, dtype=torch.int32, device=DEV), wts=torch.zeros(T, per, device=DEV),
             offsets=torch.zeros(E + more + 1, dtype=torch.int32, device=DEV), pairs=torch.zeros(T * per, dtype=torch.int32, device=DEV),
             in_wts=torch.zeros(T, per, device=DEV))
    if apart:
        o.update(gate_out=torch.zeros(T, device=DEV))
        if norm is not None:
            o.update(norm_out=torch.zeros(T, device=DEV))
    K.route(dev(logits), top, always=always, scores="sigmoid", n_experts=E, gate_col=gate_col, norm=norm, **o)
    return o


@pytest.mark.parametrize("T", [1, 9, 64, 65, 200])
@pytest.mark.parametrize("always", [False, True])
def test_router_sigmoids_on_the_experts_inputs(T, always):
    """The largest logits choose, ties go to the lower number; a weight is the sigmoid as it is and goes to the pair's
    input; the shared expert's factor comes from a column behind the experts', which is never chosen."""
    from gpullama3_java_amd.csrc import lib as K
    rng = np.random.default_rng([T, 4])
    E = 7
    logits = rng.standard_normal((T, 16)).astype(np.float32) * 2
    logits[:, E:] += 50.0                                # nothing behind the experts is a choice
    logits[:, E] = rng.standard_normal(T)                # (the shared expert's)
    logits[0, :E] = 1.0
    for top in (1, 2, 7):
        o = routed(K, logits, top, E, always, gate_col=E, apart=not always)
        idx, wts, in_wts = o["idx"].cpu().numpy(), host(o["wts"]), host(o["in_wts"])
        offsets, pairs = o["offsets"].cpu().numpy(), o["pairs"].cpu().numpy()
        z = logits.astype(np.float64)
        for t in range(T):
            order = np.argsort(-z[t, :E], kind="stable")[:top]
            assert list(idx[t, :top]) == list(order), (top, t)
            np.testing.assert_allclose(in_wts[t, :top], P.sigmoid(z[t, order]), atol=1e-6)
            assert (wts[t, :top] == 1.0).all()
            if always:
                assert idx[t, top] == E and in_wts[t, top] == 1.0
                np.testing.assert_allclose(wts[t, top], P.sigmoid(z[t, E]), atol=1e-6)
        if not always:
            np.testing.assert_allclose(host(o["gate_out"]), P.sigmoid(z[:, E]), atol=1e-6)
        per = top + (1 if always else 0)
        assert offsets[0] == 0 and offsets[-1] == T * per and sorted(pairs) == list(range(T * per))
        for e in range(E + (1 if always else 0)):
            assert all(idx.reshape(-1)[p] == e for p in pairs[offsets[e]:offsets[e + 1]])


@pytest.mark.parametrize("T, parts, d", [(1, 1, 96), (5, 17, 136), (16, 256, 2048), (64, 70, 560)])
def test_router_carries_the_norm_in_front(T, parts, d):
    from gpullama3_java_amd.csrc import lib as K
    rng = np.random.default_rng([T, parts])
    E, top, eps = 5, 2, 0.3
    logits = rng.standard_normal((T, E + 1)).astype(np.float32)
    ssq = np.zeros((parts, 64), np.float32)
    ssq[:, :T] = rng.uniform(0.1, 4.0, (parts, T))
    inv = 1.0 / np.sqrt(ssq[:, :T].astype(np.float64).sum(0) / d + eps)
    for always in (False, True):
        o = routed(K, logits, top, E, always, gate_col=E, norm=(dev(ssq), parts, d, eps), apart=not always)
        in_wts, idx = host(o["in_wts"]), o["idx"].cpu().numpy()
        s = P.sigmoid(np.take_along_axis(logits.astype(np.float64), idx[:, :top], 1))
        np.testing.assert_allclose(in_wts[:, :top], s * inv[:, None], rtol=1e-5)
        if always:
            np.testing.assert_allclose(in_wts[:, top], inv, rtol=1e-5)
        else:
            np.testing.assert_allclose(host(o["norm_out"]), inv, rtol=1e-5)


@pytest.mark.parametrize("dtype, mfma", [("float32", False), ("bfloat16", False), ("bfloat16", True)])
@pytest.mark.parametrize("E, top, T, d, F", [(5, 3, 90, 96, 40), (3, 1, 7, 64, 72), (11, 2, 300, 128, 88), (1, 1, 1, 80, 48),
                                             (4, 2, 700, 200, 136), (8, 2, 8, 1024, 520), (2, 2, 64, 320, 24), (4, 2, 100, 190, 64)])
def test_experts_weighted_on_their_inputs(E, top, T, d, F, dtype, mfma):
    """Every kernel of the grouped product (by run length): ``expert(w h)`` with factors from a hundredth to ten, and a
    single expert over all rows whose OUTPUT has a factor, beside one on its input."""
    from gpullama3_java_amd.csrc import lib as K
    rng = np.random.default_rng([E, T, d])
    h = bf16_exact(rng.standard_normal((T, d)))
    gate, up = (bf16_exact(rng.standard_normal((E, F, d)) * 1.5 / np.sqrt(d)) for _ in range(2))
    down = bf16_exact(rng.standard_normal((E, d, F)) / np.sqrt(F))
    turns = np.stack([gate, up], axis=2).reshape(E, 2 * F, d)
    logits = rng.standard_normal((T, E)).astype(np.float32)
    o = routed(K, logits, top, E, False)
    choice = o["idx"].cpu().numpy()
    w = (10.0 ** rng.uniform(-2, 0.5, (T, top))).astype(np.float32)
    hd, wd = dev(h, TD[dtype]), dev(w)
    hidden = torch.zeros(T * top, F, dtype=TD[dtype], device=DEV)
    K.expert_gemm(hd, dev(turns, TD[dtype]), hidden, gated=("silu", None, 0.0), offsets=o["offsets"], pairs=o["pairs"], a_div=top,
                  mfma=mfma, row_in=wd.view(-1))
    outs = torch.zeros(T * top, d, device=DEV)
    K.expert_gemm(hidden, dev(down, TD[dtype]), outs, offsets=o["offsets"], pairs=o["pairs"], mfma=mfma)
    y = torch.full((T, d), 2.0, device=DEV)
    K.route_combine(outs, torch.ones(T, top, device=DEV), y, accumulate=True)

    def plain_hidden(e, row):
        return P.silu(gate[e] @ row) * (up[e] @ row)

    got_hidden, ref_y = host(hidden), np.full((T, d), 2.0)
    for t in range(T):
        for j in range(top):
            e, p = choice[t, j], t * top + j
            ref = plain_hidden(e, w[t, j].astype(np.float64) * h[t])
            np.testing.assert_allclose(got_hidden[p], ref, atol=3e-5 * max(1, np.abs(ref).max()) if dtype == "float32" else 0.01, rtol=1e-5 if dtype == "float32" else 8e-3)
            ref_y[t] += down[e] @ got_hidden[p]
    np.testing.assert_allclose(host(y), ref_y, atol=(3e-5 if dtype == "float32" else 1e-3) * np.abs(ref_y).max())
    # one expert over every row in its own order, factors on input and output
    f_in, f_out = dev(rng.uniform(0.2, 2.0, T)), dev(rng.uniform(0.1, 1.0, T))
    dense = torch.zeros(T, F, dtype=TD[dtype], device=DEV)
    K.expert_gemm(hd, dev(turns[:1], TD[dtype]), dense, gated=("silu", None, 0.0), mfma=mfma, row_in=f_in, row_out=f_out)
    ref = np.stack([a * plain_hidden(0, b * h[t]) for t, (b, a) in enumerate(zip(host(f_in), host(f_out)))])
    np.testing.assert_allclose(host(dense), ref, atol=3e-5 * np.abs(ref).max() if dtype == "float32" else 0.01, rtol=1e-5 if dtype == "float32" else 8e-3)
    # an expert without a gate takes the factors the same way
    K.expert_gemm(hd, dev(gate[:1], TD[dtype]), dense, act="gelu_tanh", mfma=mfma, row_in=f_in, row_out=f_out)
    u = (h @ gate[0].T) * host(f_in)[:, None]
    ref = 0.5 * u * (1 + np.tanh(np.sqrt(2 / np.pi) * (u + 0.044715 * u ** 3))) * host(f_out)[:, None]
    np.testing.assert_allclose(host(dense), ref, atol=3e-5 * np.abs(ref).max() if dtype == "float32" else 0.01, rtol=1e-5 if dtype == "float32" else 8e-3)


@pytest.mark.parametrize("T, top, d", [(1, 1, 64), (7, 3, 96), (16, 9, 2048), (64, 2, 1500)])
def test_weighted_sum_that_leaves_what_a_folded_norm_reads(T, top, d):
    from gpullama3_java_amd.csrc import lib as K
    rng = np.random.default_rng([T, d])
    y, w = rng.standard_normal((T * top, d)).astype(np.float32), rng.uniform(0, 1, (T, top)).astype(np.float32)
    x0, g = rng.standard_normal((T, d)).astype(np.float32) * 3, (1 + 0.2 * rng.standard_normal(d)).astype(np.float32)
    x, x2 = dev(x0), dev(x0)
    ssq, xg = torch.zeros(1, 64, device=DEV), torch.zeros(T, d, dtype=torch.bfloat16, device=DEV)
    K.route_combine(dev(y), dev(w), x, accumulate=True, ssq=ssq, next_weight=dev(g), xg=xg)
    K.route_combine(dev(y), dev(w), x2, accumulate=True)
    assert torch.equal(x, x2)
    ref = x0 + np.einsum("tj,tjd->td", w.astype(np.float64), y.reshape(T, top, d))
    np.testing.assert_allclose(host(x), ref, atol=2e-5)
    np.testing.assert_allclose(host(ssq)[0, :T], (ref * ref).sum(-1), rtol=1e-5)
    np.testing.assert_allclose(host(xg), ref * g, rtol=6e-3, atol=1e-3)


# ----------------------------------------------------------------- whole models through the engine
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_whole_prompt_and_every_layer(name, dtype):
    eng, cfg, W = engine(name, dtype)
    toks = tokens(name, 1, 210)                       # beyond every window, over four pages
    seq = P.Sequence(cfg, W)
    ref = seq.feed(toks)
    seen = []
    eng.after_block = lambda i, x: seen.append(x.float().cpu().numpy())
    s = eng.take_slot()
    got = eng.step([(s, toks)], want="all").cpu().numpy()
    eng.after_block = None
    assert len(seen) == len(seq.rows[0]) == len(cfg["layers"])
    for r, (a, b) in enumerate(zip(seen, seq.rows[0])):     # the first layer that differs names the mechanism
        near(a, b, dtype, f"layer {r}")
    close(got, ref, dtype, name)
    # the first tokens of a sequence, each alone from an empty slot
    for n in (1, 2, 3):
        s2 = eng.take_slot()
        close(eng.step([(s2, toks[:n])], want="all").cpu().numpy(), ref[:n], dtype, f"{name} first {n}")
        eng.give_back_slot(s2)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_prompt_then_token_by_token(name, dtype):
    """Decoding passes every window's edge, every temperature's steps and two page borders; the decoded rows are those
    of the whole prompt."""
    eng, cfg, W = engine(name, dtype)
    toks = tokens(name, 2, 200)
    ref = P.forward(cfg, W, toks)
    s = eng.take_slot()
    rows = [eng.step([(s, toks[:3])], want="all").cpu().numpy()]
    for t in toks[3:]:
        rows.append(eng.step([(s, [t])]).cpu().numpy())
    close(np.concatenate(rows), ref, dtype, name)
    assert eng.cache.length(s) == 200


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name, cuts", [("mixed", [2, 4, 7, 31, 33, 36, 38, 64, 66, 89, 91, 128, 129, 131, 190]),
                                        ("reordered", [1, 3, 5, 7, 19, 21, 63, 65, 67, 100, 102, 190]),
                                        ("bare", [19, 21, 23, 64, 190]),
                                        ("tiled", [17, 49, 51, 99, 101, 130, 131, 133, 190])])
def test_portions_of_a_prompt(name, cuts, dtype):
    eng, cfg, W = engine(name, dtype)
    toks = tokens(name, 3, 190)
    ref = P.forward(cfg, W, toks)
    s = eng.take_slot()
    rows, lo = [], 0
    for hi in cuts:
        rows.append(eng.step([(s, toks[lo:hi])], want="all").cpu().numpy())
        lo = hi
    close(np.concatenate(rows), ref, dtype, name)
    if dtype == "float32":
        # nothing but rounding hangs on the cut: against the same prompt in one step
        s2 = eng.take_slot()
        whole = eng.step([(s2, toks)], want="all").cpu().numpy()
        assert row_errors(np.concatenate(rows), whole).max() < 1e-5


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_unequal_requests_in_one_batch_and_slots_used_again(name, dtype):
    eng, cfg, W = engine(name, dtype, n_slots=4, max_tokens=1024)
    lens = [1, 70, 131, 9]
    prompts = [tokens(name, 10 + i, n + 12) for i, n in enumerate(lens)]
    refs = [P.forward(cfg, W, p) for p in prompts]
    for time in range(2):                             # the second time takes the slots and pages that the first gave back
        slots = [eng.take_slot() for _ in lens]
        order = list(range(4)) if time == 0 else [2, 0, 3, 1]
        got = eng.step([(slots[i], prompts[i][:lens[i]]) for i in order], want="all").cpu().numpy()
        lo = 0
        for i in order:
            close(got[lo:lo + lens[i]], refs[i][:lens[i]], dtype, f"{name} prompt {i} time {time}")
            lo += lens[i]
        live = list(order)
        for step in range(12):
            if step == 5:                             # one request ends earlier
                eng.give_back_slot(slots[live.pop(0)])
            got = eng.step([(slots[i], [prompts[i][lens[i] + step]]) for i in live]).cpu().numpy()
            for r, i in enumerate(live):
                close(got[r:r + 1], refs[i][lens[i] + step:lens[i] + step + 1], dtype, f"{name} request {i} step {step}")
        for i in live:
            eng.give_back_slot(slots[i])
    assert eng.slots_free() == 4


def test_a_windowed_layer_gives_pages_back():
    """The cache of a windowed attention holds the window only: pages in front of it go back to the pool as the
    sequence grows and are used again by another sequence; the logits stay those of the plain implementation."""
    eng, cfg, W = engine("mixed", "float32", n_slots=2, max_tokens=700)
    toks, other = tokens("mixed", 40, 330), tokens("mixed", 41, 100)
    ref, ref_other = P.forward(cfg, W, toks), P.forward(cfg, W, other)
    a = eng.take_slot()
    rows = [eng.step([(a, toks[:150])], want="all").cpu().numpy()]
    windowed = {group.need.window: g for g, group in enumerate(eng.cache.groups) if group.need.window}
    assert set(windowed) == {37, 64, 90}
    assert len([p for p in eng.cache.slots.pages[a][windowed[37]] if p]) <= 2       # only the last pages are still held
    b = eng.take_slot()
    rows_b = [eng.step([(b, other[:60])], want="all").cpu().numpy()]
    for j in range(150, 330):
        entries = [(a, [toks[j]])] + ([(b, [other[60 + j - 150]])] if 60 + j - 150 < 100 else [])
        out = eng.step(entries).cpu().numpy()
        rows.append(out[:1])
        if len(entries) > 1:
            rows_b.append(out[1:])
    close(np.concatenate(rows), ref, "float32", "the long request")
    close(np.concatenate(rows_b), ref_other, "float32", "the one that took its pages")


@pytest.mark.parametrize("name, dtype", [("mixed", "float32"), ("tiled", "bfloat16")])
def test_long_decoding(name, dtype):
    eng, cfg, W = engine(name, dtype)
    toks = tokens(name, 4, 420)
    ref = P.forward(cfg, W, toks)
    s = eng.take_slot()
    rows = [eng.step([(s, toks[:2])], want="all").cpu().numpy()]
    for t in toks[2:]:
        rows.append(eng.step([(s, [t])]).cpu().numpy())
    close(np.concatenate(rows), ref, dtype, name)


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_far_key_that_stands_out_in_a_whole_model(dtype):
    """One token's embedding is far longer along the direction that one layer's keys and queries share, so it is found
    from everywhere inside the window: the logits of the last position that sees it and of the first that does not."""
    import copy
    import tempfile
    from gpullama3_java_amd.engine import Engine
    from lusalix_models import TILED, write_model
    cfg = copy.deepcopy(TILED)
    cfg["layers"] = cfg["layers"][:1]
    cfg["layers"][0]["mixer"]["softcap"] = 40.0
    W = {k: np.array(v) for k, v in P.make_weights(cfg, 9).items()}
    d, m, loud, at = cfg["width"], cfg["layers"][0]["mixer"], 5, 40
    W["embed"][loud] = 0.0
    W["embed"][loud, 0] = 16.0                             # after the norm: sqrt(d) along dimension 0
    W["embed"][np.arange(cfg["vocab"]) != loud, 1] = 2.0    # every other token: a part along dimension 1
    W["l0.norm1"][:] = 1.0
    W["l0.mix.k"][:, 0] = W["l0.mix.q"][:, 1] = 0.5        # keys of dimension 0 meet queries of dimension 1
    W["l0.mix.v"][:, 0] = 1.0                              # and bring a value of their own
    W = {k: bf16_exact(v) for k, v in W.items()}
    folder = tempfile.mkdtemp(prefix="lusalix-far-")
    write_model(folder, cfg, W)
    rng = np.random.default_rng(3)
    toks = [int(t) for t in rng.integers(6, cfg["vocab"], 170)]
    toks[at] = loud
    last = at + m["mask"]["size"] - 1
    ref = P.forward(cfg, W, toks)
    quiet = list(toks)
    quiet[at] = 6
    moved = row_errors(ref, P.forward(cfg, W, quiet))
    assert moved[last] > 0.3 and moved[last + 1] == 0.0      # the plain logits: seen, then not
    eng = Engine.from_folder(folder, dtype=dtype, max_tokens=1024, n_slots=4)
    tol = {"float32": 5e-5, "bfloat16": 0.1}[dtype]               # (random tokens: a 16-bit engine may flip one close choice)
    s = eng.take_slot()
    whole = row_errors(eng.step([(s, toks)], want="all").cpu().numpy(), ref)
    s = eng.take_slot()
    rows = [eng.step([(s, toks[:at + 1])], want="all").cpu().numpy()] + [eng.step([(s, [t])]).cpu().numpy() for t in toks[at + 1:]]
    decoded = row_errors(np.concatenate(rows), ref)
    for e in (whole, decoded):
        assert np.median(e) < tol and e[[last - 1, last, last + 1, last + 2]].max() < max(tol, moved[last] / 3)


def test_every_fast_path_gives_the_same_numbers_within_rounding():
    """A bfloat16 engine without one family of fast paths after another: norms folded into products and pairs' factors,
    the matrix-core attention kernels, the copies in operand order."""
    eng, cfg, W = engine("tiled", "bfloat16")
    toks = tokens("tiled", 2, 200)
    ref = P.forward(cfg, W, toks)
    for without in ("fused", "attn_decode,attn_prefill", "tiled", "mfma", "skinny,wide"):
        eng, _, _ = engine("tiled", "bfloat16", without=without)
        s = eng.take_slot()
        rows = [eng.step([(s, toks[:120])], want="all").cpu().numpy()] + [eng.step([(s, [t])]).cpu().numpy() for t in toks[120:150]]
        close(np.concatenate(rows), ref[:150], "bfloat16", f"tiled without {without}")


def test_greedy_generation_through_the_scheduler():
    """The engine's own entry point and scheduler: three prompts of unequal lengths, greedy, in 32-bit (a bfloat16
    engine may choose another expert on a close call of a token that it generated itself)."""
    eng, cfg, W = engine("mixed", "float32")
    prompts = [tokens("mixed", 20, 5), tokens("mixed", 21, 45), tokens("mixed", 22, 1)]
    out = eng.generate(prompts, max_new_tokens=20, temperature=0.0)
    for p, r in zip(prompts, out):
        assert len(r.tokens) == 20
        seq = list(p)
        for t in r.tokens:
            logits = P.forward(cfg, W, seq)[-1]
            best = int(np.argmax(logits))
            assert t == best or logits[best] - logits[t] < 1e-4 * np.abs(logits).max(), (len(seq), t, best)
            seq.append(t)
    assert eng.slots_free() == eng.n_slots


def test_generation_in_bfloat16_runs_captured_steps():
    """A bfloat16 engine decodes from captured graphs: the same tokens come out of eager steps, run after run."""
    eng, cfg, W = engine("tiled", "bfloat16")
    assert eng.use_graphs
    prompts = [tokens("tiled", 23, 9), tokens("tiled", 24, 70)]
    first = [r.tokens for r in eng.generate(prompts, max_new_tokens=24, temperature=0.0)]
    again = [r.tokens for r in eng.generate(prompts, max_new_tokens=24, temperature=0.0)]
    plain, _, _ = engine("tiled", "bfloat16", use_graphs=False)
    eager = [r.tokens for r in plain.generate(prompts, max_new_tokens=24, temperature=0.0)]
    assert first == again == eager


def test_the_command_line_takes_the_model(capsys):
    from gpullama3_java_amd import cli
    folder, cfg, W = model("reordered")
    prompt = tokens("reordered", 30, 6)
    rc = cli.main(["--model", folder, "--prompt-ids", ",".join(map(str, prompt)), "--max-tokens", "12", "--temperature", "0",
                   "--dtype", "float32", "--stream", "false"])
    assert not rc
    words = capsys.readouterr().out.split()
    got = [int(w) for w in words if w.lstrip("-").isdigit()]
    seq = list(prompt)
    for t in got[:3]:
        assert t == int(np.argmax(P.forward(cfg, W, seq)[-1]))
        seq.append(t)
    assert len(got) >= 3


def test_the_trace_runner_replays_a_model_of_this_design(tmp_path):
    """bin/trace_run as a user drives it: a request whole, one with its last tokens one by one, two of unequal lengths
    in one batch that end at different times; the model class comes from the folder's config.json."""
    from test_gpu_replay import Replay
    name = "mixed"
    folder, cfg, W = model(name)
    V = cfg["vocab"]
    reqs = {"a": tokens(name, 50, 90), "b": tokens(name, 51, 140), "c": tokens(name, 52, 7)}
    ref = {k: P.forward(cfg, W, t) for k, t in reqs.items()}
    rp = Replay(folder, "float32", tmp_path, max_tokens=400)
    t = reqs["a"]
    close(rp.step([("a", t, list(range(len(t))))], end=["a"]).reshape(-1, V), ref["a"], "float32", "whole")
    t = reqs["b"]
    rows = [rp.step([("b", t[:100], [0, 50, 99])]).reshape(-1, V)]
    for j in range(100, len(t)):
        rows.append(rp.step([("b", [t[j]], [0])], end=["b"] if j == len(t) - 1 else []).reshape(-1, V))
    close(np.concatenate(rows), ref["b"][[0, 50, 99] + list(range(100, len(t)))], "float32", "decoded")
    got = {"a": [], "c": []}
    out = rp.step([("c", reqs["c"][:3], [0, 1, 2]), ("a", reqs["a"][:70], [69])]).reshape(-1, V)
    got["c"].append(out[:3]); got["a"].append(out[3:])
    for j in range(20):
        live = [k for k in ("c", "a") if (3 if k == "c" else 70) + j < len(reqs[k])]
        at = {k: (3 if k == "c" else 70) + j for k in live}
        out = rp.step([(k, [reqs[k][at[k]]], [0]) for k in live], end=[k for k in live if at[k] + 1 == len(reqs[k])]).reshape(-1, V)
        for r, k in enumerate(live):
            got[k].append(out[r:r + 1])
    close(np.concatenate(got["c"]), ref["c"], "float32", "the shorter of a batch")
    close(np.concatenate(got["a"]), ref["a"][69:90], "float32", "the longer of a batch")
    rp.close()


# ----------------------------------------------------------------- seeded random configurations
def random_config(seed):
    """A configuration drawn from a seed: widths, head counts and sizes that no tile need divide (values larger and
    smaller than keys), windows, caps, temperatures (small ones: scores in the tens make a softmax pick single keys, and
    then the rounding of 16-bit queries and keys is the row), blends, experts and shared experts of any size, or none
    of each."""
    from lusalix_models import _attn, _model, _moe
    rng = np.random.default_rng([seed, 78])
    pick = lambda *a: a[int(rng.integers(0, len(a)))]
    kv, vdim = int(pick(1, 2, 3)), int(pick(6, 8, 16, 20, 24, 48, 64))      # (of the layers that blend their values)

    def mlp():
        if rng.random() < 0.2:
            return None
        experts = int(pick(1, 2, 3, 5, 8, 17))
        ff = int(pick(8, 24, 33, 40, 64))
        return _moe(experts, int(rng.integers(1, min(experts, 4) + 1)), ff, pick(None, ff, int(pick(16, 24, 40)), 72))

    def layer():
        mix = bool(rng.random() < 0.6)
        G, Dv = (kv, vdim) if mix else (int(pick(1, 2, 3)), int(pick(8, 12, 32, 64, 100)))
        dim = int(pick(8, 10, 16, 32, 40, 64, 112, 140))
        return _attn(G * int(pick(1, 2, 4)), G, dim, Dv, float(dim ** -0.5 * rng.uniform(0.7, 1.4)), pick(None, 1.5, 4.0, 30.0),
                     pick(None, (0.1, 1), (float(rng.uniform(0.1, 0.6)), int(pick(5, 16, 33, 64, 100)))),
                     pick(None, 1, 2, 7, 33, 64, 65, 100), mix, mlp())

    return _model(int(pick(97, 150, 256, 301)), int(pick(48, 64, 72, 90, 100, 104, 128)), float(pick(1e-6, 1e-5)), float(pick(0.5, 1.0, 4.0)),
                  [layer() for _ in range(int(rng.integers(2, 6)))])


@pytest.mark.parametrize("seed", range(16))
def test_seeded_random_configurations(seed, tmp_path):
    """Whole, in portions with the last tokens one by one, and as one of a batch of three: 32-bit against the plain
    implementation to rounding, bfloat16 within three times what rounding alone does to the same row."""
    from gpullama3_java_amd.engine import Engine
    from lusalix_models import rounding, write_model
    cfg = random_config(seed)
    W = P.make_weights(cfg, seed)
    folder = str(tmp_path / "model")
    write_model(folder, cfg, W)
    toks = P.tokens_with_clear_choices(cfg, W, seed, 150)
    others = [P.tokens_with_clear_choices(cfg, W, seed + 100 + i, n) for i, n in enumerate((40, 9))]
    ref = P.forward(cfg, W, toks)
    refs = [P.forward(cfg, W, t) for t in others]
    alone = rounding(cfg, W, toks, ref)
    alones = [rounding(cfg, W, t, r) for t, r in zip(others, refs)]
    for dtype in DTYPES:
        eng = Engine.from_folder(folder, dtype=dtype, max_tokens=1024, n_slots=4)
        s = eng.take_slot()
        what = f"seed {seed} {dtype}"
        close(eng.step([(s, toks)], want="all").cpu().numpy(), ref, dtype, what + " whole", alone=alone)
        eng.give_back_slot(s)
        s = eng.take_slot()
        rows = [eng.step([(s, toks[:70])], want="all").cpu().numpy(), eng.step([(s, toks[70:72])], want="all").cpu().numpy(),
                eng.step([(s, toks[72:140])], want="all").cpu().numpy()]
        rows += [eng.step([(s, [t])]).cpu().numpy() for t in toks[140:]]
        close(np.concatenate(rows), ref, dtype, what + " in portions", alone=alone)
        eng.give_back_slot(s)
        slots = [eng.take_slot() for _ in range(3)]
        got = eng.step([(slots[0], others[0][:30]), (slots[1], toks[:100]), (slots[2], others[1][:3])], want="all").cpu().numpy()
        close(got[:30], refs[0][:30], dtype, what + " batch 0", alone=alones[0][:30])
        close(got[30:130], ref[:100], dtype, what + " batch 1", alone=alone[:100])
        close(got[130:], refs[1][:3], dtype, what + " batch 2", alone=alones[1][:3])
        for j in range(6):
            got = eng.step([(slots[0], [others[0][30 + j]]), (slots[1], [toks[100 + j]]), (slots[2], [others[1][3 + j]])]).cpu().numpy()
            close(got[0:1], refs[0][30 + j:31 + j], dtype, what + f" decode 0 step {j}", alone=alones[0][30 + j])
            close(got[1:2], ref[100 + j:101 + j], dtype, what + f" decode 1 step {j}", alone=alone[100 + j])
            close(got[2:3], refs[1][3 + j:4 + j], dtype, what + f" decode 2 step {j}", alone=alones[1][3 + j])
        del eng
