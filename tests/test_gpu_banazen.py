"""The Banazen decoder on the GPU against the plain implementation (``plain_banazen.py``): each mechanism's kernels alone,
with inputs made so that a fault shows, then whole models through the engine's step function, its cache, its batching and
its generation loop."""
import copy
import functools
import tempfile

import numpy as np
import pytest
import torch

import plain_banazen as P
from banazen_models import (CONFIGS, TILED, close, decoder, dense, latent, model, moe, near, ranks, rounding, row_errors, sides,
                            tokens, write_model)
from cache_order import tile_keys, untile_keys, untile_values

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


@functools.lru_cache(maxsize=None)
def reference(name, seed, n):
    """(tokens, plain logits, each row's error by rounding alone)."""
    _, cfg, W = model(name)
    toks = tokens(name, seed, n)
    ref = P.forward(cfg, W, toks)
    return toks, ref, rounding(cfg, W, toks, ref)


# ----------------------------------------------------------------- queries, keys and values behind a convolution
def tables(n, dims, base):
    from gpullama3_java_amd.config.specs import RotarySpec
    from gpullama3_java_amd.parts.rotary import Rotary
    r = Rotary(RotarySpec(head_dim=dims, theta=base, pairing="adjacent", max_positions=n), DEV)
    return dims, r.cos, r.sin


CONV_CASES = [  # H, G, D, Dv, stored D, stored Dv, taps, rot, norm with weights
    (4, 2, 24, 40, 32, 48, 4, 12, False), (3, 3, 16, 16, 16, 16, 1, 16, True), (6, 1, 64, 64, 64, 64, 3, 64, False),
    (2, 2, 40, 24, 64, 64, 7, None, True), (5, 5, 128, 96, 128, 96, 2, 32, False), (1, 1, 34, 200, 48, 208, 9, 34, None)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H, G, D, Dv, hs, vd, taps, rot, weights", CONV_CASES)
def test_heads_behind_a_convolution(H, G, D, Dv, hs, vd, taps, rot, weights, dtype):
    """Three sequences of unequal lengths fed in pieces (down to one token each, cuts inside the convolution's reach and
    inside groups of eight positions), slots and pages in another order than the sequences, page borders inside; the
    caches, the queries and the held inputs against the equations. ``weights`` None: no norm."""
    from gpullama3_java_amd.csrc import lib as K
    rng = np.random.default_rng([H, D, taps])
    page, eps, lens = 32, 1e-2, [45, 7, 20]
    C = (H + G) * hs + G * vd
    table = np.array([[3, 6], [1, 4], [5, 2], [0, 0]])          # rows are slots
    slots = [2, 0, 1]
    u = []
    for n in lens:
        rows = np.zeros((n, C + 16), np.float32)
        for c0, heads, d, dp in ((0, H, D, hs), (H * hs, G, D, hs), ((H + G) * hs, G, Dv, vd)):
            part = np.zeros((n, heads, dp))
            part[..., :d] = rng.standard_normal((n, heads, d))
            rows[:, c0:c0 + heads * dp] = part.reshape(n, -1)
        u.append(bf16_exact(rows))
    w = np.zeros((C, taps), np.float32)
    w[:] = rng.standard_normal((C, taps)) * 0.7
    qw, kw = (1 + 0.3 * rng.standard_normal(hs) for _ in range(2))
    base = 700.0
    state_off, width = 8, 8 + -(-C * (taps - 1) // 4) * 4 + 4
    state = torch.zeros(4, width, device=DEV)
    kc = torch.zeros(7, G, page, hs, dtype=TD[dtype], device=DEV)
    vc = torch.zeros(7, G, vd, page, dtype=TD[dtype], device=DEV)
    rotation = tables(64, rot, base) if rot else None
    norm = None if weights is None else (eps, D, dev(qw) if weights else None, dev(kw) if weights else None)
    q_got = [[] for _ in lens]
    cuts = [[1, 2, 5, 13, 14, 37, 38, 45], [1, 3, 7], [9, 11, 12, 13, 20]]
    at = [0, 0, 0]
    for step in range(8):
        who = [b for b in range(3) if step < len(cuts[b])]
        n = [cuts[b][step] - at[b] for b in who]
        T = sum(n)
        rows = dev(np.concatenate([u[b][at[b]:at[b] + k] for b, k in zip(who, n)]), TD[dtype])
        positions = np.concatenate([np.arange(at[b], at[b] + k) for b, k in zip(who, n)])
        seq = np.repeat(np.arange(len(who)), n)
        q = torch.full((T, H * hs), 9.0, dtype=TD[dtype], device=DEV)
        K.conv_heads(rows, dev(w.T), state, state_off, i32(np.concatenate([[0], np.cumsum(n)])), i32(seq), i32([slots[b] for b in who]),
                     i32(positions), i32([slots[who[s]] for s in seq]), i32(table), rotation, q, kc, vc, H, G, hs, vd, page, norm=norm,
                     one_token_each=max(n) == 1)
        lo = 0
        for b, k in zip(who, n):
            q_got[b].append(host(q)[lo:lo + k])
            lo += k
            at[b] += k
    gk, gv, held = untile_keys(host(kc)), untile_values(host(vc)), host(state)
    atol = 2e-5 if dtype == "float32" else 0.04
    for b, n in enumerate(lens):
        y, left = P.short_conv(u[b][:, :C].astype(np.float64), w.astype(np.float64))
        np.testing.assert_allclose(held[slots[b], state_off:state_off + C * (taps - 1)].reshape(taps - 1, C), left, atol=1e-6)
        parts = []
        for c0, heads, nw in ((0, H, qw), (H * hs, G, kw)):
            x = y[:, c0:c0 + heads * hs].reshape(n, heads, hs)
            if rot:
                x = P.rotate(x, np.arange(n), rot, base)
            if weights is not None:
                x = x / np.sqrt((x ** 2).sum(-1, keepdims=True) / D + eps) * (nw if weights else 1.0)
            parts.append(x)
        np.testing.assert_allclose(np.concatenate(q_got[b]).reshape(n, H, hs), parts[0], atol=atol)
        v = y[:, (H + G) * hs:].reshape(n, G, vd)
        for i in range(n):
            pg, ip = table[slots[b], i // page], i % page
            np.testing.assert_allclose(gk[pg, :, ip], parts[1][i], atol=atol)
            np.testing.assert_allclose(gv[pg, :, :, ip], v[i], atol=atol)
    assert not held[3].any() and not held[:, :state_off].any() and not gk[0].any() and not gv[0].any()
    assert not held[:, state_off + C * (taps - 1):].any()


def test_a_convolution_refuses_what_it_is_not_built_for():
    from gpullama3_java_amd.csrc import lib as K
    T, H, G, hs = 4, 2, 1, 16
    C = (H + G) * hs + G * hs
    kc, vc = torch.zeros(2, G, 32, hs, device=DEV), torch.zeros(2, G, hs, 32, device=DEV)

    def run(rows=None, w=None, state=None, norm=None, one=False):
        K.conv_heads(torch.zeros(T, C, device=DEV) if rows is None else rows, torch.zeros(3, C, device=DEV) if w is None else w,
                     torch.zeros(2, 2 * C, device=DEV) if state is None else state, 0, i32([0, T]), i32([0] * T), i32([0]), i32(range(T)),
                     i32([0] * T), i32([[1]]), None, torch.zeros(T, H * hs, device=DEV), kc, vc, H, G, hs, hs, 32, norm=norm,
                     one_token_each=one)
    run()
    run(one=True)                                # (four tokens of one sequence: not one each, the plain way is taken)
    for bad in (dict(rows=torch.zeros(T, C - 16, device=DEV)), dict(w=torch.zeros(3, C + 16, device=DEV)),
                dict(state=torch.zeros(2, 2 * C - 4, device=DEV)), dict(norm=(1e-5, 17, None, None)),
                dict(norm=(1e-5, 16, torch.zeros(8, device=DEV), None)), dict(rows=torch.zeros(T, C, dtype=torch.bfloat16, device=DEV))):
        with pytest.raises(K.KernelError):
            run(**bad)


# ----------------------------------------------------------------- the delta rule with a decay per key channel
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T, H, D, Dv, ra, rg", [(1, 3, 16, 24, 8, 12), (16, 2, 40, 32, 33, 7), (17, 4, 64, 64, 64, 64), (150, 1, 20, 130, 100, 200),
                                                 (70, 6, 128, 16, 5, 32)])
def test_second_steps_of_decay_and_gate(T, H, D, Dv, ra, rg, dtype):
    from gpullama3_java_amd.csrc import lib as K
    rng = np.random.default_rng([T, H, D])
    ca, cg = 3, 3 + ra + 2
    proj = bf16_exact(rng.standard_normal((T, cg + rg + 5)))
    a2, g2 = bf16_exact(rng.standard_normal((H * D, ra)) / np.sqrt(ra)), bf16_exact(rng.standard_normal((H * Dv, rg)) / np.sqrt(rg))
    A, bias = rng.uniform(-4, 0.5, H).astype(np.float32), rng.uniform(-3, 1, H * D).astype(np.float32)
    Na, Ng, Rp = -(-H * D // 64) * 64, -(-H * Dv // 64) * 64, -(-max(ra, rg) // 32) * 32
    w2 = np.zeros((Na + Ng, Rp), np.float32)
    w2[:H * D, :ra], w2[Na:Na + H * Dv, :rg] = a2, g2
    decay, gate = torch.full((T, H * D), 9.0, device=DEV), torch.full((T, H * Dv), 9.0, device=DEV)
    K.delta_inner(dev(proj), ca, ra, cg, rg, dev(w2, TD[dtype]), Na, dev(A), dev(bias), decay, gate, H, D, Dv)
    p64 = proj.astype(np.float64)
    s = p64[:, ca:ca + ra] @ a2.T.astype(np.float64) + bias
    ref = np.exp(-np.exp(A.astype(np.float64))[:, None] * P.softplus(s.reshape(T, H, D)))
    np.testing.assert_allclose(host(decay).reshape(T, H, D), ref, atol=3e-6)
    np.testing.assert_allclose(host(gate), p64[:, cg:cg + rg] @ g2.T.astype(np.float64), atol=2e-5)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H, G, D, Dv", [(4, 2, 24, 40), (3, 3, 64, 64), (2, 1, 128, 128), (2, 2, 7, 16), (1, 1, 200, 96), (4, 4, 32, 130), (1, 1, 256, 256),
                                         (130, 65, 48, 20)])
def test_delta_rule_with_channel_decays_whole_and_in_pieces(H, G, D, Dv, dtype):
    """Two sequences in one step, whole, in pieces and with tokens one by one, from the state in slots that are not in the
    sequences' order; decays from almost one to almost zero, so that a decay on the wrong channel shows; the gate is a
    sigmoid. Values and read-outs that the norm would hide are compared before it, too."""
    from gpullama3_java_amd.csrc import lib as K
    rng = np.random.default_rng([H, D, Dv])
    lens, eps, taps = [37, 21], 1e-5, 3
    C = 2 * G * D + H * Dv
    n_state = -(-K.delta_state_floats(H, G, D, Dv, taps) // 4) * 4
    q, k = (P.unit_length(rng.standard_normal((sum(lens), G, D))) for _ in range(2))
    q = q * D ** -0.5
    v = rng.standard_normal((sum(lens), H, Dv))
    g = np.exp(-10.0 ** rng.uniform(-3, 0.7, (sum(lens), H, D)))
    beta = rng.uniform(0, 1, (sum(lens), H))
    gate, nw = rng.standard_normal((sum(lens), H * Dv)) * 2, 1 + 0.2 * rng.standard_normal(Dv)
    act = np.concatenate([q.reshape(-1, G * D), k.reshape(-1, G * D), v.reshape(-1, H * Dv)], 1).astype(np.float32)
    strengths = np.concatenate([np.full((sum(lens), H), 77.0), beta], 1).astype(np.float32)     # (the first half is not looked at)
    first = [0, lens[0]]
    ref = np.zeros((sum(lens), H, Dv))
    S_ref = np.zeros((2, H, D, Dv))
    f32 = lambda a: a.astype(np.float32).astype(np.float64)
    for b in range(2):
        sl = slice(first[b], first[b] + lens[b])
        for h in range(H):
            c = h // (H // G)
            ref[sl, h], S_ref[b, h] = P.delta_rule(f32(q)[sl, c], f32(k)[sl, c], f32(v)[sl, h], f32(g)[sl, h], f32(beta)[sl, h], np.zeros((D, Dv)))
    out_ref = P.rms_norm(ref, nw, eps) * P.sigmoid(gate.reshape(-1, H, Dv))
    one_by_one = [list(range(1, 38)), list(range(1, 22))]
    for cuts, one in (([[37], [21]], False), ([[3, 5, 20, 37], [16, 17, 18, 21]], False), (one_by_one, False), (one_by_one, True)):
        state = torch.zeros(3, n_state, device=DEV)
        got, raw = np.zeros((sum(lens), H * Dv)), np.zeros((sum(lens), H * Dv))
        at = [0, 0]
        for step in range(max(len(c) for c in cuts)):
            who = [b for b in range(2) if step < len(cuts[b])]
            n = [cuts[b][step] - at[b] for b in who]
            idx = np.concatenate([np.arange(first[b] + at[b], first[b] + at[b] + m) for b, m in zip(who, n)])
            T = len(idx)
            o, y = torch.zeros(T, H * Dv, device=DEV), torch.zeros(T, H * Dv, dtype=TD[dtype], device=DEV)
            K.delta_recurrence(dev(act[idx]), dev(strengths[idx]), state, i32(np.concatenate([[0], np.cumsum(n)])), i32([[2, 0][b] for b in who]),
                               o, dev(gate[idx]), 0, dev(nw), y, H, G, D, Dv, taps, eps, decay=dev(g.reshape(-1, H * D)[idx]), gate_act="sigmoid",
                               one_token_each=one)
            got[idx], raw[idx] = host(y), host(o)
            for b, m in zip(who, n):
                at[b] += m
        if not one:      # (the kernel for steps of one token each keeps its read-outs to itself)
            np.testing.assert_allclose(raw.reshape(ref.shape), ref, atol=3e-5 * np.abs(ref).max())
        np.testing.assert_allclose(got.reshape(ref.shape), out_ref, atol=2e-4 if dtype == "float32" else 0.03)
        st = host(state)
        CT = -(-Dv // 16)
        for b, slot in enumerate([2, 0]):
            S = st[slot, :H * CT * D * 16].reshape(H, CT, D, 16).transpose(0, 2, 1, 3).reshape(H, D, CT * 16)[..., :Dv]
            np.testing.assert_allclose(S, S_ref[b], atol=3e-5 * np.abs(S_ref[b]).max())
        assert not st[1].any()


# ----------------------------------------------------------------- attention over cached latents in a window
def paged_latents(c, dk, page, dtype):
    """One sequence's latents [S, rank] as a paged cache of rows of dk; its pages lie in another order than its positions."""
    S, rank = c.shape
    n = -(-S // page)
    table = 1 + (np.arange(n) * 3 + 1) % n if n % 3 else 1 + np.arange(n)[::-1]
    kc = np.zeros((n + 1, 1, page, dk), np.float32)
    for j in range(S):
        kc[table[j // page], 0, j % page, :rank] = c[j]
    return dev(tile_keys(kc), TD[dtype]), i32(table[None])


@pytest.mark.parametrize("kernel", ["any", "matrix 1", "matrix 3", "matrix prompt", "any prompt"])
@pytest.mark.parametrize("H, rank, window", [(3, 64, 37), (8, 96, 64), (16, 128, 33), (2, 256, 100), (40, 32, 9), (5, 64, 1), (4, 64, None)])
def test_a_window_over_cached_latents(H, rank, window, kernel):
    """A marked latent that every query finds if it may see it: positions at both edges of its window, at page borders and
    chunk edges, decoded (each query a sequence of its own) and as a portion of a prompt that passes the edge."""
    from gpullama3_java_amd.csrc import lib as K
    rng = np.random.default_rng([H, rank])
    S, at, scale, dk = 330, 150, 0.3, -(-rank // 32) * 32
    c = bf16_exact(rng.standard_normal((S, rank)) * 0.3)
    c[at] = bf16_exact(30.0 / np.sqrt(rank) * np.ones(rank))
    w = window or 10 ** 6
    if "prompt" in kernel:
        lo = at + w - 40 if window is not None and at + w + 20 < S else at - 30
        positions = list(range(lo, min(S, lo + 90)))
    else:
        positions = sorted({p for p in (0, 1, 31, 32, 63, 64, at - 1, at, at + 1, at + w - 2, at + w - 1, at + w, at + w + 1, 255, 256, S - 1) if p < S})
    T = len(positions)
    q = bf16_exact(rng.standard_normal((T, H, rank)) * 0.2 + 1.0 / np.sqrt(rank))
    ref = np.zeros((T, H, rank))
    for t, i in enumerate(positions):
        lo = P.first_seen(i, window)
        for a in range(H):
            ref[t, a] = P.softmax_over(q[t, a].astype(np.float64), c[lo:i + 1].astype(np.float64), c[lo:i + 1].astype(np.float64), scale)
    if window is not None and at + w in positions and window > 1:
        assert np.abs(ref[positions.index(at + w - 1)]).mean() > 2 * np.abs(ref[positions.index(at + w)]).mean()      # seen, then not
    for dtype in (["bfloat16"] if "matrix" in kernel else DTYPES):
        kc, table = paged_latents(c, dk, 64, dtype)
        qa = np.zeros((T, H, dk), np.float32)
        qa[..., :rank] = q
        qd, out = dev(qa.reshape(T, -1), TD[dtype]), torch.zeros(T, H * rank, dtype=TD[dtype], device=DEV)
        if "matrix" in kernel:
            if kernel == "matrix prompt":
                K.latent_attention(qd, kc, i32([0, T]), i32([positions[0]]), table, out, T, H, rank, scale, window=window)
            else:
                n = int(kernel.split()[1])
                part_o = torch.zeros(T * H * n * rank, device=DEV) if n > 1 else None
                part_ml = torch.zeros(T * H * n * 2, device=DEV) if n > 1 else None
                K.latent_attention(qd, kc, i32(range(T + 1)), i32(positions), table, out, 1, H, rank, scale, seq_rows=i32([0] * T),
                                   n_splits=n, part_o=part_o, part_ml=part_ml, window=window)
        else:
            K.attention_generic(qd, kc, None, i32(positions), i32([0] * T), table, out, H, 1, dk, 64, window, scale, v_head_dim=rank,
                                values_in_keys=0)
        np.testing.assert_allclose(host(out).reshape(T, H, rank), ref, atol=3e-5 if dtype == "float32" else 0.05)


@pytest.mark.parametrize("dtype", DTYPES)
def test_queries_and_latents_from_one_product(dtype):
    """The rows of the stacked product without a query latent, with and without latents of the layer's own."""
    from gpullama3_java_amd.csrc import lib as K
    rng = np.random.default_rng(4)
    T, H, D, rank, page = 7, 3, 5, 32, 32          # (a layer that only reads has fewer columns than a latent)
    proj = rng.standard_normal((T, 80)).astype(np.float32)
    w = (1 + 0.2 * rng.standard_normal(rank)).astype(np.float32)
    positions, table = [0, 1, 2, 31, 32, 33, 5], np.array([[2, 1], [3, 4]])
    seqs = [0, 0, 0, 0, 0, 0, 1]
    for own in (True, False):
        cq = torch.zeros(T, H * D, dtype=TD[dtype], device=DEV)
        kc = torch.full((5, 1, page, 32), 5.0, dtype=TD[dtype], device=DEV)
        runs, rows = torch.zeros(H + 1, dtype=torch.int32, device=DEV), torch.zeros(T * H, dtype=torch.int32, device=DEV)
        K.latent_prep(dev(proj if own else proj[:, :16]), 1, H * D, 33 if own else None, rank, 0, None, dev(w) if own else None, 1e-2, i32(positions), i32(seqs), i32(table),
                      None, None, cq, kc, page, H, runs, rows)
        np.testing.assert_allclose(host(cq), proj[:, 1:1 + H * D], rtol=5e-3 if dtype == "bfloat16" else 1e-7)
        np.testing.assert_array_equal(host(runs), np.arange(H + 1) * T)
        np.testing.assert_array_equal(host(rows).reshape(H, T), np.arange(T)[None] * H + np.arange(H)[:, None])
        got = untile_keys(host(kc))
        if own:
            c = P.rms_norm(proj[:, 33:33 + rank], w, 1e-2)
            for t in range(T):
                row = got[table[seqs[t], positions[t] // page], 0, positions[t] % page]
                np.testing.assert_allclose(row[:rank], c[t], atol=2e-2 if dtype == "bfloat16" else 2e-6)
                assert not row[rank:].any()
        else:
            assert (got == 5.0).all()


# ----------------------------------------------------------------- experts from the best groups
def routed(K, logits, top, E, always=False, gate_col=None, **kw):
    T, more = logits.shape[0], 1 if always else 0
    o = dict(idx=torch.zeros(T, top + more, dtype=torch.int32, device=DEV), wts=torch.zeros(T, top + more, device=DEV),
             offsets=torch.zeros(E + more + 1, dtype=torch.int32, device=DEV),
             pairs=torch.zeros(T * (top + more), dtype=torch.int32, device=DEV))
    gate_out = torch.zeros(T, device=DEV) if gate_col is not None and not always else None
    K.route(dev(logits), top, always=always, scores=True, n_experts=E, gate_col=gate_col, gate_out=gate_out, **o, **kw)
    return o, gate_out


@pytest.mark.parametrize("T", [1, 7, 64, 65, 300])
@pytest.mark.parametrize("E, top, count, keep", [(6, 2, 3, 2), (12, 4, 4, 3), (9, 4, 3, 2), (8, 3, 8, 5), (64, 6, 8, 2), (256, 8, 8, 4), (130, 5, 65, 3),
                                                 (1, 1, 1, 1), (5, 5, 1, 1), (1024, 16, 512, 100)])
def test_router_with_groups(T, E, top, count, keep):
    """Choice scores may be negative (a closed group's experts still count as less than any of them), ties go to the lower
    number, the weights leave the correction out, the shared expert's factor is not scaled; every pair once in its run."""
    from gpullama3_java_amd.csrc import lib as K
    rng = np.random.default_rng([T, E])
    logits = np.zeros((T, -(-(E + 1) // 16) * 16), np.float32)
    logits[:, :E] = rng.standard_normal((T, E)) * 1.5
    logits[:, E:] = 30.0
    logits[:, E] = rng.standard_normal(T)
    correction = (rng.standard_normal(E) * 0.6 / np.sqrt(E) - 0.4).astype(np.float32)           # most choice scores are negative
    router = {"experts": E, "top": top, "groups": {"count": count, "keep": keep}}
    z = logits[:, :E].astype(np.float64)
    s = np.exp(z - z.max(-1, keepdims=True))
    s /= s.sum(-1, keepdims=True)
    for always in (False, True):
        if always and (top >= 16 or E >= 1024):
            continue
        o, gate = routed(K, logits, top, E, always, E, correction=dev(correction), sum_eps=1e-20, groups=(count, keep), weight_scale=2.5)
        idx, wts, pairs, offsets = o["idx"].cpu().numpy(), host(o["wts"]), o["pairs"].cpu().numpy(), o["offsets"].cpu().numpy()
        unclear = 0
        for t in range(T):
            want, gap = P.choose(s[t] + correction, router)
            if gap < 2e-6:                      # (scores that 32-bit cannot tell apart)
                unclear += 1
                continue
            assert list(idx[t, :top]) == list(want) or gap < 1e-5 and set(idx[t, :top]) == set(want), t
            np.testing.assert_allclose(wts[t, :top], s[t, idx[t, :top]] / s[t, want].sum() * 2.5, rtol=2e-5, atol=1e-7)
            factor = P.sigmoid(logits[t, E].astype(np.float64))
            np.testing.assert_allclose(wts[t, top] if always else host(gate)[t], factor, atol=1e-6)
            if always:
                assert idx[t, top] == E
        assert unclear <= max(1, T // 20) * (1 + (E > 100) * 10)
        per = top + always
        assert offsets[0] == 0 and offsets[-1] == T * per and sorted(pairs) == list(range(T * per))
        for e in range(E + always):
            assert all(idx.reshape(-1)[p] == e for p in pairs[offsets[e]:offsets[e + 1]])


def test_router_ties_and_equal_groups():
    """All scores equal: the first groups stay open and the first experts are chosen; with corrections of two values the
    groups that hold the larger one."""
    from gpullama3_java_amd.csrc import lib as K
    for T in (3, 100):
        o, _ = routed(K, np.zeros((T, 12), np.float32), 3, 12, groups=(4, 2))
        assert (o["idx"].cpu().numpy() == [0, 1, 2]).all()
        np.testing.assert_allclose(host(o["wts"]), 1 / 3, rtol=1e-6)
        corr = np.array([0, 0, 0, 0, 0, 0, -1, -1, 0.5, -3, -3, 0.5], np.float32)
        o, _ = routed(K, np.zeros((T, 12), np.float32), 3, 12, groups=(4, 2), correction=dev(corr))
        assert (o["idx"].cpu().numpy() == [8, 11, 6]).all()       # (groups 6..8 and 9..11 are the best: the zeros are closed)
        o, _ = routed(K, np.zeros((T, 12), np.float32), 3, 12, groups=(6, 2), correction=dev(corr))
        assert (o["idx"].cpu().numpy() == [8, 11, 9]).all()       # (a closed group's 0 is not chosen in place of -3)
    with pytest.raises(K.KernelError):
        routed(K, np.zeros((3, 12), np.float32), 7, 12, groups=(4, 2))
    with pytest.raises(K.KernelError):
        routed(K, np.zeros((3, 12), np.float32), 2, 12, groups=(5, 2))


# ----------------------------------------------------------------- a token's side row
@pytest.mark.parametrize("dtype, mfma", [("float32", False), ("bfloat16", False), ("bfloat16", True)])
@pytest.mark.parametrize("T, d, dim, pad", [(1, 96, 10, 32), (8, 256, 64, 64), (17, 100, 24, 32), (300, 128, 33, 64), (33, 520, 96, 96), (2, 2048, 128, 128)])
def test_side_gate(T, d, dim, pad, dtype, mfma):
    from gpullama3_java_amd.csrc import lib as K
    rng = np.random.default_rng([T, d])
    x = (rng.standard_normal((T, d)) * 2).astype(np.float32)
    w, table = bf16_exact(rng.standard_normal((dim, d)) * 1.5 / np.sqrt(d)), bf16_exact(rng.standard_normal((50, 3 * dim + 1)))
    ids = rng.integers(0, 50, T)
    out = torch.full((T, pad), 3.0, dtype=TD[dtype], device=DEV)
    K.side_gate(dev(x), dev(w, TD[dtype]), dev(table, TD[dtype]), dim + 1, i32(ids), out, mfma=mfma)
    xr = x if dtype == "float32" else bf16_exact(x)
    ref = P.gelu_tanh(xr.astype(np.float64) @ w.T) * table[ids, dim + 1:2 * dim + 1]
    got = host(out)
    np.testing.assert_allclose(got[:, :dim], ref, atol=3e-5 if dtype == "float32" else 0.03, rtol=1e-5 if dtype == "float32" else 8e-3)
    assert not got[:, dim:].any()


@pytest.mark.parametrize("T, d", [(1, 64), (9, 96), (64, 2048), (70, 4100), (5, 20000)])
def test_norm_added_with_what_the_next_norm_makes(T, d):
    from gpullama3_java_amd.csrc import lib as K
    rng = np.random.default_rng([T, d])
    x0, y = (rng.standard_normal((T, d)).astype(np.float32) * s for s in (2.0, 0.01))
    w, nw = ((1 + 0.2 * rng.standard_normal(d)).astype(np.float32) for _ in range(2))
    eps, neps = 1e-4, 1e-2
    ref = x0 + P.rms_norm(y, w, eps)
    for dt, tol in ((torch.float32, 1e-5), (torch.bfloat16, 2e-2)):
        x, h = dev(x0), torch.zeros(T, d, dtype=dt, device=DEV)
        ssq, xg = (torch.zeros(64, device=DEV), torch.zeros(T, d, dtype=torch.bfloat16, device=DEV)) if T <= 64 else (None, None)
        K.norm_add_next(x, dev(y), dev(w), eps, dev(nw), neps, h=h, xg=xg, ssq=ssq)
        np.testing.assert_allclose(host(x), ref, atol=1e-5)
        np.testing.assert_allclose(host(h), P.rms_norm(ref, nw, neps), atol=tol, rtol=5e-3 if dt == torch.bfloat16 else 0)
        if ssq is not None:
            np.testing.assert_allclose(host(ssq)[:T], (ref * ref).sum(-1), rtol=1e-5)
            np.testing.assert_allclose(host(xg), ref * nw, rtol=6e-3, atol=1e-3)
    x = dev(x0)
    K.norm_add_next(x, dev(y), dev(w), eps)
    np.testing.assert_allclose(host(x), ref, atol=1e-5)


# ----------------------------------------------------------------- whole models through the engine
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_whole_prompt_and_every_layer(name, dtype):
    eng, cfg, W = engine(name, dtype)
    toks, ref, alone = reference(name, 1, 210)        # beyond every window, over four pages
    seq = P.Sequence(cfg, W)
    seq.feed(toks)
    seen = []
    eng.after_block = lambda i, x: seen.append(x.float().cpu().numpy())
    s = eng.take_slot()
    got = eng.step([(s, toks)], want="all").cpu().numpy()
    eng.after_block = None
    assert len(seen) == len(seq.rows[0]) == len(cfg["layers"])
    for r, (a, b) in enumerate(zip(seen, seq.rows[0])):     # the first layer that differs names the mechanism
        near(a, b, dtype, f"layer {r}")
    close(got, ref, dtype, name, alone)
    # the first tokens of a sequence, each alone from an empty slot
    for n in (1, 2, 3):
        s2 = eng.take_slot()
        close(eng.step([(s2, toks[:n])], want="all").cpu().numpy(), ref[:n], dtype, f"{name} first {n}", alone[:n])
        eng.give_back_slot(s2)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_prompt_then_token_by_token(name, dtype):
    """Decoding passes every window's edge and three page borders; the decoded rows are those of the whole prompt. The first
    tokens are fewer than the convolutions reach back."""
    eng, cfg, W = engine(name, dtype)
    toks, ref, alone = reference(name, 2, 200)
    s = eng.take_slot()
    rows = [eng.step([(s, toks[:2])], want="all").cpu().numpy()]
    for t in toks[2:]:
        rows.append(eng.step([(s, [t])]).cpu().numpy())
    close(np.concatenate(rows), ref, dtype, name, alone)
    assert eng.cache.length(s) == 200


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name, cuts", [("mixed", [2, 4, 7, 31, 33, 36, 38, 63, 65, 89, 91, 128, 129, 131, 190]),
                                        ("reordered", [1, 3, 5, 12, 19, 21, 63, 65, 67, 100, 102, 190]),
                                        ("bare", [19, 21, 23, 64, 190]),
                                        ("tiled", [17, 49, 51, 99, 101, 130, 131, 133, 190])])
def test_portions_of_a_prompt(name, cuts, dtype):
    eng, cfg, W = engine(name, dtype)
    toks, ref, alone = reference(name, 3, 190)
    s = eng.take_slot()
    rows, lo = [], 0
    for hi in cuts:
        rows.append(eng.step([(s, toks[lo:hi])], want="all").cpu().numpy())
        lo = hi
    close(np.concatenate(rows), ref, dtype, name, alone)
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
    refs = [reference(name, 10 + i, n + 12) for i, n in enumerate(lens)]
    prompts = [r[0] for r in refs]
    for time in range(2):                             # the second time takes the slots and pages that the first gave back
        slots = [eng.take_slot() for _ in lens]
        order = list(range(4)) if time == 0 else [2, 0, 3, 1]
        got = eng.step([(slots[i], prompts[i][:lens[i]]) for i in order], want="all").cpu().numpy()
        lo = 0
        for i in order:
            close(got[lo:lo + lens[i]], refs[i][1][:lens[i]], dtype, f"{name} prompt {i} time {time}", refs[i][2][:lens[i]])
            lo += lens[i]
        live = list(order)
        for step in range(12):
            if step == 5:                             # one request ends earlier
                eng.give_back_slot(slots[live.pop(0)])
            got = eng.step([(slots[i], [prompts[i][lens[i] + step]]) for i in live]).cpu().numpy()
            for r, i in enumerate(live):
                at = lens[i] + step
                close(got[r:r + 1], refs[i][1][at:at + 1], dtype, f"{name} request {i} step {step}", refs[i][2][at:at + 1])
        for i in live:
            eng.give_back_slot(slots[i])
    assert eng.slots_free() == 4


@pytest.mark.parametrize("B", [5, 20, 40])
def test_batches_on_every_kernel_family(B):
    """Decode steps of few rows, of 17 to 32 and of more: each row against the same request alone."""
    eng, cfg, W = engine("tiled", "bfloat16", n_slots=B, max_tokens=64 * B)
    refs = [reference("tiled", 60 + i % 3, 20 + 3 * (i % 3)) for i in range(B)]
    lens = [len(r[0]) - 6 - i % 4 for i, r in enumerate(refs)]
    slots = [eng.take_slot() for _ in range(B)]
    eng.step([(s, r[0][:n]) for s, r, n in zip(slots, refs, lens)], want="none")
    for j in range(6):
        got = eng.step([(s, [r[0][n + j]]) for s, r, n in zip(slots, refs, lens)]).cpu().numpy()
        for i in range(B):
            at = lens[i] + j
            close(got[i:i + 1], refs[i][1][at:at + 1], "bfloat16", f"request {i} of {B} step {j}", refs[i][2][at:at + 1])


def test_windows_over_shared_latents_give_pages_back():
    """A source's cache reaches as far back as the widest of its readers sees (37 itself, 64 the reader): pages in front of
    that go back to the pool as the sequence grows and are used by another sequence; a source that some layer reads
    without a window keeps everything."""
    eng, cfg, W = engine("mixed", "float32", n_slots=2, max_tokens=700)
    toks, ref, _ = reference("mixed", 40, 330)
    other, ref_other, _ = reference("mixed", 41, 100)
    windows = {e: eng.cache.groups[g].need.window for e, (g, _) in eng.cache.group_of.items()}
    assert windows == {0: 64, 1: None, 3: None, 5: None}
    g = eng.cache.group_of[0][0]
    a = eng.take_slot()
    rows = [eng.step([(a, toks[:150])], want="all").cpu().numpy()]
    assert len([p for p in eng.cache.slots.pages[a][g] if p]) <= 2       # only the last pages are still held
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


@pytest.mark.parametrize("name, dtype", [("mixed", "float32"), ("reordered", "float32"), ("tiled", "bfloat16")])
def test_long_decoding(name, dtype):
    eng, cfg, W = engine(name, dtype)
    toks, ref, alone = reference(name, 4, 400)
    s = eng.take_slot()
    rows = [eng.step([(s, toks[:2])], want="all").cpu().numpy()]
    for t in toks[2:]:
        rows.append(eng.step([(s, [t])]).cpu().numpy())
    close(np.concatenate(rows), ref, dtype, name, alone)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("reader", [0, 1])
def test_one_loud_token_at_the_edge_of_a_window(reader, dtype):
    """One token's latent is far longer than any other and every query points to it: the last position that sees it and
    the first that does not, through the source's own window or (``reader``) through a wider one of a layer that reads
    the same latents, whose own weights make the other layer's output vanish."""
    from gpullama3_java_amd.engine import Engine
    cfg = decoder(120, 128, 1e-5, 1.0, 1.0, 0, [latent(4, 32, 32, 64, 1.0, 70, None), latent(4, 32, 32, 64, 1.0, 101, None, kv_from=0)])
    W = {k: np.array(v) for k, v in P.make_weights(cfg, 9).items()}
    loud, at, size = 5, 40, [70, 101][reader]
    W["embed"][loud] = 0.0
    W["embed"][loud, 0] = 12.0
    W["embed"][:, 1] = np.where(np.arange(cfg["vocab"]) == loud, 0.0, 2.0)
    W["l0.norm1"][:] = W["l1.norm1"][:] = 1.0
    W["l0.mix.dkv"][:, 0] = np.where(np.arange(64) < 32, 3.0, 0.0)              # the loud token's latent: its first half
    for i in (0, 1):
        W[f"l{i}.mix.uk"][:, :32] = 0.1
        W[f"l{i}.mix.q"][:, 1] = 0.25                                            # everyone else's queries meet such keys
        if i != reader:
            W[f"l{i}.mix.o"][:] = 0.0
    W = {k: bf16_exact(v) for k, v in W.items()}
    folder = tempfile.mkdtemp(prefix="banazen-far-")
    write_model(folder, cfg, W)
    rng = np.random.default_rng(3)
    toks = [int(t) for t in rng.integers(6, cfg["vocab"], 180)]
    toks[at] = loud
    last = at + size - 1
    ref = P.forward(cfg, W, toks)
    quiet = list(toks)
    quiet[at] = 6
    moved = row_errors(ref, P.forward(cfg, W, quiet))
    assert moved[last] > 0.1 and moved[last + 1] == 0.0      # the plain logits: seen, then not
    tol = {"float32": 5e-5, "bfloat16": 0.04}[dtype]
    eng = Engine.from_folder(folder, dtype=dtype, max_tokens=1024, n_slots=4)
    s = eng.take_slot()
    whole = row_errors(eng.step([(s, toks)], want="all").cpu().numpy(), ref)
    s = eng.take_slot()
    rows = [eng.step([(s, toks[:at + 1])], want="all").cpu().numpy()] + [eng.step([(s, [t])]).cpu().numpy() for t in toks[at + 1:]]
    decoded = row_errors(np.concatenate(rows), ref)
    for e in (whole, decoded):
        assert np.median(e) < tol and e[last - 1:last + 3].max() < max(tol, moved[last] / 10), e[last - 1:last + 3]


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_far_token_stays_in_the_state(dtype):
    """A delta rule that hardly decays and an attention over all earlier keys both still show one token hundreds of
    positions later: another token in its place moves the last logits, and the engine follows, prompt and decoded."""
    from gpullama3_java_amd.engine import Engine
    cfg = decoder(100, 64, 1e-5, 1.0, 1.0, 8, [sides((4, 2, 16, 16, 3, (100.0, 16), 0.3), (4, 2, 16, 16, 3), None)])
    W = {k: np.array(v) for k, v in P.make_weights(cfg, 5).items()}
    W["l0.mix.right.A_log"][:] = -7.0
    W["l0.mix.right.b"][:] *= 3.0
    W = {k: bf16_exact(v) for k, v in W.items()}
    folder = tempfile.mkdtemp(prefix="banazen-state-")
    write_model(folder, cfg, W)
    rng = np.random.default_rng(8)
    toks = [int(t) for t in rng.integers(0, 8, 330)]
    toks[3] = 90
    toks[-1] = 90                                             # the same key once more: what was written under it is read
    ref = P.forward(cfg, W, toks)
    other = list(toks)
    other[3] = 91
    assert row_errors(ref, P.forward(cfg, W, other))[-1] > 3e-3
    alone = rounding(cfg, W, toks, ref)
    eng = Engine.from_folder(folder, dtype=dtype, max_tokens=1024, n_slots=2)
    s = eng.take_slot()
    close(eng.step([(s, toks)], want="all").cpu().numpy(), ref, dtype, "whole", alone)
    s = eng.take_slot()
    rows = [eng.step([(s, toks[:250])], want="all").cpu().numpy()] + [eng.step([(s, [t])]).cpu().numpy() for t in toks[250:]]
    close(np.concatenate(rows), ref, dtype, "decoded", alone)


def test_every_fast_path_gives_the_same_numbers_within_rounding():
    """A bfloat16 engine without one family of fast paths after another."""
    _, cfg, W = model("tiled")
    toks, ref, alone = reference("tiled", 2, 200)
    for without in ("fused", "attn_decode,attn_prefill", "tiled", "mfma", "skinny,wide"):
        eng, _, _ = engine("tiled", "bfloat16", without=without)
        s = eng.take_slot()
        rows = [eng.step([(s, toks[:120])], want="all").cpu().numpy()] + [eng.step([(s, [t])]).cpu().numpy() for t in toks[120:150]]
        close(np.concatenate(rows), ref[:150], "bfloat16", f"tiled without {without}", alone[:150])


def test_greedy_generation_through_the_scheduler():
    """The engine's own entry point and scheduler: three prompts of unequal lengths, greedy, in 32-bit (a bfloat16
    engine may choose another expert on a close call of a token that it generated itself)."""
    eng, cfg, W = engine("mixed", "float32")
    prompts = [tokens("mixed", 20, 5), tokens("mixed", 21, 45), tokens("mixed", 22, 1)]
    out = eng.generate(prompts, max_new_tokens=20, temperature=0.0)
    for p, r in zip(prompts, out):
        assert len(r.tokens) == 20
        logits = P.forward(cfg, W, list(p) + r.tokens)
        for j, t in enumerate(r.tokens):
            row = logits[len(p) - 1 + j]
            assert t == int(np.argmax(row)) or row.max() - row[t] < 1e-4 * np.abs(row).max(), (len(p), j, t)
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


def test_a_model_of_random_weights_runs(tmp_path):
    """The random-weights mode: inner sizes that no weights give yet are chosen, written, and read back from the shapes."""
    import gpullama3_java_amd as g
    from gpullama3_java_amd.engine import Engine
    cfg = g.config_from_dict(TILED)
    g.write_random_model(str(tmp_path), cfg, 7, norm_std=0.05)
    eng = Engine.from_folder(str(tmp_path), dtype="bfloat16", max_tokens=256, n_slots=2)
    assert len(eng.generate([[1, 2, 3]], max_new_tokens=4, temperature=0.0)[0].tokens) == 4


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
    """A configuration drawn from a seed: widths, head counts and sizes that no tile need divide, layers in any order,
    readers of earlier latents with windows and heads of their own, groups, experts and shared experts of any size, or
    none of each. Returns (configuration, the inner sizes per layer)."""
    rng = np.random.default_rng([seed, 91])
    pick = lambda *a: a[int(rng.integers(0, len(a)))]

    def mlp():
        kind = rng.random()
        if kind < 0.15:
            return None
        if kind < 0.4:
            return dense(int(pick(16, 40, 66, 100, 128)))
        count = int(pick(1, 2, 3, 4))
        experts = count * int(pick(1, 2, 3, 4))
        keep = int(rng.integers(1, count + 1))
        top = int(rng.integers(1, min(4, keep * experts // count) + 1))
        ff, limit = int(pick(8, 24, 33, 40, 64)), float(pick(0.5, 1.0, 3.0))
        shared = pick(None, (ff, limit), (int(pick(16, 24, 72)), float(pick(0.3, 2.0))))
        return moe(experts, top, ff, limit, float(pick(0.5, 1.0, 2.5)), pick(None, (count, keep), (count, keep)) if top <= keep else (count, keep), shared)

    layers, sources = [], []
    for i in range(int(rng.integers(2, 6))):
        size, scale = pick(None, 1, 2, 9, 33, 64, 65, 100), lambda n: float(n ** -0.5 * rng.uniform(0.7, 1.3))
        if rng.random() < 0.45:
            G, D, Dv = int(pick(1, 2, 3)), int(pick(8, 10, 16, 32, 40, 64, 140)), int(pick(8, 12, 32, 64, 100))
            rot = pick(None, (float(pick(20.0, 1000.0, 5e5)), D), (300.0, 2 * int(rng.integers(1, D // 2 + 1))))
            Gr = int(pick(1, 2, 3))
            layers.append(sides((G * int(pick(1, 2, 4)), G, D, Dv, int(pick(1, 2, 3, 4, 6)), rot, scale(D) * 0.6),
                                (Gr * int(pick(1, 2)), Gr, int(pick(4, 16, 20, 32, 64, 96)), int(pick(8, 16, 24, 64)), int(pick(1, 2, 4, 5))), mlp()))
            continue
        H, D, Dv = int(pick(1, 2, 3, 4, 8)), int(pick(6, 8, 16, 32, 40)), int(pick(8, 12, 16, 64))
        if sources and rng.random() < 0.6:
            j, rank = pick(*sources)
            layers.append(latent(H, D, Dv, rank, scale(D), size, mlp(), kv_from=j))
        else:
            rank = int(pick(16, 24, 32, 40, 64, 96, 300))
            sources.append((i, rank))
            layers.append(latent(H, D, Dv, rank, scale(D), size, mlp()))
    inner = [(int(pick(3, 8, 24, 40)), int(pick(4, 16, 33, 64))) for _ in layers]
    return decoder(int(pick(97, 150, 256, 301)), int(pick(48, 64, 72, 90, 100, 104, 128)), float(pick(1e-6, 1e-5)), float(pick(0.5, 1.0, 4.0)),
                   float(pick(0.5, 1.0, 2.0)), int(pick(0, 6, 16, 33)), layers), inner


@pytest.mark.parametrize("seed", range(16))
def test_seeded_random_configurations(seed, tmp_path):
    """Whole, in portions with the last tokens one by one, and as one of a batch of three: 32-bit against the plain
    implementation to rounding, bfloat16 within three times what rounding alone does to the same row."""
    from gpullama3_java_amd.engine import Engine
    cfg, inner = random_config(seed)
    W = P.make_weights(cfg, seed, lambda i: inner[i])
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
