"""A plain, slow implementation of the Banazen decoder in numpy float64, one function per mechanism, written from the
design's equations and sharing nothing with the package: what the GPU tests compare the engine with.

Notation: T tokens of ONE sequence; W maps a stored tensor name to a float array; linear weights are [out, in].
A ``Sequence`` keeps what the design carries from token to token and can be fed in pieces.

Every layer reads one norm of its residual row twice: x <- x + mixer(h) + ff(h). Behind that a small network of the
token's own row of a second embedding table adds a normed vector. A mixer is either an attention over cached latents in
a sliding window, possibly over an earlier layer's latents, or two mixers side by side: an attention behind short
convolutions, and a gated delta rule that decays each key channel by itself.
"""
from __future__ import annotations

import math
import zlib

import numpy as np


# ----------------------------------------------------------------- small functions
def rms_unit(x, eps):
    x = np.asarray(x, np.float64)
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps)


def rms_norm(x, w, eps):
    return rms_unit(x, eps) * np.asarray(w, np.float64)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-np.asarray(z, np.float64)))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.logaddexp(0.0, z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def exact(a):
    return a


def to_16_bits(a):
    """Rounded to bfloat16: what a 16-bit engine does to the activations between its parts. Every function here takes
    such a rounding as ``r`` (``exact``: none), so that the error that rounding alone makes in a model can be known."""
    import torch
    return torch.as_tensor(np.asarray(a, np.float64)).to(torch.bfloat16).double().numpy()


def linear(x, w):
    return np.asarray(x, np.float64) @ np.asarray(w, np.float64).T


def short_conv(u, w, held=None):
    """u [T, C] over time, w [C, taps] (the last column is the current token's), ``held`` the taps - 1 inputs before
    u[0], oldest first (None: zeros). Returns (the sums [T, C], the new held inputs)."""
    T, taps = u.shape[0], w.shape[1]
    held = np.zeros((taps - 1, u.shape[1])) if held is None else held
    past = np.concatenate([held, u])
    y = sum(past[j:j + T] * w[:, j] for j in range(taps))
    return y, past[len(past) - (taps - 1):]


def rotate(x, positions, dims, base):
    """x [T, heads, D]: the pairs (2i, 2i + 1) of the first ``dims`` elements turned by position * base^(-2i/dims)."""
    out = np.array(x, np.float64)
    for i in range(dims // 2):
        a = np.asarray(positions, np.float64)[:, None] * base ** (-2.0 * i / dims)
        u, v = x[:, :, 2 * i], x[:, :, 2 * i + 1]
        out[:, :, 2 * i] = u * np.cos(a) - v * np.sin(a)
        out[:, :, 2 * i + 1] = v * np.cos(a) + u * np.sin(a)
    return out


def softmax_over(q, keys, values, scale):
    """One query over the keys it sees."""
    s = keys @ q * scale
    e = np.exp(s - s.max())
    return (e / e.sum()) @ values


def first_seen(i, size):
    """The first position that position i sees."""
    return 0 if size is None else max(0, i - size + 1)


# ----------------------------------------------------------------- the mixers
def latents(h, W, p, eps, r=exact):
    """What a layer with latents of its own caches for its tokens."""
    return r(rms_norm(linear(h, W[p + "dkv"]), W[p + "dkv.norm"], eps))


def latent_attention(h, positions, W, p, m, c, r=exact):
    """``c``: the latents [n, kv_rank] of all positions so far, this piece's included."""
    T, H, D, Dv = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = r(linear(h, W[p + "q"])).reshape(T, H, D)
    k = r(linear(c, W[p + "uk"])).reshape(-1, H, D)
    v = r(linear(c, W[p + "uv"])).reshape(-1, H, Dv)
    size = (m.get("mask") or {}).get("size")
    out = np.zeros((T, H, Dv))
    for t, i in enumerate(int(x) for x in positions):
        lo = first_seen(i, size)
        for a in range(H):
            out[t, a] = softmax_over(q[t, a], k[lo:i + 1, a], v[lo:i + 1, a], m["scale"])
    return linear(r(out).reshape(T, H * Dv), W[p + "o"])


def conv_attention(h, positions, W, p, m, eps, state, r=exact):
    """``state``: {"q", "k", "v": held inputs of the convolutions, "keys", "values"}, empty at a sequence's start."""
    T, H, G, D, Dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    u = {}
    for n in ("q", "k", "v"):
        u[n], state[n] = short_conv(r(linear(h, W[p + n])), W[p + n + ".conv"], state.get(n))
    q, k, v = u["q"].reshape(T, H, D), u["k"].reshape(T, G, D), r(u["v"]).reshape(T, G, Dv)
    rot = m.get("rot")
    if rot is not None:
        q, k = (rotate(x, positions, rot["dims"], rot["base"]) for x in (q, k))
    q, k = r(rms_unit(q, eps)), r(rms_unit(k, eps))
    state["keys"] = k if "keys" not in state else np.concatenate([state["keys"], k])
    state["values"] = v if "values" not in state else np.concatenate([state["values"], v])
    out = np.zeros((T, H, Dv))
    for t, i in enumerate(int(x) for x in positions):
        for a in range(H):
            g = a // (H // G)
            out[t, a] = softmax_over(q[t, a], state["keys"][:i + 1, g], state["values"][:i + 1, g], m["scale"])
    return linear(r(out).reshape(T, H * Dv), W[p + "o"])


def unit_length(x, eps=1e-6):
    return x / np.sqrt((x * x).sum(-1, keepdims=True) + eps)


def delta_rule(q, k, v, g, beta, S):
    """One head: q, k, g [T, D], v [T, Dv], beta [T], S [D, Dv]. Returns (o [T, Dv], S)."""
    o = np.zeros((q.shape[0], v.shape[1]))
    for t in range(q.shape[0]):
        S = g[t][:, None] * S
        S = S + np.outer(k[t], beta[t] * (v[t] - S.T @ k[t]))
        o[t] = S.T @ q[t]
    return o, S


def delta_decay(h, W, p, H, D, r=exact):
    """The factor on each row of every head's matrix, [T, H, D]."""
    a = linear(r(linear(h, W[p + "a1"])), W[p + "a2"]) + W[p + "dt_bias"]
    return np.exp(-np.exp(W[p + "A_log"])[:, None] * softplus(a.reshape(-1, H, D)))


def delta_mixer(h, W, p, m, eps, state, r=exact):
    """``state``: {"q", "k", "v": held inputs, "S": [H, D, Dv]}, empty at a sequence's start."""
    T, H, G, D, Dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    u = {}
    for n in ("q", "k", "v"):
        y, state[n] = short_conv(r(linear(h, W[p + n])), W[p + n + ".conv"], state.get(n))
        u[n] = r(silu(y))
    q, k, v = u["q"].reshape(T, G, D), u["k"].reshape(T, G, D), u["v"].reshape(T, H, Dv)
    q, k = unit_length(q) * D ** -0.5, unit_length(k)
    beta = sigmoid(linear(h, W[p + "b"]))
    g = delta_decay(h, W, p, H, D, r)
    S = state.get("S", np.zeros((H, D, Dv)))
    o, S_new = np.zeros((T, H, Dv)), np.zeros((H, D, Dv))
    for a in range(H):
        c = a // (H // G)
        o[:, a], S_new[a] = delta_rule(q[:, c], k[:, c], v[:, a], g[:, a], beta[:, a], S[a])
    state["S"] = S_new
    gate = sigmoid(linear(r(linear(h, W[p + "g1"])), W[p + "g2"])).reshape(T, H, Dv)
    return linear(r(rms_norm(o, W[p + "norm"], eps) * gate).reshape(T, H * Dv), W[p + "o"])


def two_mixers(h, positions, W, p, m, eps, state, r=exact):
    left = conv_attention(h, positions, W, p + "left.", m["left"], eps, state.setdefault("left", {}), r)
    right = delta_mixer(h, W, p + "right.", m["right"], eps, state.setdefault("right", {}), r)
    return 0.5 * (rms_norm(left, W[p + "left.out"], eps) + rms_norm(right, W[p + "right.out"], eps))


# ----------------------------------------------------------------- feed-forward
def dense(h, W, p, r=exact):
    return linear(r(silu(linear(h, W[p + "gate"])) * linear(h, W[p + "up"])), W[p + "down"])


def expert(h, W, p, limit, r=exact):
    g = np.minimum(linear(h, W[p + "gate"]), limit)
    u = np.clip(linear(h, W[p + "up"]), -limit, limit)
    return linear(r(g * sigmoid(1.702 * g) * (u + 1.0)), W[p + "down"])


def choose(c, router, s=None):
    """The chosen experts of ONE token from its choice scores c [experts], and the margin of the choice: by how much the
    last group kept and the last expert chosen lie above the next ones, with ``s`` (the scores themselves) as a fraction of
    the larger score of the two that compete, which is what a rounding moves."""
    E, top, groups = router["experts"], router["top"], router.get("groups") or {"count": 1, "keep": 1}
    n, keep = groups["count"], groups["keep"]

    def margin(a, b):
        return (c[a] - c[b]) / (1.0 if s is None else max(s[a], s[b]))

    leaders = c.reshape(n, E // n).argmax(-1) + np.arange(n) * (E // n)
    order = np.argsort(-c[leaders], kind="stable")
    open_ = np.zeros(n, bool)
    open_[order[:keep]] = True
    left = np.where(np.repeat(open_, E // n), c, -np.inf)
    ranked = np.argsort(-left, kind="stable")
    gap = margin(leaders[order[keep - 1]], leaders[order[keep]]) if keep < n else math.inf
    if top < E and left[ranked[top]] > -np.inf:
        gap = min(gap, margin(ranked[top - 1], ranked[top]))
    return ranked[:top], gap


def route(h, W, p, router):
    """Per token: the chosen experts, their weights, and the margin of the choice."""
    z = linear(h, W[p + "router"])
    s = np.exp(z - z.max(-1, keepdims=True))
    s = s / s.sum(-1, keepdims=True)
    out = []
    for row in s:
        idx, gap = choose(row + W[p + "correction"], router, row)
        out.append((idx, row[idx] / (row[idx].sum() + 1e-20) * router["scale"], gap))
    return out


def mixture(h, W, p, mlp, note=None, r=exact):
    """``note`` (a list) receives the margin of every token's choice."""
    out = np.zeros_like(h, dtype=np.float64)
    for t, (idx, w, gap) in enumerate(route(h, W, p, mlp["router"])):
        if note is not None:
            note.append(gap)
        for e, a in zip(idx, w):
            out[t] += a * expert(h[t:t + 1], W, f"{p}e{e}.", mlp["expert"]["limit"], r)[0]
    if mlp.get("shared") is not None:
        out += sigmoid(linear(h, W[p + "shared.sg"])) * expert(h, W, p + "shared.", mlp["shared"]["limit"], r)
    return out


def feed_forward(h, W, p, mlp, note=None, r=exact):
    return dense(h, W, p, r) if mlp["kind"] == "dense" else mixture(h, W, p, mlp, note, r)


def token_side(x, e, W, p, eps, r=exact):
    """What a token's own row ``e`` [T, dim] of the side table adds to its residual row."""
    g = r(gelu_tanh(linear(r(x), W[p + "gate"])) * e)
    return rms_norm(linear(g, W[p + "proj"]), W[p + "norm"], eps)


# ----------------------------------------------------------------- the decoder
class Sequence:
    """One sequence that is fed in pieces. ``rows`` collects, per piece, the residual rows after every layer."""

    def __init__(self, cfg, W, r=exact):
        self.cfg, self.W, self.r = cfg, {k: np.asarray(v, np.float64) for k, v in W.items()}, r
        self.n = 0
        self.states = [dict() for _ in cfg["layers"]]
        self.rows = []
        self.gaps = []          # of every router's choices so far (``mixture``)

    def copy(self):
        """A sequence that goes on from here by itself (a piece replaces a state's arrays and changes none)."""
        def twin(s):
            return {k: twin(v) if isinstance(v, dict) else v for k, v in s.items()}
        out = Sequence(self.cfg, {}, self.r)
        out.W, out.n, out.states = self.W, self.n, [twin(s) for s in self.states]
        return out

    def feed(self, tokens):
        cfg, W, eps, r = self.cfg, self.W, self.cfg["norm"]["eps"], self.r
        tokens = np.asarray(tokens)
        positions = np.arange(self.n, self.n + len(tokens))
        self.n += len(tokens)
        x = W["embed"][tokens] * cfg["embedding"]["scale"]
        side = (cfg.get("token_side") or {}).get("dim")
        rows = []
        for i, lay in enumerate(cfg["layers"]):
            p, m, state = f"l{i}.", lay["mixer"], self.states[i]
            h = r(rms_norm(x, W[p + "norm1"], eps))
            if lay["type"] == "parallel":
                y = two_mixers(h, positions, W, p + "mix.", m, eps, state, r)
            else:
                if m.get("kv_from") is None:
                    c = latents(h, W, p + "mix.", eps, r)
                    state["c"] = c if "c" not in state else np.concatenate([state["c"], c])
                else:
                    state = self.states[m["kv_from"]]
                y = latent_attention(h, positions, W, p + "mix.", m, state["c"], r)
            if lay.get("mlp") is not None:
                y = y + feed_forward(h, W, p + "mlp.", lay["mlp"], self.gaps, r)
            x = x + y
            if side:
                x = x + token_side(x, W["side.embed"][tokens, i * side:(i + 1) * side], W, p + "side.", eps, r)
            rows.append(x)
        self.rows.append(np.stack(rows))
        return linear(r(rms_norm(x, W["final.norm"], eps)), W["head"]) * cfg.get("logit_scale", 1.0)


def forward(cfg, W, tokens):
    """Logits [T, vocab] of one sequence fed whole."""
    return Sequence(cfg, W).feed(tokens)


# ----------------------------------------------------------------- models for tests
def tensor_shapes(cfg, ranks=lambda i: (8, 12)):
    """Stored name -> shape of every tensor of a model of this design; ``ranks``: a layer's inner sizes of the decay's
    and of the read-out gate's two-step projection, which only the weights give."""
    d, V = cfg["width"], cfg["vocab"]
    out = {"embed": (V, d), "final.norm": (d,), "head": (V, d)}
    side = (cfg.get("token_side") or {}).get("dim")
    if side:
        out["side.embed"] = (V, side * len(cfg["layers"]))
    for i, lay in enumerate(cfg["layers"]):
        p, m, mlp = f"l{i}.", lay["mixer"], lay.get("mlp")
        q = p + "mix."
        out[p + "norm1"] = (d,)
        if lay["type"] == "latent_attention":
            H, D, Dv, R = m["heads"], m["dim"], m["vdim"], m["kv_rank"]
            out.update({q + "q": (H * D, d), q + "uk": (H * D, R), q + "uv": (H * Dv, R), q + "o": (d, H * Dv)})
            if m.get("kv_from") is None:
                out.update({q + "dkv": (R, d), q + "dkv.norm": (R,)})
        else:
            a, b = m["left"], m["right"]
            sizes = {"q": a["heads"] * a["dim"], "k": a["kv_heads"] * a["dim"], "v": a["kv_heads"] * a["vdim"]}
            for n, c in sizes.items():
                out.update({f"{q}left.{n}": (c, d), f"{q}left.{n}.conv": (c, a["conv"])})
            out[q + "left.o"] = (d, a["heads"] * a["vdim"])
            H, D, Dv = b["heads"], b["dim"], b["vdim"]
            sizes = {"q": b["kv_heads"] * D, "k": b["kv_heads"] * D, "v": H * Dv}
            for n, c in sizes.items():
                out.update({f"{q}right.{n}": (c, d), f"{q}right.{n}.conv": (c, b["conv"])})
            ra, rg = ranks(i)
            out.update({q + "right.b": (H, d), q + "right.A_log": (H,), q + "right.norm": (Dv,), q + "right.a1": (ra, d),
                        q + "right.a2": (H * D, ra), q + "right.dt_bias": (H * D,), q + "right.g1": (rg, d),
                        q + "right.g2": (H * Dv, rg), q + "right.o": (d, H * Dv), q + "left.out": (d,), q + "right.out": (d,)})
        if mlp is not None:
            q = p + "mlp."
            forms = [(q, mlp["ff"])] if mlp["kind"] == "dense" else \
                [(f"{q}e{e}.", mlp["expert"]["ff"]) for e in range(mlp["router"]["experts"])]
            if mlp["kind"] == "moe":
                out.update({q + "router": (mlp["router"]["experts"], d), q + "correction": (mlp["router"]["experts"],)})
                if mlp.get("shared") is not None:
                    forms.append((q + "shared.", mlp["shared"]["ff"]))
                    out[q + "shared.sg"] = (1, d)
            for pre, ff in forms:
                out.update({pre + "gate": (ff, d), pre + "up": (ff, d), pre + "down": (d, ff)})
        if side:
            out.update({p + "side.gate": (side, d), p + "side.proj": (d, side), p + "side.norm": (d,)})
    return out


def make_weights(cfg, seed, ranks=lambda i: (8, 12), overrides=None):
    """float32 weights that bfloat16 holds exactly, sized so that every mechanism moves the logits: matrices
    N(0, 1.5/sqrt(fan-in)), norm weights around one, a wide spread of decays, corrections of the size of the scores.
    ``overrides``: name suffix -> factor on a tensor's values."""
    import torch
    out = {}
    for name, shape in tensor_shapes(cfg, ranks).items():
        rng = np.random.default_rng([seed, zlib.crc32(name.encode())])
        last = name.split(".")[-1]
        if last in ("norm1", "norm", "out"):
            a = 1.0 + 0.2 * rng.standard_normal(shape)
        elif last == "A_log":
            a = rng.uniform(-4.0, 0.5, shape)
        elif last == "dt_bias":
            a = rng.uniform(-3.0, 1.0, shape)
        elif last == "conv":
            a = 0.6 * rng.standard_normal(shape)
            a[:, -1] += 0.5
        elif last == "correction":
            a = rng.standard_normal(shape) * (0.5 / shape[0])
        elif name in ("embed", "side.embed"):
            a = 0.7 * rng.standard_normal(shape)
        else:
            a = rng.standard_normal(shape) * (1.5 / np.sqrt(shape[-1]))
        for suffix, factor in (overrides or {}).items():
            if name.endswith(suffix):
                a = a * factor
        out[name] = torch.tensor(a, dtype=torch.float32).to(torch.bfloat16).float().numpy()
    return out


def tokens_with_clear_choices(cfg, W, seed, n, gap=0.12):
    """n token ids drawn from a seed at which no router makes a close call: at every token and layer the margin of the
    groups and of the experts (``choose``) is at least ``gap``, so an engine that rounds to 16 bits chooses the same
    experts."""
    rng = np.random.default_rng([seed, 11])
    seq, out = Sequence(cfg, W), []
    while len(out) < n:
        best = None
        for _ in range(150):
            t = int(rng.integers(0, cfg["vocab"]))
            trial = seq.copy()
            trial.feed([t])
            least = min(trial.gaps) if trial.gaps else math.inf
            if best is None or least > best[0]:
                best = (least, t, trial)
            if least >= gap:
                break
        if best[0] < gap / 4:
            raise RuntimeError("no token without a close call found")
        seq = best[2]
        out.append(best[1])
    return out
