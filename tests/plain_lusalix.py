"""A plain, slow implementation of the Lusalix decoder in numpy float64, one function per mechanism, written from
the design's equations and sharing nothing with the package: what the GPU tests compare the engine with.

Notation: T tokens of ONE sequence; W maps a stored tensor name to a float array; linear weights are [out, in].
A ``Sequence`` keeps what the design carries from token to token (keys and mixed values) and can be fed in pieces.

Pre-norm layers. The mixer is an attention without a rotation: queries are made longer with the position (a
"temperature" that steps up every so many tokens), scores pass a soft cap and lose a slope times the distance, a window
bounds what is seen, values are blended with the first such layer's values of the same token, and the heads' outputs
are gated element by element. The feed-forward is a mixture of gated experts whose weights are plain sigmoids that
multiply the experts' INPUT, beside a shared expert with a gate of its own.
"""
from __future__ import annotations

import math

import numpy as np


# ----------------------------------------------------------------- small functions
def rms_norm(x, w, eps):
    x = np.asarray(x, np.float64)
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps) * np.asarray(w, np.float64)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-np.asarray(z, np.float64)))


def silu(z):
    return z * sigmoid(z)


def exact(a):
    return a


def to_16_bits(a):
    """Rounded to bfloat16: what a 16-bit engine does to the activations between its parts. Every function here takes
    such a rounding as ``r`` (``exact``: none), so that the error that rounding alone makes in a model can be known."""
    import torch
    return torch.as_tensor(np.asarray(a, np.float64)).to(torch.bfloat16).double().numpy()


def linear(x, w):
    return np.asarray(x, np.float64) @ np.asarray(w, np.float64).T


# ----------------------------------------------------------------- the attention's pieces
def temperature(positions, coef, every):
    """The factor on the query at each position: 1 over the first ``every`` positions but one, then a step up at every
    position p with p + 1 a multiple of ``every``."""
    return np.array([1.0 + coef * math.log((int(p) + 1) // every + 1) for p in positions])


def slopes(H):
    return np.array([2.0 ** (-8.0 * (h + 1) / H) for h in range(H)])


def score(q, keys, i, j, m, h):
    """Scores of ONE query (position i, head h, temperature applied) and keys [n, dim] at positions j [n]."""
    s = keys @ q * m["scale"]
    cap = m.get("softcap")
    if cap is not None:
        s = cap * np.tanh(s / cap)
    return s - slopes(m["heads"])[h] * (i - np.asarray(j, np.float64))


def visible(i, size):
    """The first position that position i sees."""
    return 0 if size is None else max(0, i - size + 1)


def blend(v, first, lam):
    return (1.0 - lam) * v + lam * first


def attention(h, positions, W, p, m, state, first=None, r=exact):
    """``state``: {"k": [n, G, dim], "v": [n, G, vdim]} so far. ``first``: None where the layer's values stay as they
    are, else the values of the same tokens that they are blended with. Returns (output, the values as projected)."""
    T = h.shape[0]
    H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = r(linear(h, W[p + "q"])).reshape(T, H, D)
    if m.get("q_temp") is not None:
        q = q * temperature(positions, m["q_temp"]["coef"], m["q_temp"]["every"])[:, None, None]
    k = r(linear(h, W[p + "k"])).reshape(T, G, D)
    own = r(linear(h, W[p + "v"])).reshape(T, G, Dv)
    v = own if first is None else r(blend(own, first, float(W[p + "vmix"])))
    state["k"] = k if "k" not in state else np.concatenate([state["k"], k])
    state["v"] = v if "v" not in state else np.concatenate([state["v"], v])
    size = (m.get("mask") or {}).get("size")
    out = np.zeros((T, H, Dv))
    for t in range(T):
        i = int(positions[t])
        lo = visible(i, size)
        j = np.arange(lo, i + 1)
        for a in range(H):
            g = a // (H // G)
            s = score(q[t, a], state["k"][lo:i + 1, g], i, j, m, a)
            e = np.exp(s - s.max())
            out[t, a] = (e / e.sum()) @ state["v"][lo:i + 1, g]
    y = r(out.reshape(T, H * Dv) * sigmoid(r(linear(h, W[p + "g"]))))
    return linear(y, W[p + "o"]), own


# ----------------------------------------------------------------- feed-forward
def expert(h, W, p, r=exact):
    return linear(r(silu(linear(h, W[p + "gate"])) * linear(h, W[p + "up"])), W[p + "down"])


def route(h, W, p, router):
    """Per token the chosen experts and their scores, which are their weights as they are."""
    s = sigmoid(linear(h, W[p + "router"]))
    idx = np.argsort(-s, axis=-1, kind="stable")[:, :router["top"]]
    return idx, np.take_along_axis(s, idx, -1), s


def mixture(h, W, p, mlp, note=None, r=exact):
    """``note`` (a list) receives, per token, how far the last chosen expert's score lies above the first left out."""
    top = mlp["router"]["top"]
    idx, w, s = route(h, W, p, mlp["router"])
    if note is not None and s.shape[-1] > top:
        ranked = -np.sort(-s, axis=-1)
        note.extend((ranked[:, top - 1] - ranked[:, top]).tolist())
    out = np.zeros_like(h, dtype=np.float64)
    for t in range(h.shape[0]):
        for e, a in zip(idx[t], w[t]):
            out[t] += expert(a * h[t:t + 1], W, f"{p}e{e}.", r)[0]
    if mlp.get("shared") is not None:
        out += sigmoid(linear(h, W[p + "shared.sg"])) * expert(h, W, p + "shared.", r)
    return out


# ----------------------------------------------------------------- the decoder
class Sequence:
    """One sequence that is fed in pieces. ``rows`` collects, per piece, the residual rows after every layer; ``after``
    (optional) is called with (layer, "mixer" or "ffn", the rows)."""

    def __init__(self, cfg, W, after=None, r=exact):
        self.cfg, self.W, self.after, self.r = cfg, {k: np.asarray(v, np.float64) for k, v in W.items()}, after, r
        self.n = 0
        self.states = [dict() for _ in cfg["layers"]]
        self.rows = []
        self.gaps = []          # of every router's choices so far (``mixture``)

    def feed(self, tokens):
        cfg, W, eps, r = self.cfg, self.W, self.cfg["norm"]["eps"], self.r
        positions = np.arange(self.n, self.n + len(tokens))
        self.n += len(tokens)
        x = W["embed"][np.asarray(tokens)] * cfg["embedding"]["scale"]
        rows, first = [], None
        for i, lay in enumerate(cfg["layers"]):
            p, m = f"l{i}.", lay["mixer"]
            mixes = bool(m.get("v_mix"))
            y, own = attention(r(rms_norm(x, W[p + "norm1"], eps)), positions, W, p + "mix.", m, self.states[i],
                               first if mixes else None, r)
            if mixes and first is None:
                first = own
            x = x + y
            if self.after:
                self.after(i, "mixer", x)
            if lay.get("mlp") is not None:
                x = x + mixture(r(rms_norm(x, W[p + "norm2"], eps)), W, p + "mlp.", lay["mlp"], self.gaps, r)
                if self.after:
                    self.after(i, "ffn", x)
            rows.append(x)
        self.rows.append(np.stack(rows))
        return linear(r(rms_norm(x, W["final.norm"], eps)), W["head"])


def forward(cfg, W, tokens):
    """Logits [T, vocab] of one sequence fed whole."""
    return Sequence(cfg, W).feed(tokens)


# ----------------------------------------------------------------- models for tests
def tensor_shapes(cfg):
    """Stored name -> shape of every tensor of a model of this design."""
    d = cfg["width"]
    out = {"embed": (cfg["vocab"], d), "final.norm": (d,), "head": (cfg["vocab"], d)}
    for i, lay in enumerate(cfg["layers"]):
        p, m, mlp = f"l{i}.", lay["mixer"], lay.get("mlp")
        H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        out.update({p + "norm1": (d,), p + "mix.q": (H * D, d), p + "mix.k": (G * D, d), p + "mix.v": (G * Dv, d),
                    p + "mix.g": (H * Dv, d), p + "mix.o": (d, H * Dv)})
        if m.get("v_mix"):
            out[p + "mix.vmix"] = ()
        if mlp is None:
            continue
        q, E = p + "mlp.", mlp["router"]["experts"]
        out.update({p + "norm2": (d,), q + "router": (E, d)})
        forms = [(f"{q}e{e}.", mlp["expert"]["ff"]) for e in range(E)]
        if mlp.get("shared") is not None:
            forms.append((q + "shared.", mlp["shared"]["ff"]))
            out[q + "shared.sg"] = (1, d)
        for pre, ff in forms:
            out.update({pre + "gate": (ff, d), pre + "up": (ff, d), pre + "down": (d, ff)})
    return out


def make_weights(cfg, seed, overrides=None):
    """float32 weights that bfloat16 holds exactly, sized so that every mechanism moves the logits: matrices
    N(0, 1.5/sqrt(fan-in)), norm weights around one, value blends between 0.2 and 0.8. ``overrides``: name suffix ->
    factor on a tensor's values (long queries for the soft cap, for instance)."""
    import zlib
    import torch
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        rng = np.random.default_rng([seed, zlib.crc32(name.encode())])
        last = name.split(".")[-1]
        if last in ("norm1", "norm2", "norm"):
            a = 1.0 + 0.2 * rng.standard_normal(shape)
        elif last == "vmix":
            a = rng.uniform(0.2, 0.8)
        else:
            a = rng.standard_normal(shape) * (1.5 / np.sqrt(shape[-1]))
        for suffix, factor in (overrides or {}).items():
            if name.endswith(suffix):
                a = a * factor
        out[name] = torch.tensor(a, dtype=torch.float32).to(torch.bfloat16).float().numpy()
    return out


def tokens_with_clear_choices(cfg, W, seed, n, gap=0.03):
    """n token ids drawn from a seed at which no router makes a close call: at every token and layer the last chosen
    expert's score lies at least ``gap`` above the first one left out, so an engine that rounds to 16 bits chooses the
    same experts."""
    rng = np.random.default_rng([seed, 11])
    seq, out = Sequence(cfg, W), []
    while len(out) < n:
        best = None
        for _ in range(150):
            t = int(rng.integers(0, cfg["vocab"]))
            trial = Sequence(cfg, {})
            trial.W, trial.n = seq.W, seq.n
            trial.states = [dict(s) for s in seq.states]      # (a piece replaces a state's arrays and changes none)
            trial.feed([t])
            least = min(trial.gaps) if trial.gaps else math.inf
            if best is None or least > best[0]:
                best = (least, t, trial)
            if least >= gap:
                break
        if best[0] < gap / 5:
            raise RuntimeError("no token without a close call found")
        seq = best[2]
        out.append(best[1])
    return out
