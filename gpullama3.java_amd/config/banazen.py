"""Typed configuration of the Banazen decoder, read from its config.json.

Banazen's layers are parallel: one RMS norm whose output feeds mixer and feed-forward, both of which add into the residual
row, and behind them a small network of the token's own row of a side table that adds a normed vector. Mixers:

  latent_attention:  queries W_q h; keys and values expanded per head from an RMS-normed latent of ``kv_rank`` numbers, which
                 is all that is cached; no positions; a sliding window. A layer with ``kv_from`` has no latents of its own
                 and reads that layer's through its own expansions and window;
  parallel:      two mixers side by side, half the sum of their outputs, each RMS-normed over the model width. Left: grouped
                 causal attention whose q, k and v pass a short convolution over time, q and k then a rotation (adjacent
                 pairs, the first ``rot.dims`` elements) and a division by their root mean square. Right: a gated delta rule
                 (short convolutions with silu, unit queries and keys) with one decay per head and key channel and a
                 sigmoid gate, both from two-step projections whose inner sizes only the weights give.

Feed-forward: dense and gated, or a mixture of bounded gated experts chosen by softmax scores plus a correction from the
best groups, beside a shared expert with a factor of its own; or none.

config.json: ``architecture`` "Banazen", ``vocab``, ``width``, ``norm.eps``, ``embedding.scale``, ``logit_scale``,
``token_side.dim`` (absent or null: no side table) and ``layers``, a list of ``{"type", "mixer": {...}, "mlp": {...} | null}``:
  latent_attention: ``heads``, ``dim``, ``vdim``, ``kv_rank``, ``scale``, ``mask``: ``size`` (absent: every earlier key),
                 ``kv_from``: the number of an earlier layer;
  parallel:      ``left``: ``heads``, ``kv_heads``, ``dim``, ``vdim``, ``conv``, ``rot``: ``base``, ``dims`` (absent: none),
                 ``scale``; ``right``: ``heads``, ``kv_heads``, ``dim``, ``vdim``, ``conv``;
  mlp:           ``{"kind": "dense", "ff"}`` or ``{"kind": "moe", "router": {"experts", "top", "scale", "groups": {"count",
                 "keep"}}, "expert": {"ff", "limit"}, "shared": {"ff", "limit"} | null}``; without ``scale``, ``groups`` or
                 ``limit`` (absent or null) there is none.
The folder names no longest sequence: ``max_positions`` (ours, optional) bounds it, else ``DEFAULT_MAX_POSITIONS``.
Tensor names: ``embed``, ``side.embed``, ``final.norm``, ``head``, and per layer i ``l<i>.norm1``, ``l<i>.mix.*``,
``l<i>.mlp.*``, ``l<i>.side.*``.
"""
from __future__ import annotations

import copy
from dataclasses import dataclass, replace
from typing import Optional

from .registry import ConfigError, _as_ids, register_architecture
from .specs import (AttentionSpec, BlockSpec, ExpertSpec, GatedDeltaSpec, GatedFeedForwardSpec, LatentAttentionSpec,
                    ModelSpec, NormSpec, RotarySpec, RoutedFeedForwardSpec, Run, SideBySideSpec, TokenSideSpec)

# what the design fixes
DENSE_ACTIVATION = "silu"
EXPERT_ACTIVATION = "quick_gelu"      # z * sigmoid(1.702 z)
EXPERT_UP_SHIFT = 1.0
ROUTER_SUM_EPS = 1e-20
UNIT_EPS = 1e-6                       # inside the root of the delta rule's unit queries and keys
SIDES_WEIGHT = 0.5                    # of the sum of two mixers side by side
DEFAULT_MAX_POSITIONS = 1 << 17       # a folder sets no bound on a sequence's length; the engine's caches need one
TYPES = ("latent_attention", "parallel")


def _int(d, key, where, least=1):
    v = d.get(key) if isinstance(d, dict) else None
    if isinstance(v, bool) or not isinstance(v, int) or v < least:
        raise ConfigError(f"config.json: {where}'{key}' must be an integer of at least {least}, found {v!r}")
    return v


def _number(d, key, where):
    v = d.get(key) if isinstance(d, dict) else None
    if isinstance(v, bool) or not isinstance(v, (int, float)):
        raise ConfigError(f"config.json: {where}'{key}' must be a number, found {v!r}")
    return float(v)


def _positive(d, key, where):
    v = _number(d, key, where)
    if not v > 0:
        raise ConfigError(f"config.json: {where}'{key}' must be a positive number, found {v!r}")
    return v


def _check_heads(m, where):
    heads, kv = _int(m, "heads", where), _int(m, "kv_heads", where)
    if heads % kv:
        raise ConfigError(f"config.json: {where}{heads} heads are not a multiple of {kv} kv_heads")
    _int(m, "dim", where), _int(m, "vdim", where), _int(m, "conv", where)


def _check_latent(i, m, layers, where):
    for k in ("heads", "dim", "vdim", "kv_rank"):
        _int(m, k, where)
    _positive(m, "scale", where)
    if m.get("mask") is not None:
        _int(m["mask"], "size", where + "mask: ")
    if m.get("kv_from") is None:
        return
    j = _int(m, "kv_from", where, 0)
    other = layers[j] if j < i else None
    if other is None or other.get("type") != "latent_attention" or other["mixer"].get("kv_from") is not None:
        raise ConfigError(f"config.json: {where}'kv_from' {j} is not an earlier layer with latents of its own")
    if other["mixer"]["kv_rank"] != m["kv_rank"]:
        raise ConfigError(f"config.json: {where}latents of {m['kv_rank']} read from layer {j}, whose latents have "
                          f"{other['mixer']['kv_rank']}")


def _check_parallel(m, where):
    for side in ("left", "right"):
        if not isinstance(m.get(side), dict):
            raise ConfigError(f"config.json: {where}'{side}' must be an object")
        _check_heads(m[side], where + side + ": ")
    left = m["left"]
    _positive(left, "scale", where + "left: ")
    if left.get("rot") is not None:
        w = where + "left: rot: "
        _positive(left["rot"], "base", w)
        dims = _int(left["rot"], "dims", w, 2)
        if dims % 2 or dims > left["dim"]:
            raise ConfigError(f"config.json: {w}'dims' must be an even number up to the heads' {left['dim']}, found {dims}")


def _check_mlp(mlp, where):
    if mlp is None:
        return
    if not isinstance(mlp, dict) or mlp.get("kind") not in ("dense", "moe"):
        raise ConfigError(f"config.json: {where}'mlp' must be null or an object of kind 'dense' or 'moe'")
    if mlp["kind"] == "dense":
        _int(mlp, "ff", where)
        return
    r, w = mlp.get("router"), where + "router: "
    experts, top = _int(r, "experts", w), _int(r, "top", w)
    if r.get("scale") is not None:
        _number(r, "scale", w)
    can = experts
    if r.get("groups") is not None:
        count, keep = _int(r["groups"], "count", w + "groups: "), _int(r["groups"], "keep", w + "groups: ")
        if experts % count or keep > count:
            raise ConfigError(f"config.json: {w}the best {keep} of {count} groups of {experts} experts")
        can = keep * (experts // count)
    if top > can:
        raise ConfigError(f"config.json: {w}the {top} largest of {can} experts")
    for k in ("expert", "shared"):
        if k == "expert" or mlp.get(k) is not None:
            _int(mlp.get(k), "ff", where + k + ": ")
            if mlp[k].get("limit") is not None:
                _positive(mlp[k], "limit", where + k + ": ")


@dataclass(frozen=True)
class BanazenConfiguration:
    vocab_size: int
    width: int
    norm_eps: float
    embedding_scale: float
    logit_scale: float
    side_dim: int                           # 0: no side table
    layers: tuple                           # the checked entries of config.json's 'layers', as they stand there
    ranks: tuple = ()                       # per layer (inner size of the decay's projection, of the gate's), from the weights
    max_positions: int = DEFAULT_MAX_POSITIONS
    context_length: Optional[int] = None
    stop_ids: tuple = ()
    architecture: str = "Banazen"

    @property
    def max_position_embeddings(self):
        return self.max_positions if self.context_length is None else min(self.context_length, self.max_positions)

    @property
    def hidden_size(self):
        return self.width

    def __hash__(self):
        return hash((self.vocab_size, self.width, self.norm_eps, self.embedding_scale, self.logit_scale, self.side_dim,
                     repr(self.layers), self.ranks, self.max_positions, self.context_length, self.stop_ids))

    # ------------------------------------------------------------------ reading
    @classmethod
    def from_dict(cls, d):
        layers_in = d.get("layers")
        if not isinstance(layers_in, list) or not layers_in:
            raise ConfigError("config.json: 'layers' must be a list with at least one layer")
        for i, lay in enumerate(layers_in):
            where = f"layers[{i}]: "
            if not isinstance(lay, dict) or lay.get("type") not in TYPES:
                raise ConfigError(f"config.json: {where}'type' must be one of {TYPES}")
            if not isinstance(lay.get("mixer"), dict):
                raise ConfigError(f"config.json: {where}'mixer' must be an object")
            if lay["type"] == "parallel":
                _check_parallel(lay["mixer"], where)
            else:
                _check_latent(i, lay["mixer"], layers_in, where)
            _check_mlp(lay.get("mlp"), where + "mlp: ")
        ranks = d.get("inner_sizes") or ()
        return cls(vocab_size=_int(d, "vocab", ""), width=_int(d, "width", ""),
                   norm_eps=_positive(d.get("norm"), "eps", "norm: "),
                   embedding_scale=_number(d["embedding"], "scale", "embedding: ") if d.get("embedding") is not None else 1.0,
                   logit_scale=_number(d, "logit_scale", "") if d.get("logit_scale") is not None else 1.0,
                   side_dim=_int(d["token_side"], "dim", "token_side: ") if d.get("token_side") is not None else 0,
                   layers=tuple(copy.deepcopy(layers_in)), ranks=tuple(tuple(int(n) for n in r) for r in ranks),
                   max_positions=_int(d, "max_positions", "") if d.get("max_positions") is not None else DEFAULT_MAX_POSITIONS,
                   stop_ids=_as_ids(d.get("eos_token_id")))

    def to_dict(self):
        d = {"architecture": self.architecture, "vocab": self.vocab_size, "width": self.width,
             "norm": {"eps": self.norm_eps}, "embedding": {"scale": self.embedding_scale}, "logit_scale": self.logit_scale,
             "layers": copy.deepcopy(list(self.layers))}
        if self.side_dim:
            d["token_side"] = {"dim": self.side_dim}
        if self.ranks:      # (ours: for a model whose weights are still to be drawn)
            d["inner_sizes"] = [list(r) for r in self.ranks]
        if self.max_positions != DEFAULT_MAX_POSITIONS:
            d["max_positions"] = self.max_positions
        if self.stop_ids:
            d["eos_token_id"] = list(self.stop_ids)
        return d

    def with_tensor_shapes(self, shapes):
        """Sizes that only the weights give: the inner sizes of the delta rule's two-step projections
        (``l<i>.mix.right.a1`` and ``.g1`` are [rank, width]). ``shapes``: stored name -> shape."""
        ranks = []
        for i in range(len(self.layers)):
            a, g = (shapes.get(f"l{i}.mix.right.{n}1") for n in ("a", "g"))
            ranks.append(tuple(int(s[0]) if s is not None and len(s) == 2 else 0 for s in (a, g)))
        return replace(self, ranks=tuple(ranks)) if any(any(r) for r in ranks) else self

    # ------------------------------------------------------------------ what the engine asks
    def chat_format(self, tokenizer):
        raise ConfigError("a Banazen model folder brings no chat format: give the prompt as token ids")

    def with_stop_ids(self, ids):
        return replace(self, stop_ids=tuple(ids))

    def with_context_length(self, n):
        if n is None or n < 0:
            return self
        return replace(self, context_length=min(n, self.max_positions))

    def run_order(self):
        return tuple(Run(layer=i, reads=lay["mixer"].get("kv_from") if lay["type"] == "latent_attention" else None)
                     for i, lay in enumerate(self.layers))

    def _inner(self, i):
        """The inner sizes of layer i's two-step projections: the weights', else something to draw weights with."""
        a, g = self.ranks[i] if i < len(self.ranks) else (0, 0)
        return a or max(8, self.width // 16), g or max(8, self.width // 16)

    @staticmethod
    def _window(m):
        return m["mask"]["size"] if m.get("mask") is not None else None

    def _latent(self, i, m):
        p = f"l{i}.mix."
        names = {k: p + k for k in ("q", "uk", "uv", "o")}
        kept = None
        if m.get("kv_from") is None:
            names.update({"dkv": p + "dkv", "dkv_norm": p + "dkv.norm"})
            readers = [self._window(lay["mixer"]) for lay in self.layers
                       if lay["type"] == "latent_attention" and lay["mixer"].get("kv_from") == i]
            windows = readers + [self._window(m)]
            kept = 0 if any(w is None for w in windows) else max(windows)
        return LatentAttentionSpec(
            hidden=self.width, n_heads=m["heads"], head_dim=m["dim"], v_head_dim=m["vdim"], kv_rank=m["kv_rank"],
            scale=float(m["scale"]), norm_eps=self.norm_eps, names=names, window=self._window(m), kept_window=kept)

    def _parallel(self, i, m):
        p, a, b = f"l{i}.mix.", m["left"], m["right"]
        left = {k: p + "left." + k for k in ("q", "k", "v", "o")}
        left.update({k + "_conv": p + f"left.{k}.conv" for k in ("q", "k", "v")})
        rot = None
        if a.get("rot") is not None:
            rot = RotarySpec(head_dim=a["rot"]["dims"], theta=float(a["rot"]["base"]), pairing="adjacent",
                             max_positions=self.max_position_embeddings)
        right = {k: p + "right." + k for k in ("q", "k", "v", "b", "A_log", "norm", "a1", "a2", "dt_bias", "g1", "g2", "o")}
        right.update({k + "_conv": p + f"right.{k}.conv" for k in ("q", "k", "v")})
        ra, rg = self._inner(i)
        return SideBySideSpec(
            hidden=self.width, norm_eps=self.norm_eps, weight=SIDES_WEIGHT,
            names={"left_norm": p + "left.out", "right_norm": p + "right.out"},
            left=AttentionSpec(hidden=self.width, n_heads=a["heads"], n_kv_heads=a["kv_heads"], head_dim=a["dim"],
                               v_head_dim=a["vdim"], position=rot, scale=float(a["scale"]), conv_taps=a["conv"],
                               qk_norm_eps=self.norm_eps, names=left),
            right=GatedDeltaSpec(hidden=self.width, n_heads=b["heads"], n_kv_heads=b["kv_heads"], key_dim=b["dim"],
                                 value_dim=b["vdim"], conv_taps=b["conv"], unit_eps=UNIT_EPS, norm_eps=self.norm_eps,
                                 decay_rank=ra, gate_rank=rg, gate_activation="sigmoid", names=right))

    def _ffn(self, i, mlp):
        q = f"l{i}.mlp."
        if mlp["kind"] == "dense":
            return GatedFeedForwardSpec(hidden=self.width, intermediate=mlp["ff"], activation=DENSE_ACTIVATION,
                                        names={k: q + k for k in ("gate", "up", "down")})

        def expert(e):
            return ExpertSpec(e["ff"], EXPERT_ACTIVATION, gated=True, limit=float(e["limit"]) if e.get("limit") is not None else None,
                              up_shift=EXPERT_UP_SHIFT)

        names = {"router": q + "router", "correction": q + "correction", "expert_gate": q + "e{e}.gate",
                 "expert_up": q + "e{e}.up", "expert_down": q + "e{e}.down"}
        shared = mlp.get("shared")
        if shared is not None:
            names.update({"shared_gate": q + "shared.gate", "shared_up": q + "shared.up", "shared_down": q + "shared.down",
                          "shared_weight": q + "shared.sg"})
        r = mlp["router"]
        groups = r.get("groups")
        return RoutedFeedForwardSpec(
            hidden=self.width, n_experts=r["experts"], top=r["top"], expert=expert(mlp["expert"]),
            shared=expert(shared) if shared is not None else None, names=names, weights="scores", sum_eps=ROUTER_SUM_EPS,
            groups=(groups["count"], groups["keep"]) if groups is not None else None,
            weight_scale=float(r["scale"]) if r.get("scale") is not None else 1.0)

    def model_spec(self):
        def norm(name):
            return NormSpec(dim=self.width, eps=self.norm_eps, names={"weight": name})

        blocks = []
        for i, lay in enumerate(self.layers):
            p, m, mlp, side = f"l{i}.", lay["mixer"], lay.get("mlp"), None
            if self.side_dim:
                side = TokenSideSpec(
                    hidden=self.width, dim=self.side_dim, rows=self.vocab_size, columns=self.side_dim * len(self.layers),
                    index=i, norm_eps=self.norm_eps, names={"embed": "side.embed", "gate": p + "side.gate",
                                                            "proj": p + "side.proj", "norm": p + "side.norm"})
            blocks.append(BlockSpec(
                kind="parallel", mixer_norm=norm(p + "norm1"), side=side,
                mixer=self._parallel(i, m) if lay["type"] == "parallel" else self._latent(i, m),
                ffn=self._ffn(i, mlp) if mlp is not None else None))
        return ModelSpec(
            architecture=self.architecture, vocab_size=self.vocab_size, hidden=self.width, layers=tuple(blocks),
            run_order=self.run_order(), final_norm=norm("final.norm"), max_positions=self.max_position_embeddings,
            tie_embeddings=False, embedding_name="embed", head_name="head", stop_ids=self.stop_ids,
            embedding_scale=self.embedding_scale, logit_scale=self.logit_scale if self.logit_scale != 1.0 else None)


register_architecture("Banazen", BanazenConfiguration)
