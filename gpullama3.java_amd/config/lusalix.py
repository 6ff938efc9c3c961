"""Typed configuration of the Lusalix decoder, read from its config.json.

Lusalix is a pre-norm decoder (RMS norms, an embedding times a constant, a head of its own) with one kind of layer:

  attention:     grouped heads without a rotation; the query at position p counts ``1 + coef ln(floor((p + 1) / every) +
                 1)`` times; the scaled score passes ``cap tanh(score / cap)``, then a slope per head times the distance is
                 taken off; a sliding window; an ordinary softmax. Every layer with ``v_mix`` but the first of them
                 caches ``(1 - lambda) v + lambda v_first``, with that first layer's values of the same token and a
                 stored ``lambda``. The heads' outputs are multiplied element by element with sigmoid of a projection of
                 the mixer's input, then the output projection;
  feed-forward:  a mixture of experts ``down(silu(gate h) * up h)``: the ``top`` largest router outputs choose, a chosen
                 expert reads the token's row times sigmoid of its router output (not divided by anything), and a shared
                 expert of the same form runs for every token, its output times sigmoid of one more product.

config.json: ``architecture`` "Lusalix", ``vocab``, ``width``, ``norm.eps``, ``embedding.scale`` and ``layers``, a list of
``{"type": "attention", "mixer": {...}, "mlp": {...} | null}`` with
  mixer:  ``heads``, ``kv_heads``, ``dim``, ``vdim``, ``scale``, ``softcap``, ``q_temp``: ``coef``, ``every``; ``mask``: ``size``;
          ``v_mix``. Without ``softcap``, ``q_temp``, ``mask`` or ``v_mix`` (absent, null or false) there is none.
  mlp:    ``{"kind": "moe", "router": {"experts", "top"}, "expert": {"ff"}, "shared": {"ff"} | null}``.
The folder names no longest sequence: ``max_positions`` (ours, optional) bounds it, else ``DEFAULT_MAX_POSITIONS``.
Tensor names: ``embed``, ``final.norm``, ``head``, and per layer i ``l<i>.norm1``, ``l<i>.norm2``, ``l<i>.mix.*``
(``q``, ``k``, ``v``, ``vmix``, ``g``, ``o``), ``l<i>.mlp.*`` (``router``, ``e<j>.*``, ``shared.*``, ``shared.sg``).
"""
from __future__ import annotations

import copy
from dataclasses import dataclass, replace
from typing import Optional

from .registry import ConfigError, _as_ids, register_architecture
from .specs import (AttentionSpec, BlockSpec, DistanceBias, ExpertSpec, ModelSpec, NormSpec, QueryTemperature,
                    RoutedFeedForwardSpec, Run, ValueMix)

# what the design fixes
EXPERT_ACTIVATION = "silu"
SLOPES = DistanceBias(base=2.0, exponent=8.0)     # head h of H: 2 ** (-8 (h + 1) / H)
DEFAULT_MAX_POSITIONS = 1 << 17       # a folder sets no bound on a sequence's length; the engine's caches need one
TYPES = ("attention",)


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


def _check_mixer(m, where):
    if not isinstance(m, dict):
        raise ConfigError(f"config.json: {where}'mixer' must be an object")
    heads, kv = _int(m, "heads", where), _int(m, "kv_heads", where)
    if heads % kv:
        raise ConfigError(f"config.json: {where}{heads} heads are not a multiple of {kv} kv_heads")
    _int(m, "dim", where), _int(m, "vdim", where), _positive(m, "scale", where)
    if m.get("softcap") is not None:
        _positive(m, "softcap", where)
    if m.get("q_temp") is not None:
        _number(m["q_temp"], "coef", where + "q_temp: "), _int(m["q_temp"], "every", where + "q_temp: ")
    if m.get("mask") is not None:
        _int(m["mask"], "size", where + "mask: ")
    if m.get("v_mix") is not None and not isinstance(m["v_mix"], bool):
        raise ConfigError(f"config.json: {where}'v_mix' must be true or false, found {m['v_mix']!r}")


def _check_mlp(mlp, where):
    if mlp is None:
        return
    if not isinstance(mlp, dict) or mlp.get("kind") != "moe":
        raise ConfigError(f"config.json: {where}'mlp' must be null or an object of kind 'moe'")
    r = mlp.get("router")
    experts, top = _int(r, "experts", where + "router: "), _int(r, "top", where + "router: ")
    if top > experts:
        raise ConfigError(f"config.json: {where}router: the {top} largest of {experts} experts")
    _int(mlp.get("expert"), "ff", where + "expert: ")
    if mlp.get("shared") is not None:
        _int(mlp["shared"], "ff", where + "shared: ")


@dataclass(frozen=True)
class LusalixConfiguration:
    vocab_size: int
    width: int
    norm_eps: float
    embedding_scale: float
    layers: tuple                           # the checked entries of config.json's 'layers', as they stand there
    max_positions: int = DEFAULT_MAX_POSITIONS
    context_length: Optional[int] = None
    stop_ids: tuple = ()
    architecture: str = "Lusalix"

    @property
    def max_position_embeddings(self):
        return self.max_positions if self.context_length is None else min(self.context_length, self.max_positions)

    @property
    def hidden_size(self):
        return self.width

    def __hash__(self):
        return hash((self.vocab_size, self.width, self.norm_eps, self.embedding_scale, repr(self.layers), self.max_positions,
                     self.context_length, self.stop_ids))

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
            _check_mixer(lay.get("mixer"), where)
            _check_mlp(lay.get("mlp"), where + "mlp: ")
        mixing = [(i, lay["mixer"]) for i, lay in enumerate(layers_in) if lay["mixer"].get("v_mix")]
        for i, m in mixing[1:]:
            if any(m[k] != mixing[0][1][k] for k in ("kv_heads", "vdim")):
                raise ConfigError(f"config.json: layers[{i}]: values blended with layer {mixing[0][0]}'s have that layer's "
                                  "kv_heads and vdim")
        scale = d.get("embedding")
        return cls(vocab_size=_int(d, "vocab", ""), width=_int(d, "width", ""),
                   norm_eps=_positive(d.get("norm"), "eps", "norm: "),
                   embedding_scale=_number(scale, "scale", "embedding: ") if scale is not None else 1.0,
                   layers=tuple(copy.deepcopy(layers_in)),
                   max_positions=_int(d, "max_positions", "") if d.get("max_positions") is not None else DEFAULT_MAX_POSITIONS,
                   stop_ids=_as_ids(d.get("eos_token_id")))

    def to_dict(self):
        d = {"architecture": self.architecture, "vocab": self.vocab_size, "width": self.width,
             "norm": {"eps": self.norm_eps}, "embedding": {"scale": self.embedding_scale},
             "layers": copy.deepcopy(list(self.layers))}
        if self.max_positions != DEFAULT_MAX_POSITIONS:
            d["max_positions"] = self.max_positions
        if self.stop_ids:
            d["eos_token_id"] = list(self.stop_ids)
        return d

    # ------------------------------------------------------------------ what the engine asks
    def chat_format(self, tokenizer):
        raise ConfigError("a Lusalix model folder brings no chat format: give the prompt as token ids")

    def with_stop_ids(self, ids):
        return replace(self, stop_ids=tuple(ids))

    def with_context_length(self, n):
        if n is None or n < 0:
            return self
        return replace(self, context_length=min(n, self.max_positions))

    def run_order(self):
        return tuple(Run(layer=i) for i in range(len(self.layers)))

    def _mixer(self, i, m, first_mixing):
        p = f"l{i}.mix."
        names = {k: p + k for k in ("q", "k", "v", "o")}
        names["gate"] = p + "g"
        mix = None
        if m.get("v_mix"):
            mix = ValueMix(first=i == first_mixing)
            if not mix.first:
                names["v_mix"] = p + "vmix"
        t = m.get("q_temp")
        return AttentionSpec(
            hidden=self.width, n_heads=m["heads"], n_kv_heads=m["kv_heads"], head_dim=m["dim"], v_head_dim=m["vdim"],
            position=None, window=m["mask"]["size"] if m.get("mask") is not None else None, scale=float(m["scale"]),
            distance_bias=SLOPES, score_softcap=float(m["softcap"]) if m.get("softcap") is not None else None,
            query_temperature=QueryTemperature(float(t["coef"]), int(t["every"])) if t is not None else None,
            value_mix=mix, names=names)

    def _ffn(self, i, mlp):
        q = f"l{i}.mlp."

        def expert(e):
            return ExpertSpec(e["ff"], EXPERT_ACTIVATION, gated=True)

        names = {"router": q + "router", "expert_gate": q + "e{e}.gate", "expert_up": q + "e{e}.up",
                 "expert_down": q + "e{e}.down"}
        shared = mlp.get("shared")
        if shared is not None:
            names.update({"shared_gate": q + "shared.gate", "shared_up": q + "shared.up", "shared_down": q + "shared.down",
                          "shared_weight": q + "shared.sg"})
        r = mlp["router"]
        return RoutedFeedForwardSpec(
            hidden=self.width, n_experts=r["experts"], top=r["top"], expert=expert(mlp["expert"]),
            shared=expert(shared) if shared is not None else None, names=names, weights="sigmoid", weight_on="input")

    def model_spec(self):
        def norm(name):
            return NormSpec(dim=self.width, eps=self.norm_eps, names={"weight": name})

        first_mixing = next((i for i, lay in enumerate(self.layers) if lay["mixer"].get("v_mix")), None)
        blocks, unused = [], []
        for i, lay in enumerate(self.layers):
            p, mlp = f"l{i}.", lay.get("mlp")
            if not lay["mixer"].get("v_mix") or i == first_mixing:
                unused.append(p + "mix.vmix")      # (a folder may hold the number of a layer that blends nothing)
            if mlp is None:
                unused.append(p + "norm2")         # (and the second norm of a layer without a feed-forward)
            blocks.append(BlockSpec(
                kind="prenorm", mixer_norm=norm(p + "norm1"), mixer=self._mixer(i, lay["mixer"], first_mixing),
                ffn_norm=norm(p + "norm2") if mlp is not None else None, ffn=self._ffn(i, mlp) if mlp is not None else None))
        return ModelSpec(
            architecture=self.architecture, vocab_size=self.vocab_size, hidden=self.width, layers=tuple(blocks),
            run_order=self.run_order(), final_norm=norm("final.norm"), max_positions=self.max_position_embeddings,
            tie_embeddings=False, embedding_name="embed", head_name="head", stop_ids=self.stop_ids,
            embedding_scale=self.embedding_scale, unused_tensor_names=tuple(unused))


register_architecture("Lusalix", LusalixConfiguration)
