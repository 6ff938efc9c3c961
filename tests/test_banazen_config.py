"""The Banazen configuration on the CPU: reader, descriptions, expected tensors, cache and state needs, errors, and the plain
implementation's own consistency (a sequence fed whole and in pieces, cases worked by hand)."""
import copy
import math

import numpy as np
import pytest
import torch

import plain_banazen as P
from banazen_models import BARE, CONFIGS, MIXED, REORDERED, TILED, model, ranks

from gpullama3_java_amd.config import ConfigError, config_from_dict, load_config
from gpullama3_java_amd.parts import DecoderModel, expected_tensors


def with_shapes(cfg):
    return config_from_dict(cfg).with_tensor_shapes(P.tensor_shapes(cfg, ranks))


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_expected_tensors_are_the_design_s(name):
    cfg = with_shapes(CONFIGS[name])
    exp, shapes = expected_tensors(cfg.model_spec()), P.tensor_shapes(CONFIGS[name], ranks)
    assert set(exp) == set(shapes)
    for k in exp:
        assert tuple(exp[k].shape) == tuple(shapes[k]), k
    again = config_from_dict(cfg.to_dict())
    assert again.to_dict() == cfg.to_dict() and again == cfg and hash(again) == hash(cfg)
    folder, _, _ = model(name)
    assert load_config(folder) == cfg                     # (the inner sizes come from the file's header)


def test_descriptions():
    spec = with_shapes(MIXED).model_spec()
    assert (spec.embedding_scale, spec.logit_scale, len(spec.layers)) == (2.5, 0.7, 6) and all(b.kind == "parallel" for b in spec.layers)
    assert [r.reads for r in spec.run_order] == [None, None, 0, None, 3, None]
    a = spec.layers[0].mixer
    assert (a.kind, a.n_heads, a.head_dim, a.v_head_dim, a.kv_rank, a.scale) == ("latent_attention", 3, 24, 40, 40, 0.2)
    assert (a.q_rank, a.rot_dim, a.position) == (0, 0, None) and not {"g", "dq", "uq"} & set(a.names)
    # (a source keeps as far back as the widest of its readers sees; all of it where one sees everything)
    assert [(b.mixer.window, b.mixer.kept_window) for b in spec.layers if b.mixer.kind == "latent_attention"] == \
        [(37, 64), (64, None), (None, 0), (21, None)]
    assert "dkv" in a.names and "dkv" not in spec.layers[2].mixer.names
    two = spec.layers[1].mixer
    assert two.kind == "side_by_side" and two.weight == 0.5 and two.names == {"left_norm": "l1.mix.left.out", "right_norm": "l1.mix.right.out"}
    left, right = two.left, two.right
    assert (left.n_heads, left.n_kv_heads, left.head_dim, left.v_head_dim, left.conv_taps, left.scale, left.window) == (4, 2, 24, 40, 4, 0.25, None)
    assert (left.position.head_dim, left.position.theta, left.position.pairing) == (12, 900.0, "adjacent") and left.qk_norm_eps == 1e-5
    assert "q_norm" not in left.names and left.names["v_conv"] == "l1.mix.left.v.conv"
    assert (right.n_heads, right.n_kv_heads, right.key_dim, right.value_dim, right.conv_taps) == (4, 2, 24, 40, 2)
    assert (right.decay_rank, right.gate_rank, right.gate_activation, right.unit_eps) == ranks(1) + ("sigmoid", 1e-6)
    assert spec.layers[5].mixer.left.position is None and spec.layers[5].mixer.left.conv_taps == 1
    moe = spec.layers[0].ffn
    assert (moe.n_experts, moe.top, moe.weights, moe.sum_eps, moe.groups, moe.weight_scale) == (6, 2, "scores", 1e-20, (3, 2), 2.5)
    assert (moe.expert.activation, moe.expert.limit, moe.expert.up_shift) == ("quick_gelu", 0.7, 1.0)
    assert (moe.shared.intermediate, moe.shared.limit) == (24, 1.3) and moe.names["shared_weight"] == "l0.mlp.shared.sg"
    assert spec.layers[1].ffn.kind == "gated" and spec.layers[1].ffn.activation == "silu" and spec.layers[2].ffn is None
    assert spec.layers[4].ffn.shared is None and spec.layers[4].ffn.groups is None
    side = spec.layers[3].side
    assert (side.dim, side.columns, side.index, side.rows, side.names["embed"]) == (10, 60, 3, 300, "side.embed")
    bare = config_from_dict(REORDERED).model_spec()
    assert all(b.side is None for b in bare.layers) and bare.logit_scale == 3.0 and config_from_dict(BARE).model_spec().logit_scale is None
    loose = copy.deepcopy(MIXED)
    loose["layers"][0]["mlp"]["router"].pop("scale")
    loose["layers"][0]["mlp"]["shared"].pop("limit")
    ffn = config_from_dict(loose).model_spec().layers[0].ffn
    assert ffn.weight_scale == 1.0 and ffn.shared.limit is None and ffn.expert.limit == 0.7


def test_cache_and_state_needs():
    kv, state = DecoderModel(with_shapes(MIXED).model_spec(), torch.float32, "cpu").cache_needs()
    # (latents: one row a position, padded to 32s; keys and values behind a convolution: heads padded to 16s)
    assert [None if n is None else (n.n_kv_heads, n.head_dim, n.v_head_dim, n.window, n.values) for n in kv] == \
        [(1, 64, None, 64, False), (2, 32, 48, None, True), None, (1, 32, None, None, False), None, (1, 48, 32, None, True)]
    conv = (4 + 2) * 32 + 2 * 48
    delta = 4 * 3 * 24 * 16 + (2 * 2 * 24 + 4 * 40)
    assert [None if n is None else n.elements for n in state] == [None, 3 * conv + delta, None, None, None, 4 + 3 * 20 * 16 + 4 * (2 * 3 * 20 + 3 * 12)]
    kv, _ = DecoderModel(with_shapes(TILED).model_spec(), torch.bfloat16, "cpu").cache_needs()
    # (bfloat16: keys and values in one size that the matrix-core kernels are built for)
    assert [None if n is None else (n.n_kv_heads, n.head_dim, n.v_head_dim) for n in kv] == \
        [(2, 64, None), (1, 96, None), None, (2, 96, None), (1, 128, None)]


@pytest.mark.parametrize("change, says", [
    (lambda c: c["layers"][0].update(type="gru"), "'type'"),
    (lambda c: c.update(layers=[]), "'layers'"),
    (lambda c: c["layers"][0].pop("mixer"), "'mixer'"),
    (lambda c: c["layers"][1]["mixer"].pop("right"), "'right'"),
    (lambda c: c["layers"][1]["mixer"]["left"].update(kv_heads=3), "kv_heads"),
    (lambda c: c["layers"][1]["mixer"]["right"].pop("vdim"), "vdim"),
    (lambda c: c["layers"][1]["mixer"]["left"].update(conv=0), "conv"),
    (lambda c: c["layers"][1]["mixer"]["left"]["rot"].update(dims=26), "dims"),
    (lambda c: c["layers"][1]["mixer"]["left"]["rot"].update(dims=11), "dims"),
    (lambda c: c["layers"][1]["mixer"]["left"].update(scale=0), "scale"),
    (lambda c: c["layers"][0]["mixer"]["mask"].update(size=0), "size"),
    (lambda c: c["layers"][0]["mixer"].pop("kv_rank"), "kv_rank"),
    (lambda c: c["layers"][2]["mixer"].update(kv_from=1), "kv_from"),
    (lambda c: c["layers"][2]["mixer"].update(kv_from=3), "kv_from"),
    (lambda c: c["layers"][4]["mixer"].update(kv_from=2), "kv_from"),
    (lambda c: c["layers"][2]["mixer"].update(kv_rank=48), "latents of 48"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(top=5), "largest of 4"),
    (lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(count=4), "groups"),
    (lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(keep=4), "groups"),
    (lambda c: c["layers"][0]["mlp"]["expert"].update(limit=0), "limit"),
    (lambda c: c["layers"][0]["mlp"]["shared"].pop("ff"), "ff"),
    (lambda c: c["layers"][1]["mlp"].update(kind="sparse"), "'mlp'"),
    (lambda c: c["token_side"].update(dim=0), "dim"),
    (lambda c: c["norm"].update(eps=0), "eps"),
    (lambda c: c["embedding"].update(scale=None), "scale"),
    (lambda c: c.pop("width"), "'width'"),
])
def test_errors_name_the_key(change, says):
    c = copy.deepcopy(MIXED)
    change(c)
    with pytest.raises(ConfigError, match=says):
        config_from_dict(c)


def test_max_positions_and_context():
    cfg = config_from_dict(dict(MIXED, max_positions=500))
    assert cfg.max_position_embeddings == 500 and cfg.with_context_length(100).model_spec().max_positions == 100
    assert config_from_dict(cfg.to_dict()).max_positions == 500
    with pytest.raises(ConfigError, match="token ids"):
        cfg.chat_format(None)


def test_inner_sizes_before_there_are_weights(tmp_path):
    """The random-weights mode writes two-step projections of a size of its own, which the folder's shapes then give."""
    import gpullama3_java_amd as g
    g.write_random_model(str(tmp_path), config_from_dict(BARE), 5)
    cfg = load_config(str(tmp_path))
    assert cfg.ranks == ((0, 0), (8, 8))
    assert config_from_dict(dict(BARE, inner_sizes=[[1, 1], [5, 7]])).model_spec().layers[1].mixer.right.gate_rank == 7


def test_descriptions_that_are_not_built_say_so():
    from dataclasses import replace
    from gpullama3_java_amd.parts import build_part
    spec = with_shapes(MIXED).model_spec()
    kw = dict(dtype=torch.float32, device="cpu")
    right = spec.layers[1].mixer.right
    left = spec.layers[1].mixer.left
    for bad in (replace(right, gate_rank=0), replace(left, position=replace(left.position, pairing="half")), replace(left, values_are_keys=True)):
        with pytest.raises(ValueError):
            build_part("mixer", bad, **kw)
    with pytest.raises(ValueError):
        build_part("ffn", replace(spec.layers[0].ffn, groups=(4, 2)), **kw)
    with pytest.raises(ValueError):
        build_part("ffn", replace(spec.layers[0].ffn, weights="sigmoid"), **kw)
    with pytest.raises(ValueError):
        build_part("side", replace(spec.layers[0].side, activation="erf"), **kw)


# ----------------------------------------------------------------- the plain implementation
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_plain_sequence_in_pieces(name):
    _, cfg, W = model(name)
    toks = np.random.default_rng(1).integers(0, cfg["vocab"], 120).tolist()
    whole = P.forward(cfg, W, toks)
    seq = P.Sequence(cfg, W)
    rows = [seq.feed(toks[:2]), seq.feed(toks[2:70])] + [seq.feed([t]) for t in toks[70:]]
    np.testing.assert_allclose(np.concatenate(rows), whole, atol=1e-9)


def test_plain_cases_by_hand():
    # a convolution of three taps over 1, 2, 3 and then 4: the last weight is the current token's
    y, held = P.short_conv(np.array([[1.0], [2.0], [3.0]]), np.array([[100.0, 10.0, 1.0]]))
    np.testing.assert_array_equal(y[:, 0], [1, 12, 123])
    y, held = P.short_conv(np.array([[4.0]]), np.array([[100.0, 10.0, 1.0]]), held)
    assert y[0, 0] == 234 and held[:, 0].tolist() == [3, 4]
    # a quarter turn: pairs are neighbours, what lies behind the rotated part stays
    x = np.array([[[1.0, 0.0, 5.0]]])
    np.testing.assert_allclose(P.rotate(x, [math.pi / 2], 2, 10.0), [[[0.0, 1.0, 5.0]]], atol=1e-15)
    # the delta rule: the decay acts on a key's row before the correction, and the read-out sees the token's own write
    o, S = P.delta_rule(np.array([[1.0, 0.0]]), np.array([[1.0, 0.0]]), np.array([[2.0]]), np.array([[0.5, 0.25]]), np.array([0.5]),
                        np.array([[4.0], [8.0]]))
    np.testing.assert_allclose(S, [[2.0 + 0.5 * (2.0 - 2.0)], [2.0]])
    assert o[0, 0] == 2.0
    # a window of 3: position 5 sees 3, 4, 5
    assert (P.first_seen(5, 3), P.first_seen(1, 3), P.first_seen(5, None), P.first_seen(5, 1)) == (3, 0, 0, 5)
    # choice: of the groups {0, 1}, {2, 3}, {4, 5} the best two by their best; a closed group's zero loses to an open group's -3
    router = {"experts": 6, "top": 3, "groups": {"count": 3, "keep": 2}}
    idx, gap = P.choose(np.array([0.9, -3.0, 0.0, -0.1, 0.5, -2.0]), router)
    assert idx.tolist() == [0, 4, 5] and gap == pytest.approx(0.5)
    # the weights leave the correction out, and are scaled after the division
    W = {"router": np.array([[1.0], [0.0]]), "correction": np.array([0.0, 5.0])}
    (idx, w, _), = P.route(np.array([[1.0]]), W, "", {"experts": 2, "top": 1, "scale": 1.5})
    assert idx.tolist() == [1] and w[0] == pytest.approx(1.5)
    # an expert: the gate bounded from above only, the up value on both sides, then shifted by one
    W = {"gate": np.array([[1.0]]), "up": np.array([[-4.0]]), "down": np.array([[2.0]])}
    np.testing.assert_allclose(P.expert(np.array([[3.0]]), W, "", 0.5), [[2.0 * 0.5 / (1 + math.exp(-1.702 * 0.5)) * 0.5]])
