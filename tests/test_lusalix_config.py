"""The Lusalix configuration on the CPU: reader, descriptions, expected tensors, cache needs, errors, and the plain
implementation's own consistency (a sequence fed whole and in pieces, cases worked by hand)."""
import copy
import math

import numpy as np
import pytest
import torch

import plain_lusalix as P
from lusalix_models import BARE, CONFIGS, MIXED, REORDERED, TILED, model, write_model

from gpullama3_java_amd.config import ConfigError, config_from_dict
from gpullama3_java_amd.parts import DecoderModel, expected_tensors


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_expected_tensors_are_the_design_s(name):
    cfg = config_from_dict(CONFIGS[name])
    spec = cfg.model_spec()
    exp = expected_tensors(spec)
    shapes = P.tensor_shapes(CONFIGS[name])
    mixing = [i for i, lay in enumerate(CONFIGS[name]["layers"]) if lay["mixer"]["v_mix"]]
    unread = {f"l{mixing[0]}.mix.vmix"} if mixing else set()      # the first blending layer's number: stored, read by nothing
    assert set(exp) == set(shapes) - unread and unread <= set(spec.unused_tensor_names)
    for k in exp:
        assert tuple(exp[k].shape) == tuple(shapes[k]), k
    assert config_from_dict(cfg.to_dict()).to_dict() == cfg.to_dict()


def test_descriptions():
    spec = config_from_dict(MIXED).model_spec()
    assert spec.embedding_scale == 2.5 and len(spec.layers) == 4 and all(b.kind == "prenorm" for b in spec.layers)
    a = spec.layers[0].mixer
    assert (a.n_heads, a.n_kv_heads, a.head_dim, a.v_head_dim, a.window, a.scale, a.position) == (4, 2, 24, 40, 37, 0.2, None)
    assert (a.score_softcap, a.query_temperature.coef, a.query_temperature.every) == (6.0, 0.4, 33)
    assert a.names["gate"] == "l0.mix.g" and a.distance_bias.slopes(4) == [2.0 ** -2, 2.0 ** -4, 2.0 ** -6, 2.0 ** -8]
    mixes = [b.mixer.value_mix for b in spec.layers]
    assert [m if m is None else m.first for m in mixes] == [True, None, False, False]
    assert "v_mix" not in spec.layers[0].mixer.names and spec.layers[3].mixer.names["v_mix"] == "l3.mix.vmix"
    assert spec.layers[2].mixer.score_softcap is None and spec.layers[2].mixer.query_temperature is None
    moe = spec.layers[0].ffn
    assert (moe.n_experts, moe.top, moe.weights, moe.weight_on) == (5, 3, "sigmoid", "input")
    assert moe.expert.gated and (moe.expert.activation, moe.expert.limit, moe.expert.up_shift) == ("silu", None, 0.0)
    assert moe.shared.intermediate == 24 and moe.names["shared_weight"] == "l0.mlp.shared.sg"
    assert spec.layers[2].ffn is None and spec.layers[3].ffn.shared is None
    assert [b.mixer.value_mix for b in config_from_dict(BARE).model_spec().layers] == [None, None]
    # which layer hands its values out follows from the order alone
    assert [m if m is None else m.first for m in (b.mixer.value_mix for b in config_from_dict(REORDERED).model_spec().layers)] \
        == [None, True, None, False]


def test_cache_needs():
    kv, state = DecoderModel(config_from_dict(MIXED).model_spec(), torch.float32, "cpu").cache_needs()
    assert state == [None] * 4
    # (32-bit: heads padded to 16s; bfloat16: to one size for keys and values that the matrix-core kernels take)
    assert [(n.n_kv_heads, n.head_dim, n.v_head_dim, n.window) for n in kv] == \
        [(2, 32, 48, 37), (1, 48, 16, None), (2, 16, 48, 64), (2, 32, 48, 90)]
    kv, _ = DecoderModel(config_from_dict(TILED).model_spec(), torch.bfloat16, "cpu").cache_needs()
    assert [(n.n_kv_heads, n.head_dim, n.v_head_dim, n.window) for n in kv] == \
        [(2, 64, None, 100), (2, 96, None, None), (2, 128, None, 130), (1, 96, None, 33)]
    big = copy.deepcopy(BARE)
    big["layers"][0]["mixer"].update(dim=160, vdim=48)      # larger than any of them: the kernel for any sizes, as stored
    kv, _ = DecoderModel(config_from_dict(big).model_spec(), torch.bfloat16, "cpu").cache_needs()
    assert (kv[0].head_dim, kv[0].v_head_dim) == (160, 48)


@pytest.mark.parametrize("change, says", [
    (lambda c: c["layers"][0].update(type="gru"), "'type'"),
    (lambda c: c.update(layers=[]), "'layers'"),
    (lambda c: c["layers"][0].pop("mixer"), "'mixer'"),
    (lambda c: c["layers"][0]["mixer"].update(kv_heads=3), "kv_heads"),
    (lambda c: c["layers"][1]["mixer"].pop("vdim"), "vdim"),
    (lambda c: c["layers"][1]["mixer"].update(scale=0), "scale"),
    (lambda c: c["layers"][1]["mixer"].update(softcap=-1.0), "softcap"),
    (lambda c: c["layers"][1]["mixer"]["q_temp"].update(every=0), "every"),
    (lambda c: c["layers"][1]["mixer"]["q_temp"].pop("coef"), "coef"),
    (lambda c: c["layers"][0]["mixer"]["mask"].update(size=0), "size"),
    (lambda c: c["layers"][0]["mixer"].update(v_mix=1), "v_mix"),
    (lambda c: c["layers"][3]["mixer"].update(vdim=24), "layer 0's"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(top=6), "largest"),
    (lambda c: c["layers"][0]["mlp"].update(kind="dense"), "'mlp'"),
    (lambda c: c["layers"][0]["mlp"]["shared"].pop("ff"), "ff"),
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


def test_stored_numbers_that_nothing_reads_are_allowed(tmp_path):
    """A folder may hold a blend for every layer and a second norm for a layer without a feed-forward."""
    from gpullama3_java_amd.weights.loader import load_weights
    _, cfg, W = model("mixed")
    W = dict(W, **{"l1.mix.vmix": np.float32(0.5), "l2.norm2": np.ones(96, np.float32)})
    write_model(str(tmp_path), cfg, W)
    spec = config_from_dict(cfg).model_spec()
    out = load_weights(str(tmp_path), expected_tensors(spec), torch.float32, "cpu", ignore=spec.unused_tensor_names)
    assert out["l2.mix.vmix"].shape == () and float(out["l2.mix.vmix"]) == float(W["l2.mix.vmix"])
    assert "l0.mix.vmix" not in out and "l2.norm2" not in out


def test_random_weights_mode(tmp_path):
    import gpullama3_java_amd as g
    g.write_random_model(str(tmp_path), config_from_dict(TILED), 5)
    from safetensors.torch import load_file
    W = load_file(str(tmp_path / "model.safetensors"))
    assert 0.0 < float(W["l2.mix.vmix"]) < 1.0 and W["l2.mix.vmix"].shape == ()


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
    # the temperature: 1 up to the last but one of the first `every` positions, then ln 2, ln 3 more
    np.testing.assert_allclose(P.temperature([0, 2, 3, 6, 7, 10, 11], 0.5, 4),
                               1 + 0.5 * np.log([1, 1, 2, 2, 3, 3, 4]))
    # a score: the cap bends before the slope is taken off (head 1 of 2: slope 2^-8)
    m = {"scale": 0.5, "softcap": 2.0, "heads": 2}
    s = P.score(np.array([2.0, 0.0]), np.array([[4.0, 1.0], [-1.0, 0.0]]), 10, [6, 10], m, 1)
    np.testing.assert_allclose(s, [2 * math.tanh(2.0) - 4 / 256, 2 * math.tanh(-0.5)])
    # a window of 3: position 5 sees 3, 4, 5
    assert (P.visible(5, 3), P.visible(1, 3), P.visible(5, None), P.visible(5, 1)) == (3, 0, 0, 5)
    # a weight on the input of a gated expert is not a weight on its output
    rng = np.random.default_rng(0)
    W = {"gate": rng.standard_normal((3, 4)), "up": rng.standard_normal((3, 4)), "down": rng.standard_normal((4, 3))}
    h = rng.standard_normal((1, 4))
    g, u = W["gate"] @ (0.5 * h[0]), W["up"] @ (0.5 * h[0])
    np.testing.assert_allclose(P.expert(0.5 * h, W, "")[0], W["down"] @ (g / (1 + np.exp(-g)) * u))
    assert np.abs(P.expert(0.5 * h, W, "") - 0.5 * P.expert(h, W, "")).max() > 1e-2
    # the scores are sigmoids as they are: three chosen with scores over a half sum to more than one
    idx, w, _ = P.route(np.array([[1.0]]), {"router": np.array([[0.5], [2.0], [1.0], [-1.0]])}, "", {"top": 3})
    assert list(idx[0]) == [1, 2, 0] and w.sum() > 2.0
    # values are blended with the first blending layer's own, not with blended ones
    np.testing.assert_allclose(P.blend(np.array([1.0]), np.array([5.0]), 0.25), [2.0])
