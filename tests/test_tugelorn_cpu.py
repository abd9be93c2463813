"""Tugelorn without a GPU: the configurations the builder takes and refuses, and the plain statement checked by hand."""
import json

import numpy as np
import pytest

import plain_tugelorn as pt
import tugelorn_models as tm
import ug_amd


def test_the_registry_knows_it(cpu):
    for cfg in tm.MODELS.values():
        assert ug_amd.Decoder.random(cpu, cfg, bf16=False).vocab == cfg["vocab"]
    no_loop = {k: v for k, v in tm.ODD.items() if k != "loop"}
    assert ug_amd.Decoder.random(cpu, no_loop, bf16=False).vocab == 101
    assert ug_amd.Decoder.random(cpu, {**no_loop, "loop": None}, bf16=False).vocab == 101


@pytest.mark.parametrize("change, message", [
    (lambda c: c["layers"][0].update(type="mamba2"), "unknown mixer 'mamba2'"),
    (lambda c: c["layers"][0]["mlp"].update(kind="moe"), "unknown feed-forward 'moe'"),
    (lambda c: c["layers"][0]["mlp"].pop("limit"), "'limit' is missing"),
    (lambda c: c["layers"][0]["mlp"].update(limit=0.0), "the limit 0"),
    (lambda c: c["layers"][0]["mixer"].update(kv_heads=4), "6 heads on 4"),
    (lambda c: c["layers"][0]["mixer"].update(conv=0), "behind 0 taps"),
    (lambda c: c["layers"][1]["mixer"].update(kv_heads=5), "6 heads on 5"),
    (lambda c: c["layers"][1]["mixer"]["rot"].update(dims=24), "rotates 24 elements of 22"),
    (lambda c: c["layers"][1]["mixer"]["rot"].update(dims=13), "rotates 13"),
    (lambda c: c["layers"][1]["mixer"]["rot"].pop("scaling"), "'scaling' is missing"),
    (lambda c: c["layers"][1]["mixer"]["mask"].update(size=0), "a window of no positions"),
    (lambda c: c["layers"][2]["mixer"]["q_temp"].update(every=0), "every 0"),
    (lambda c: c["layers"][2]["mixer"].update(dim=300), "heads of 300"),
    (lambda c: c["layers"][2]["mixer"].pop("scale"), "'scale' is missing"),
    (lambda c: c["loop"].update(stop=6), "layers 1 .. 6 of 5"),
    (lambda c: c["loop"].update(start=5), "layers 5 .. 4"),
    (lambda c: c["loop"].update(times=0), "run 0 times"),
    (lambda c: c.pop("residual_mult"), "'residual_mult' is missing"),
])
def test_configurations_that_make_no_model_are_refused(cpu, change, message):
    cfg = json.loads(json.dumps(tm.ODD))
    change(cfg)
    with pytest.raises(ug_amd.UgError, match=message):
        ug_amd.Decoder.random(cpu, cfg, bf16=False)


@pytest.mark.parametrize("name, shape", [("l0.mix.a2", (108, 8)), ("l0.mix.q.conv", (36, 4)), ("l2.mix.k.b", (18,)), ("l1.norm2b", (91,))])
def test_a_tensor_of_another_shape_is_refused(cpu, tmp_path, name, shape):
    w = tm.weights(tm.ODD, tm.RANKS["odd"], 3)
    w[name] = np.zeros(shape)
    with pytest.raises(ug_amd.UgError, match=name.replace(".", r"\.")):
        ug_amd.Decoder.load(cpu, tm.write(tmp_path / "m", tm.ODD, w), bf16=False)


def test_ranks_come_from_the_tensors(cpu, tmp_path):
    """The same configuration with other ranks of the decay's and the output gate's matrices."""
    for ranks in ({0: (7, 5), 3: (12, 33)}, {0: (1, 64), 3: (9, 2)}):
        ug_amd.Decoder.load(cpu, tm.write(tmp_path / str(ranks[0][0]), tm.ODD, tm.weights(tm.ODD, ranks, 3)), bf16=False)


@pytest.mark.parametrize("name", ["odd", "even", "ones"])
def test_the_plain_statement_is_causal(name):
    cfg = tm.MODELS[name]
    w = tm.weights(cfg, tm.RANKS[name], 5)
    tokens = np.arange(50) * 7 % cfg["vocab"]
    np.testing.assert_allclose(pt.forward(cfg, w, tokens)[:21], pt.forward(cfg, w, tokens[:21]), rtol=1e-9, atol=1e-11)


def test_plain_mechanisms_by_hand():
    x = np.array([[[1.0, 2.0, 3.0, 4.0, 9.0]]])
    out = pt.rotate_pairs(x, [6], 100.0, 4, 3.0)       # pairs (0, 1) and (2, 3), angles 6 / 3 and 6 / 10 / 3
    np.testing.assert_allclose(out[0, 0], [np.cos(2) - 2 * np.sin(2), 2 * np.cos(2) + np.sin(2), 3 * np.cos(.2) - 4 * np.sin(.2), 4 * np.cos(.2) + 3 * np.sin(.2), 9.0])
    np.testing.assert_allclose(pt.query_temperature([0, 2, 3, 7, 8], 0.5, 4), 1 + 0.5 * np.log([1, 1, 2, 3, 3]))
    # a window of two over equal scores: the mean of what is seen; query head 1 and 2 of four share with 0 and 3
    v = np.arange(4.0).reshape(4, 1, 1) * [[[1.0], [10.0]]]
    got = pt.grouped_attention(np.zeros((4, 4, 2)), np.zeros((4, 2, 2)), v, 1.0, window=2)[:, :, 0]
    np.testing.assert_allclose(got[:, 0], [0, 0.5, 1.5, 2.5])
    np.testing.assert_allclose(got, got[:, :1] * [1, 1, 10, 10])
    np.testing.assert_allclose(pt.grouped_attention(np.zeros((1, 1, 2)), np.zeros((4, 1, 2)), v[:, :1], 1.0, first=3)[0, 0], [1.5])
    np.testing.assert_allclose(pt.clamped_glu(np.array([5.0, -5.0, 1.0]), np.array([3.0, -3.0, 0.5]), 2.0),
                               [2 / (1 + np.exp(-3.404)) * 3, -5 / (1 + np.exp(8.51)) * -1, 1 / (1 + np.exp(-1.702)) * 1.5])
    # one channel, one column: S = g S, then the error towards v corrected by beta along k
    q, k, v = np.full((2, 1, 1), 2.0), np.ones((2, 1, 1)), np.array([[[3.0]], [[5.0]]])
    o = pt.delta_scan(q, k, v, np.log(np.array([[[0.9]], [[0.5]]])), np.array([[0.25], [0.5]]))
    s1 = 0.25 * 3.0
    np.testing.assert_allclose(o[:, 0, 0], [2 * s1, 2 * (0.5 * s1 + 0.5 * (5.0 - 0.5 * s1))])
    assert pt.layer_runs(tm.ODD) == [(0, False), (1, False), (2, False), (3, False), (1, True), (2, False), (3, False), (1, True), (2, False), (3, False), (4, False)]
    assert pt.layer_runs({"layers": [0, 0]}) == [(0, False), (1, False)]
