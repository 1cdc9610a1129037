"""CPU: the Kazedra oracle against hand-worked facts, how sensitive the test models are, and the host side of the model
(registry, tables, shapes, cache layout)."""
import json
import math

import pytest
import torch

import kazedra_models as K
import lusatar_models as M
from oracle import kazedra as O


# ---- oracle -------------------------------------------------------------------------------------------------------------
def test_the_sink_takes_its_share_and_the_values_are_plain_keys():
    v = torch.tensor([[[2.0, 0.0]], [[0.0, 4.0]]]).double()
    q, rel, sink = torch.zeros(2, 1, 2).double(), torch.zeros(4, 1).double(), torch.tensor([math.log(2.0)]).double()
    o = O.tied_attention(q, torch.zeros_like(v), v, 1.0, rel, 9, sink)
    assert torch.allclose(o[0, 0], v[0, 0] / 3) and torch.allclose(o[1, 0], (v[0, 0] + v[1, 0]) / 4)


def test_distances_share_logarithmic_buckets():
    got = [O.distance_bucket(n, 8, 64) for n in (0, 3, 4, 7, 8, 15, 16, 31, 32, 63, 64, 5000)]
    assert got == [0, 3, 4, 4, 5, 5, 6, 6, 7, 7, 7, 7]


def test_the_delta_rule_replaces_what_a_key_held():
    k = torch.tensor([[[1.0, 0.0]], [[1.0, 0.0]], [[0.0, 1.0]]]).double()
    v = torch.tensor([[[3.0]], [[5.0]], [[7.0]]]).double()
    one = torch.ones(3, 1).double()
    o, S = O.delta_rule(k, k, v, one, one)
    assert o[:, 0, 0].tolist() == [3.0, 5.0, 7.0] and S[0, :, 0].tolist() == [5.0, 7.0]
    o, S = O.delta_rule(k, k, v, one * 0.5, one * 0.25)        # decay first, then a quarter of the way to the value
    assert o[0, 0, 0] == 0.75 and abs(float(o[1, 0, 0]) - (0.375 + 0.25 * (5 - 0.375))) < 1e-12


def test_convolution_last_tap_is_the_token_itself():
    x = torch.arange(1.0, 6.0).view(5, 1).double()
    assert O.causal_conv(x, torch.tensor([[100.0, 10.0, 1.0]]).double())[:, 0].tolist() == [1.0, 12.0, 123.0, 234.0, 345.0]


def test_temperature_steps_after_whole_groups():
    t = [O.temperature(p, 0.5, 4) for p in range(9)]
    assert t[:3] == [1.0] * 3 and t[3:7] == [1 + 0.5 * math.log(2)] * 4 and t[7] == 1 + 0.5 * math.log(3)


def _spoilt(name, cfg, w):
    """The same model with one mistake, planted in what the oracle is given."""
    c, v = json.loads(json.dumps(cfg)), dict(w)
    m = c["layers"][0]["mixer"]
    if name == "sink":
        v["l0.mix.left.sink"] = w["l0.mix.left.sink"] - 50
    elif name == "buckets":
        m["left"]["bias_max"] += 12
    elif name == "bias":
        v["l0.mix.left.rel"] = torch.zeros_like(w["l0.mix.left.rel"])
    elif name == "temperature":
        m["left"]["q_temp"]["every"] += 1
    elif name == "key norm":
        v["l0.mix.left.k.norm"] = w["l0.mix.left.k.norm"].flip(0)
    elif name == "bias of the output":
        v["l0.mix.left.o.b"] = w["l0.mix.left.o.b"] * 0
    elif name == "taps":
        v["l0.mix.right.k.conv"] = w["l0.mix.right.k.conv"].flip(1)
    elif name == "decay":
        v["l0.mix.right.A_log"] = w["l0.mix.right.A_log"] - 20
    elif name == "step size":
        v["l0.mix.right.dt_bias"], v["l0.mix.right.b"] = w["l0.mix.right.dt_bias"], w["l0.mix.right.b"] * 0
    elif name == "scales":
        m["left_scale"], m["right_scale"] = m["right_scale"], m["left_scale"]
    elif name == "norm weights":
        v["l1.norm1"] = w["l1.norm1"] - 1
    elif name == "groups":
        q = w["l0.mix.right.q"].view(3, 20, -1)
        v["l0.mix.right.q"] = q.roll(1, 0).reshape(60, -1)
    return c, v


@pytest.mark.parametrize("name", ["sink", "buckets", "bias", "temperature", "key norm", "bias of the output", "taps", "decay", "step size",
                                  "scales", "norm weights", "groups"])
def test_test_models_show_a_mistake(name):
    cfg = K.CONFIGS["mixed"]
    w, t = K.weights(cfg), M.tokens(cfg, 48)
    want, _ = O.forward(cfg, w, t)
    got, _ = O.forward(*_spoilt(name, cfg, w), t)
    assert float(M.rel_rms(got, want).max()) > 0.02      # against 1e-4 that the fp32 comparisons allow


# ---- product host side ---------------------------------------------------------------------------------------------------
def test_distance_tables():
    from sglang_security_amd.layers.position_bias import LOG2E, bucket_starts, distance_table

    for buckets, longest in ((2, 40), (7, 90), (8, 64), (10, 40), (16, 128), (32, 1000), (64, 256), (16, 100.5), (6, 3.5)):
        starts = bucket_starts(buckets, longest)
        assert len(starts) == buckets
        rel = torch.randn(buckets, 3)
        for context in (5, 50, 2000):
            t = distance_table(rel, longest, context)
            assert t.shape[1] <= context
            for n in range(context):
                want = rel[O.distance_bucket(n, buckets, longest)] * LOG2E
                assert torch.allclose(t[:, min(n, t.shape[1] - 1)], want, rtol=1e-6), (buckets, longest, n)
    for bad in ((1, 9), (8, 4), (8, 2)):
        with pytest.raises(ValueError):
            bucket_starts(*bad)


def test_temperature_tables():
    from sglang_security_amd.layers.position_bias import temperature

    for coef, every in ((0.3, 7), (1.1, 64), (0.0, 1), (0.5, 2.5)):
        t = temperature({"coef": coef, "every": every}, 300, "cpu")
        assert torch.allclose(t.double(), torch.tensor([O.temperature(p, coef, every) for p in range(300)], dtype=torch.float64), rtol=1e-7)
    assert bool((temperature(None, 9, "cpu") == 1).all())


def test_registry_shapes_and_sources():
    from sglang_security_amd import models
    from sglang_security_amd.models.kazedra import Kazedra, tensor_shapes

    assert models.model_class({"architecture": "Kazedra"}) is Kazedra
    assert "rglru.hip" not in models.kernel_sources({"architecture": "Kazedra"})
    for cfg in K.CONFIGS.values():
        shapes, w = tensor_shapes(cfg), K.weights(cfg)
        assert set(shapes) == set(w)
        assert all(a is None or a == b for n in w for a, b in zip(shapes[n], w[n].shape))
    bad = json.loads(json.dumps(K.CONFIGS["mixed"]))
    bad["layers"][1]["mixer"]["left"]["vdim"] = 8
    with pytest.raises(ValueError, match="layer 1"):
        tensor_shapes(bad)
    bad["layers"][1]["type"] = "attention"
    with pytest.raises(ValueError, match="unknown mixer"):
        tensor_shapes(bad)


def test_open_sizes_come_from_the_tensor():
    from sglang_security_amd.model_loader import Weights

    ws = Weights({"rel": torch.zeros(5, 3)}, torch.float32, "cpu")
    assert ws.get("rel", (None, 3)).shape == (5, 3)
    for shape in ((None, 4), (None,), (5, None, 3)):
        with pytest.raises(ValueError, match="shape"):
            ws.get("rel", shape)


def test_cache_of_parallel_mixers():
    from sglang_security_amd.mem_cache.memory_pool import HybridCache

    c = HybridCache([("parallel", [("tied", 48), ("matrix", 64, 4, (2, 32, 16))]), ("recurrent", 32, 3)], 10, 3, 20, torch.bfloat16, "cpu")
    tied, matrix = c.layers[0]
    assert tied.rows.shape == (11, 48) and tied.rms.shape == (11,) and tied.rms.dtype == torch.float32
    assert matrix.state.shape == (3, 2, 32, 16) and matrix.state.dtype == torch.float32 and matrix.conv.shape == (3, 3, 64)
    assert c.layers[1].state.shape == (3, 32)
    assert c.get_size_bytes() == 11 * (96 + 4) + 3 * (2 * 32 * 16 * 4 + 3 * 64 * 2) + 3 * (32 * 4 + 2 * 32 * 2)
    with pytest.raises(ValueError, match="unknown kind"):
        HybridCache([("paged", 1)], 1, 1, 1, torch.float32, "cpu")
