"""Sorulix on the CPU: the configuration's round trip, sizes read from stored shapes and errors, the plan (order of calls,
entries into a run of layers, memory), and the plain model whole against in pieces."""
import copy
import math

import numpy as np
import pytest
import torch

from plain import sorulix_plain as plain
from sorulix_helpers import SOR, as_f64, make_weights, random_config, random_tokens, stored_config, tensor_shapes

from minivllm_amd.config.model_config import ConfigError, SorulixConfig
from minivllm_amd.models import config_from_dict, expected_tensors


def completed(name):
    shapes = tensor_shapes(SOR[name])
    arch, cfg = config_from_dict(stored_config(SOR[name]))
    return arch, cfg.completed(lambda n: shapes.get(n))


@pytest.mark.parametrize("name", sorted(SOR))
def test_round_trip_and_tensor_names(name):
    arch, cfg = completed(name)
    assert arch.name == "Sorulix" and SorulixConfig.from_dict(cfg.to_dict()) == cfg
    expected, stored = expected_tensors(arch, cfg), tensor_shapes(SOR[name])
    assert set(expected) == set(stored) and all(tuple(expected[n].shape) == tuple(stored[n]) for n in expected)


def test_configurations_drawn_at_random_parse():
    for seed in range(30):
        raw = random_config(np.random.default_rng(seed), fast_sizes=seed % 2 == 0)
        shapes = tensor_shapes(raw)
        arch, cfg = config_from_dict(stored_config(raw))
        assert set(expected_tensors(arch, cfg.completed(lambda n: shapes.get(n)))) == set(shapes)


@pytest.mark.parametrize("name", sorted(SOR))
def test_sizes_left_out_are_read_from_the_stored_shapes(name):
    _, full = completed(name)
    raw = copy.deepcopy(stored_config(SOR[name]))
    del raw["vocab"], raw["width"]
    for layer in raw["layers"]:
        m = layer["mixer"]
        if layer["type"] == "parallel":
            for key in ("kv_heads", "dim", "vdim"):
                m["left"].pop(key)
            for key in ("heads", "dim", "vdim"):
                m["right"].pop(key)
        else:
            m.clear()
        if layer["mlp"] is not None:
            layer["mlp"].pop("ff")
    shapes = tensor_shapes(SOR[name])
    thin = SorulixConfig.from_dict(raw)
    assert thin.vocab_size == -1
    assert thin.completed(lambda n: shapes.get(n)) == full
    with pytest.raises(ConfigError):
        thin.completed()


@pytest.mark.parametrize("name, edit", [
    ("A", lambda c: c["layers"][0].update(type="delta")),
    ("A", lambda c: c["layers"][1]["mixer"]["left"].update(kv_heads=3)),
    ("A", lambda c: c["layers"][1]["mixer"]["left"].update(softcap=0.0)),
    ("A", lambda c: c["layers"][1]["mixer"]["left"].pop("scale")),
    ("A", lambda c: c["layers"][1]["mixer"]["left"]["q_temp"].update(every=0)),
    ("A", lambda c: c["layers"][1]["mixer"]["left"]["q_temp"].update(every=2.5)),
    ("A", lambda c: c["layers"][1]["mixer"]["right"].update(decay=[0.5])),
    ("A", lambda c: c["layers"][1]["mixer"]["right"].pop("decay")),
    ("A", lambda c: c["layers"][0]["mixer"].update(heads=3)),
    ("A", lambda c: c["layers"][0]["mixer"].update(conv=0)),
    ("A", lambda c: c["layers"][0]["mlp"].update(kind="moe")),
    ("A", lambda c: c["layers"][0]["mlp"].pop("limit")),
    ("A", lambda c: c["loop"].update(stop=5)),
    ("A", lambda c: c["loop"].update(times=0)),
    ("A", lambda c: c["loop"].pop("start")),
    ("A", lambda c: c["norm"].update(eps=0.0)),
])
def test_configuration_errors(name, edit):
    raw = copy.deepcopy(stored_config(SOR[name]))
    edit(raw)
    with pytest.raises(ConfigError):
        SorulixConfig.from_dict(raw).completed(lambda n: tensor_shapes(SOR[name]).get(n))


def test_plan_and_memory():
    from minivllm_amd.parts.base import MIXERS
    arch, cfg = completed("A")
    plan = arch.plan(cfg)
    assert [(c.layer, c.enters_pass) for c in plan.calls] == [(i, t) for i, t in plain.layer_runs(SOR["A"])]
    assert [l.mixer.kind for l in plan.layers] == ["channel_delta", "parallel", "channel_delta", "parallel"]
    assert plan.layers[1].ffn is None and plan.entry.times == 3
    m = plan.layers[1].mixer
    need = MIXERS.get(m.kind).cache_need(m)
    assert need.retention.keeps_everything and need.page_shapes(16) == {"k": (2, 16, 16), "v": (2, 24, 16)}
    assert MIXERS.get(m.kind).state_shapes(m) == {"state": ((3, 20, 12), torch.float32)}
    d = plan.layers[0].mixer
    assert MIXERS.get(d.kind).cache_need(d) is None
    assert MIXERS.get(d.kind).state_shapes(d) == {"state": ((4, 24, 16), torch.float32), "conv": ((2, 2 * 2 * 16 + 4 * 24), None)}
    arch, cfg = completed("B")
    assert arch.plan(cfg).entry is None and all(c.enters_pass is None for c in arch.plan(cfg).calls)
    assert "conv" not in MIXERS.get("channel_delta").state_shapes(arch.plan(cfg).layers[1].mixer)       # one tap: nothing is kept


@pytest.mark.parametrize("name", sorted(SOR))
def test_plain_model_in_pieces(name):
    cfg = SOR[name]
    w = as_f64(make_weights(cfg, seed=3))
    toks = random_tokens(cfg, 23, seed=1)
    whole, _ = plain.forward(cfg, w, toks)
    state, rows, p = None, [], 0
    for n in (5, 1, 2, 9, 1, 1, 4):
        logits, state = plain.forward(cfg, w, toks[p:p + n], state=state)
        rows.append(logits)
        p += n
    assert torch.allclose(torch.cat(rows), whole, atol=1e-9, rtol=0)


def test_plain_mechanisms_by_hand():
    """The sink: one score of 0 against it gives a half; a query that likes nothing attends to nothing. The distance bias
    halves with the head count's share; the temperature steps where the position is one short of a multiple."""
    p = plain.sink_softmax(torch.tensor([[0.0, -math.inf], [-50.0, -60.0]], dtype=torch.float64))
    assert torch.allclose(p[0], torch.tensor([0.5, 0.0], dtype=torch.float64)) and float(p[1].sum()) < 1e-20
    assert plain.distance_slope(0, 8) == 0.5 and plain.distance_slope(7, 8) == 2.0 ** -8 and plain.distance_slope(0, 1) == 2.0 ** -8
    assert plain.query_temperature(6, 0.5, 8) == 1.0
    assert plain.query_temperature(7, 0.5, 8) == 1.0 + 0.5 * math.log(2.0) == plain.query_temperature(14, 0.5, 8)
