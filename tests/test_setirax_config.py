"""Setirax on the CPU: the configuration's round trip, sizes read from stored shapes and errors, the plan (whose tensors a
layer runs, memory), rotary frequencies by wavelength, the plain model whole against in pieces, its mechanisms by hand, and
that the suites' bounds would notice each mechanism done wrong."""
import copy
import math

import numpy as np
import pytest
import torch

from helpers import BF16_FLOOR, rel_err
from plain import setirax_plain as plain
from setirax_helpers import (SET, as_f64, make_weights, plain_logits, plain_logits_bf16, random_config, random_tokens, sharpened,
                             stored_config, tensor_shapes)

from minivllm_amd.config.model_config import ConfigError, SetiraxConfig
from minivllm_amd.models import config_from_dict, expected_tensors


def completed(name):
    shapes = tensor_shapes(SET[name])
    arch, cfg = config_from_dict(stored_config(SET[name]))
    return arch, cfg.completed(lambda n: shapes.get(n))


@pytest.mark.parametrize("name", sorted(SET))
def test_round_trip_and_tensor_names(name):
    arch, cfg = completed(name)
    assert arch.name == "Setirax" and SetiraxConfig.from_dict(cfg.to_dict()) == cfg
    expected, stored = expected_tensors(arch, cfg), tensor_shapes(SET[name])
    assert set(expected) == set(stored) and all(tuple(expected[n].shape) == tuple(stored[n]) for n in expected)


def test_configurations_drawn_at_random_parse():
    for seed in range(40):
        raw = random_config(np.random.default_rng(seed), fast_sizes=seed % 2 == 0)
        shapes = tensor_shapes(raw)
        arch, cfg = config_from_dict(stored_config(raw))
        assert set(expected_tensors(arch, cfg.completed(lambda n: shapes.get(n)))) == set(shapes)


@pytest.mark.parametrize("name", sorted(SET))
def test_sizes_left_out_are_read_from_the_stored_shapes(name):
    _, full = completed(name)
    raw = copy.deepcopy(stored_config(SET[name]))
    del raw["vocab"], raw["width"]
    for layer in raw["layers"]:
        m = layer["mixer"]
        if layer["type"] == "parallel":
            for key in ("kv_heads", "dim", "vdim", "conv"):
                m["left"].pop(key)
            for key in ("dim", "vdim"):
                m["right"].pop(key)
        elif layer["type"] == "rglru":
            m.clear()
        else:
            for key in ("dim", "vdim", "kv_rank"):
                m.pop(key)
        if layer["mlp"] is not None:
            layer["mlp"].pop("ff")
    shapes = tensor_shapes(SET[name])
    thin = SetiraxConfig.from_dict(raw)
    assert thin.vocab_size == -1
    assert thin.completed(lambda n: shapes.get(n)) == full
    with pytest.raises(ConfigError):
        thin.completed()


@pytest.mark.parametrize("name, edit", [
    ("A", lambda c: c["layers"][0].update(type="latent")),
    ("A", lambda c: c["layers"][1]["mixer"]["left"].update(kv_heads=3)),
    ("A", lambda c: c["layers"][1]["mixer"]["left"].update(softcap=0.0)),
    ("A", lambda c: c["layers"][1]["mixer"]["left"].pop("scale")),
    ("A", lambda c: c["layers"][1]["mixer"]["left"]["mask"].update(size=0)),
    ("A", lambda c: c["layers"][1]["mixer"]["left"]["rot"].update(dims=7)),
    ("A", lambda c: c["layers"][1]["mixer"]["left"]["rot"].update(dims=18)),
    ("A", lambda c: c["layers"][1]["mixer"]["left"]["rot"].pop("base")),
    ("A", lambda c: c["layers"][1]["mixer"]["left"]["rot"]["scaling"].update(low=9.0)),
    ("A", lambda c: c["layers"][1]["mixer"]["left"]["rot"]["scaling"].pop("original")),
    ("A", lambda c: c["layers"][1]["mixer"]["left"].update(conv=0)),
    ("A", lambda c: c["layers"][1]["mixer"]["right"].update(tau=0.0)),
    ("A", lambda c: c["layers"][1]["mixer"]["right"].pop("tau")),
    ("A", lambda c: c["layers"][1]["mixer"].pop("left_scale")),
    ("A", lambda c: c["layers"][2]["mixer"].update(blocks=5)),
    ("A", lambda c: c["layers"][0]["mixer"].update(scale=-1.0)),
    ("A", lambda c: c["layers"][0]["mixer"]["mask"].update(size=2.5)),
    ("A", lambda c: c["layers"][0]["mlp"].update(kind="moe")),
    ("A", lambda c: c["layers"][3].update(weights_of=9)),
    ("A", lambda c: c["layers"][3].update(weights_of=3)),
    ("A", lambda c: c["layers"][3]["mixer"]["right"].update(tau=7.0)),
    ("A", lambda c: c["layers"][3].update(mlp=None)),
    ("A", lambda c: c["norm"].update(eps=0.0)),
    ("A", lambda c: c.update(logit_softcap=-3.0)),
    ("A", lambda c: c.update(layers=[])),
])
def test_configuration_errors(name, edit):
    raw = copy.deepcopy(stored_config(SET[name]))
    edit(raw)
    with pytest.raises(ConfigError):
        SetiraxConfig.from_dict(raw).completed(lambda n: tensor_shapes(SET[name]).get(n))


def test_plan_and_memory():
    from minivllm_amd.parts.base import MIXERS
    arch, cfg = completed("A")
    plan = arch.plan(cfg)
    # six runs of four layers' tensors
    assert [c.layer for c in plan.calls] == [0, 1, 2, 1, 2, 3]
    assert [l.mixer.kind for l in plan.layers] == ["latent_attention", "parallel_sum", "recurrent_unit", "parallel_sum"]
    assert plan.layers[2].ffn is None and plan.layers[0].ffn is not None
    part = lambda i: (MIXERS.get(plan.layers[i].mixer.kind), plan.layers[i].mixer)
    kind, m = part(0)
    need = kind.cache_need(m)
    assert need.retention.window == 13 and not need.retention.keeps_everything and kind.state_shapes(m) == {}
    kind, m = part(1)
    need = kind.cache_need(m)
    assert need.retention.window == 10 and need.page_shapes(16) == {"k": (2, 16, 16), "v": (2, 24, 16)}
    assert kind.state_shapes(m) == {"conv": ((2, 4 * 16 + 2 * (16 + 24)), None), "state": ((3, 20, 12), torch.float32)}
    kind, m = part(2)
    assert kind.cache_need(m) is None and kind.state_shapes(m) == {"state": ((48,), torch.float32), "conv": ((3, 48), None)}
    assert part(3)[0].cache_need(part(3)[1]).retention.keeps_everything
    arch, cfg = completed("B")
    plan = arch.plan(cfg)
    kind, m = part(0)
    assert "conv" not in kind.state_shapes(m)             # one tap: nothing is kept
    kind, m = part(2)
    assert kind.cache_need(m).retention.window == 0       # a query that sees itself alone
    arch, cfg = completed("E")
    assert [c.layer for c in arch.plan(cfg).calls] == [0, 0, 1, 0]


@pytest.mark.parametrize("dims, base, scaling", [(64, 10000.0, (8.0, 1.0, 4.0, 1000.0)), (8, 700.0, (4.0, 1.0, 3.0, 40.0)),
                                                 (2, 90.0, (2.0, 0.5, 2.5, 12.0)), (128, 5e5, (16.0, 2.0, 2.0, 8192.0))])
def test_frequencies_by_wavelength(dims, base, scaling):
    from minivllm_amd.parts.rope import wavelength_frequencies
    if scaling[1] < scaling[2]:
        want = plain.frequencies(dims, base, dict(zip(("factor", "low", "high", "original"), scaling)))
        got = wavelength_frequencies(dims, base, scaling)
        assert torch.allclose(got.double(), want, rtol=1e-7, atol=0)
    factor, low, high, original = scaling
    kept = wavelength_frequencies(dims, base, scaling).double() * torch.tensor([base ** (2.0 * i / dims) for i in range(dims // 2)],
                                                                               dtype=torch.float64)
    turns = torch.tensor([original * base ** (-2.0 * i / dims) / (2 * math.pi) for i in range(dims // 2)])
    assert torch.allclose(kept[turns > high], torch.ones(int((turns > high).sum()), dtype=torch.float64), atol=1e-6)
    assert torch.allclose(kept[turns < low] * factor, torch.ones(int((turns < low).sum()), dtype=torch.float64), atol=1e-6)
    assert bool((kept[1:] <= kept[:-1] + 1e-6).all())


@pytest.mark.parametrize("name", sorted(SET))
def test_plain_model_in_pieces(name):
    cfg = SET[name]
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
    f64 = torch.float64
    # a sink as large as the only score takes half; an absent sink takes nothing
    p = plain.sink_softmax(torch.tensor([[0.7, -math.inf]], dtype=f64), torch.tensor(0.7, dtype=f64))
    assert torch.allclose(p, torch.tensor([[0.5, 0.0]], dtype=f64))
    assert float(plain.sink_softmax(torch.tensor([[3.0]], dtype=f64), None)) == 1.0
    # a window of three sees the query's own position and two before it
    s = plain.windowed(torch.zeros(2, 6, dtype=f64), 4, 3)
    assert torch.isfinite(s).tolist() == [[False, False, True, True, True, False], [False, False, False, True, True, True]]
    # a convolution's last column is the current token's
    y, kept = plain.short_conv(torch.tensor([[1.0], [10.0], [100.0]], dtype=f64), torch.tensor([[0.5, 2.0]], dtype=f64))
    assert y.flatten().tolist() == [2.0, 20.5, 205.0] and kept.flatten().tolist() == [100.0]
    # the decay acts on the rows of key channels, and the read-out sees the token's own write
    o, S = plain.gated_linear_scan(torch.tensor([[1.0, 1.0]] * 2, dtype=f64), torch.tensor([[1.0, 2.0], [0.0, 1.0]], dtype=f64),
                                   torch.tensor([[3.0], [5.0]], dtype=f64), torch.tensor([[0.1, 0.1], [0.5, 1.0]], dtype=f64))
    assert o.flatten().tolist() == [9.0, 12.5] and S.flatten().tolist() == [1.5, 11.0]
    # sigmoid(0)^(1/2)
    w = {"a1": torch.zeros(1, 2, dtype=f64), "a2": torch.zeros(3, 1, dtype=f64), "a2.b": torch.zeros(3, dtype=f64)}
    assert torch.allclose(plain.channel_decay(torch.ones(1, 2, dtype=f64), w, "", 2.0), torch.full((1, 3), 0.5 ** 0.5, dtype=f64))
    o, _ = plain.linear_recurrence(torch.tensor([[0.5], [0.25]], dtype=f64), torch.tensor([[4.0], [1.0]], dtype=f64))
    assert o.flatten().tolist() == [4.0, 2.0]


def without(names):
    """The plain weights with some tensors changed: a mistake of the kind that forgets them."""
    def edit(w):
        return {k: (f(v) if (f := next((g for end, g in names if k.endswith(end)), None)) else v) for k, v in w.items()}
    return edit


def changed(path, value):
    def edit(cfg):
        cfg = copy.deepcopy(cfg)
        for layer in cfg["layers"]:
            m = layer["mixer"]
            for key in path[:-1]:
                m = m.get(key) or {}
            if path[-1] in m:
                m[path[-1]] = value(m[path[-1]])
        return cfg
    return edit


MISTAKES = {
    "a window of one key less (left)": (changed(("left", "mask", "size"), lambda s: s - 1), None),
    "a window of one key more (left)": (changed(("left", "mask", "size"), lambda s: s + 1), None),
    "a window of one key less (latent)": (changed(("mask", "size"), lambda s: s - 1), None),
    "a window of one key more (latent)": (changed(("mask", "size"), lambda s: s + 1), None),
    "no sink": (None, without([(".sink", lambda t: t - 50.0)])),
    "no cap on the scores": (changed(("left", "softcap"), lambda c: None), None),
    "no slowed frequencies": (changed(("left", "rot", "scaling"), lambda s: None), None),
    "another part of the head rotated": (changed(("left", "rot", "dims"), lambda n: n // 2), None),
    "no tau": (changed(("right", "tau"), lambda t: 1.0), None),
    "the sides' scales changed over": (changed(("left_scale",), lambda s: s + 0.1), None),
    "no convolution's past": (None, without([(".conv", lambda t: torch.cat([torch.zeros_like(t[:, :-1]), t[:, -1:]], 1))])),
    "no decay's bias": (None, without([(".a2.b", torch.zeros_like)])),
    "gates changed over": (None, without([(".ra.b", lambda t: -t)])),
    "no feed-forward biases": (None, without([(".up.b", torch.zeros_like)])),
}


@pytest.mark.parametrize("what", sorted(MISTAKES))
def test_bounds_notice_a_mistake(what):
    """Each mistake, planted in the plain model, moves logits beyond what the suites allow bfloat16 (three times what its
    rounding alone does at worst, or 1.3 times in the mean)."""
    edit_cfg, edit_w = MISTAKES[what]
    cfg = sharpened(SET["A"], 2.0)
    w = make_weights(cfg, seed=66)
    toks = random_tokens(cfg, 60, seed=100)
    want, rounded = plain_logits(cfg, w, toks), plain_logits_bf16(cfg, w, toks)
    moved = [rel_err(a, b) for a, b in zip(rounded, want)]
    wrong = plain_logits(edit_cfg(cfg) if edit_cfg else cfg, edit_w(w) if edit_w else w, toks)
    errors = [rel_err(a, b) for a, b in zip(wrong, want)]
    assert max(errors) > 3 * max(moved) + BF16_FLOOR or float(np.mean(errors)) > 1.3 * float(np.mean(moved)) + 1e-3, \
        (what, max(errors), max(moved), float(np.mean(errors)), float(np.mean(moved)))
