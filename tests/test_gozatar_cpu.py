"""Gozatar on the host: the configuration reader, the plan, what the cache manager makes of it, the plain implementation's
functions on cases worked out by hand, and how much the folders of the tests show of a mistake."""

import copy
import json
import math

import pytest
import torch

from kestrel_amd.cache.manager import CacheManager
from kestrel_amd.config.registry import resolve
from kestrel_amd.models import gozatar
from kestrel_amd.models.decoder import DecoderModel
from tests import gozatar_cases as cases
from tests import helpers
from tests.plain import gozatar_plain as plain

F64 = torch.float64


def _plan(name):
    config = cases.CONFIGS[name]
    spec = resolve(config)
    assert spec.name == "gozatar"
    return spec.build_plan(spec.read_config(config))


def test_the_configuration_survives_a_round_trip():
    for name, config in cases.CONFIGS.items():
        assert gozatar.GozatarConfig.from_dict(config).to_dict() == config, name


def test_a_configuration_without_a_name_is_recognised():
    for name, config in cases.CONFIGS.items():
        nameless = {k: v for k, v in config.items() if k != "architecture"}
        assert resolve(nameless).name == "gozatar", name


@pytest.mark.parametrize("edit, message", [
    (lambda c: c["layers"][0].update(type="attention"), "mixer 'parallel'"),
    (lambda c: c["layers"][0]["mixer"].pop("left_scale"), "left_scale missing"),
    (lambda c: c["layers"][0]["mixer"]["left"].update(kv_heads=3), "no multiple"),
    (lambda c: c["layers"][0]["mixer"]["left"]["rot"].update(dims=34), "even and at most dim"),
    (lambda c: c["layers"][0]["mixer"]["left"]["rot"].update(dims=3), "even and at most dim"),
    (lambda c: c["layers"][0]["mixer"]["left"]["mask"].update(size=0), "positive integer"),
    (lambda c: c["layers"][0]["mixer"]["right"].update(tau=0), "must be positive"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(top=5), "can be chosen"),
    (lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(count=3), "must divide"),
    (lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(keep=5), "must divide"),
    (lambda c: c["layers"][0]["mlp"]["expert"].update(limit=0.0), "must be positive"),
    (lambda c: c["layers"][1]["mlp"].update(kind="gated"), "'dense' and 'moe'"),
    (lambda c: c.pop("streams"), "'streams' missing"),
    (lambda c: c.update(streams=0), "positive integer"),
])
def test_what_the_configuration_reader_refuses(edit, message):
    config = json.loads(json.dumps(cases.CONFIGS["P"]))
    edit(config)
    with pytest.raises(ValueError, match=message):
        gozatar.GozatarConfig.from_dict(config)


def test_tensor_names_and_shapes():
    params = DecoderModel(_plan("P")).params()
    assert params["embed"].shape == (300, 128) and params["final.norm"].shape == (128,) and params["head"].shape == (300, 128)
    for q in ("1", "2"):
        assert params[f"l0.norm{q}"].shape == (128,)
        assert params[f"l0.hc{q}.in"].shape == (3,) and params[f"l0.hc{q}.out"].shape == (3,) and params[f"l0.hc{q}.mix"].shape == (3, 3)
    left, right = "l0.mix.left.", "l0.mix.right."
    assert params[left + "q"].shape == (128, 128) and params[left + "k"].shape == (64, 128) and params[left + "v"].shape == (128, 128)
    assert params[left + "q.conv"].shape == (128, 4) and params[left + "k.conv"].shape == (64, 4) and params[left + "v.conv"].shape == (128, 4)
    assert params[left + "o"].shape == (128, 256)
    assert params[right + "q"].shape == (96, 128) and params[right + "k"].shape == (96, 128) and params[right + "v"].shape == (120, 128)
    assert params[right + "g"].shape == (120, 128) and params[right + "norm"].shape == (40,) and params[right + "o"].shape == (128, 120)
    assert params[right + "a1"].shape == (16, 128) and params[right + "a2"].shape == (96, 16) and params[right + "a2.b"].shape == (96,)
    assert params["l0.mlp.e7.gate"].shape == (48, 128) and params["l0.mlp.e7.down"].shape == (128, 48) and "l0.mlp.e8.up" not in params
    assert params["l0.mlp.router"].shape == (8, 128) and params["l0.mlp.correction"].shape == (8,)
    assert params["l0.mlp.shared.up"].shape == (48, 128) and params["l2.mlp.shared.gate"].shape == (80, 128)
    assert params["l1.mlp.up"].shape == (176, 128) and params["l1.mlp.down"].shape == (128, 176) and "l1.mlp.router" not in params
    # a layer without a feed-forward has neither its norm nor its numbers; one without convolutions no taps
    assert "l3.norm2" not in params and "l3.hc2.in" not in params
    params = DecoderModel(_plan("Q")).params()
    assert "l1.mix.left.q.conv" not in params and params["l2.mix.left.q.conv"].shape == (72, 1) and "l0.mlp.shared.up" not in params


def test_the_decay_rank_may_be_left_to_the_weights():
    config = json.loads(json.dumps(cases.CONFIGS["P"]))
    for layer in config["layers"]:
        layer["mixer"]["right"].pop("decay_rank")
    spec = resolve(config)
    params = DecoderModel(spec.build_plan(spec.read_config(config))).params()
    assert params["l0.mix.right.a1"].shape == (-1, 128) and params["l0.mix.right.a2"].shape == (96, -1)


def test_streams_cache_groups_and_state():
    plan = _plan("P")
    assert plan.streams == 3 and all(layer.arrangement == "streams" for layer in plan.layers) and not plan.tied_head
    needs = DecoderModel(plan).cache_needs()
    manager = CacheManager(needs, 16, 40, 3)
    assert [len(g.entries) for g in manager.groups] == [1, 1, 1, 1]         # (four sizes of keys, values and windows)
    # the convolution's last rows and the recurrence's state lie side by side in one tensor per layer, on 16-byte places
    assert needs[0][1].shape == (3 * 320 + 3 * 32 * 40,) and needs[0][1].dtype == "float32"
    needs = DecoderModel(_plan("Q")).cache_needs()
    assert needs[0][1].shape == ((5 * (36 + 12 + 10) + 3) // 4 * 4 + (5 * 70 + 3) // 4 * 4,)
    assert needs[1][1].shape == (2 * 6 * 33,) and needs[2][1].shape == (3 * 22 * 12,)       # no taps, or one: no rows to keep


def test_a_window_gives_its_pages_back():
    manager = CacheManager(DecoderModel(_plan("P")).cache_needs(), 16, 60, 2)
    slot = manager.admit()
    manager.ensure(slot, 100)
    manager.trim(slot, 100)
    for g, group in enumerate(manager.groups):
        kept = [i for i, p in enumerate(manager.block_table(g, slot)) if p >= 0]
        first = (100 + 1 - group.spec.window) // 16
        assert kept == list(range(first, 7)), group.spec.window
    manager.check()


# ---------------------------------------------------------------------------------------------- the plain implementation
def test_plain_streams_by_hand():
    X = torch.tensor([[[1.0]], [[10.0]]], dtype=F64)
    assert float(plain.read_streams(X, torch.tensor([2.0, 0.5], dtype=F64))) == 7.0
    # from and to: the new first stream is 1 * 0.5 + 10 * 3, the new second 1 * 2 + 10 * 1
    new = plain.write_streams(X, torch.tensor([[0.5, 2.0], [3.0, 1.0]], dtype=F64), torch.tensor([1.0, -1.0], dtype=F64), torch.tensor([[100.0]], dtype=F64))
    assert new.flatten().tolist() == [130.5, -88.0]


def test_plain_recurrence_by_hand():
    q = torch.tensor([[[1.0, 2.0]], [[3.0, 0.0]], [[1.0, 1.0]]], dtype=F64)
    k = torch.tensor([[[1.0, 1.0]], [[0.0, 1.0]], [[1.0, 0.0]]], dtype=F64)
    v = torch.tensor([[[10.0]], [[20.0]], [[30.0]]], dtype=F64)
    alpha = torch.tensor([[[0.1, 0.1]], [[0.5, 1.0]], [[0.5, 0.1]]], dtype=F64)
    # S: (10, 10); (5, 10 + 20); (2.5 + 30, 3)
    assert plain.gated_sum(q, k, v, alpha).flatten().tolist() == [30.0, 15.0, 35.5]
    assert float(plain.decays(torch.tensor(0.0, dtype=F64), 2.0)) == pytest.approx(math.sqrt(0.5))


def test_plain_convolution_rotation_and_window_by_hand():
    u = torch.tensor([[1.0], [2.0], [3.0]], dtype=F64)
    assert plain.causal_conv(u, torch.tensor([[100.0, 10.0, 1.0]], dtype=F64)).flatten().tolist() == [1.0, 12.0, 123.0]
    x = torch.tensor([[[1.0, 5.0, 0.0, 7.0]]] * 2, dtype=F64)
    turned = plain.rotate_halves(x, 2, 1.0)          # channels 0 and 1, one radian a place
    assert turned[0, 0].tolist() == [1.0, 5.0, 0.0, 7.0]
    assert turned[1, 0].tolist() == pytest.approx([math.cos(1) - 5 * math.sin(1), 5 * math.cos(1) + math.sin(1), 0.0, 7.0])
    assert plain.window_mask(3, 2).tolist() == [[True, False, False], [True, True, False], [False, True, True]]


def test_plain_routing_and_expert_by_hand():
    # two groups of two: the group with the largest single score does not have the largest sum
    logit = lambda p: math.log(p / (1 - p))  # noqa: E731
    z = torch.tensor([[logit(0.8), logit(0.1), logit(0.5), logit(0.6)]], dtype=F64)
    none = torch.zeros(4, dtype=F64)
    order, weights = plain.routing(z, none, 1, (2, 1))
    assert order.tolist() == [[3]] and weights.tolist() == [[1.0]]
    order, weights = plain.routing(z, none, 2, None)
    assert order.tolist() == [[0, 3]] and weights[0].tolist() == pytest.approx([0.8 / 1.4, 0.6 / 1.4])
    # corrections that make every choice score negative: experts of groups that are not kept stay out; weights leave them out
    order, weights = plain.routing(z, torch.tensor([-3.0, -3.0, -2.0, -2.0], dtype=F64), 2, (2, 1))
    assert order.tolist() == [[3, 2]] and weights[0].tolist() == pytest.approx([0.6 / 1.1, 0.5 / 1.1])
    w = {"e.gate": torch.tensor([[3.0]], dtype=F64), "e.up": torch.tensor([[-5.0]], dtype=F64), "e.down": torch.tensor([[1.0]], dtype=F64)}
    got = float(plain.expert(torch.ones(1, 1, dtype=F64), w, "e", 1.5))
    assert got == pytest.approx(1.5 / (1 + math.exp(-1.702 * 1.5)) * (-1.5 + 1))


# ---------------------------------------------------------------------------------------------- what the folders show
def _moved(a, b):
    d = a - b
    d = d - d.mean(dim=-1, keepdim=True)
    return d.pow(2).mean(dim=-1).sqrt() / b.std(dim=-1, unbiased=False)


@pytest.mark.parametrize("layer", [0, 1, 2, 3])
def test_the_crafted_folder_shows_a_window_that_is_one_off(layer):
    """A window one too short, one too long, in the plain implementation: the row of the calling token moves by several
    times what a bfloat16 run may differ by, where the echo stands at the window's edge."""
    folder = cases.crafted(cases.folder_for("P", torch.bfloat16))
    config, weights = cases.config_of(folder), cases.stored_weights(folder)
    window = config["layers"][layer]["mixer"]["left"]["mask"]["size"]
    at = 70
    for distance, size in ((window - 1, window - 1), (window, window + 1)):
        ids = list(range(10, 90))
        ids[at], ids[at - distance] = cases.CALL, cases.ECHO
        want = plain.forward(config, weights, ids)
        wrong = copy.deepcopy(config)
        wrong["layers"][layer]["mixer"]["left"]["mask"]["size"] = size
        assert float(_moved(plain.forward(wrong, weights, ids), want)[at]) > 0.15, (distance, size)


def _patched(name, replacement, run):
    original = getattr(plain, name)
    setattr(plain, name, replacement(original))
    try:
        return run()
    finally:
        setattr(plain, name, original)


def test_the_folders_show_other_mistakes():
    """A state or a convolution's rows that are lost, a transposed mix, streams written one after the other, a clamp, a shift or a
    correction left out, groups that count by one score, a norm in the wrong place: each moves the logits by far more than a
    run may differ by."""
    folder = cases.model_dir("P")
    config, weights = cases.config_of(folder), cases.stored_weights(folder)
    ids = helpers.random_ids(7, 60, config["vocab"])
    run = lambda: plain.forward(config, weights, ids)  # noqa: E731
    want = run()
    half = len(ids) // 2

    def moved(name, replacement):
        return _moved(_patched(name, replacement, run), want)

    lost = moved("gated_sum", lambda f: lambda q, k, v, a: torch.cat([f(q[:half], k[:half], v[:half], a[:half]), f(q[half:], k[half:], v[half:], a[half:])]))
    assert float(lost[half:].median()) > 0.1
    lost = moved("causal_conv", lambda f: lambda u, w: torch.cat([f(u[:half], w), f(u[half:], w)]))
    assert float(lost[half:half + 2].min()) > 0.1
    assert float(moved("write_streams", lambda f: lambda X, m, o, y: f(X, m.T, o, y)).median()) > 0.1

    def one_by_one(_f):
        def write(X, m, o, y):
            X = X.clone()
            for t in range(X.shape[0]):
                X[t] = sum(m[s, t] * X[s] for s in range(X.shape[0])) + o[t] * y
            return X
        return write

    assert float(moved("write_streams", one_by_one).median()) > 0.05
    assert float(moved("expert", lambda f: lambda h, w, p, limit: f(h, w, p, 1e9)).median()) > 0.05
    assert float(moved("routing", lambda f: lambda z, c, top, groups: f(z, 0 * c, top, groups)).median()) > 0.05
    assert float(moved("routing", lambda f: lambda z, c, top, groups: f(z, c, top, None)).quantile(0.9)) > 0.05
    assert float(moved("decays", lambda f: lambda z, tau: f(z, 1.0)).median()) > 0.1
    assert float(moved("rotate_halves", lambda f: lambda x, dims, base: x).median()) > 0.05
