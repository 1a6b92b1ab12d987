"""Vufolorn on the host: the configuration reader, the plan, what the cache manager makes of it, the plain implementation's
functions on cases worked out by hand, and how much the crafted folder shows of a mistake."""

import copy
import json
import math

import pytest
import torch

from kestrel_amd.cache.manager import CacheManager
from kestrel_amd.config.registry import resolve
from kestrel_amd.models import vufolorn
from kestrel_amd.models.decoder import DecoderModel
from tests import helpers
from tests import vufolorn_cases as cases
from tests.plain import vufolorn_plain as plain

F64 = torch.float64


def _plan(name):
    config = cases.CONFIGS[name]
    spec = resolve(config)
    assert spec.name == "vufolorn"
    return spec.build_plan(spec.read_config(config))


def test_the_configuration_survives_a_round_trip():
    for name, config in cases.CONFIGS.items():
        assert vufolorn.VufolornConfig.from_dict(config).to_dict() == config, name


def test_a_configuration_without_a_name_is_recognised():
    for name, config in cases.CONFIGS.items():
        nameless = {k: v for k, v in config.items() if k != "architecture"}
        assert resolve(nameless).name == "vufolorn", name


@pytest.mark.parametrize("edit, message", [
    (lambda c: c["layers"][0].update(type="attention"), "this design has the mixers"),
    (lambda c: c["layers"][1]["mixer"]["decay"].pop(), "one per head"),
    (lambda c: c["layers"][1]["mixer"].update(decay=[0.5, 0.5, 0.0, 0.5]), "above 0"),
    (lambda c: c["layers"][1]["mixer"].update(decay=[0.5, 0.5, 1.5, 0.5]), "above 0"),
    (lambda c: c["layers"][0]["mixer"].pop("kv_rank"), "kv_rank missing"),
    (lambda c: c["layers"][0]["mixer"]["mask"].update(size=0), "positive integer"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(top=9), "exceeds"),
    (lambda c: c["layers"][0]["mlp"].update(kind="dense"), "kind 'moe'"),
    (lambda c: c["loop"].update(stop=9), "does not lie within"),
    (lambda c: c.pop("norm"), "'norm' missing"),
])
def test_what_the_configuration_reader_refuses(edit, message):
    config = json.loads(json.dumps(cases.CONFIGS["P"]))
    edit(config)
    with pytest.raises(ValueError, match=message):
        vufolorn.VufolornConfig.from_dict(config)


def test_tensor_names_and_shapes():
    params = DecoderModel(_plan("P")).params()
    assert params["embed"].shape == (300, 128) and params["embed.norm"].shape == (128,) and params["final.norm"].shape == (128,)
    assert params["loop.step"].shape == (2, 128) and "head" not in params
    for name in ("norm1", "norm1b", "ls1", "norm2", "norm2b", "ls2"):
        assert params["l0." + name].shape == (128,)
    # latent attention: queries directly, one gate number per head
    assert params["l0.mix.q"].shape == (64, 128) and params["l0.mix.dkv"].shape == (64, 128) and params["l0.mix.dkv.norm"].shape == (64,)
    assert params["l0.mix.uk"].shape == (64, 64) and params["l0.mix.uv"].shape == (96, 64) and params["l0.mix.g"].shape == (4, 128)
    assert params["l0.mix.o"].shape == (128, 96) and "l0.mix.k" not in params
    # the recurrence: keys and values of their own sizes, one gain over all heads
    assert params["l1.mix.q"].shape == (128, 128) and params["l1.mix.k"].shape == (128, 128) and params["l1.mix.v"].shape == (160, 128)
    assert params["l1.mix.g"].shape == (160, 128) and params["l1.mix.norm"].shape == (160,) and params["l1.mix.o"].shape == (128, 160)
    # plain experts
    assert params["l0.mlp.e5.up"].shape == (48, 128) and params["l0.mlp.e5.down"].shape == (128, 48) and "l0.mlp.e0.gate" not in params
    assert params["l0.mlp.router"].shape == (6, 128) and params["l0.mlp.router.b"].shape == (6,) and "l0.mlp.e6.up" not in params
    assert params["l0.mlp.shared.up"].shape == (32, 128) and params["l0.mlp.shared.sg"].shape == (1, 128)
    # a layer without a feed-forward has none of its norms; one without a shared expert none of its tensors
    assert "l3.norm2" not in params and "l3.ls2" not in params and "l3.mlp.router" not in params
    assert "l0.mlp.shared.up" not in DecoderModel(_plan("Q")).params()


def test_schedule_junction_cache_groups_and_state():
    plan = _plan("P")
    assert [(e.layer, e.before, e.passage) for e in plan.schedule] == [
        (0, None, 0), (1, "loop_step", 0), (2, None, 0), (1, "loop_step", 1), (2, None, 1), (3, None, 0)]
    assert plan.tied_head and plan.junctions["loop_step"].embedding_from == 1 and plan.embedding_norm is not None
    needs = DecoderModel(plan).cache_needs()
    manager = CacheManager(needs, 16, 40, 3)
    assert len(manager.groups) == 2                       # one per window and latent size; every pass has pages of its own
    assert sorted(len(g.entries) for g in manager.groups) == [1, 2]
    assert [s is not None for _c, s, _r in needs] == [False, True, False, True, False, True]
    assert needs[1][1].shape == (4 * 40 * 32,) and needs[1][1].dtype == "float32"
    assert _plan("R").junctions == {} and "loop.step" in _plan("R").ignored_prefixes
    plan = _plan("S")
    assert [e.before for e in plan.schedule] == ["loop_step", None]


def test_a_window_gives_its_pages_back():
    manager = CacheManager(DecoderModel(_plan("P")).cache_needs(), 16, 30, 2)
    slot = manager.admit()
    manager.ensure(slot, 100)
    manager.trim(slot, 100)
    for g, group in enumerate(manager.groups):
        kept = [i for i, p in enumerate(manager.block_table(g, slot)) if p >= 0]
        first = (100 + 1 - group.spec.window) // 16
        assert kept == list(range(first, 7)), group.spec.window
    manager.check()


# ---------------------------------------------------------------------------------------------- the plain implementation
def test_plain_recurrence_by_hand():
    q = torch.tensor([[[1.0, 2.0]], [[3.0, 0.0]], [[0.0, 1.0]]], dtype=F64)
    k = torch.tensor([[[1.0, 0.0]], [[0.0, 1.0]], [[1.0, 1.0]]], dtype=F64)
    v = torch.tensor([[[10.0]], [[20.0]], [[30.0]]], dtype=F64)
    # S: (10, 0); (5, 20); (2.5 + 30, 10 + 30)
    assert plain.decayed_sum(q, k, v, [0.5]).flatten().tolist() == [10.0, 15.0, 40.0]
    assert plain.decayed_sum(q, k, v, [1.0]).flatten().tolist() == [10.0, 30.0, 50.0]


def test_plain_window_and_routing_by_hand():
    seen = plain.window_mask(4, 2)
    assert seen.tolist() == [[True, False, False, False], [True, True, False, False], [False, True, True, False], [False, False, True, True]]
    assert plain.window_mask(3, None).tolist() == [[True, False, False], [True, True, False], [True, True, True]]
    order, weights = plain.routing(torch.tensor([[0.0, math.log(3.0), math.log(1.0), -5.0]], dtype=F64), 2)
    assert order.tolist() == [[1, 0]] and torch.allclose(weights, torch.tensor([[0.75, 0.25]], dtype=F64))
    assert plain.relu_squared(torch.tensor([-2.0, 3.0])).tolist() == [0.0, 9.0]


def test_plain_runs_of_the_loop():
    assert plain.runs_of({"layers": [0] * 4, "loop": {"start": 1, "stop": 3, "times": 2}}) == [
        (0, None), (1, 0), (2, None), (1, 1), (2, None), (3, None)]
    assert plain.runs_of({"layers": [0, 0]}) == [(0, None), (1, None)]


def _moved(a, b):
    d = a - b
    d = d - d.mean(dim=-1, keepdim=True)
    return d.pow(2).mean(dim=-1).sqrt() / b.std(dim=-1, unbiased=False)


@pytest.mark.parametrize("layer", [0, 2])
def test_the_crafted_folder_shows_a_window_that_is_one_off(layer):
    """A window one too short, one too long, in the plain implementation: the row of the calling token moves by several
    times what a bfloat16 run may differ by, where the echo stands at the window's edge."""
    folder = cases.crafted(cases.folder_for("P", torch.bfloat16))
    config, weights = cases.config_of(folder), cases.stored_weights(folder)
    window = config["layers"][layer]["mixer"]["mask"]["size"]
    at = 70
    for distance, size in ((window - 1, window - 1), (window, window + 1)):
        ids = list(range(10, 90))
        ids[at], ids[at - distance] = cases.CALL, cases.ECHO
        want = plain.forward(config, weights, ids)
        wrong = copy.deepcopy(config)
        wrong["layers"][layer]["mixer"]["mask"]["size"] = size
        assert float(_moved(plain.forward(wrong, weights, ids), want)[at]) > 0.15, (distance, size)


def test_the_folders_show_other_mistakes():
    """A state that is lost, an embedding that does not come back in a later pass, a pass vector of the wrong pass, a gate
    left out: each moves the logits by far more than a run may differ by."""
    folder = cases.folder_for("P", torch.bfloat16)
    config, weights = cases.config_of(folder), cases.stored_weights(folder)
    ids = helpers.random_ids(7, 60, config["vocab"])
    want = plain.forward(config, weights, ids)

    def edited(edit):
        w = dict(weights)
        edit(w)
        return float(_moved(plain.forward(config, w, ids), want)[20:].median())

    original = plain.decayed_sum

    def forgetful(q, k, v, decay):
        half = q.shape[0] // 2
        return torch.cat([original(q[:half], k[:half], v[:half], decay), original(q[half:], k[half:], v[half:], decay)])

    plain.decayed_sum = forgetful
    try:
        lost = plain.forward(config, weights, ids)
    finally:
        plain.decayed_sum = original
    assert float(_moved(lost, want)[30:].median()) > 0.1
    assert edited(lambda w: w.update({"loop.step": w["loop.step"].roll(1, 0)})) > 0.05
    assert edited(lambda w: w.update({"l0.mix.g": torch.zeros_like(w["l0.mix.g"])})) > 0.05
    assert edited(lambda w: w.update({"l1.ls1": torch.ones_like(w["l1.ls1"])})) > 0.05
    runs = plain.runs_of
    plain.runs_of = lambda c: [(i, 0 if number is not None else None) for i, number in runs(c)]
    try:
        assert float(_moved(plain.forward(config, weights, ids), want).median()) > 0.1
    finally:
        plain.runs_of = runs
