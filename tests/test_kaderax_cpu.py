"""Kaderax through the engine's host logic on the CPU (the product's model, cache, step function and generation loop
over the plain torch kernels of tests/ref_ops.py), against the plain implementation in tests/plain."""
import math
import random

import pytest
import torch

from trapetum_amd.config import ConfigError, KaderaxConfig
from trapetum_amd.engine.generate import generate
from trapetum_amd.parts.attention import Attention
from trapetum_amd.weights import write_model_folder

from . import kaderax_tiny as kt
from . import model_cases as mc
from .cpu_engine import load_cpu_model
from .plain import kaderax_plain as plain
from .tiny import random_tokens

TOL = 2e-5


def loaded(tmp_path_factory, which, tol):
    folder = kt.make_folder(tmp_path_factory.mktemp("k"), which)
    model, cfg = load_cpu_model(folder)
    pcfg, pw = plain.read_folder(folder)
    return model, cfg, pcfg, pw, tol


@pytest.fixture(scope="module", params=["P", "Q", "R", "T"])
def m(request, tmp_path_factory):
    return loaded(tmp_path_factory, request.param, TOL)


@pytest.fixture(scope="module")
def sharp(tmp_path_factory):
    return loaded(tmp_path_factory, "S", 4e-3)


def test_layout_cache_and_states(m):
    model, cfg, pcfg, _, _ = m
    names = set(model.tensor_layout())
    assert {"embed", "head", "final.norm"} <= names and ("loop.in" in names) == ("loop" in pcfg)
    cache = model.new_cache(max_tokens=64, page_size=16)
    states = model.entry_state_specs()
    order = plain.running_order(pcfg)
    assert [e.layer for e in model.schedule] == [i for i, _ in order]        # a looped layer is scheduled once per pass ...
    assert [e.before is not None for e in model.schedule] == [enters for _, enters in order]
    sites = []
    for e, (i, _) in enumerate(order):
        mx, site = pcfg["layers"][i]["mixer"], cache.site(e)
        if pcfg["layers"][i]["type"] == "parallel":
            row = max(mx["left"]["dim"], mx["left"]["vdim"])
            assert list(site.spec.tensors) == [("k", (mx["left"]["kv_heads"], row)), ("v", (mx["left"]["kv_heads"], row))]
            r = mx["right"]
            assert states[e]["mixer.right.memory"].shape == (r["heads"], r["vdim"], r["dim"])
        else:
            assert list(site.spec.tensors) == [("latent", (1, mx["rot_dim"] + mx["kv_rank"]))]
        sites.append((site.group_index, site.index_in_group))
    assert len(set(sites)) == len(sites)                                     # ... with a cache of its own for each
    assert len({id(p) for p in model.added if p is not None}) <= 1           # the passes share one matrix


def test_config_errors():
    for path, value, match in [(("layers", 1, "mixer", "left", "kv_heads"), 3, "no multiple"),
                               (("layers", 1, "mixer", "left", "softcap"), 0.0, "positive"),
                               (("layers", 1, "mixer", "left", "q_temp", "every"), 0, "positive"),
                               (("layers", 1, "mixer", "left", "bias_max"), 0, "positive"),
                               (("layers", 1, "mixer", "right", "decay"), [0.5], "list of 3"),
                               (("layers", 1, "mixer", "right", "decay"), [0.5, 1.5, 0.5], "between"),
                               (("layers", 0, "mixer", "rot", "dims"), 10, "at most"),
                               (("layers", 0, "mixer", "q_rank"), 0, "positive"),
                               (("layers", 0, "mlp", "kind"), "moe", "dense"), (("layers", 0, "mlp", "ff"), 0, "positive"),
                               (("layers", 0, "type"), "other", "mixers are"),
                               (("loop", "stop"), 6, "inside"), (("loop", "start"), 4, "below"), (("loop", "times"), 0, "positive")]:
        bad = kt.config_p()
        at = bad
        for k in path[:-1]:
            at = at[k]
        at[path[-1]] = value
        with pytest.raises(ConfigError, match=match):
            KaderaxConfig.from_dict(bad)
    for key, where in (("norm", None), ("residual_mult", None), ("scale", ("layers", 0, "mixer")), ("left_scale", ("layers", 1, "mixer")),
                       ("coef", ("layers", 1, "mixer", "left", "q_temp")), ("decay", ("layers", 1, "mixer", "right")), ("times", ("loop",))):
        d = kt.config_p()
        at = d
        for k in where or ():
            at = at[k]
        del at[key]
        with pytest.raises(ConfigError, match=key):
            KaderaxConfig.from_dict(d)


@pytest.mark.parametrize("rows,reach", [(2, 3), (8, 5), (20, 90), (32, 129), (32, 17), (64, 1000), (24, 96)])
def test_buckets_of_distances(rows, reach):
    """Every distance below half the rows has its own; from there on the rows follow logarithmically and none is skipped
    backwards; from the reach on it is the last one, the same as the table by distance holds."""
    got = [Attention.bucket_of_distance(n, rows, reach) for n in range(3 * reach)]
    assert got == [plain.bucket(n, rows, reach) for n in range(3 * reach)]
    assert got[:rows // 2] == list(range(rows // 2))
    assert all(b >= a for a, b in zip(got, got[1:])) and set(got[reach:]) == {rows - 1}
    part = Attention(8, 2, 1, 4, 1.0, distance_bias="rel", bias_reach=reach)
    table = torch.randn(rows, 2, generator=torch.Generator().manual_seed(1))
    wide = part._table_by_distance(table)
    assert wide.shape == (2, reach + 1)
    for n in range(2 * reach):
        assert torch.equal(wide[:, min(n, reach)], table[got[n]])


def test_bias_table_that_does_not_reach():
    for rows, reach in ((1, 10), (32, 16), (32, 3)):
        with pytest.raises(ValueError, match="does not reach"):
            Attention(8, 2, 1, 4, 1.0, distance_bias="rel", bias_reach=reach)._table_by_distance(torch.zeros(rows, 2))


def test_temperature_of_the_query():
    assert plain.query_temperature(0, {"coef": 0.5, "every": 4}) == 1.0          # positions 0 .. 2: floor((p + 1) / 4) = 0
    assert plain.query_temperature(2, {"coef": 0.5, "every": 4}) == 1.0
    assert plain.query_temperature(3, {"coef": 0.5, "every": 4}) == 1.0 + 0.5 * math.log(2.0)


def test_whole_and_token_by_token(m):
    mc.whole_and_token_by_token(m, n=60)


def test_prompt_then_decode(m):
    mc.prompt_then_decode(m, n=80, tail=45)


def test_portions(m):
    mc.portions(m)


def test_unequal_batches_and_reuse(m):
    mc.unequal_batches_and_reuse(m)


def test_slot_after_a_longer_sequence(m):
    mc.slot_after_a_longer_sequence(m)


def test_sharp_scores(sharp):
    mc.sharp_scores_far_keys(sharp, n=90)


def test_greedy_generation_through_the_loop(m):
    model, cfg, pcfg, pw, _ = m
    prompts = [random_tokens(n, cfg.vocab_size, 70 + n) for n in (7, 1, 19, 4)]
    want = [plain.greedy_generate(pcfg, pw, p, 6) for p in prompts]
    cache = model.new_cache(max_tokens=64 * 2, page_size=64)             # room for two sequences at a time: slots are used again
    assert generate(model, cache, prompts, max_tokens=6, stop_ids=()) == want
    assert cache.live_slots() == [] and cache.tokens_held() == 0


@pytest.mark.parametrize("case", range(8))
def test_random_configuration(case, tmp_path):
    """A configuration drawn at random: a prompt whole, then in two portions and single tokens."""
    rng = random.Random(1300 + case)
    cfg = kt.draw(rng)
    folder = str(tmp_path)
    write_model_folder(KaderaxConfig.from_dict(cfg), folder, seed=case, sigma=0.1, sigma_norm=0.2)
    model, c = load_cpu_model(folder)
    pcfg, pw = plain.read_folder(folder)
    assert pcfg == cfg
    toks = random_tokens(57, c.vocab_size, case)
    ref = plain.forward(pcfg, pw, toks)
    cache = model.new_cache(max_tokens=128, page_size=16)
    s = cache.acquire()
    got = [model.step(cache, [s], toks[:20], counts=[20], want=list(range(20))),
           model.step(cache, [s], toks[20:47], counts=[27], want=list(range(27)))]
    got += [model.step(cache, [s], [t]) for t in toks[47:]]
    mc.rows_close(torch.cat(got), ref, 5e-5, cfg)
