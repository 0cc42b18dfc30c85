"""Sosuvik's configuration on the CPU: keys, refusals, the round trip, the model as a list of parts, the order of running with
a loop, tensor names and shapes, the pages of chunked attention, and step costs."""
import copy

import pytest
import torch

from plain import sosuvik_plain as P
from pulse_infer_amd.cache.manager import CacheManager
from pulse_infer_amd.cache.specs import PagedKVSpec
from pulse_infer_amd.config import ConfigError, SosuvikConfig, config_from_dict
from pulse_infer_amd.models.causal_lm import expected_tensors
from pulse_infer_amd.models.cost import step_cost
from pulse_infer_amd.ops.attention_mfma import CHUNK_SLACK, split_span

SCALING = {"factor": 4.0, "original": 512.0, "fast": 16.0, "slow": 2.0}
ATTENTION = {"dim": 32, "heads": 6, "kv_heads": 3, "mask": {"size": 21}, "rot": {"base": 1e4, "dims": 16, "scaling": SCALING},
             "scale": 0.2, "softcap": 7.0, "vdim": 16}
LATENT = {"dim": 16, "heads": 5, "kv_rank": 40, "rot": {"base": 500.0, "dims": 8}, "rot_dim": 8, "scale": 0.3, "vdim": 20}
MOE = {"expert": {"ff": 56, "limit": 0.9}, "kind": "moe",
       "router": {"experts": 10, "groups": {"count": 5, "keep": 2}, "scale": 1.25, "top": 3}}
CONFIG = {
    "architecture": "Sosuvik", "norm": {"eps": 1e-5}, "vocab": 311, "width": 96, "logit_scale": 1.5,
    "loop": {"start": 1, "stop": 3, "times": 2},
    "layers": [
        {"type": "attention", "mixer": ATTENTION, "mlp": MOE},
        {"type": "latent_attention", "mixer": LATENT, "mlp": None},
        {"type": "attention", "mixer": dict(ATTENTION, mask={"size": 50}), "mlp": MOE},
        {"type": "latent_attention", "mixer": dict(LATENT, heads=2), "mlp": MOE},
    ],
}


def broken(path, value):
    data = copy.deepcopy(CONFIG)
    at = data
    for key in path[:-1]:
        at = at[key]
    if value is KeyError:
        del at[path[-1]]
    else:
        at[path[-1]] = value
    return data


def test_round_trip_and_registry():
    cfg = config_from_dict(CONFIG)
    assert isinstance(cfg, SosuvikConfig)
    assert cfg.to_dict() == CONFIG
    assert SosuvikConfig.from_dict(cfg.to_dict()).to_dict() == CONFIG
    assert (cfg.vocab_size, cfg.width, cfg.norm_eps, cfg.logit_scale) == (311, 96, 1e-5, 1.5)


@pytest.mark.parametrize("path,value", [
    (("layers", 0, "type"), "convolution"),
    (("layers", 0, "mlp", "kind"), "dense"),
    (("layers", 0, "mlp", "expert", "ff"), 0),
    (("layers", 0, "mlp", "expert", "limit"), KeyError),
    (("layers", 0, "mlp", "expert", "limit"), 0.0),
    (("layers", 0, "mlp", "router"), None),
    (("layers", 0, "mlp", "router", "top"), 0),
    (("layers", 0, "mlp", "router", "top"), 5),              # two groups of two hold four
    (("layers", 0, "mlp", "router", "experts"), 9),          # no five equal groups
    (("layers", 0, "mlp", "router", "experts"), 2000),
    (("layers", 0, "mlp", "router", "groups", "keep"), 6),
    (("layers", 0, "mlp", "router", "groups", "keep"), 0),
    (("layers", 0, "mixer", "kv_heads"), 4),
    (("layers", 0, "mixer", "rot", "dims"), 34),
    (("layers", 0, "mixer", "rot", "dims"), 15),
    (("layers", 0, "mixer", "rot", "scaling", "factor"), 0.0),
    (("layers", 0, "mixer", "rot", "scaling", "slow"), KeyError),
    (("layers", 0, "mixer", "mask", "size"), 0),
    (("layers", 0, "mixer", "scale"), KeyError),
    (("layers", 0, "mixer", "softcap"), -1.0),
    (("layers", 1, "mixer", "rot_dim"), 6),
    (("layers", 1, "mixer", "kv_rank"), KeyError),
    (("layers", 1, "mixer", "rot"), None),
    (("loop", "times"), 0),
    (("loop", "stop"), 5),
    (("loop", "start"), 4),                                  # behind its stop
    (("loop", "start"), KeyError),
    (("layers",), []),
    (("norm",), KeyError),
    (("vocab",), KeyError),
])
def test_refusals(path, value):
    with pytest.raises(ConfigError):
        SosuvikConfig.from_dict(broken(path, value))


def test_the_model_as_parts():
    spec = SosuvikConfig.from_dict(CONFIG).model_spec()
    assert [layer.mixer.kind for layer in spec.layers] == ["attention_rows", "latent_attention"] * 2
    assert [layer.ffn.kind if layer.ffn else None for layer in spec.layers] == ["routed_experts", None, "routed_experts", "routed_experts"]
    assert all(layer.block.kind == "parallel_pair" for layer in spec.layers)
    mixer = spec.layers[0].mixer.params
    assert (mixer["chunk"], mixer["fixed_sink"], mixer["score_cap"], mixer["scale"], mixer["value_dim"]) == (21, 0.0, 7.0, 0.2, 16)
    assert spec.positions[mixer["position"]].params == {"theta": 1e4, "rotary_dim": 16, "head_dim": 32, "pairing": "half", "yarn": SCALING}
    latent = spec.layers[1].mixer.params
    assert (latent["latent_dim"], latent["rotary_dim"], latent["head_dim"], latent["value_dim"]) == (40, 8, 16, 20)
    assert spec.positions[latent["position"]].params["pairing"] == "interleaved"
    moe = spec.layers[0].ffn.params
    assert moe["groups"] == {"count": 5, "keep": 2} and (moe["weight_scale"], moe["limit"], moe["top"]) == (1.25, 0.9, 3)
    assert spec.head.params["scale"] == 1.5 and spec.rejoins == ["loop.in"] and spec.offsets == {"loop.step": 2}


def test_without_groups_masks_caps_or_a_loop():
    data = copy.deepcopy(CONFIG)
    del data["loop"], data["logit_scale"], data["layers"][0]["mlp"]["router"]["groups"]
    del data["layers"][0]["mixer"]["mask"], data["layers"][0]["mixer"]["softcap"]
    spec = SosuvikConfig.from_dict(data).model_spec()
    assert spec.layers[0].ffn.params["groups"] is None and spec.layers[0].mixer.params["chunk"] is None
    assert spec.layers[0].mixer.params["score_cap"] == 0.0 and spec.head.params["scale"] == 1.0
    assert [r.layer for r in spec.order] == [0, 1, 2, 3] and not spec.rejoins and not spec.offsets
    assert "loop.in" not in expected_tensors(spec)


@pytest.mark.parametrize("start,stop,times", [(1, 3, 2), (0, 4, 3), (3, 4, 1), (0, 1, 4), (2, 2, 3)])
def test_the_order_of_running(start, stop, times):
    data = broken(("loop",), {"start": start, "stop": stop, "times": times})
    spec = SosuvikConfig.from_dict(data).model_spec()
    want = P.run_order(data)
    assert [(r.layer, r.offset[1] if r.offset else None) for r in spec.order] == want
    assert all((r.rejoin == "loop.in") == (r.offset is not None) for r in spec.order)
    assert all(r.cache_of is None for r in spec.order)        # every pass keeps a cache of its own
    assert ("loop.step" in expected_tensors(spec)) == (stop > start)


def test_tensor_names_and_shapes():
    names = expected_tensors(SosuvikConfig.from_dict(CONFIG).model_spec())
    shape = lambda n: tuple(names[n].shape)
    assert shape("embed") == (311, 96) and shape("head") == (311, 96) and shape("final.norm") == (96,)
    assert shape("loop.in") == (96, 192) and shape("loop.step") == (2, 96)
    assert shape("l0.norm1") == shape("l0.norm2") == shape("l1.norm1") == (96,) and "l1.norm2" not in names
    assert shape("l0.mix.q") == (192, 96) and shape("l0.mix.k") == (96, 96) and shape("l0.mix.v") == (48, 96)
    assert shape("l0.mix.o") == (96, 96)
    assert shape("l1.mix.q") == (120, 96) and shape("l1.mix.dkv") == (48, 96) and shape("l1.mix.dkv.norm") == (40,)
    assert shape("l1.mix.uk") == (80, 40) and shape("l1.mix.uv") == (100, 40) and shape("l1.mix.o") == (96, 100)
    assert shape("l0.mlp.router") == (10, 96) and shape("l0.mlp.correction") == (10,)
    assert shape("l0.mlp.e9.gate") == shape("l0.mlp.e0.up") == (56, 96) and shape("l0.mlp.e4.down") == (96, 56)
    for extra in ("l0.mix.q.b", "l0.mix.sink", "l1.mix.sink", "l1.mix.g", "l1.mix.dq", "l0.mlp.e10.gate"):
        assert extra not in names


def test_a_chunk_that_is_over_gives_its_pages_back():
    cache = CacheManager([PagedKVSpec(3, 32, None, chunk=21), PagedKVSpec(3, 32, None, chunk=50), PagedKVSpec(1, 48, None)],
                         page_size=4, num_pages=40, max_requests=2)
    first, second, whole = cache.groups
    cache.add_request("a")
    for computed in (20, 21, 22, 41, 42, 43, 49, 50, 60, 99, 100, 101, 105, 106):
        cache.reserve("a", computed)
        cache.advance("a", computed)
        for group, chunk in ((first, 21), (second, 50)):
            # the token at position `computed` comes next: it needs its own chunk's keys
            low = computed // chunk * chunk
            table = group.tables["a"]
            assert [p >= 0 for p in table] == [(i + 1) * 4 > low for i in range(len(table))], (computed, chunk)
        assert all(p >= 0 for p in whole.tables["a"])
        cache.check()
    cache.free_request("a")
    cache.check()
    assert all(g.pool.num_free == 40 for g in cache.groups)


def test_the_keys_that_splits_must_cover():
    assert split_span(1000, 0) == 1000 and split_span(1000, 200) == 200 + CHUNK_SLACK and split_span(100, 200) == 100
    # a block's rounding (31) and up to 16 tokens of an item behind a chunk's first key
    assert CHUNK_SLACK >= 31 + 15


def test_step_costs():
    spec = SosuvikConfig.from_dict(CONFIG).model_spec()
    decode, prompt = step_cost(spec, [(100, 1)], 1), step_cost(spec, [(0, 101)], 1)
    assert 0 < decode.flops < prompt.flops and decode.weight_bytes > 0 and decode.cache_bytes > 0
    # from one place in both chunks to another (1050 periods of 21 and of 50 later) only the latent rows are more, in each
    # of the two passes and in the last layer
    later = step_cost(spec, [(100 + 21 * 50, 1)], 1)
    from pulse_infer_amd.parts.latent import latent_stored_width
    assert later.cache_bytes - decode.cache_bytes == pytest.approx(3 * 2 * latent_stored_width(40, 8) * 2 * 21 * 50)
    # every pass costs its layers once more, and the product that brings the embedding's output back
    once = step_cost(SosuvikConfig.from_dict(broken(("loop", "times"), 1)).model_spec(), [(100, 1)], 1)
    assert decode.weight_bytes - once.weight_bytes >= 2 * (96 * 192 + 56 * 96 * 3 * 3)


def test_the_plain_router_takes_groups_by_their_two_best():
    w = {"m.router": torch.eye(6, dtype=torch.float64), "m.correction": torch.tensor([0., 0., 0., 0., 0., -2.], dtype=torch.float64)}
    s = torch.tensor([[.9, .1, .6, .55, .5, .99]], dtype=torch.float64)
    x = torch.log(s / (1 - s))
    router = {"experts": 6, "top": 2, "groups": {"count": 3, "keep": 1}}
    got, c, left = P.choice_scores(x, w, "m", router)
    assert torch.allclose(got, s) and c[0, 5] == pytest.approx(-1.01)
    assert torch.isinf(left[0]).tolist() == [True, True, False, False, True, True]
    assert float(P.router_margin(x, w, "m", {"router": router})[0]) == pytest.approx(1.15 - 1.0)
