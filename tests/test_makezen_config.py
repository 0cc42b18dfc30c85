"""Makezen's configuration on the CPU: keys, refusals, the round trip, the model as a list of parts, tensor names and
shapes, the blended frequencies, the cache of its runs (rows kept for the layers that read them), and step costs."""
import copy
import types

import pytest
import torch

from plain import makezen_plain as P
from pulse_infer_amd.cache.manager import CacheManager
from pulse_infer_amd.cache.specs import CombinedSpec, PagedKVSpec, StateSpec
from pulse_infer_amd.config import ConfigError, MakezenConfig, config_from_dict
from pulse_infer_amd.models.causal_lm import expected_tensors
from pulse_infer_amd.models.cost import step_cost
from pulse_infer_amd.ops import kernels
from pulse_infer_amd.parts.rope import RotaryEmbedding

SCALING = {"factor": 4.0, "original": 512.0, "fast": 16.0, "slow": 2.0}
LEFT = {"dim": 32, "heads": 6, "kv_heads": 3, "rot": {"base": 1e4, "dims": 16, "scaling": SCALING}, "scale": 0.2,
        "softcap": 7.0, "vdim": 16}
RIGHT = {"conv": 4, "dim": 16, "heads": 4, "kv_heads": 2, "vdim": 24}
LATENT = {"dim": 16, "heads": 3, "kv_rank": 40, "mask": {"size": 7}, "q_rank": 24, "rot": {"base": 500.0, "dims": 8},
          "rot_dim": 8, "scale": 0.3, "vdim": 20}
READER = dict(copy.deepcopy(LATENT), heads=5, dim=8, vdim=12, q_rank=36, mask={"size": 29}, kv_from=1)
CONFIG = {
    "architecture": "Makezen", "norm": {"eps": 1e-5}, "vocab": 311, "width": 96,
    "layers": [
        {"type": "parallel", "mixer": {"left": LEFT, "right": RIGHT}, "mlp": {"kind": "dense", "ff": 160}},
        {"type": "latent_attention", "mixer": LATENT, "mlp": None},
        {"type": "delta", "mixer": {"conv": 2, "dim": 24, "heads": 3, "kv_heads": 1, "vdim": 40}, "mlp": None},
        {"type": "latent_attention", "mixer": READER, "mlp": {"kind": "dense", "ff": 112}},
    ],
}


def test_round_trip_and_registry():
    cfg = config_from_dict(CONFIG)
    assert isinstance(cfg, MakezenConfig)
    assert cfg.to_dict() == CONFIG
    assert MakezenConfig.from_dict(cfg.to_dict()).to_dict() == CONFIG
    assert (cfg.vocab_size, cfg.width, cfg.norm_eps) == (311, 96, 1e-5)


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


@pytest.mark.parametrize("path,value", [
    (("layers", 0, "type"), "convolution"),
    (("layers", 0, "mlp", "kind"), "moe"),
    (("layers", 0, "mlp", "ff"), 0),
    (("layers", 0, "mixer", "left", "kv_heads"), 4),
    (("layers", 0, "mixer", "left", "rot", "dims"), 34),
    (("layers", 0, "mixer", "left", "rot", "dims"), 15),
    (("layers", 0, "mixer", "left", "rot", "scaling", "factor"), 0.0),
    (("layers", 0, "mixer", "left", "rot", "scaling", "slow"), KeyError),
    (("layers", 0, "mixer", "left", "rot", "base"), 1.0),
    (("layers", 0, "mixer", "left", "scale"), KeyError),
    (("layers", 0, "mixer", "left", "softcap"), -1.0),
    (("layers", 0, "mixer", "right", "kv_heads"), 3),
    (("layers", 0, "mixer", "right", "dim"), 300),
    (("layers", 0, "mixer", "right", "conv"), 0),
    (("layers", 2, "mixer", "conv"), 17),
    (("layers", 1, "mixer", "mask", "size"), 0),
    (("layers", 1, "mixer", "rot_dim"), 6),
    (("layers", 1, "mixer", "q_rank"), KeyError),
    (("layers", 1, "mixer", "rot"), None),
    (("layers", 3, "mixer", "kv_from"), 2),         # no latent attention
    (("layers", 3, "mixer", "kv_from"), 3),         # itself
    (("layers", 3, "mixer", "kv_from"), -1),
    (("layers", 1, "mixer", "kv_from"), 3),         # a later one
    (("layers", 3, "mixer", "kv_rank"), 48),        # another form of rows
    (("layers", 3, "mixer", "rot", "base"), 600.0),
    (("layers",), []),
    (("norm",), KeyError),
    (("vocab",), KeyError),
])
def test_refusals(path, value):
    with pytest.raises(ConfigError):
        MakezenConfig.from_dict(broken(path, value))


def test_a_reader_of_a_reader_is_refused():
    data = copy.deepcopy(CONFIG)
    data["layers"].append({"type": "latent_attention", "mixer": dict(READER, kv_from=3), "mlp": None})
    with pytest.raises(ConfigError):
        MakezenConfig.from_dict(data)
    data["layers"][-1]["mixer"]["kv_from"] = 1
    assert [run.cache_of for run in MakezenConfig.from_dict(data).model_spec().order] == [None, None, None, 1, 1]


def test_the_model_as_parts():
    spec = MakezenConfig.from_dict(CONFIG).model_spec()
    assert [layer.mixer.kind for layer in spec.layers] == ["side_by_side", "latent_attention", "gated_delta", "latent_attention"]
    assert [layer.ffn.kind if layer.ffn else None for layer in spec.layers] == ["mlp", None, None, "mlp"]
    assert all(layer.block.kind == "sandwich" for layer in spec.layers)
    assert all(n.kind == "layernorm" and n.params["bias"] is False for layer in spec.layers for n in layer.norms.values())
    mixer = spec.layers[0].mixer.params
    assert mixer["branch_norm"] == {"tensor": "out", "eps": 1e-5, "factor": 0.5}
    left, right = (b["params"] for b in mixer["branches"])
    assert [b["kind"] for b in mixer["branches"]] == ["attention_rows", "gated_delta"]
    assert (left["score_cap"], left["value_dim"], left["bias"], left["qk_norm"], left["qk_norm_weights"]) == (7.0, 16, True, "head", True)
    assert spec.positions[left["position"]].params == {"theta": 1e4, "rotary_dim": 16, "head_dim": 32, "pairing": "half",
                                                       "yarn": SCALING}
    assert (right["num_heads"], right["num_groups"], right["head_dim"], right["value_dim"], right["conv"]) == (4, 2, 16, 24, 4)
    own, reader = spec.layers[1].mixer.params, spec.layers[3].mixer.params
    assert (own["window"], own["cache_window"], own["reads_rows"], own["query_dim"], own["output_gate"]) == (7, 29, False, 24, "head")
    assert (reader["window"], reader["reads_rows"], reader["query_dim"]) == (29, True, 36)
    assert [run.cache_of for run in spec.order] == [None, None, None, 1]
    assert spec.embedding.params["norm"] == {"kind": "layernorm", "tensor": "embed.norm", "eps": 1e-5}
    assert spec.head.params["tied"] and spec.final_norm.kind == "layernorm"


def test_rows_are_kept_for_the_widest_reader():
    cfg = MakezenConfig.from_dict(CONFIG)
    assert cfg.rows_kept(1) == 29
    narrow = copy.deepcopy(CONFIG)
    narrow["layers"][3]["mixer"]["mask"]["size"] = 3
    assert MakezenConfig.from_dict(narrow).rows_kept(1) == 7
    whole = copy.deepcopy(CONFIG)
    del whole["layers"][3]["mixer"]["mask"]
    assert MakezenConfig.from_dict(whole).rows_kept(1) == 0       # a reader without a window: every row stays


def test_tensor_names_and_shapes():
    names = expected_tensors(MakezenConfig.from_dict(CONFIG).model_spec())
    shape = lambda n: tuple(names[n].shape)
    assert shape("embed") == (311, 96) and shape("embed.norm") == (96,) and shape("final.norm") == (96,)
    assert shape("l0.norm1") == shape("l0.norm1b") == shape("l0.norm2") == shape("l0.norm2b") == (96,)
    assert "l1.norm2" not in names and "l1.norm2b" not in names and "l1.norm1b" in names
    assert shape("l0.mix.left.q") == (192, 96) and shape("l0.mix.left.k.b") == (96,) and shape("l0.mix.left.v") == (48, 96)
    assert shape("l0.mix.left.q.norm") == shape("l0.mix.left.k.norm") == (32,) and shape("l0.mix.left.o") == (96, 96)
    assert shape("l0.mix.left.out") == shape("l0.mix.right.out") == (96,)
    assert shape("l0.mix.right.q") == (32, 96) and shape("l0.mix.right.q.conv") == (32, 4) and shape("l0.mix.right.v.conv") == (96, 4)
    assert shape("l0.mix.right.b") == shape("l0.mix.right.a") == (4, 96) and shape("l0.mix.right.norm") == (24,)
    assert shape("l0.mix.right.A_log") == shape("l0.mix.right.dt_bias") == (4,) and shape("l0.mix.right.g") == (96, 96)
    assert shape("l2.mix.q") == (24, 96) and shape("l2.mix.v") == (120, 96) and shape("l2.mix.o") == (96, 120)
    assert shape("l1.mix.dq") == (24, 96) and shape("l1.mix.uq") == (72, 24) and shape("l1.mix.dkv") == (48, 96)
    assert shape("l1.mix.uk") == (48, 40) and shape("l1.mix.uv") == (60, 40) and shape("l1.mix.g") == (3, 96)
    assert "l3.mix.dkv" not in names and "l3.mix.dkv.norm" not in names
    assert shape("l3.mix.uk") == (40, 40) and shape("l3.mix.sink") == (5,) and shape("l3.mix.dq.norm") == (36,)
    assert "l1.mix.q" not in names and names["head"].optional


@pytest.mark.parametrize("base,dims,scaling", [
    (1e4, 64, {"factor": 8.0, "original": 4096, "fast": 32.0, "slow": 1.0}),
    (5e5, 128, {"factor": 32.0, "original": 8192, "fast": 32.0, "slow": 1.0}),
    (100.0, 8, {"factor": 2.0, "original": 64, "fast": 4.0, "slow": 1.0}),
    (1e4, 16, {"factor": 1.0, "original": 2048, "fast": 32.0, "slow": 1.0}),
    (20.0, 6, {"factor": 3.0, "original": 1 << 20, "fast": 2.0, "slow": 1.0}),     # both ends beyond the last index
    (1e6, 32, {"factor": 4.0, "original": 16, "fast": 32.0, "slow": 8.0}),         # both ends before the first one
    (1e4, 32, None),
])
def test_blended_frequencies(base, dims, scaling):
    params = {"theta": base, "rotary_dim": dims, "pairing": "half"}
    if scaling:
        params["yarn"] = scaling
    part = RotaryEmbedding(params, types.SimpleNamespace(device="cpu"))
    rot = {"base": base, "dims": dims, "scaling": scaling}
    want = torch.tensor(P.frequencies(rot), dtype=torch.float64)
    assert torch.allclose(part.inv_freq, want, rtol=1e-12, atol=0.0)
    assert part.magnitude == pytest.approx(P.magnitude(rot), rel=1e-12)


def test_the_cache_keeps_rows_as_long_as_a_reader_needs_them():
    cfg = MakezenConfig.from_dict(CONFIG)
    own = cfg.model_spec().layers[1].mixer.params
    rows = PagedKVSpec(1, 48, own["cache_window"])
    left = PagedKVSpec(3, 32, None)
    state = StateSpec((kernels.delta_slot_floats(4, 2, 16, 24, 4),), "float32")
    alone = StateSpec((kernels.delta_slot_floats(3, 1, 24, 40, 2),), "float32")
    cache = CacheManager([CombinedSpec((left, state)), rows, alone, None], page_size=4, num_pages=64, max_requests=2)
    group = next(g for g in cache.groups if g.window == 29)
    cache.add_request("a")
    cache.reserve("a", 60)
    cache.advance("a", 60)
    # position 60 of the wider reader sees 32 .. 60
    assert all(p == -1 for p in group.tables["a"][:8]) and all(p >= 0 for p in group.tables["a"][8:15])
    assert all(p >= 0 for p in next(g for g in cache.groups if g.window is None).tables["a"])
    cache.free_request("a")
    cache.check()


def test_slot_sizes():
    assert kernels.delta_slot_floats(4, 2, 16, 24, 4) == 4 * 16 * 24 + 4 * (2 * 2 * 16 + 4 * 24)
    assert kernels.delta_slot_floats(1, 1, 3, 5, 1) == 28 and kernels.delta_slot_floats(1, 1, 3, 5, 1) % 4 == 0   # 26 values
    assert kernels.delta_decode_takes(128, 128) and kernels.delta_decode_takes(24, 20)
    assert not kernels.delta_decode_takes(16, 10) and not kernels.delta_decode_takes(300, 64)


def test_step_costs():
    spec = MakezenConfig.from_dict(CONFIG).model_spec()
    decode, prompt = step_cost(spec, [(100, 1)], 1), step_cost(spec, [(0, 101)], 1)
    assert 0 < decode.flops < prompt.flops and decode.weight_bytes > 0 and decode.cache_bytes > 0
    # only the left attention reads more of a longer context: windows and states do not grow
    grown = step_cost(spec, [(1000, 1)], 1).cache_bytes - decode.cache_bytes
    assert grown == pytest.approx(2 * 3 * 32 * 2 * 900)
