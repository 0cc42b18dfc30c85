"""Linear attention whose state is corrected towards every new value: the gated delta rule, behind short convolutions.

For a token with input x: q = Wq x and k = Wk x (``num_groups`` x dim), v = Wv x (``num_heads`` x vdim); each passes a
causal convolution along the sequence (``conv`` taps a channel, no bias, zeros before a sequence's start) and silu; then
every head of q and k is divided by its length (with 1e-6 added to the sum of squares), and q multiplied by dim^(-1/2).
Query head h uses q and k of group h // (num_heads // num_groups).  With beta = sigmoid(Wb x) and g = exp(-exp(A_log) softplus(Wa x + dt_bias)),
one of each a head, every head keeps a state S [dim, vdim] per request, zero at the request's start:

    D = g S           r = v - D^T k           S = D + beta k r^T           o = S^T q

Every head's o is divided by its own root mean square, multiplied by a weight [vdim] that the heads share and by
silu(Wg x); the heads side by side are projected by Wo.

The six input projections are one product with the row-stacked weight.  A step of single tokens runs everything between
that product and the output projection in one kernel; other steps prepare float32 rows (convolutions, unit vectors,
decays), run the recurrence over them (portions of 64 tokens and more in chunks on the matrix cores, in float32; the
others token by token) and norm and gate the heads (``csrc/delta.hip``).  A request's slot holds one
float32 row: the states and the last ``conv`` inputs of the convolutions, which are kept as projected.

Parameters: ``hidden_size``, ``num_heads``, ``num_groups``, ``head_dim``, ``value_dim``, ``conv``, ``norm_eps``, ``names``
(tensor names below the prefix), ``out_scale`` (a factor on the result).  It answers the protocol of a branch of
``side_by_side``.
"""
from __future__ import annotations

from typing import Any, Dict, List, Tuple

import torch

from ..cache.specs import StateSpec, StateView
from ..ops import kernels
from ..weights.store import TensorSpec
from .base import MIXERS, BuildContext, Part, StepContext, StepCost, joined
from .linear import Linear


@MIXERS.register("gated_delta")
class GatedDelta(Part):
    NAMES = {"q": "q", "k": "k", "v": "v", "gate": "g", "beta": "b", "decay": "a", "q_conv": "q.conv", "k_conv": "k.conv",
             "v_conv": "v.conv", "a_log": "A_log", "dt_bias": "dt_bias", "norm": "norm", "o": "o"}
    ROW_PAD = 16    # rows of the stacked weight are filled up with zero rows to a multiple of this

    @classmethod
    def tensor_names(cls, params: Dict[str, Any]) -> Dict[str, str]:
        return {**cls.NAMES, **params.get("names", {})}

    @classmethod
    def weight_specs(cls, params: Dict[str, Any]) -> Dict[str, TensorSpec]:
        hidden, heads, groups, d, dv, taps = (params[k] for k in ("hidden_size", "num_heads", "num_groups", "head_dim",
                                                                  "value_dim", "conv"))
        n = cls.tensor_names(params)
        return {
            n["q"]: TensorSpec((groups * d, hidden), fan_in=hidden),
            n["k"]: TensorSpec((groups * d, hidden), fan_in=hidden),
            n["v"]: TensorSpec((heads * dv, hidden), fan_in=hidden),
            n["q_conv"]: TensorSpec((groups * d, taps), fan_in=taps),
            n["k_conv"]: TensorSpec((groups * d, taps), fan_in=taps),
            n["v_conv"]: TensorSpec((heads * dv, taps), fan_in=taps),
            n["gate"]: TensorSpec((heads * dv, hidden), fan_in=hidden),
            n["beta"]: TensorSpec((heads, hidden), fan_in=hidden),
            n["decay"]: TensorSpec((heads, hidden), fan_in=hidden),
            n["a_log"]: TensorSpec((heads,), fan_in=4),
            n["dt_bias"]: TensorSpec((heads,), fan_in=1),
            n["norm"]: TensorSpec((dv,), kind="norm"),
            n["o"]: TensorSpec((hidden, heads * dv), fan_in=heads * dv),
        }

    @classmethod
    def step_cost(cls, params: Dict[str, Any], entries: List[Tuple[int, int]], weight_bytes: int,
                  cache_bytes: int) -> StepCost:
        """The projections; the recurrence (three multiply-adds and a product a state element and token) and the
        convolutions; every request's state and convolution inputs read and written once, in float32."""
        cost = super().step_cost(params, entries, weight_bytes, cache_bytes)
        heads, d, dv, taps = (params[k] for k in ("num_heads", "head_dim", "value_dim", "conv"))
        channels = 2 * params["num_groups"] * d + heads * dv
        cost.flops += 7.0 * heads * d * dv * sum(count for _, count in entries)   # (the taps are counted as matrices)
        cost.cache_bytes += 4.0 * (2 * heads * d * dv + taps * channels) * len(entries)
        return cost

    def __init__(self, params: Dict[str, Any], prefix: str, build: BuildContext):
        self.hidden = int(params["hidden_size"])
        self.heads = int(params["num_heads"])
        self.groups = int(params["num_groups"])
        self.d = int(params["head_dim"])
        self.dv = int(params["value_dim"])
        self.taps = int(params["conv"])
        if min(self.heads, self.groups, self.d, self.dv) <= 0 or self.heads % self.groups:
            raise ValueError(f"the delta rule's {self.heads} heads cannot be shared out evenly over {self.groups} groups")
        if self.d > kernels.DELTA_MAX_DIM:
            raise ValueError(f"the delta rule's kernels take at most {kernels.DELTA_MAX_DIM} key channels a head, got {self.d}")
        if not 1 <= self.taps <= kernels.DELTA_MAX_TAPS:
            raise ValueError(f"the convolution's kernels take 1 to {kernels.DELTA_MAX_TAPS} taps, got {self.taps}")
        self.eps = float(params["norm_eps"])
        self.out_scale = float(params.get("out_scale", 1.0))
        load = build.loader
        n = {k: joined(prefix, v) for k, v in self.tensor_names(params).items()}
        weight = load.get_concat([n["q"], n["k"], n["v"], n["gate"], n["beta"], n["decay"]])
        pad = -weight.shape[0] % self.ROW_PAD
        if pad:
            weight = torch.cat([weight, weight.new_zeros(pad, self.hidden)], dim=0).contiguous()
        self.proj = Linear(weight, build.mode)
        # columns of the projection output: q, k, v (what is convolved), gate, strength, decay
        self.channels = 2 * self.groups * self.d + self.heads * self.dv
        self.gate0 = self.channels
        self.beta0 = self.gate0 + self.heads * self.dv
        self.decay0 = self.beta0 + self.heads
        f32 = lambda t: t.to(torch.float32).contiguous()
        self.conv = f32(load.get_concat([n["q_conv"], n["k_conv"], n["v_conv"]]).t())   # [taps, channels]
        self.a_log, self.dt_bias, self.norm_weight = (f32(load.get(n[k])) for k in ("a_log", "dt_bias", "norm"))
        self._o_weight = load.get(n["o"])
        self._o = None
        self.mode = build.mode
        self.act_dtype = build.act_dtype
        self.inner_width = self.heads * self.dv
        walk_only = build.options.get("delta", "auto") == "walk"
        self.decodes = not walk_only and kernels.delta_decode_takes(self.d, self.dv)
        self.chunked = not walk_only and kernels.delta_chunks_takes(self.d, self.dv)

    CHUNKED_MIN_TOKENS = 64  # portions from here on go through the recurrence in chunks
    records_cleanly = True   # slots, starts, positions and rows are read on the device

    def cache_spec(self) -> StateSpec:
        return StateSpec((kernels.delta_slot_floats(self.heads, self.groups, self.d, self.dv, self.taps),), "float32")

    def out_weight(self) -> torch.Tensor:
        return self._o_weight

    def forward_inner(self, x: torch.Tensor, ctx: StepContext, cache: StateView, out: torch.Tensor) -> None:
        """The mixer up to its output projection: ``out`` [T, inner_width] (rows may be strided) receives the normed,
        gated heads times ``out_scale``."""
        tokens = x.shape[0]
        ws = ctx.workspace
        y = ws.buffer("delta.proj", tokens, self.proj.out_features, self.act_dtype)
        self.proj.forward(x, y)
        if "static:delta.single_tokens" not in ctx.extras:
            ctx.extras["static:delta.single_tokens"] = all(e.count == 1 for e in ctx.entries)
        if self.decodes and ctx.extras["static:delta.single_tokens"]:
            kernels.delta_decode(y, self.gate0, self.beta0, self.decay0, self.conv, self.a_log, self.dt_bias,
                                 self.norm_weight, cache.state, out, ctx.positions, ctx.token_entry, ctx.entry_slot,
                                 self.heads, self.groups, self.d, self.dv, self.eps, self.out_scale)
            return
        rows = ws.buffer("delta.rows", tokens, self.channels, torch.float32)
        gates = ws.buffer("delta.gates", tokens, 2 * self.heads, torch.float32)
        kernels.delta_prepare(y, self.beta0, self.decay0, self.conv, self.a_log, self.dt_bias, cache.state, rows, gates,
                              ctx.positions, ctx.token_entry, ctx.entry_start, ctx.entry_first_row, ctx.entry_slot,
                              self.heads, self.groups, self.d, self.dv)
        o = ws.buffer("delta.heads", tokens, self.heads * self.dv, torch.float32)
        # long portions 64 tokens at a time on the matrix cores, the other entries token by token (the lists depend on the
        # step's shape alone)
        key = "static:delta.chunks"
        if key not in ctx.extras:
            chunks, runs, others = kernels.delta_chunk_lists(ctx.entries, self.CHUNKED_MIN_TOKENS)
            dev = lambda flat: ctx.to_device(flat) if flat else None
            ctx.extras[key] = (dev(chunks), dev(runs), dev(others), len(others))
        chunks, runs, others, walkers = ctx.extras[key]
        if chunks is not None and self.chunked:
            scratch = ws.buffer("delta.chunks", chunks.numel() // 4 * self.heads, kernels.delta_chunk_floats(self.d, self.dv),
                                torch.float32)
            kernels.delta_chunks(rows, gates, o, cache.state, ctx.entry_start, ctx.entry_slot, chunks, runs, scratch, self.heads,
                                 self.groups, self.d, self.dv, self.taps)
        else:
            others, walkers = None, len(ctx.entries)
        if walkers:
            kernels.delta_walk(rows, gates, o, cache.state, ctx.entry_first_row, ctx.entry_start, ctx.entry_slot, self.heads,
                               self.groups, self.d, self.dv, self.taps,
                               kernels.delta_row_groups(walkers, self.heads, self.d, self.dv), which=others)
        kernels.group_norm_gate(o, self.norm_weight, y[:, self.gate0:self.gate0 + self.heads * self.dv], out, self.heads,
                                self.eps, self.out_scale, "silu")

    def forward(self, x: torch.Tensor, ctx: StepContext, cache: StateView) -> torch.Tensor:
        if self._o is None:
            self._o = Linear(self._o_weight, self.mode)
        ws = ctx.workspace
        inner = ws.buffer("delta.inner", x.shape[0], self.inner_width, self.act_dtype)
        self.forward_inner(x, ctx, cache, inner)
        return self._o.forward(inner, ws.buffer("delta.out", x.shape[0], self.hidden, self.act_dtype))
