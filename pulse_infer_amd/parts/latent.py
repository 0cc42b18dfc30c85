"""Attention whose keys and values come from one latent row a token ("latent attention").

For a token with input x: q = Wq x, laid out head by head as [dim plain | rot_dim turned]; [c_raw | k_rot] = Wd x with
``latent_dim`` + ``rotary_dim`` rows; c = c_raw / rms(c_raw) * w (the latent row) and k_rot, turned by the token's
position, are all that is cached.  Head h's key is [W_uk,h c | k_rot] (the turned part is shared by all heads), its
value W_uv,h c; scores are (q . key) * scale over all earlier tokens, softmax with an optional sink per head; the
heads' results, side by side, are multiplied element by element by sigmoid(Wg x) (optional) and projected by Wo.

Scores and weighted sums are linear in c, so the part works in the latent space and paged attention kernels serve it
as they are (those of ``attention`` where they are compiled for rows this wide, else ``pulse_attn_wide``, else the
generic one): one kv head whose stored key is [c | k_rot] and whose stored value is c, query head
h = [W_uk,h^T q_plain,h | q_rot,h], and W_uv,h applied to the weighted sum of latent rows afterwards.  Keys and values
are stored ``stored`` = latent_dim + rotary_dim (rounded up to 16) channels wide, the rest zeros.

Parameters: ``hidden_size``, ``num_heads``, ``head_dim`` (plain channels of a head), ``rotary_dim``, ``value_dim``,
``latent_dim``, ``scale``, ``norm_eps``, ``position`` (a rotary encoding of ``rotary_dim`` channels), ``sink``,
``output_gate`` (True: by channel; "head": one number a head, sigmoid(Wg x)_h), ``names``, ``out_scale``.

Variations: ``query_dim``: the queries come from a latent of their own, q = W_uq (W_dq x / rms * w) (tensors ``q_down``,
``q_down_norm``, ``q_up`` in place of ``q``).  ``window``: a token sees itself and the ``window`` - 1 tokens before it.
``cache_window`` (default ``window``): how far back the cached rows must stay readable, where runs with wider windows read
them too (0: all of them).  ``reads_rows`` True: the part has no down projection; its run reads the latent rows and turned
key parts that another run of the order caches (``RunSpec.cache_of``), with its own up projections.

Where the rows are wider than the compiled attention kernels take, long portions of prompts go another way: the rows they
see are gathered from the pages, expanded to every head's keys and values by one product with [W_uk; W_uv], and the
prompt-portion kernel of ``attention`` runs on those (``EXPAND_MIN_TOKENS``; a third of the arithmetic at a latent row of
512 and heads of 128, on a kernel that shares keys through LDS).  What is cached stays the same.

Kernels: ``pulse_latent_rows`` (norm of the latent row, turns, page write), ``pulse_rms_rows``
(norm of the queries' latent), ``pulse_heads_product`` (bfloat16: both
products a head on the matrix cores) or ``pulse_latent_absorb`` / ``pulse_latent_expand`` (queries into the latent
space, values out of it with the gate), and the attention kernels between them; ``pulse_latent_queries`` / ``gather`` /
``pages`` / ``compact`` around the expanded form.  It answers the
protocol of a branch of ``side_by_side``.
"""
from __future__ import annotations

from typing import Any, Dict, List, Optional, Tuple

import torch

from ..cache.manager import PagedKVSpec
from ..ops import attention_mfma, kernels
from ..weights.store import TensorSpec
from .attention import PagedAttention, keys_seen
from .base import MIXERS, BuildContext, PagedCacheView, Part, StepContext, StepCost, joined
from .linear import Linear


def latent_stored_width(rank: int, rot: int) -> int:
    return (rank + rot + 15) // 16 * 16


@MIXERS.register("latent_attention")
class LatentAttention(PagedAttention):
    NAMES = {"q": "q", "q_down": "dq", "q_down_norm": "dq.norm", "q_up": "uq", "down": "dkv", "down_norm": "dkv.norm",
             "up_k": "uk", "up_v": "uv", "gate": "g", "sink": "sink", "o": "o"}
    GATES = (False, None, True, "channel", "head")

    @classmethod
    def weight_specs(cls, params: Dict[str, Any]) -> Dict[str, TensorSpec]:
        hidden, heads, d, rot, dv, rank = (params[k] for k in ("hidden_size", "num_heads", "head_dim", "rotary_dim",
                                                               "value_dim", "latent_dim"))
        n = cls.tensor_names(params)
        specs = {}
        query = params.get("query_dim")
        if query:
            specs[n["q_down"]] = TensorSpec((query, hidden), fan_in=hidden)
            specs[n["q_down_norm"]] = TensorSpec((query,), kind="norm")
            specs[n["q_up"]] = TensorSpec((heads * (d + rot), query), fan_in=query)
        else:
            specs[n["q"]] = TensorSpec((heads * (d + rot), hidden), fan_in=hidden)
        if not params.get("reads_rows", False):
            specs[n["down"]] = TensorSpec((rank + rot, hidden), fan_in=hidden)
            specs[n["down_norm"]] = TensorSpec((rank,), kind="norm")
        specs.update({
            n["up_k"]: TensorSpec((heads * d, rank), fan_in=rank),
            n["up_v"]: TensorSpec((heads * dv, rank), fan_in=rank),
            n["o"]: TensorSpec((hidden, heads * dv), fan_in=heads * dv),
        })
        gate = params.get("output_gate", False)
        if gate:
            specs[n["gate"]] = TensorSpec((heads if gate == "head" else heads * dv, hidden), fan_in=hidden)
        if params.get("sink", False):
            specs[n["sink"]] = TensorSpec((heads,), kind="linear", fan_in=4)
        return specs

    @classmethod
    def step_cost(cls, params: Dict[str, Any], entries, weight_bytes: int, cache_bytes: int) -> StepCost:
        """The projections (the two up projections a head and row); scores and weighted sums in the latent space over
        every token seen; every request's visible stored rows read once."""
        cost = Part.step_cost.__func__(cls, params, entries, weight_bytes, cache_bytes)
        heads, rot, rank = params["num_heads"], params["rotary_dim"], params["latent_dim"]
        stored = latent_stored_width(rank, rot)
        window = params.get("window")
        for start, count in entries:
            seen, kept = keys_seen(start, count, window)
            cost.flops += 2.0 * heads * (2 * rank + rot) * seen
            cost.cache_bytes += 2.0 * stored * cache_bytes * kept
        return cost

    def __init__(self, params: Dict[str, Any], prefix: str, build: BuildContext):
        self.hidden = int(params["hidden_size"])
        self.nq = int(params["num_heads"])
        self.nkv = 1
        self.plain_dim = int(params["head_dim"])
        self.rot_dim = int(params["rotary_dim"])
        self.v_dim = int(params["value_dim"])
        self.rank = int(params["latent_dim"])
        if min(self.nq, self.plain_dim, self.rot_dim, self.v_dim, self.rank) <= 0 or self.rot_dim % 2:
            raise ValueError("latent attention needs positive sizes and an even rotary_dim")
        self.d = latent_stored_width(self.rank, self.rot_dim)    # what the cache and the attention kernels see
        self.scale = float(params["scale"])
        self.window = params.get("window")
        if self.window is not None and int(self.window) <= 0:
            raise ValueError(f"an attention window must be positive, got {self.window}")
        keep = params.get("cache_window", self.window)
        self.cache_window = int(keep) if keep else None
        if self.cache_window is not None and (self.window is None or self.cache_window < int(self.window)):
            raise ValueError(f"rows kept for {self.cache_window} tokens do not serve a window of {self.window}")
        self.reads_rows = bool(params.get("reads_rows", False))
        self.query_dim = int(params.get("query_dim") or 0)
        self.eps = float(params["norm_eps"])
        self.out_scale = float(params.get("out_scale", 1.0))
        self._read_score_form(params)
        self.position = params.get("position")
        self.encodings = build.positions
        if self.position is None or self.position not in self.encodings:
            raise KeyError(f"latent attention needs a position encoding of the model, got '{self.position}' "
                           f"(the model defines {sorted(self.encodings)})")
        load = build.loader
        n = {k: joined(prefix, v) for k, v in self.tensor_names(params).items()}
        gate = params.get("output_gate", False)
        if gate not in self.GATES:
            raise ValueError(f"latent attention has an output gate by 'channel', by 'head' or none, got {gate!r}")
        self.gated = bool(gate)
        self.gate_heads = gate == "head"
        stacked = [n["q_down"] if self.query_dim else n["q"]] + ([] if self.reads_rows else [n["down"]]) \
            + ([n["gate"]] if self.gated else [])
        weight = load.get_concat(stacked)
        pad = -weight.shape[0] % self.GATE_PAD if self.gate_heads else 0
        if pad:   # (the product's rows stay 16-byte aligned)
            weight = torch.cat([weight, weight.new_zeros(pad, self.hidden)], dim=0).contiguous()
        self.proj = Linear(weight, build.mode)
        # columns of the projection output: the queries (or their latent), the down projection, the gate
        self.down_col0 = self.query_dim or self.nq * (self.plain_dim + self.rot_dim)
        self.gate_col0 = self.down_col0 + (0 if self.reads_rows else self.rank + self.rot_dim)
        self.gate_cols = self.nq * (1 if self.gate_heads else self.v_dim)
        self.q_up = Linear(load.get(n["q_up"]), build.mode) if self.query_dim else None
        self.q_norm_weight = load.get(n["q_down_norm"]) if self.query_dim else None
        self.norm_weight = None if self.reads_rows else load.get(n["down_norm"])
        up = load.get_concat([n["up_k"], n["up_v"]])
        self.w_uk, self.w_uv = up[:self.nq * self.plain_dim], up[self.nq * self.plain_dim:]
        self.up = Linear(up, build.mode)
        self.expanded = (max(self.plain_dim + self.rot_dim, self.v_dim) + 15) // 16 * 16   # channels of an expanded head
        # for the matrix cores: a head's rows side by side ([heads, out, in]); w_uk transposed once, so that both
        # products walk their inner dimension along a row (a layout choice, not new maths)
        self.w_uk_t = self.w_uv_h = None
        if build.mode == "bfloat16" and self.w_uk.dtype == torch.bfloat16 and self.plain_dim % 8 == 0 and self.rank % 8 == 0:
            self.w_uk_t = self.w_uk.view(self.nq, self.plain_dim, self.rank).transpose(1, 2).contiguous()
            self.w_uv_h = self.w_uv.view(self.nq, self.v_dim, self.rank)
        self.sink = self._load_sink(load, n["sink"]) if params.get("sink", False) else None
        self._o_weight = load.get(n["o"])
        self._o = None
        self.mode = build.mode
        self.inner_width = self.nq * self.v_dim
        self.act_dtype = build.act_dtype
        self.options = build.options
        # what the inherited kernel choice asks about (none of it applies here)
        self.qk_norm = self.plain_norm = self.values_are_keys = self.output_gate = False
        self.q_temperature = None
        self.q_w = self.k_w = None

    accepts_residual = True
    accepts_lazy_input = False
    records_cleanly = True

    def cache_spec(self) -> PagedKVSpec:
        return PagedKVSpec(1, self.d, self.cache_window)

    def out_weight(self) -> torch.Tensor:
        return self._o_weight

    def decodes_from_raw(self, ctx, cache, qkv, tables) -> bool:
        return False

    def takes_lazy_input(self, x, cache) -> bool:
        return False

    def forward_inner(self, x: torch.Tensor, ctx: StepContext, cache: PagedCacheView, out: torch.Tensor) -> None:
        tokens = x.shape[0]
        ws = ctx.workspace
        if cache.writable == self.reads_rows:
            raise ValueError("latent attention caches rows of its own exactly if it has a down projection")
        y = ws.buffer("latent.proj", tokens, self.proj.out_features, self.act_dtype)
        self.proj.forward(x, y)
        raw = y    # the matrix whose first columns are the queries as projected
        if self.query_dim:
            latent = ws.buffer("latent.queries", tokens, self.query_dim, self.act_dtype)
            kernels.rms_rows(y, 0, self.q_norm_weight, self.eps, latent)
            raw = self.q_up.forward(latent, ws.buffer("latent.raw_q", tokens, self.q_up.out_features, self.act_dtype))
        tables = ctx.position_product(self.position, self.encodings)
        if tables.rotary_dim != self.rot_dim:
            raise ValueError(f"latent attention turns {self.rot_dim} channels, its position encoding {tables.rotary_dim}")
        table = ctx.block_tables[cache.group]
        gate = y[:, self.gate_col0:self.gate_col0 + self.gate_cols] if self.gated else None
        plan = self._expansion(ctx, cache)
        runs = plan["others"] if plan is not None else [(0, tokens)]
        q = ws.buffer("latent.q", tokens, self.nq * self.d, self.act_dtype) if runs else None
        if runs or cache.writable:
            kernels.latent_rows(raw, 0, self.down_col0, q, self.norm_weight, tables.cos, tables.sin, tables.pairing,
                                cache.keys, cache.values, ctx.positions, ctx.token_entry, table, self.nq, self.plain_dim,
                                self.rot_dim, self.rank, self.d, self.eps, write=cache.writable, down=y)
        if runs:
            self._absorbed(raw, q, gate, ctx, cache, table, out, runs, plan)
        if plan is not None:
            self._expanded(raw, gate, ctx, cache, table, tables, out, plan)

    def _absorbed(self, raw, q, gate, ctx: StepContext, cache: PagedCacheView, table, out, runs: List[Tuple[int, int]],
                  plan: Optional[Dict[str, Any]]) -> None:
        """Attention in the latent space, of the rows in ``runs`` (all of them without a plan)."""
        ws = ctx.workspace
        tokens = q.shape[0]
        q_head = self.plain_dim + self.rot_dim
        for a, b in runs:
            if self.w_uk_t is not None and kernels.heads_product_takes(raw[a:b], self.w_uk_t, q[a:b], q_head):
                kernels.heads_product(raw[a:b], q_head, self.w_uk_t, None, q[a:b], self.d)
            else:
                kernels.latent_absorb(raw[a:b], 0, q_head, self.w_uk, q[a:b], self.d, self.nq, self.plain_dim, self.rank)
        window = int(self.window) if self.window is not None else 0
        # the weighted latent rows: from the matrix-core kernels of ``attention`` where they are compiled for rows this
        # wide (the activations' type), else in float32 from the matrix-core kernel for wide values or the generic one
        if self.uses_matrix_cores(q, cache):
            o = ws.buffer("latent.rows", tokens, self.nq * self.d, self.act_dtype)
            self.attend(q, o, ctx, cache, table)
        elif self._wide(q, cache):
            o = ws.buffer("latent.rows", tokens, self.nq * self.d, torch.float32)
            key = f"static:latent.wide_items:{self.nq}:{'some' if plan else 'all'}"
            if key not in ctx.extras:
                row_tiles = kernels.attn_wide_row_tiles(ctx.num_tokens)
                entries = [e for i, e in enumerate(ctx.entries) if plan is None or i not in plan["at"]]
                flat, hp = kernels.attn_wide_items(entries, self.nq, 1, row_tiles)
                ctx.extras[key] = (ctx.to_device(flat), hp, row_tiles)
            items, hp, row_tiles = ctx.extras[key]
            wv = (self.rank + 15) // 16 * 16
            seen = min(ctx.max_context, window + 32) if window else ctx.max_context
            splits = kernels.attn_wide_splits(items.numel() // 4, (wv + 255) // 256, seen) if row_tiles == 1 else 1
            if plan is not None:
                splits = 1     # (the merge of splits covers every row of the step)
            part = part_ml = None
            if splits > 1:
                part = ws.buffer("attn_wide.part", tokens * self.nq * splits, self.d, torch.float32)
                part_ml = ws.buffer("attn_wide.part_ml", tokens * self.nq * splits, 2, torch.float32)
            kernels.attn_wide(q, o, self.nq, 1, self.d, wv, False, cache.keys, cache.values, ctx.positions,
                              ctx.token_entry, table, items, hp, self.scale, window, 0, self.sink, self.score_cap, row_tiles,
                              splits, part, part_ml)
        else:
            o = ws.buffer("latent.rows", tokens, self.nq * self.d, torch.float32)
            kernels.attn_generic(q, o, self.nq, 1, self.d, cache.keys, cache.values, ctx.positions, ctx.token_entry,
                                 table, self.scale, window, sink=self.sink, softcap=self.score_cap)
        for a, b in runs:
            some = gate[a:b] if gate is not None else None
            if self.w_uv_h is not None and kernels.heads_product_takes(o[a:b], self.w_uv_h, out[a:b], self.d):
                kernels.heads_product(o[a:b], self.d, self.w_uv_h, some, out[a:b], self.v_dim, self.out_scale, self.gate_heads)
            else:
                kernels.latent_expand(o[a:b], self.d, self.w_uv, some, out[a:b], self.nq, self.v_dim, self.rank, self.out_scale,
                                      self.gate_heads)

    def _wide(self, q: torch.Tensor, cache: PagedCacheView) -> bool:
        return self.options.get("attention", "auto") != "generic" and kernels.attn_wide_takes(q, cache.keys, self.d)

    EXPAND_MIN_TOKENS = 64             # portions from here on attend to expanded keys and values
    EXPAND_MAX_BYTES = 1 << 31         # of the expanded keys of a step, and of its values

    def _expansion(self, ctx: StepContext, cache: PagedCacheView) -> Optional[Dict[str, Any]]:
        """How this step's long portions attend to expanded keys and values; None: no portion does.  The lists depend on the
        step's shape and positions; every layer with this window and these sizes shares them."""
        if not any(e.count >= self.EXPAND_MIN_TOKENS for e in ctx.entries):
            return None
        form = self.options.get("latent", "auto")
        if (form == "absorbed" or self.w_uk_t is None or self.options.get("attention", "auto") == "generic"
                or not attention_mfma.supported(self.expanded, kernels.EXPANDED_PAGE, self.act_dtype, cache.keys.dtype)):
            return None
        if attention_mfma.supported(self.d, cache.page_size, self.act_dtype, cache.keys.dtype):
            return None      # (narrow rows: the compiled kernels take them as they are)
        window = int(self.window) if self.window is not None else 0
        key = f"latent.expansion:{window}:{self.nq}:{self.expanded}"
        if key not in ctx.extras:
            ctx.extras[key] = self._plan(ctx, window)
        return ctx.extras[key]

    def _plan(self, ctx: StepContext, window: int) -> Optional[Dict[str, Any]]:
        numbered = [(i, e) for i, e in enumerate(ctx.entries) if e.count >= self.EXPAND_MIN_TOKENS]
        flat, at = kernels.latent_expand_pages(numbered, window)
        n_pages = len(flat) // 4
        if 2 * n_pages * self.nq * kernels.EXPANDED_PAGE * self.expanded > self.EXPAND_MAX_BYTES:
            return None
        width = max((e.start + e.count + kernels.EXPANDED_PAGE - 1) // kernels.EXPANDED_PAGE for _, e in numbered)
        rows = [[-1] * width for _ in ctx.entries]
        for (index, e) in numbered:
            low, first = at[index]
            last = (e.start + e.count + kernels.EXPANDED_PAGE - 1) // kernels.EXPANDED_PAGE
            rows[index][low:last] = range(first, first + last - low)
        others: List[Tuple[int, int]] = []     # the other entries' rows, neighbours together
        for i, e in enumerate(ctx.entries):
            if i in at:
                continue
            if others and others[-1][1] == e.first_row:
                others[-1] = (others[-1][0], e.first_row + e.count)
            else:
                others.append((e.first_row, e.first_row + e.count))
        portion = attention_mfma.portion_tokens(1, self.expanded)
        split_size, splits = attention_mfma.choose_prefill_splits(numbered, portion, self.nq, 1, self.expanded, window)
        return {"at": at, "n_pages": n_pages, "pages": ctx.to_device(flat), "others": others,
                "table": ctx.to_device([p for row in rows for p in row]).view(len(rows), width),
                "items": ctx.to_device(attention_mfma.build_items(numbered, portion)),
                "spans": [(e.first_row, e.first_row + e.count) for _, e in numbered], "split_size": split_size, "splits": splits}

    def _expanded(self, raw, gate, ctx: StepContext, cache: PagedCacheView, table, tables, out, plan: Dict[str, Any]) -> None:
        """Attention of the long portions over keys and values expanded to every head."""
        ws = ctx.workspace
        tokens, w, page, n = raw.shape[0], self.expanded, kernels.EXPANDED_PAGE, plan["n_pages"]
        bf16 = self.act_dtype
        q = ws.buffer("latent.expanded_q", tokens, self.nq * w, bf16)
        kernels.latent_queries(raw, 0, q, tables.cos, tables.sin, tables.pairing, self.nq, self.plain_dim, self.rot_dim, w)
        rows = ws.buffer("latent.gathered", n * page, self.rank, bf16)
        kernels.latent_gather(cache.keys, table, plan["pages"], rows, self.rot_dim)
        up = self.up.forward(rows, ws.buffer("latent.up", n * page, self.up.out_features, bf16))
        keys = ws.buffer("latent.expanded_k", n * self.nq * page, w, bf16).view(n, self.nq, page, w)
        values = ws.buffer("latent.expanded_v", n * self.nq * w, page, bf16).view(n, self.nq, w, page)
        kernels.latent_pages(cache.keys, table, plan["pages"], up, keys, values, self.plain_dim, self.rot_dim, self.v_dim, self.rank)
        direct = w == self.v_dim and self.out_scale == 1.0
        o = out if direct else ws.buffer("latent.expanded_o", tokens, self.nq * w, bf16)
        part_o = part_ml = None
        if plan["splits"] > 1:
            part_o = ws.buffer("attention.portion_part_o", tokens * self.nq * plan["splits"], w, torch.float32)
            part_ml = ws.buffer("attention.portion_part_ml", tokens * self.nq * plan["splits"], 2, torch.float32)
        attention_mfma.attn_prefill(q, o, self.nq, self.nq, w, keys, values, ctx.positions, plan["table"], plan["items"],
                                    self.scale, int(self.window) if self.window is not None else 0, plan["split_size"],
                                    plan["splits"], part_o, part_ml, gate=gate,
                                    gate_width=0 if self.gate_heads else (self.v_dim if gate is not None else 0),
                                    sink=self.sink, softcap=self.score_cap)
        if not direct:
            for a, b in plan["spans"]:
                kernels.latent_compact(o[a:b], w, out[a:b], self.nq, self.v_dim, self.out_scale)

    def forward(self, x: torch.Tensor, ctx: StepContext, cache: PagedCacheView, residual: Optional[torch.Tensor] = None,
                next_scale: Optional[torch.Tensor] = None, next_offset: float = 0.0, leave_stats: bool = True):
        if self._o is None:
            self._o = Linear(self._o_weight, self.mode)
        ws = ctx.workspace
        inner = ws.buffer("latent.inner", x.shape[0], self.inner_width, self.act_dtype)
        self.forward_inner(x, ctx, cache, inner)
        result = ws.buffer("latent.out", x.shape[0], self.hidden, self.act_dtype)
        if residual is not None:
            return self._o.add_into(inner, residual, result, ws, next_scale, next_offset, leave_stats)
        return self._o.forward(inner, result)
