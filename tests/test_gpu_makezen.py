"""Makezen on the GPU against the plain implementation (tests/plain/makezen_plain.py), in 32-bit and in bfloat16.

Small configurations of their own and seeded random weights: one whose layers all differ (keys wider than values and the
other way round, grouped and ungrouped heads, 1 to 4 taps, latent rows read by layers with wider and with narrower
windows, layers without a feed-forward), one whose constants are one and whose sizes coincide, and one at widths where the
serving kernels run.  Each mechanism alone at its kernels, with inputs made so that a fault shows; window edges by what a
changed token may and may not reach; then whole prompts, token-by-token decoding, portions down to two tokens, mixed
batches with pages and slots used again, long prompts and long decoding, greedy generation through the scheduler, the
command line and the trace replay program.
"""
import json
import os
import random
import subprocess
import sys

import pytest
import torch

from conftest import ROOT, token_ids
from plain import makezen_plain as P
from test_gpu_model import SPLIT_TOL, close, mixed_trace, pages_were_used_again, run_alone, run_mixed

pytestmark = pytest.mark.gpu

DEV = "cuda:0"
F64 = torch.float64
TOL = {"float32": 3e-5, "bfloat16": 5e-2}


def scaling(factor, original, fast=32.0, slow=1.0):
    return {"factor": factor, "fast": fast, "original": original, "slow": slow}


def rot(base, dims, scale=None):
    out = {"base": base, "dims": dims}
    if scale is not None:
        out["scaling"] = scale
    return out


def delta(heads, kv_heads, dim, vdim, conv):
    return "delta", {"conv": conv, "dim": dim, "heads": heads, "kv_heads": kv_heads, "vdim": vdim}


def parallel(heads, kv_heads, dim, vdim, turn, scale, cap, right):
    left = {"dim": dim, "heads": heads, "kv_heads": kv_heads, "rot": turn, "scale": scale, "softcap": cap, "vdim": vdim}
    return "parallel", {"left": left, "right": right[1]}


def latent(heads, dim, rot_dim, vdim, q_rank, kv_rank, window, base, scale, scaled=None, kv_from=None):
    out = {"dim": dim, "heads": heads, "kv_rank": kv_rank, "mask": {"size": window}, "q_rank": q_rank,
           "rot": rot(base, rot_dim, scaled), "rot_dim": rot_dim, "scale": scale, "vdim": vdim}
    if kv_from is not None:
        out["kv_from"] = kv_from
    return "latent_attention", out


def layer(mixer, ff):
    return {"mixer": mixer[1], "mlp": None if ff is None else {"ff": ff, "kind": "dense"}, "type": mixer[0]}


def config(vocab, width, eps, layers):
    return {"architecture": "Makezen", "layers": layers, "norm": {"eps": eps}, "vocab": vocab, "width": width}


SLOW = scaling(4.0, 64, 8.0, 1.0)
# every layer another shape; layer 1's rows are read with a wider and with a narrower window, layer 4's with a narrower one
MIXED = config(311, 96, 1e-5, [
    layer(parallel(6, 3, 32, 16, rot(1e4, 16, scaling(8.0, 256, 16.0, 1.0)), 0.2, 7.0, delta(4, 2, 16, 32, 4)), 160),
    layer(latent(3, 16, 8, 24, 20, 40, 7, 500.0, 0.3, SLOW), None),
    layer(delta(3, 1, 24, 20, 2), None),
    layer(latent(2, 24, 8, 16, 28, 40, 29, 500.0, 0.2, SLOW, kv_from=1), 112),
    layer(latent(4, 8, 16, 40, 32, 24, 16, 1e4, 0.25), 72),
    layer(delta(2, 2, 40, 10, 3), 96),
    layer(latent(5, 16, 16, 8, 16, 24, 5, 1e4, 0.25, kv_from=4), None),
    layer(latent(1, 32, 8, 48, 24, 40, 1, 500.0, 0.3, SLOW, kv_from=1), 64),
])
# constants that are one, sizes that coincide, a window no prompt of the tests reaches, a convolution of one tap
EQUAL = config(515, 128, 1e-6, [
    layer(delta(2, 2, 64, 64, 1), 128),
    layer(parallel(2, 2, 64, 64, rot(1e4, 64, scaling(1.0, 1024)), 1.0, 1.0, delta(2, 2, 64, 64, 4)), 128),
    layer(latent(2, 64, 64, 64, 64, 64, 1000, 1e4, 0.125, scaling(1.0, 1024)), 128),
    layer(latent(2, 64, 64, 64, 64, 64, 1000, 1e4, 0.125, scaling(1.0, 1024), kv_from=2), None),
])
# widths of a real model's layers
WIDE = config(300, 1024, 1e-6, [
    layer(parallel(8, 2, 128, 128, rot(1e6, 64, scaling(4.0, 4096)), 0.09, 30.0, delta(4, 2, 128, 128, 4)), 2048),
    layer(latent(8, 64, 32, 64, 384, 256, 64, 1e5, 0.1, scaling(2.0, 2048)), 1024),
    layer(delta(8, 4, 128, 128, 4), None),
    layer(latent(8, 64, 32, 64, 256, 256, 100, 1e5, 0.1, scaling(2.0, 2048), kv_from=1), 2048),
])
CONFIGS = {"mixed": MIXED, "equal": EQUAL, "wide": WIDE}


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    if not torch.cuda.is_available():
        pytest.skip("no GPU visible")
    from pulse_infer_amd.config import MakezenConfig
    from pulse_infer_amd.weights import write_model_folder

    out = {}
    for seed, (name, cfg) in enumerate(CONFIGS.items()):
        out[name] = write_model_folder(MakezenConfig.from_dict(cfg), str(tmp_path_factory.mktemp(name)), seed=370 + seed)
    return out


class Oracle:
    """The plain implementation of every folder, its logits and fragile positions remembered."""

    def __init__(self, folders):
        self.models = {name: P.PlainMakezen.from_folder(folder) for name, folder in folders.items()}
        self.memo = {}

    def _kept(self, what, name, ids, make):
        key = (what, name, tuple(ids))
        if key not in self.memo:
            self.memo[key] = make(list(ids))
        return self.memo[key]

    def __call__(self, name, ids):
        return self._kept("logits", name, ids, self.models[name].logits)

    def fragile(self, name, ids):
        return self._kept("fragile", name, ids, self.models[name].fragile_positions)


@pytest.fixture(scope="module")
def plain(folders):
    return Oracle(folders)


def agree(got, want, dtype, what, fragile=(), first=0, tol=TOL, loose=False):
    """``close``, without the positions whose logits hang on cancellations.  ``loose`` (in bfloat16, for models with narrow
    delta heads: a head's few values are divided by their own size, which multiplies bfloat16's roundings where they
    cancel): the median position within the bound, none beyond three times it."""
    keep = [i for i in range(want.shape[0]) if i + first not in fragile]
    assert len(keep) >= 0.7 * want.shape[0] or want.shape[0] < 10, f"{what}: too many fragile positions to say anything"
    if not keep:
        return
    if loose and dtype == "bfloat16":
        rows = (got[keep].double().cpu() - want[keep].double().cpu()).abs().max(dim=1).values
        bound = tol[dtype] * max(1.0, float(want.abs().max()))
        assert torch.isfinite(rows).all(), what
        assert float(rows.median()) <= bound and float(rows.max()) <= 3.0 * bound, \
            f"{what}: median {float(rows.median()):.3e}, worst {float(rows.max()):.3e}, bound {bound:.3e}"
        return
    close(got[keep], want[keep], dtype, what, tol)


@pytest.fixture(scope="module")
def runners(folders):
    from pulse_infer_amd.engine.runner import ModelRunner
    from pulse_infer_amd.models.factory import load_model

    made = {}

    def get(name, dtype, page=16, tokens=512):
        key = (name, dtype, page, tokens)
        if key not in made:
            _, model = load_model(folders[name], mode=dtype)
            made[key] = ModelRunner(model, page_size=page, num_pages=tokens // page, max_requests=4)
        return made[key]

    return get


# ------------------------------------------------------------------------------------------- mechanisms alone
def rnd(*shape, seed=0, scale=1.0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=torch.float32) * scale


def stored(x, dtype):
    dev = x.to(dtype).to(DEV)
    return dev, dev.cpu().to(F64)


def tol(dtype):
    return dict(atol=2e-5, rtol=2e-5) if dtype == torch.float32 else dict(atol=2e-2, rtol=2e-2)


def ints(values):
    return torch.tensor(values, dtype=torch.int32, device=DEV)


def near(got, want, dtype, what=""):
    got = got.cpu().to(F64)
    assert torch.allclose(got, want, **tol(dtype)), (what, float((got - want).abs().max()))


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("hidden", [96, 50, 1000, 4096, 9216])
def test_a_norm_before_and_after_in_one_step(dtype, hidden):
    """The update's own norm (layer norm, RMS norm, none; of a result or of the normed terms of one or two), the sum and
    the norm that reads the residual next, of all rows and of gathered ones (which leave the residual as it is)."""
    from pulse_infer_amd.ops import kernels

    eps, tokens = 1e-3, 11
    weights = [stored(1.0 + rnd(hidden, seed=10 + i, scale=0.3), dtype) for i in range(5)]
    bias, bias_ref = stored(rnd(hidden, seed=20), dtype)
    ys = [stored(rnd(tokens, hidden, seed=i + 1, scale=2.0) + 0.7, dtype) for i in range(2)]
    norms = {"layernorm": lambda x, w: P.layer_norm(x, w, eps), "rmsnorm": lambda x, w: P.unit_rms(x, eps) * w}
    for terms in (0, 1, 2):
        for post in ("layernorm", "rmsnorm", None):
            for pre in ("layernorm", "rmsnorm", None):
                h0 = rnd(tokens, hidden, seed=5) * 3.0 + 1.0
                if terms:
                    y = 0.5 * sum(P.unit_rms(ys[i][1], eps) * weights[i][1] for i in range(terms))
                    given = [(ys[i][0], weights[i][0]) for i in range(terms)]
                else:
                    y, given = ys[0][1], [(ys[0][0], None)]
                if post:
                    y = norms[post](y, weights[2][1]) + bias_ref
                want_h = h0.to(F64) + y
                want = norms[pre](want_h, weights[3][1]) if pre else None
                step = dict(post=(post, weights[2][0], bias, eps) if post else None, term_scale=0.5, term_eps=eps,
                            norm=(pre, weights[3][0], None, eps) if pre else None)
                h = h0.to(DEV)
                out = torch.full((tokens, hidden), float("nan"), dtype=dtype, device=DEV) if pre else None
                kernels.sandwich_step(h, given, out=out, **step)
                assert torch.allclose(h.cpu().to(F64), want_h, atol=3e-5, rtol=3e-5), (terms, post, pre)
                if pre is None:
                    continue
                near(out, want, dtype, (terms, post, pre))
                rows = [7, 0, 10, 3]
                h = h0.to(DEV)
                picked = torch.full((len(rows), hidden), float("nan"), dtype=dtype, device=DEV)
                kernels.sandwich_step(h, given, out=picked, rows=ints(rows), **step)
                near(picked, want[rows], dtype, (terms, post, pre, "rows"))
                assert torch.equal(h.cpu(), h0)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_the_embedding_with_a_norm(dtype):
    from pulse_infer_amd.ops import kernels

    for hidden in (50, 96, 1000, 4096):
        table, ref = stored(rnd(40, hidden, seed=1) + 0.5, dtype)
        w, wref = stored(1.0 + rnd(hidden, seed=2, scale=0.2), dtype)
        ids = [3, 39, 0, 3, 17]
        for kind, norm in (("layernorm", P.layer_norm), ("rmsnorm", lambda x, w, eps: P.unit_rms(x, eps) * w)):
            out = torch.full((len(ids), hidden), float("nan"), dtype=torch.float32, device=DEV)
            bad = torch.zeros(1, dtype=torch.int32, device=DEV)
            kernels.embed_norm(ints(ids), table, w, kind, 1e-4, out, bad, 2.5)
            assert torch.allclose(out.cpu().to(F64), norm(ref[ids] * 2.5, wref, 1e-4), atol=2e-5, rtol=2e-5)
            assert int(bad.item()) == 0
    kernels.embed_norm(ints([1, 40]), table, w, "layernorm", 1e-4, out[:2], bad)
    assert int(bad.item()) == 1 and torch.isnan(out[1]).all() and torch.isfinite(out[0]).all()


def test_blended_rotation_tables():
    from types import SimpleNamespace

    from pulse_infer_amd.ops import kernels
    from pulse_infer_amd.parts.rope import RotaryEmbedding

    positions = [0, 1, 5, 63, 64, 2047, 100000]
    for r in (rot(1e4, 64, scaling(8.0, 4096)), rot(500.0, 8, SLOW), rot(1e6, 32)):
        part = RotaryEmbedding({"theta": r["base"], "rotary_dim": r["dims"], "pairing": "half", "yarn": r.get("scaling")},
                               SimpleNamespace(device=DEV))
        cos, sin = (torch.empty(len(positions), r["dims"] // 2, dtype=torch.float32, device=DEV) for _ in range(2))
        kernels.rope_table(ints(positions), part.inv_freq, cos, sin, part.magnitude)
        x = torch.zeros(len(positions), 1, r["dims"], dtype=F64)
        x[..., :r["dims"] // 2] = 1.0
        want = P.turn(x, positions, r)[:, 0]        # (1, 0) turned: cos in the first half, sin in the second
        got = torch.cat([cos, sin], dim=1).cpu().to(F64)
        assert torch.allclose(got, want, atol=1e-6, rtol=0)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_short_convolution_ring_and_recurrence(dtype):
    """The gated delta rule from its projections on against the plain mixer with identity projections: earlier portions,
    then one step that holds a long portion, a fresh prompt in a slot full of NaN, two tokens and single tokens (token by
    token, with the rows of the state shared out over 4 and over 16 lanes, and the longer ones in chunks), then a step of
    single tokens through the one-launch kernel and through prepared rows."""
    from types import SimpleNamespace

    from pulse_infer_amd.ops import kernels

    for heads, groups, d, dv, taps in [(4, 2, 16, 32, 4), (3, 1, 24, 20, 2), (2, 2, 40, 10, 3), (2, 2, 64, 64, 1),
                                       (6, 3, 128, 128, 4), (2, 1, 256, 256, 5), (1, 1, 8, 4, 16), (2, 2, 33, 12, 4), (2, 1, 100, 52, 4)]:
        eps, scale = 1e-5, 1.3
        gd, hv = groups * d, heads * dv
        channels = 2 * gd + hv
        g0, b0, a0 = channels, channels + hv, channels + hv + heads
        width = a0 + heads
        eye = torch.eye(width, dtype=F64)
        taps_all = rnd(channels, taps, seed=1, scale=0.7)
        taps_ref = taps_all.to(F64)
        a_log, dt = rnd(heads, seed=2, scale=0.5), rnd(heads, seed=3)
        norm_w = 1.0 + rnd(dv, seed=4, scale=0.2)
        w = {"m.q": eye[:gd], "m.k": eye[gd:2 * gd], "m.v": eye[2 * gd:channels], "m.g": eye[g0:b0], "m.b": eye[b0:a0],
             "m.a": eye[a0:], "m.q.conv": taps_ref[:gd], "m.k.conv": taps_ref[gd:2 * gd], "m.v.conv": taps_ref[2 * gd:],
             "m.A_log": a_log.to(F64), "m.dt_bias": dt.to(F64), "m.norm": norm_w.to(F64), "m.o": torch.eye(hv, dtype=F64)}
        sizes = {"heads": heads, "kv_heads": groups, "dim": d, "vdim": dv}
        counts, starts, slots = [150, 64, 2, 1, 1], [33, 0, 5, 17, 0], [3, 0, 4, 1, 6]
        y_of, wants = [], []
        for r in range(5):
            y, ref = stored(rnd(starts[r] + counts[r] + 3, width, seed=40 + r), dtype)
            y_of.append(y)
            wants.append(P.delta_mixer(ref, w, "m", sizes, eps) * scale)
        dev = lambda t: t.to(torch.float32).to(DEV).contiguous()
        conv, a_log, dt, norm_w = dev(taps_all.t()), dev(a_log), dev(dt), dev(norm_w)
        slot_floats = kernels.delta_slot_floats(heads, groups, d, dv, taps)

        def step(state, which, cut, lens, one_launch=False, row_groups=None):
            """Rows cut[r] .. cut[r] + lens[r] of every request in ``which``."""
            x = torch.cat([y_of[r][cut[r]:cut[r] + lens[r]] for r in which]).contiguous()
            n = x.shape[0]
            positions = ints([p for r in which for p in range(cut[r], cut[r] + lens[r])])
            entry = ints([i for i, r in enumerate(which) for _ in range(lens[r])])
            firsts = [0]
            for r in which:
                firsts.append(firsts[-1] + lens[r])
            first, start, slot = ints(firsts), ints([cut[r] for r in which]), ints([slots[r] for r in which])
            out = torch.full((n, hv), float("nan"), dtype=dtype, device=DEV)
            if one_launch:
                kernels.delta_decode(x, g0, b0, a0, conv, a_log, dt, norm_w, state, out, positions, entry, slot, heads, groups,
                                     d, dv, eps, scale)
                return out
            rows = torch.full((n, channels), float("nan"), dtype=torch.float32, device=DEV)
            gates = torch.full((n, 2 * heads), float("nan"), dtype=torch.float32, device=DEV)
            kernels.delta_prepare(x, b0, a0, conv, a_log, dt, state, rows, gates, positions, entry, start, first, slot, heads,
                                  groups, d, dv)
            o = torch.full((n, hv), float("nan"), dtype=torch.float32, device=DEV)
            others = None
            if row_groups == "chunks":
                entries = [SimpleNamespace(first_row=firsts[i], count=lens[r]) for i, r in enumerate(which)]
                chunks, runs, others = kernels.delta_chunk_lists(entries, 2)
                scratch = torch.full((len(chunks) // 4 * heads, kernels.delta_chunk_floats(d, dv)), float("nan"),
                                     dtype=torch.float32, device=DEV)
                kernels.delta_chunks(rows, gates, o, state, start, slot, ints(chunks), ints(runs), scratch, heads, groups, d, dv,
                                     taps)
                others = ints(others)
            if others is None or others.numel():
                kernels.delta_walk(rows, gates, o, state, first, start, slot, heads, groups, d, dv, taps,
                                   row_groups if isinstance(row_groups, int) else kernels.delta_row_groups(len(which), heads, d, dv),
                                   which=others)
            kernels.group_norm_gate(o, norm_w, x[:, g0:g0 + hv], out, heads, eps, scale, "silu")
            return out

        ends = {}
        for row_groups in (4, 16) + ("chunks",) * kernels.delta_chunks_takes(d, dv):
            state = torch.full((7, slot_floats), float("nan"), dtype=torch.float32, device=DEV)
            earlier = [r for r in range(5) if starts[r]]
            step(state, earlier, {r: 0 for r in earlier}, {r: starts[r] for r in earlier}, row_groups=row_groups)
            got = step(state, range(5), starts, counts, row_groups=row_groups)
            want = torch.cat([wants[r][starts[r]:starts[r] + counts[r]] for r in range(5)])
            near(got, want, dtype, (heads, groups, d, dv, taps, row_groups))
            ends[row_groups] = state
            if row_groups != 4:       # the states and the convolutions' inputs that are left behind
                used = [s for s in slots]
                assert torch.allclose(state[used], ends[4][used], atol=1e-4, rtol=1e-4, equal_nan=True), (heads, d, dv, row_groups)
        one_launch = [True] if kernels.delta_decode_takes(d, dv) else []
        for fused in [False] + one_launch:
            state = ends[4].clone()
            for i in range(3):     # three single tokens each, over what the portions left
                cut = {r: starts[r] + counts[r] + i for r in range(5)}
                got = step(state, range(5), cut, {r: 1 for r in range(5)}, one_launch=fused)
                near(got, torch.cat([wants[r][cut[r]:cut[r] + 1] for r in range(5)]), dtype, (heads, d, dv, "fused" if fused else "rows", i))
        if one_launch:             # first tokens in slots that hold NaN
            state = torch.full((7, slot_floats), float("nan"), dtype=torch.float32, device=DEV)
            for i in range(4):
                got = step(state, range(5), {r: i for r in range(5)}, {r: 1 for r in range(5)}, one_launch=True)
                near(got, torch.cat([wants[r][i:i + 1] for r in range(5)]), dtype, (heads, d, dv, "first", i))


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_a_far_write_is_read_back(dtype):
    """Decays of almost one and a key that no other token comes near: the value written at the start is read 300 tokens
    later, in a prompt and after decoding; its write strength counts."""
    from pulse_infer_amd.ops import kernels

    heads, d, dv, taps, n = 1, 32, 16, 1, 301
    channels, hv = 2 * d + dv, dv
    g0, b0, a0 = channels, channels + hv, channels + hv + 1
    y = torch.zeros(n, a0 + 1)
    y[:, :2 * d] = rnd(n, 2 * d, seed=1)
    y[:, 0] = y[:, d] = 0.0                      # channel 0 of q and k belongs to the far pair
    y[0, d:2 * d] = 0.0
    y[0, d] = 30.0
    y[n - 1, :d] = 0.0
    y[n - 1, 0] = 30.0
    y[:, 2 * d:channels] = rnd(n, dv, seed=2, scale=0.1)
    y[0, 2 * d:channels] = rnd(dv, seed=3, scale=4.0)
    y[:, g0:b0] = 5.0
    y[:, a0] = -12.0
    x, ref = stored(y, dtype)
    one = torch.ones(channels, 1)
    w = {"m." + k: torch.eye(a0 + 1, dtype=F64)[lo:hi] for k, lo, hi in
         (("q", 0, d), ("k", d, 2 * d), ("v", 2 * d, channels), ("g", g0, b0), ("b", b0, a0), ("a", a0, a0 + 1))}
    w.update({"m.q.conv": one[:d].to(F64), "m.k.conv": one[:d].to(F64), "m.v.conv": one[:dv].to(F64), "m.o": torch.eye(hv, dtype=F64),
              "m.A_log": torch.zeros(1, dtype=F64), "m.dt_bias": torch.zeros(1, dtype=F64), "m.norm": torch.ones(dv, dtype=F64)})
    want = P.delta_mixer(ref, w, "m", {"heads": 1, "kv_heads": 1, "dim": d, "vdim": dv}, 1e-6)
    state = torch.full((1, kernels.delta_slot_floats(1, 1, d, dv, taps)), float("nan"), dtype=torch.float32, device=DEV)
    args = (one.t().contiguous().to(DEV), torch.zeros(1, device=DEV), torch.zeros(1, device=DEV))
    out = torch.empty(1, hv, dtype=dtype, device=DEV)
    for t in range(n):
        kernels.delta_decode(x[t:t + 1], g0, b0, a0, *args, torch.ones(dv, device=DEV), state, out, ints([t]), ints([0]), ints([0]),
                             1, 1, d, dv, 1e-6)
    near(out, want[-1:], dtype, "decoded")
    first = P.silu(ref[0, 2 * d:channels])
    cosine = torch.dot(out.cpu().to(F64)[0], first) / (out.cpu().to(F64)[0].norm() * first.norm())
    assert float(cosine) > 0.98, "the read-out does not point at the first value"


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("nq,nkv,d,dv,dims", [(6, 3, 32, 16, 16), (2, 2, 64, 64, 64), (8, 2, 128, 128, 64), (3, 1, 20, 44, 8)])
def test_biased_projections_with_a_weighted_norm_of_every_head(dtype, nq, nkv, d, dv, dims):
    """Biases, the norm of every head with one weight vector for q and one for k, the blended rotation: prepared queries
    and what is stored in the pages (filled with NaN before)."""
    from pulse_infer_amd.ops import kernels
    from pulse_infer_amd.parts.attention_rows import stored_width

    n, page, eps = 37, 8, 1e-4
    D = stored_width(d, dv)
    cols = nq * d + nkv * (d + dv)
    x, ref = stored(rnd(n, cols, seed=1), dtype)
    biases = [stored(rnd(k, seed=2 + i, scale=0.8), dtype) for i, k in enumerate((nq * d, nkv * d, nkv * dv))]
    weights = [stored(1.0 + rnd(d, seed=7 + i, scale=0.4), dtype) for i in range(2)]
    r = rot(1e4, dims, scaling(4.0, 128, 8.0, 1.0))
    positions = list(range(100, 100 + n))
    half = dims // 2
    basis = torch.zeros(n, 1, dims, dtype=F64)
    basis[..., :half] = 1.0
    cs = P.turn(basis, positions, r)[:, 0]
    cos, sin = cs[:, :half].float().to(DEV).contiguous(), cs[:, half:].float().to(DEV).contiguous()
    pages = (positions[-1] + page) // page
    perm = torch.randperm(pages, generator=torch.Generator().manual_seed(3))
    kc = torch.full((pages, nkv, page, D), float("nan"), dtype=dtype, device=DEV)
    vc = torch.full((pages, nkv, D, page), float("nan"), dtype=dtype, device=DEV)
    q = torch.full((n, nq * D), float("nan"), dtype=dtype, device=DEV)
    kernels.qkv_rows(x, q, nq, nkv, d, dv, D, tuple(b[0] for b in biases), tuple(w[0] for w in weights), eps, cos, sin, dims, 1,
                     kc, vc, ints(positions), ints([0] * n), perm.to(torch.int32).view(1, -1).to(DEV), norm="head")
    q_ref = P.turn(P.unit_rms((ref[:, :nq * d] + biases[0][1]).view(n, nq, d), eps) * weights[0][1], positions, r)
    k_ref = P.turn(P.unit_rms((ref[:, nq * d:(nq + nkv) * d] + biases[1][1]).view(n, nkv, d), eps) * weights[1][1], positions, r)
    v_ref = (ref[:, (nq + nkv) * d:] + biases[2][1]).view(n, nkv, dv)
    q = q.cpu().view(n, nq, D)
    near(q[..., :d], q_ref, dtype, "q")
    assert float(q[..., d:].abs().sum()) == 0.0
    for i, p in enumerate(positions):
        pg, slot = int(perm[p // page]), p % page
        near(kc[pg, :, slot, :d], k_ref[i], dtype, "k")
        near(vc[pg, :, :dv, slot], v_ref[i], dtype, "v")


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_latent_helpers(dtype):
    """The norm of some columns of strided rows; a gate of one number a head behind both expansions; queries prepared
    without rows being written."""
    from pulse_infer_amd.ops import kernels

    heads, d, dr, dv, rank, n, D = 5, 16, 8, 24, 40, 19, 48
    x, ref = stored(rnd(n, 90, seed=1), dtype)
    w, wref = stored(1.0 + rnd(40, seed=2, scale=0.3), dtype)
    out = torch.full((n, 40), float("nan"), dtype=dtype, device=DEV)
    kernels.rms_rows(x, 17, w, 1e-3, out)
    near(out, P.unit_rms(ref[:, 17:57], 1e-3) * wref, dtype)

    o, oref = stored(rnd(n, heads * D, seed=3), dtype)
    w_uv, uv = stored(rnd(heads * dv, rank, seed=4, scale=rank ** -0.5), dtype)
    gate, gref = stored(rnd(n, 32, seed=5), dtype)
    want = torch.stack([(oref.view(n, heads, D)[:, h, :rank] @ uv[h * dv:(h + 1) * dv].T) * torch.sigmoid(gref[:, h:h + 1])
                        for h in range(heads)], dim=1).reshape(n, heads * dv) * 1.2
    y = torch.full((n, heads * dv), float("nan"), dtype=dtype, device=DEV)
    kernels.latent_expand(o, D, w_uv, gate[:, :heads], y, heads, dv, rank, 1.2, gate_heads=True)
    near(y, want, dtype, "expand")
    per_head = w_uv.view(heads, dv, rank)
    if kernels.heads_product_takes(o, per_head, y, D):
        y.fill_(float("nan"))
        kernels.heads_product(o, D, per_head, gate[:, :heads], y, dv, 1.2, gate_heads=True)
        near(y, want, dtype, "heads_product")

    raw, raw_ref = stored(rnd(n, heads * (d + dr), seed=6), dtype)
    r, positions = rot(500.0, dr, SLOW), list(range(60, 60 + n))
    basis = torch.zeros(n, 1, dr, dtype=F64)
    basis[..., :dr // 2] = 1.0
    cs = P.turn(basis, positions, r)[:, 0]
    cos, sin = cs[:, :dr // 2].float().to(DEV).contiguous(), cs[:, dr // 2:].float().to(DEV).contiguous()
    kc = torch.full((4, 1, 16, D), float("nan"), dtype=dtype, device=DEV)
    vc = torch.full((4, 1, D, 16), float("nan"), dtype=dtype, device=DEV)
    q = torch.full((n, heads * D), float("nan"), dtype=dtype, device=DEV)
    kernels.latent_rows(raw, 0, 0, q, None, cos, sin, 1, kc, vc, ints(positions), ints([0] * n), ints([[0, 1, 2, 3]]), heads, d,
                        dr, rank, D, 1e-5, write=False)
    assert torch.isnan(kc.float()).all() and torch.isnan(vc.float()).all()
    near(q.view(n, heads, D)[..., rank:rank + dr], P.turn(raw_ref.view(n, heads, d + dr)[..., d:], positions, r), dtype, "turned")


# ------------------------------------------------------------------------------------------------ what stands out
def edited_folder(cfg, folder, seed, edit):
    """A model folder whose random weights ``edit(tensors)`` has changed."""
    from safetensors.torch import load_file

    from pulse_infer_amd.config import MakezenConfig
    from pulse_infer_amd.weights import write_model_folder
    from pulse_infer_amd.weights.safetensors_io import write_safetensors

    write_model_folder(MakezenConfig.from_dict(cfg), folder, seed=seed)
    path = os.path.join(folder, "model.safetensors")
    tensors = load_file(path)
    edit(tensors)
    write_safetensors(path, {k: v.contiguous() for k, v in tensors.items()})
    return folder


def new_runner(folder, dtype, page=16, tokens=512):
    from pulse_infer_amd.engine.runner import ModelRunner
    from pulse_infer_amd.models.factory import load_model

    _, model = load_model(folder, mode=dtype)
    return ModelRunner(model, page_size=page, num_pages=tokens // page, max_requests=4)


@pytest.mark.parametrize("page", [4, 16])
@pytest.mark.parametrize("windows,width", [((9,), 64), ((16, 16), 64), ((6, 21), 96), ((21, 6), 64), ((1, 33), 64)])
def test_what_a_token_reaches_at_a_windows_edge(tmp_path, windows, width, page):
    """One latent layer, or one and a layer that reads its rows: a position's logits depend on exactly the tokens its
    windows cover.  Changing the token just inside the edge changes them, changing the one just outside does not, at every
    position of a prompt and of decoded tokens (the edge then lies at every place of a page), and both are what the plain
    implementation says.  (A reader sees rows formed from the stream before the first layer's attention reached it only
    through that layer's input, so its reach is its own window.)"""
    from pulse_infer_amd.config import MakezenConfig
    from pulse_infer_amd.weights import write_model_folder

    layers = [layer(latent(3, 16, 8, 16, 24, 32, windows[0], 500.0, 0.15, SLOW), None)]
    if len(windows) > 1:
        layers.append(layer(latent(2, 24, 8, 16, 24, 32, windows[1], 500.0, 0.15, SLOW, kv_from=0), None))
    cfg = config(97, width, 1e-5, layers)
    folder = write_model_folder(MakezenConfig.from_dict(cfg), str(tmp_path / "m"), seed=5)
    oracle = P.PlainMakezen.from_folder(folder)
    runner = new_runner(folder, "float32", page, 192)
    n = 70
    ids = token_ids(97, n, seed=3)
    # rows (c, turned part) are formed from layer 0's input, the embedding alone: both layers see tokens, not sums
    reach = max(windows)
    base = {"prompt": run_alone(runner, ids, [n]), "decoded": run_alone(runner, ids, [20] + [1] * (n - 20))}
    want = oracle.logits(ids)
    for got in base.values():
        close(got, want, "float32", "base", TOL)
    for j in (0, 3, 4, 15, 16, 17, 31, 32, 40):
        changed = list(ids)
        changed[j] = (ids[j] + 41) % 97
        want = oracle.logits(changed)
        for kind, cuts in (("prompt", [n]), ("decoded", [20] + [1] * (n - 20))):
            got = run_alone(runner, changed, cuts)
            close(got, want, "float32", f"{kind}, token {j} changed", TOL)
            moved = (got - base[kind]).abs().max(dim=1).values.cpu()
            inside, outside = moved[j:j + reach], torch.cat([moved[:j], moved[j + reach:]])
            assert float(inside[-1]) > 1e-4 and float(inside.min()) > 1e-5, (kind, j, inside)
            assert float(outside.max()) < 1e-6 * float(want.abs().max()) + 1e-6, (kind, j, float(outside.max()))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_far_token_stands_out_in_capped_attention(tmp_path, dtype):
    """Keys made of the queries' own weights with the sign turned, and a token whose embedding is another one's with the
    sign turned: when the second comes, the first takes most of the weight wherever it stands (far back, at a page's border,
    at the very start), in prompts, at a portion's end and decoded."""
    cfg = config(131, 96, 1e-5, [layer(parallel(3, 3, 32, 32, rot(1e6, 8), 3.0, 40.0, delta(2, 1, 16, 16, 3)), 96)])
    asks, answers = 125, 126

    def edit(t):
        t["l0.mix.left.k"] = -t["l0.mix.left.q"]
        t["l0.mix.left.q.b"] = torch.zeros_like(t["l0.mix.left.q.b"])
        t["l0.mix.left.k.b"] = torch.zeros_like(t["l0.mix.left.k.b"])
        t["l0.mix.left.k.norm"] = t["l0.mix.left.q.norm"].clone()
        t["l0.mix.left.out"] *= 4.0
        t["embed"][answers] = -t["embed"][asks]
    folder = edited_folder(cfg, str(tmp_path / "m"), 7, edit)
    oracle = P.PlainMakezen.from_folder(folder)
    runner = new_runner(folder, dtype, 16, 512)
    n = 330
    for far in (0, 2, 15, 16, 31, 32, n - 3):
        ids = token_ids(120, n, seed=9)
        other = list(ids)
        ids[far] = answers
        ids[-1] = other[-1] = asks
        want, without = oracle.logits(ids), oracle.logits(other)
        assert float((want[-1] - without[-1]).abs().max()) > 0.1 * float(want[-1].abs().max()), far
        for cuts in ([n], [n - 1, 1], [100, n - 102, 2], [n - 20] + [1] * 20):
            got = run_alone(runner, ids, cuts)
            close(got[-1:], want[-1:], dtype, f"far token at {far}, {cuts}", TOL)


def test_sinks_and_score_caps_count(tmp_path):
    """Sinks of several sizes (one that takes almost everything) and scores far beyond the cap, against the plain
    implementation; leaving them out would show."""
    cfg = config(97, 64, 1e-5, [layer(latent(4, 16, 8, 16, 24, 32, 9, 500.0, 0.6, SLOW), None),
                                layer(parallel(4, 2, 16, 16, rot(1e4, 8, SLOW), 6.0, 2.5, delta(2, 2, 16, 16, 2)), 64)])

    def edit(t):
        t["l0.mix.sink"] = torch.tensor([6.0, -3.0, 0.5, 2.0], dtype=t["l0.mix.sink"].dtype)
    folder = edited_folder(cfg, str(tmp_path / "m"), 11, edit)
    oracle = P.PlainMakezen.from_folder(folder)
    ids = token_ids(97, 60, seed=4)
    want = oracle.logits(ids)
    for leave_out in ("sink", "cap"):
        w, c = dict(oracle.w), json.loads(json.dumps(cfg))
        if leave_out == "sink":
            w["l0.mix.sink"] = torch.full((4,), -1e9, dtype=F64)
        else:
            c["layers"][1]["mixer"]["left"]["softcap"] = 1e9
        assert float((P.forward(c, w, ids) - want).abs().max()) > 1e-2 * float(want.abs().max()), leave_out
    for dtype in ("float32", "bfloat16"):
        runner = new_runner(folder, dtype, 16, 128)
        close(run_alone(runner, ids, [60]), want, dtype, "whole", TOL)
        close(run_alone(runner, ids, [9, 2, 29] + [1] * 20), want, dtype, "cut", TOL)


# ------------------------------------------------------------------------------------------------ whole models
LENGTH = {"mixed": 150, "equal": 130, "wide": 170}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name,page", [("mixed", 16), ("mixed", 4), ("equal", 16), ("equal", 64), ("wide", 16)])
def test_whole_tail_and_portions(runners, plain, name, page, dtype):
    ids = token_ids(CONFIGS[name]["vocab"], LENGTH[name], seed=3)
    want, fragile = plain(name, ids), plain.fragile(name, ids)
    runner = runners(name, dtype, page)
    n = len(ids)
    whole = run_alone(runner, ids, [n])
    agree(whole, want, dtype, f"{name} whole", fragile, loose=name == "mixed")
    tail = run_alone(runner, ids, [n - 40] + [1] * 40)               # prefill against token-by-token decoding
    agree(tail, want, dtype, f"{name} tail", fragile, loose=name == "mixed")
    agree(tail, whole, dtype, f"{name} tail against whole", fragile, tol=SPLIT_TOL, loose=name == "mixed")
    for cuts in ([2, 3, 31, 2, 17, n - 57, 2], [1, 1, 1, 31, n - 34], [n - 2, 2], [7] * (n // 7) + [n % 7 or 7][:n % 7 > 0]):
        cuts = [c for c in cuts if c]
        portions = run_alone(runner, ids, cuts)
        agree(portions, want, dtype, f"{name} portions {cuts}", fragile, loose=name == "mixed")
        agree(portions, whole, dtype, f"{name} portions against whole", fragile, tol=SPLIT_TOL, loose=name == "mixed")
    first = run_alone(runner, ids[:3], [1, 1, 1])                     # the first tokens of a sequence
    agree(first, want[:3], dtype, f"{name} first tokens", fragile)


@pytest.mark.parametrize("name", ["mixed", "equal"])
def test_the_stream_after_every_layer(runners, plain, name):
    from pulse_infer_amd.engine.runner import StepEntry

    ids = token_ids(CONFIGS[name]["vocab"], 37, seed=8)
    runner = runners(name, "float32")
    model, seen = runner.model, []
    originals = [b.forward for b in model.blocks]

    def watched(forward):
        def run(stream, ctx, cache):
            forward(stream, ctx, cache)
            stream.settle()
            seen.append(stream.h.clone())
        return run

    try:
        for block, forward in zip(model.blocks, originals):
            block.forward = watched(forward)
        runner.add_request("layers")
        runner.reserve("layers", len(ids))
        runner.step([StepEntry("layers", ids, [])])
    finally:
        for block, forward in zip(model.blocks, originals):
            block.forward = forward
        runner.free_request("layers")
    want = plain.models[name].residuals(ids)
    assert len(seen) == len(want) == len(CONFIGS[name]["layers"])
    for i, (got, ref) in enumerate(zip(seen, want)):
        close(got, ref, "float32", f"{name} after layer {i}", TOL)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name,page", [("mixed", 16), ("equal", 16), ("equal", 32), ("wide", 16)])
def test_mixed_batches_with_pages_and_slots_used_again(runners, plain, name, page, dtype):
    """Up to four live requests over a pool of 256 tokens and four slots, portions of some beside single tokens of
    others: every request's logits are what it gets alone, whoever held its pages and its state's slot before."""
    ids, steps = mixed_trace(CONFIGS[name]["vocab"], seed=6, sizes=(2, 3, 5, 8, 13, 21, 34))
    runner = runners(name, dtype, page, tokens=256)
    got, pages_seen, most_live = run_mixed(runner, steps)
    assert most_live == 4 and pages_were_used_again(pages_seen)
    for k, mine in got.items():
        agree(mine, plain(name, ids[k]), dtype, f"{name} mixed request {k}", plain.fragile(name, ids[k]), loose=name == "mixed")


def test_slots_and_pages_are_used_again_by_requests_of_other_lengths(runners, plain):
    from pulse_infer_amd.engine.runner import StepEntry

    name = "mixed"
    runner = runners(name, "float32", 16, tokens=160)
    for storage in runner.cache.state.values():       # whatever a slot held before must not show
        storage.fill_(float("nan"))
    for g in runner.cache.groups:
        for t in g.spec.tensors(g.storage):
            t.fill_(float("nan"))
    lengths = [70, 3, 64, 17, 1, 80, 33, 16, 65, 48]
    for i in range(0, len(lengths), 2):
        pair = {f"q{i + j}": token_ids(CONFIGS[name]["vocab"], n, seed=40 + i + j) for j, n in enumerate(lengths[i:i + 2])}
        for rid, ids in pair.items():
            runner.add_request(rid)
            runner.reserve(rid, len(ids))
        logits = runner.step([StepEntry(rid, ids, [len(ids) - 1]) for rid, ids in pair.items()])
        for row, (rid, ids) in enumerate(pair.items()):
            close(logits[row:row + 1], plain(name, ids)[-1:], "float32", f"request {rid} of {len(ids)} tokens", TOL)
            runner.free_request(rid)
        runner.cache.check()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_long_prompt_far_beyond_the_windows(runners, plain, dtype):
    """400 tokens through windows of 1 to 29 (pages below the widest reader's window go back to the pool while the request
    runs), through states that keep everything and through attention that sees all of them: whole, with the last 60
    tokens decoded, and in a pool that holds no more than one such request's live pages of a window group."""
    name = "mixed"
    ids = token_ids(CONFIGS[name]["vocab"], 400, seed=21)
    want, fragile = plain(name, ids), plain.fragile(name, ids)
    runner = runners(name, dtype, 16, tokens=512)
    agree(run_alone(runner, ids, [400]), want, dtype, "whole", fragile, loose=name == "mixed")
    agree(run_alone(runner, ids, [150, 190] + [1] * 60), want, dtype, "decoded tail", fragile, loose=name == "mixed")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_portions_beside_single_tokens(runners, plain, dtype):
    """Steps that hold portions of 64 tokens and more (which attend to keys and values expanded to every head, behind
    windows of 64 and 100 tokens whose pages have gone back to the pool) beside short portions and single tokens of other
    requests (which attend in the latent space), and a step of two long portions."""
    from pulse_infer_amd.engine.runner import StepEntry

    name = "wide"
    vocab = CONFIGS[name]["vocab"]
    lengths = {"a": 420, "b": 90, "c": 300}
    ids = {k: token_ids(vocab, n, seed=30 + i) for i, (k, n) in enumerate(lengths.items())}
    runner = runners(name, dtype, 16, tokens=1024)
    steps = [{"a": 64, "b": 30}, {"a": 200, "b": 1}, {"b": 1, "a": 63, "c": 70}, {"c": 2, "b": 20, "a": 90}, {"c": 130, "a": 1},
             {"a": 1, "c": 65, "b": 38}, {"a": 1, "c": 1}, {"c": 32}]
    fed, got = {k: 0 for k in ids}, {k: [] for k in ids}
    for k in ids:
        runner.add_request(k)
    for step in steps:
        for k, n in step.items():
            runner.reserve(k, fed[k] + n)
        logits = runner.step([StepEntry(k, ids[k][fed[k]:fed[k] + n], list(range(n))) for k, n in step.items()])
        row = 0
        for k, n in step.items():
            got[k].append(logits[row:row + n])
            fed[k], row = fed[k] + n, row + n
    assert fed == lengths
    for k in ids:
        runner.free_request(k)
        agree(torch.cat(got[k]), plain(name, ids[k]), dtype, f"request {k}", plain.fragile(name, ids[k]))
        agree(run_alone(runner, ids[k], [lengths[k]]), plain(name, ids[k]), dtype, f"request {k} whole", plain.fragile(name, ids[k]))


@pytest.mark.parametrize("gate_heads", [True, False])
@pytest.mark.parametrize("heads,d,dr,dv,rank,window", [(4, 64, 32, 64, 256, 0), (4, 64, 32, 64, 256, 70), (3, 16, 8, 24, 264, 33),
                                                       (2, 128, 64, 128, 512, 64), (2, 96, 16, 112, 232, 1)])
def test_latent_rows_expanded_to_every_head(heads, d, dr, dv, rank, window, gate_heads):
    """Long portions over gathered and expanded pages against the plain mixer's attention: portions that start inside a
    page and beyond the window, whose earlier pages are gone from the block table (and hold NaN), with a key planted just
    inside the window of one query and another just outside."""
    from types import SimpleNamespace

    from pulse_infer_amd.ops import attention_mfma as M
    from pulse_infer_amd.ops import kernels
    from pulse_infer_amd.parts.latent import latent_stored_width

    dtype, bs, scale = torch.bfloat16, 16, 0.2
    D, w = latent_stored_width(rank, dr), (max(d + dr, dv) + 15) // 16 * 16
    lens, counts = [300, 90, 131], [170, 90, 67]
    up_w, up_ref = stored(rnd(heads * (d + dv), rank, seed=1, scale=rank ** -0.5), dtype)
    sink = rnd(heads, seed=2)
    entries = [SimpleNamespace(start=n - c, count=c, first_row=sum(counts[:i])) for i, (n, c) in enumerate(zip(lens, counts))]
    per = [(n + bs - 1) // bs for n in lens]
    kc = torch.full((sum(per) + 1, 1, bs, D), float("nan"), dtype=dtype, device=DEV)
    perm = torch.randperm(sum(per) + 1, generator=torch.Generator().manual_seed(4)).tolist()
    table = torch.full((3, max(per)), -1, dtype=torch.int32)
    q, qref = stored(rnd(sum(counts), heads * (d + dr), seed=5), dtype)
    gate_cols = heads * (1 if gate_heads else dv)
    gate, gref = stored(rnd(sum(counts), gate_cols, seed=6), dtype)
    wants, at = [], 0
    for r, (n, e) in enumerate(zip(lens, entries)):
        c, cref = stored(rnd(n, rank + dr, seed=10 + r), dtype)
        if window > 1:     # one query's own direction as a key: seen by it, and by nobody `window` later
            t = e.start + 40
            row = qref[e.first_row + 40].view(heads, d + dr)[0]
            far = torch.cat([up_ref[:d].T @ row[:d], row[d:]]) * 4.0
            for j in (t - window + 1, t - window):
                if j >= 0:
                    c[j], cref[j] = stored(far.float(), dtype)
        low = max(0, e.start - window + 1) if window else 0
        for i in range(per[r]):
            if (i + 1) * bs <= low:
                continue                     # gone back to the pool
            page = perm[at + i]
            table[r, i] = page
            here = c[i * bs:min(n, (i + 1) * bs)]
            kc[page, 0, :here.shape[0]] = float("nan")
            kc[page, 0, :here.shape[0], :rank + dr] = here
        at += per[r]
        k_plain = (cref[:, :rank] @ up_ref[:heads * d].T).view(n, heads, d)
        v = (cref[:, :rank] @ up_ref[heads * d:].T).view(n, heads, dv)
        mine = qref[e.first_row:e.first_row + e.count].view(e.count, heads, d + dr)
        scores = torch.stack([mine[:, h, :d] @ k_plain[:, h].T + mine[:, h, d:] @ cref[:, rank:].T for h in range(heads)]) * scale
        full = torch.full((heads, n, n), 0.0, dtype=F64)
        full[:, e.start:] = scores
        a = P.softmax_weights(full, P.visible(n, window or None), sink.to(F64))[:, e.start:]
        o = torch.stack([a[h] @ v[:, h] for h in range(heads)], dim=1)
        g = torch.sigmoid(gref[e.first_row:e.first_row + e.count]).view(e.count, heads, -1)
        wants.append((o * g).reshape(e.count, heads * dv))
    numbered = list(enumerate(entries))
    flat, where = kernels.latent_expand_pages(numbered, window)
    n_pages, page = len(flat) // 4, kernels.EXPANDED_PAGE
    rows = torch.full((n_pages * page, rank), float("nan"), dtype=dtype, device=DEV)
    kernels.latent_gather(kc, table.to(DEV), ints(flat), rows, dr)
    assert torch.isfinite(rows).all()
    up = (rows.float() @ up_w.float().t()).to(dtype)
    keys = torch.full((n_pages, heads, page, w), float("nan"), dtype=dtype, device=DEV)
    values = torch.full((n_pages, heads, w, page), float("nan"), dtype=dtype, device=DEV)
    kernels.latent_pages(kc, table.to(DEV), ints(flat), up, keys, values, d, dr, dv, rank)
    assert torch.isfinite(keys).all() and torch.isfinite(values).all()
    wide_table = torch.full((3, max((n + page - 1) // page for n in lens)), -1, dtype=torch.int32)
    for r, e in numbered:
        low, first = where[r]
        last = (lens[r] + page - 1) // page
        wide_table[r, low:last] = torch.arange(first, first + last - low, dtype=torch.int32)
    positions = [p for e in entries for p in range(e.start, e.start + e.count)]
    cos, sin = torch.ones(len(positions), dr // 2, device=DEV), torch.zeros(len(positions), dr // 2, device=DEV)
    qx = torch.full((len(positions), heads * w), float("nan"), dtype=dtype, device=DEV)
    kernels.latent_queries(q, 0, qx, cos, sin, 1, heads, d, dr, w)
    o = torch.full((len(positions), heads * w), float("nan"), dtype=dtype, device=DEV)
    items = ints(M.build_items(numbered, M.portion_tokens(1, w)))
    M.attn_prefill(qx, o, heads, heads, w, keys, values, ints(positions), wide_table.to(DEV), items, scale, window, gate=gate,
                   gate_width=0 if gate_heads else dv, sink=sink.to(DEV))
    out = torch.full((len(positions), heads * dv), float("nan"), dtype=dtype, device=DEV)
    kernels.latent_compact(o, w, out, heads, dv)
    near(out, torch.cat(wants), dtype)


# ------------------------------------------------------------------------------------ seeded random configurations
def random_config(rng):
    """Layers drawn one by one, in any order: head sizes that are no multiples of 16 or of 4, keys wider or narrower than
    values, any grouping of heads, windows from one token on, latent rows that are no multiples of 8 and layers that read
    earlier ones', rotations on a part of a head and on all of it, with and without blended frequencies, 1 to 7 taps."""
    width = rng.choice([64, 96, 160, 256])

    def one_delta():
        groups = rng.choice([1, 2, 3])
        return delta(groups * rng.choice([1, 2, 3]), groups, rng.choice([8, 16, 24, 33, 64]), rng.choice([4, 10, 16, 32, 72]),
                     rng.choice([1, 2, 3, 4, 7]))

    def turn(dims):
        s = rng.choice([None, scaling(rng.choice([1.0, 4.0, 16.0]), rng.choice([32, 256, 4096]), rng.choice([8.0, 32.0]), 1.0)])
        return rot(rng.choice([100.0, 1e4, 5e5]), dims, s)

    layers = []
    for i in range(rng.choice([2, 3, 4])):
        kind = rng.choice(["delta", "parallel", "latent", "latent"])
        if kind == "delta":
            mixer = one_delta()
        elif kind == "parallel":
            groups, dim = rng.choice([1, 2, 3]), rng.choice([16, 24, 32, 64])
            mixer = parallel(groups * rng.choice([1, 2, 4, 18]), groups, dim, rng.choice([8, 16, 40, 64]),
                             turn(rng.choice([x for x in (2, 8, 16, dim) if x <= dim])), rng.choice([0.1, dim ** -0.5, 0.5]),
                             rng.choice([1.5, 10.0, 50.0]), one_delta())
        else:
            sources = [j for j, l in enumerate(layers) if l["type"] == "latent_attention" and "kv_from" not in l["mixer"]]
            heads, dim, vdim = rng.choice([1, 2, 4, 20]), rng.choice([8, 16, 24, 40]), rng.choice([8, 16, 20, 48])
            q_rank, window, scale = rng.choice([12, 24, 32, 100]), rng.choice([1, 5, 16, 33, 100, 500]), rng.choice([0.1, 0.3])
            if sources and rng.random() < 0.6:
                j = rng.choice(sources)
                s = layers[j]["mixer"]
                mixer = ("latent_attention", dict(s, heads=heads, dim=dim, vdim=vdim, q_rank=q_rank, mask={"size": window}, scale=scale,
                                                  kv_from=j))
            else:
                rot_dim = rng.choice([2, 8, 16, 32])
                mixer = latent(heads, dim, rot_dim, vdim, q_rank, rng.choice([12, 24, 32, 64, 100]), window, 1.0, scale)
                mixer[1]["rot"] = turn(rot_dim)
        layers.append(layer(mixer, rng.choice([None, 32, 100, 256])))
    return config(rng.choice([257, 300, 1000]), width, rng.choice([1e-6, 1e-5]), layers)


@pytest.mark.parametrize("seed", range(12))
def test_random_configurations(tmp_path, seed):
    """Whole, with the last 20 tokens one by one, and in portions of 2 to 70 tokens, in 32-bit and in bfloat16."""
    if not torch.cuda.is_available():
        pytest.skip("no GPU visible")
    from pulse_infer_amd.config import MakezenConfig
    from pulse_infer_amd.weights import write_model_folder

    rng = random.Random(4100 + seed)
    cfg = random_config(rng)
    length = rng.choice([90, 150])
    folder = write_model_folder(MakezenConfig.from_dict(cfg), str(tmp_path / "m"), seed=seed)
    oracle = P.PlainMakezen.from_folder(folder)
    ids = token_ids(cfg["vocab"], length, seed=seed)
    want, fragile = oracle.logits(ids), oracle.fragile_positions(ids)
    what = f"{cfg} length {length}"
    print(what, flush=True)
    for dtype in ("float32", "bfloat16"):
        runner = new_runner(folder, dtype, 16, 256)
        whole = run_alone(runner, ids, [length])
        agree(whole, want, dtype, f"whole: {what}", fragile, loose=True)
        tail = run_alone(runner, ids, [length - 20] + [1] * 20)
        agree(tail, want, dtype, f"tail: {what}", fragile, loose=True)
        cuts, left_over, sizes = [], length, [40, 2, 17, 3, 70, 5, 19]
        while left_over:
            n = min(sizes[len(cuts) % len(sizes)], left_over)
            cuts.append(n)
            left_over -= n
        portions = run_alone(runner, ids, cuts)
        agree(portions, want, dtype, f"portions {cuts}: {what}", fragile, loose=True)
        agree(tail, whole, dtype, f"tail against whole: {what}", fragile, loose=True)
        agree(portions, whole, dtype, f"portions against whole: {what}", fragile, loose=True)
        del runner
    torch.cuda.empty_cache()


# ------------------------------------------------------------------------------------------------ long decoding
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["mixed", "wide"])
def test_long_decoding_of_three_requests(runners, plain, name, dtype):
    """Three requests of unequal prompts decode 100 tokens together, over page borders and out of every window; in
    bfloat16 the steps are recorded and replayed."""
    from pulse_infer_amd.engine.runner import StepEntry

    vocab, new = CONFIGS[name]["vocab"], 100
    runner = runners(name, dtype, 16, tokens=704)
    prompt = {"d0": 1, "d1": 30, "d2": 47}
    ids = {k: token_ids(vocab, n + new, seed=60 + i) for i, (k, n) in enumerate(prompt.items())}
    got = {k: [] for k in ids}
    for k in ids:
        runner.add_request(k)
        runner.reserve(k, prompt[k])
    first = runner.step([StepEntry(k, ids[k][:prompt[k]], [prompt[k] - 1]) for k in ids])
    for row, k in enumerate(ids):
        got[k].append(first[row:row + 1])
    replays = runner.graph_replays
    for step in range(new):
        for k in ids:
            runner.reserve(k, prompt[k] + step + 1)
        logits = runner.step([StepEntry(k, [ids[k][prompt[k] + step]], [0]) for k in ids])
        for row, k in enumerate(ids):
            got[k].append(logits[row:row + 1])
    assert (runner.graph_replays > replays) == (dtype == "bfloat16")
    for k in ids:
        runner.free_request(k)
        agree(torch.cat(got[k]), plain(name, ids[k])[prompt[k] - 1:], dtype, f"{name} decoding request {k}",
              plain.fragile(name, ids[k]), first=prompt[k] - 1, loose=name == "mixed")


# --------------------------------------------------------------------------- generation through the scheduler
@pytest.mark.parametrize("name", ["mixed", "equal"])
def test_greedy_generation_through_the_engine(folders, plain, name):
    """In 32-bit the greedy choice does not depend on the batch: requests generated together, in small portions and
    with a pool so tight that some are preempted and recomputed (their states start again from zero), give what
    each gives alone and what the plain implementation chooses."""
    from pulse_infer_amd import LLM

    vocab, new, page = CONFIGS[name]["vocab"], 12, 16
    prompts = [token_ids(vocab, n, seed=80 + i) for i, n in enumerate((1, 5, 18, 40, 77))]
    make = lambda **kw: LLM.from_pretrained(folders[name], dtype="float32", page_size=page, **kw)
    alone = [make(max_batch_size=1, chunk_size=256, num_pages=32).generate([p], max_new_tokens=new, ignore_eos=True)[0]
             for p in prompts]
    assert alone == [plain.models[name].greedy(p, new) for p in prompts]
    roomy = make(max_batch_size=4, chunk_size=16, num_pages=64, max_num_batched_tokens=24)
    assert roomy.generate(prompts, max_new_tokens=new, ignore_eos=True) == alone
    need = max((len(p) + new + page - 1) // page for p in prompts)
    tight = make(max_batch_size=4, chunk_size=16, num_pages=need + 2)
    assert tight.generate(prompts, max_new_tokens=new, ignore_eos=True) == alone
    tight.engine.runner.cache.check()


def test_bfloat16_generation_stays_within_rounding_of_the_plain_choice(folders, plain):
    """Every token that the bfloat16 engine chooses is, for the plain implementation, within rounding of the best one."""
    from pulse_infer_amd import LLM

    name, new = "wide", 10
    prompts = [token_ids(CONFIGS[name]["vocab"], n, seed=90 + i) for i, n in enumerate((3, 21))]
    llm = LLM.from_pretrained(folders[name], dtype="bfloat16", max_batch_size=2, chunk_size=8, page_size=16, num_pages=32)
    for prompt, out in zip(prompts, llm.generate(prompts, max_new_tokens=new, ignore_eos=True)):
        assert len(out) == new
        for t, token in enumerate(out):
            row = plain(name, prompt + out[:t])[-1]
            assert float(row[token]) >= float(row.max()) - TOL["bfloat16"] * float(row.abs().max())


def test_the_command_line_generates(folders, plain):
    name = "equal"
    prompt = token_ids(CONFIGS[name]["vocab"], 9, seed=99)
    run = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "pulse_infer"), folders[name], "--dtype", "float32",
                          "--prompt-ids", ",".join(map(str, prompt)), "--max-new-tokens", "6", "--greedy",
                          "--ignore-eos", "--max-positions", "64"], capture_output=True, text=True, timeout=300)
    assert run.returncode == 0, run.stderr[-2000:]
    out = json.loads(run.stdout.strip().splitlines()[0])
    assert out["output_ids"] == plain.models[name].greedy(prompt, 6)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_replay_program(folders, plain, tmp_path, dtype):
    import numpy as np

    name = "mixed"
    vocab = CONFIGS[name]["vocab"]
    a, b = token_ids(vocab, 70, seed=1), token_ids(vocab, 21, seed=2)
    steps = [
        {"step": 0, "entries": [{"id": "a", "tokens": a[:50], "want": [0, 49]}], "end": []},
        {"step": 1, "entries": [{"id": "a", "tokens": a[50:69], "want": []}, {"id": "b", "tokens": b[:20], "want": [19]}],
         "end": []},
        {"step": 2, "entries": [{"id": "b", "tokens": b[20:], "want": [0]}, {"id": "a", "tokens": a[69:], "want": [0]}],
         "end": ["a", "b"]},
    ]
    out = tmp_path / f"out_{dtype}"
    run = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", folders[name], "--dtype", dtype,
                          "--out", str(out), "--max-tokens", "192"], input="\n".join(json.dumps(s) for s in steps) + "\n",
                         capture_output=True, text=True, timeout=300)
    assert run.returncode == 0, run.stderr[-2000:]
    assert [line for line in run.stdout.splitlines() if line.startswith("done")] == ["done 0", "done 1", "done 2"]
    la, lb = plain(name, a), plain(name, b)
    read = lambda i: torch.from_numpy(np.fromfile(out / f"{i}.f32", dtype="<f4").reshape(-1, vocab).copy())
    fragile = {id(la): plain.fragile(name, a), id(lb): plain.fragile(name, b)}
    judged = 0
    for step, rows in ((0, [(la, 0), (la, 49)]), (1, [(lb, 19)]), (2, [(lb, 20), (la, 69)])):
        got = read(step)
        assert got.shape[0] == len(rows) and torch.isfinite(got).all()
        for i, (want, at) in enumerate(rows):
            if at in fragile[id(want)]:
                continue
            close(got[i:i + 1], want[at:at + 1], dtype, f"step {step} row {i}", TOL)
            judged += 1
    assert judged >= 3
