"""Sosuvik on the GPU against the plain implementation (tests/plain/sosuvik_plain.py), in 32-bit and in bfloat16.

Small configurations of their own and seeded random weights: one whose layers all differ (keys wider than values and the
other way round, grouped and ungrouped heads, chunks of 7 to 50 positions, a loop over some of the layers, layers without a
feed-forward), one whose constants are one and whose sizes coincide, one without a loop and without groups of experts, and
one at widths where the serving kernels run.  Each mechanism alone at its kernels, with inputs made so that a fault shows;
chunk borders by what a changed token may and may not reach; then whole prompts, token-by-token decoding, portions down to
two tokens, mixed batches with pages used again, long prompts and long decoding, greedy generation through the scheduler,
the command line and the trace replay program.
"""
import json
import os
import random
import subprocess
import sys

import pytest
import torch

from conftest import ROOT, token_ids
from plain import sosuvik_plain as P
from test_gpu_model import SPLIT_TOL, close, mixed_trace, pages_were_used_again, run_alone, run_mixed

pytestmark = pytest.mark.gpu

DEV = "cuda:0"
F64 = torch.float64
TOL = {"float32": 3e-5, "bfloat16": 4e-2}


def scaling(factor, original, fast=32.0, slow=1.0):
    return {"factor": factor, "fast": fast, "original": original, "slow": slow}


def rot(base, dims, scale=None):
    out = {"base": base, "dims": dims}
    if scale is not None:
        out["scaling"] = scale
    return out


def attention(heads, kv_heads, dim, vdim, chunk, turn, scale, cap):
    return "attention", {"dim": dim, "heads": heads, "kv_heads": kv_heads, "mask": {"size": chunk}, "rot": turn, "scale": scale,
                         "softcap": cap, "vdim": vdim}


def latent(heads, dim, rot_dim, vdim, kv_rank, base, scale):
    return "latent_attention", {"dim": dim, "heads": heads, "kv_rank": kv_rank, "rot": rot(base, rot_dim), "rot_dim": rot_dim,
                                "scale": scale, "vdim": vdim}


def moe(experts, groups, top, ff, limit, scale):
    router = {"experts": experts, "scale": scale, "top": top}
    if groups:
        router["groups"] = {"count": groups[0], "keep": groups[1]}
    return {"expert": {"ff": ff, "limit": limit}, "kind": "moe", "router": router}


def layer(mixer, mlp):
    return {"mixer": mixer[1], "mlp": mlp, "type": mixer[0]}


def config(vocab, width, eps, logit_scale, loop, layers):
    out = {"architecture": "Sosuvik", "layers": layers, "logit_scale": logit_scale, "norm": {"eps": eps}, "vocab": vocab,
           "width": width}
    if loop:
        out["loop"] = dict(zip(("start", "stop", "times"), loop))
    return out


SLOW = scaling(4.0, 64, 8.0, 1.0)
# every layer another shape; layers 1 and 2 run three times
MIXED = config(311, 96, 1e-5, 1.7, (1, 3, 3), [
    layer(attention(6, 3, 32, 16, 24, rot(1e4, 16, scaling(8.0, 256, 16.0, 1.0)), 0.2, 7.0), moe(9, (3, 2), 3, 40, 0.8, 2.5)),
    layer(latent(3, 16, 8, 24, 40, 500.0, 0.3), None),
    layer(attention(4, 1, 24, 48, 7, rot(500.0, 24, SLOW), 0.25, 20.0), moe(8, (4, 3), 5, 72, 1.2, 0.7)),
    layer(latent(5, 8, 16, 40, 24, 1e4, 0.25), moe(6, (2, 1), 2, 56, 2.0, 1.0)),
    layer(attention(2, 2, 40, 20, 50, rot(1e4, 8), 0.15, 3.0), None),
])
# constants that are one, sizes that coincide, a chunk no prompt of the tests leaves, one pass, every expert chosen
EQUAL = config(515, 128, 1e-6, 1.0, (0, 1, 1), [
    layer(latent(2, 64, 64, 64, 64, 1e4, 0.125), moe(4, (1, 1), 4, 128, 1.0, 1.0)),
    layer(attention(2, 2, 64, 64, 1000, rot(1e4, 64, scaling(1.0, 1024)), 1.0, 1.0), moe(4, (4, 4), 1, 128, 1.0, 1.0)),
])
# no loop, no groups, a chunk of one token, the last layer a latent one
STRAIGHT = config(257, 80, 1e-4, 0.5, None, [
    layer(attention(3, 3, 20, 44, 1, rot(100.0, 4), 0.3, 5.0), moe(7, None, 2, 24, 0.5, 3.0)),
    layer(attention(9, 3, 48, 48, 33, rot(1e5, 48, scaling(16.0, 32, 4.0, 2.0)), 0.14, 30.0), None),
    layer(latent(4, 32, 16, 8, 96, 300.0, 0.2), moe(5, None, 3, 100, 3.0, 1.0)),
])
# widths of a real model's layers
WIDE = config(300, 1024, 1e-6, 2.0, (0, 2, 2), [
    layer(attention(8, 2, 128, 128, 64, rot(1e6, 128, scaling(4.0, 4096)), 0.09, 30.0), moe(8, (4, 2), 2, 512, 1.5, 1.5)),
    layer(latent(8, 64, 32, 64, 256, 1e5, 0.1), None),
    layer(attention(16, 4, 64, 64, 100, rot(1e6, 32), 0.125, 50.0), moe(8, (2, 1), 2, 256, 1.5, 2.0)),
])
CONFIGS = {"mixed": MIXED, "equal": EQUAL, "straight": STRAIGHT, "wide": WIDE}


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    if not torch.cuda.is_available():
        pytest.skip("no GPU visible")
    from pulse_infer_amd.config import SosuvikConfig
    from pulse_infer_amd.weights import write_model_folder

    out = {}
    for seed, (name, cfg) in enumerate(CONFIGS.items()):
        out[name] = write_model_folder(SosuvikConfig.from_dict(cfg), str(tmp_path_factory.mktemp(name)), seed=470 + seed)
    return out


CLOSE_CALL = 0.008      # a router's margin under which bfloat16 may choose otherwise


def clear_ids(model, vocab, count, seed, rounds=60):
    """Random tokens none of which leaves a router a close call (tokens that do are drawn again)."""
    gen = torch.Generator().manual_seed(seed)
    ids = torch.randint(0, vocab, (count,), generator=gen).tolist()
    for _ in range(rounds):
        bad = (model.router_margins(ids) < CLOSE_CALL).nonzero().flatten().tolist()
        if not bad:
            break
        for p in bad:
            ids[p] = int(torch.randint(0, vocab, (1,), generator=gen))
    return ids


class Oracle:
    """The plain implementation of every folder; tokens and logits remembered."""

    def __init__(self, folders):
        self.folders = folders
        self.models = {name: P.PlainSosuvik.from_folder(folder) for name, folder in folders.items()}
        self.memo = {}

    def _kept(self, key, make):
        if key not in self.memo:
            self.memo[key] = make()
        return self.memo[key]

    def __call__(self, name, ids):
        return self._kept(("logits", name, tuple(ids)), lambda: self.models[name].logits(list(ids)))

    def ids(self, name, count, seed):
        return self._kept(("ids", name, count, seed), lambda: clear_ids(self.models[name], CONFIGS[name]["vocab"], count, seed))

    def close_calls(self, name, ids):
        return self._kept(("calls", name, tuple(ids)), lambda: close_calls(self.models[name], ids))


def close_calls(model, ids):
    return set((model.router_margins(list(ids)) < CLOSE_CALL).nonzero().flatten().tolist())


@pytest.fixture(scope="module")
def plain(folders):
    return Oracle(folders)


def agree(got, want, dtype, what, calls=(), first=0, tol=TOL):
    """``close``; in bfloat16 a router's close call (``calls``, positions in the sequence; row 0 of ``got`` is position
    ``first``) may go the other way and reach later positions through the attention: the positions before the first one are
    compared one by one, and of the rest the median error."""
    if dtype == "bfloat16" and calls:
        cut = max(0, min(min(calls) - first, want.shape[0]))
        if cut:
            close(got[:cut], want[:cut], dtype, what + " (before the first close call)", tol)
        if cut < want.shape[0]:
            rest = (got[cut:].double().cpu() - want[cut:].double().cpu()).abs().max(dim=1).values
            assert torch.isfinite(rest).all(), what
            assert float(rest.median()) <= tol[dtype] * max(1.0, float(want.abs().max())), \
                f"{what}: median error {float(rest.median()):.3e}"
        return
    close(got, want, dtype, what, tol)


@pytest.fixture(scope="module")
def runners(folders):
    made = {}

    def get(name, dtype, page=16, tokens=512):
        key = (name, dtype, page, tokens)
        if key not in made:
            made[key] = new_runner(folders[name], dtype, page, tokens)
        return made[key]

    return get


def new_runner(folder, dtype, page=16, tokens=512):
    from pulse_infer_amd.engine.runner import ModelRunner
    from pulse_infer_amd.models.factory import load_model

    _, model = load_model(folder, mode=dtype)
    return ModelRunner(model, page_size=page, num_pages=tokens // page, max_requests=4)


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
def test_updates_and_two_norms_of_one_residual(dtype, hidden):
    """Sums of none to two updates (one of them in parts), the chosen experts' weighted results and a vector, then none, one
    or two norms of the sum (or the sum itself, rounded), of all rows or of gathered ones (which leave the residual as it
    is), with outputs that are columns of a wider matrix; an index that names no expert adds nothing."""
    from pulse_infer_amd.ops import kernels

    tokens, top, experts = 11, 3, 5
    weights = [stored(1.0 + rnd(hidden, seed=10 + i, scale=0.3), dtype) for i in range(2)]
    row, row_ref = stored(rnd(hidden, seed=15), dtype)
    term, term_ref = stored(rnd(tokens, hidden, seed=16, scale=2.0), dtype)
    parts = rnd(3, tokens, hidden, seed=17)
    y = rnd(tokens * top, hidden, seed=18)
    idx = torch.randint(0, experts, (tokens, top), generator=torch.Generator().manual_seed(2)).to(torch.int32)
    idx[4, 1], idx[7, 2], idx[7, 0] = -1, experts, experts + 3
    share = torch.rand(tokens, top, generator=torch.Generator().manual_seed(3))
    counts = ((idx >= 0) & (idx < experts)).to(F64)
    fed = lambda w: (y.to(F64).view(tokens, top, hidden) * (w * counts).unsqueeze(-1)).sum(1)
    h0 = rnd(tokens, hidden, seed=5) * 3.0 + 1.0
    for n_terms, with_parts, weighted, with_row in [(0, False, None, False), (1, False, True, False), (2, True, False, True),
                                                    (1, True, None, True), (0, False, True, True), (2, False, None, False)]:
        terms, v = [], h0.to(F64)
        if n_terms:
            terms.append(parts.to(DEV) if with_parts else term)
            v = v + (parts.to(F64).sum(0) if with_parts else term_ref)
        if n_terms > 1:
            terms.append(term)
            v = v + term_ref
        chosen = None
        if weighted is not None:
            chosen = (y.to(DEV), idx.to(DEV), share.to(DEV) if weighted else None, experts)
            v = v + fed(share.to(F64) if weighted else torch.ones(tokens, top, dtype=F64))
        if with_row:
            v = v + row_ref
        args = dict(experts=chosen, row=row if with_row else None)
        for n_outs in (0, 1, 2):
            for raw in (False, True):
                wide = [torch.full((tokens, 2 * hidden + 8), float("nan"), dtype=dtype, device=DEV) for _ in range(n_outs)]
                outs = [(wide[i][:, 8 * i:8 * i + hidden], None if raw and i == 0 else weights[i][0], 1e-3 * (i + 1))
                        for i in range(n_outs)]
                want = [v if raw and i == 0 else P.rms_norm(v, weights[i][1], 1e-3 * (i + 1)) for i in range(n_outs)]
                what = (n_terms, with_parts, weighted, with_row, n_outs, raw)
                h = h0.to(DEV)
                kernels.residual_norms(h, terms, outs=outs, **args)
                assert torch.allclose(h.cpu().to(F64), v, atol=3e-5, rtol=3e-5), what
                for i in range(n_outs):
                    near(outs[i][0], want[i], dtype, what)
                    assert torch.isnan(wide[i][:, 8 * i + hidden:].float()).all()
                if not n_outs:
                    continue
                rows = [7, 0, 10, 4]
                h = h0.to(DEV)
                picked = [(torch.full((len(rows), hidden), float("nan"), dtype=dtype, device=DEV), o[1], o[2]) for o in outs]
                kernels.residual_norms(h, terms, outs=picked, rows=ints(rows), **args)
                for i in range(n_outs):
                    near(picked[i][0], want[i][rows], dtype, what)
                assert torch.equal(h.cpu(), h0)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("experts,count,keep,top", [(12, 4, 2, 3), (8, 8, 5, 4), (64, 8, 4, 8), (256, 8, 3, 8), (1024, 64, 5, 11),
                                                    (9, 3, 1, 3), (130, 2, 1, 64), (10, 1, 1, 4), (6, 2, 2, 5)])
def test_a_router_whose_outputs_form_groups(dtype, experts, count, keep, top):
    """Choices inside the best groups by the sum of their two best choice scores, weights from the scores without the
    correction; corrections of both signs and, in a second turn, so negative that every choice score is below zero (an
    output of a group that is left out must not come back as a zero); both entry points."""
    from pulse_infer_amd.ops import kernels

    tokens, hidden, factor = 70, 96, 1.75
    router = {"experts": experts, "top": top, "scale": factor, "groups": {"count": count, "keep": keep}}
    x, xref = stored(rnd(tokens, hidden, seed=1), dtype)
    w_router, wref = stored(rnd(experts, hidden, seed=2, scale=hidden ** -0.5 * 1.5), dtype)
    for shift in (0.0, -3.0):
        corr, cref = stored(rnd(experts, seed=3, scale=0.4) + shift, dtype)
        w = {"m.router": wref, "m.correction": cref}
        s, c, left = P.choice_scores(xref, w, "m", router)
        margin = P.router_margin(xref, w, "m", {"router": router})
        clear = margin > 1e-4
        assert int(clear.sum()) > tokens // 3
        want = torch.sort(left.sort(dim=-1, descending=True, stable=True).indices[:, :top], dim=-1).values
        if shift and keep < count:
            assert float(c.max()) < 0.0
        for entry in ("router", "route"):
            idx = torch.full((tokens, top), -7, dtype=torch.int32, device=DEV)
            weight = torch.full((tokens, top), float("nan"), device=DEV)
            how = dict(score="sigmoid", renormalize=True, groups=(count, keep), weight_scale=factor)
            if entry == "router":
                kernels.moe_router(x, w_router, corr, top, idx, weight, **how)
            else:
                z = torch.zeros(tokens, experts, device=DEV)
                kernels.gemm_f32(x, w_router, z)
                kernels.moe_route(z, corr, top, idx, weight, **how)
            chosen = idx.cpu().long()
            assert torch.equal(torch.sort(chosen, dim=-1).values[clear], want[clear]), (entry, shift)
            assert all(len(set(r)) == top for r in chosen.tolist())
            groups = torch.zeros(tokens, count, dtype=torch.bool).scatter(1, chosen // (experts // count), True)
            assert int(groups.sum(1).max()) <= keep
            mine = torch.gather(s, 1, chosen)
            assert torch.allclose(weight.cpu().to(F64), factor * mine / (mine.sum(1, keepdim=True) + 1e-20), atol=1e-5, rtol=1e-5)


def test_a_group_is_marked_by_its_two_best():
    """One group with the single best output and poor others, one with two good ones, one whose three are middling: the two
    best together decide, not the best one, not the sum of all."""
    from pulse_infer_amd.ops import kernels

    s = torch.tensor([[.95, .05, .05, .60, .58, .02, .45, .45, .45]])
    z = torch.log(s / (1 - s)).to(DEV)
    for keep, want in ((1, {3, 4}), (2, {0, 3})):
        idx = torch.zeros(1, 2, dtype=torch.int32, device=DEV)
        weight = torch.zeros(1, 2, device=DEV)
        kernels.moe_route(z, None, 2, idx, weight, score="sigmoid", groups=(3, keep))
        assert set(idx.cpu().tolist()[0]) == want, keep
        got = dict(zip(idx.cpu().tolist()[0], weight.cpu().tolist()[0]))
        total = sum(float(s[0, e]) for e in want)
        assert all(abs(got[e] - float(s[0, e]) / total) < 1e-5 for e in want)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("experts,top,ff,hidden,limit", [(5, 2, 48, 96, 0.7), (3, 3, 40, 80, 2.0), (4, 2, 256, 1024, 1.0)])
def test_clamped_experts_weighted_as_they_come_out(dtype, experts, top, ff, hidden, limit):
    """The clamped activation with the weight on the result: the kernels of few tokens, the grouped products of both tile
    heights with their own sum, and with the sum left to the kernel that reads the residual next."""
    from pulse_infer_amd.ops import kernels

    tokens = 90
    x, xref = stored(rnd(tokens, hidden, seed=1, scale=2.0), dtype)
    w, stacks = {}, {"gate": [], "up": [], "down": []}
    for e in range(experts):
        for i, (name, shape) in enumerate((("gate", (ff, hidden)), ("up", (ff, hidden)), ("down", (hidden, ff)))):
            dev, w[f"e{e}.{name}"] = stored(rnd(*shape, seed=10 + 3 * e + i, scale=shape[1] ** -0.5), dtype)
            stacks[name].append(dev)
    gate, up, down = (torch.stack(stacks[k]).contiguous() for k in ("gate", "up", "down"))
    idx = torch.stack([torch.randperm(experts, generator=torch.Generator().manual_seed(t))[:top] for t in range(tokens)]).to(torch.int32)
    weight = torch.rand(tokens, top, generator=torch.Generator().manual_seed(5))
    want = torch.zeros(tokens, hidden, dtype=F64)
    for t in range(tokens):
        for k in range(top):
            want[t] += float(weight[t, k]) * P.expert(xref[t:t + 1], w, f"e{int(idx[t, k])}", limit)[0]
    unclamped = sum(float(weight[0, k]) * P.expert(xref[:1], w, f"e{int(idx[0, k])}", 1e9)[0] for k in range(top))
    assert float((unclamped - want[0]).abs().max()) > 0.1      # (the clamps matter)
    idx, weight = idx.to(DEV), weight.to(DEV)
    loose = dict(atol=3e-5, rtol=3e-5) if dtype == torch.float32 else dict(atol=4e-2, rtol=4e-2)
    act = torch.full((tokens * top, ff), float("nan"), dtype=dtype, device=DEV)
    out = torch.full((tokens, hidden), float("nan"), dtype=torch.float32, device=DEV)
    kernels.moe_gate_up(x, gate, up, idx, act, activation="clamped_swish", limit=limit)
    kernels.moe_down(x, act, down, idx, weight, out)
    assert torch.allclose(out.cpu().to(F64), want, **loose), float((out.cpu().to(F64) - want).abs().max())
    if not kernels.moe_grouped_takes(x, gate, down):
        return
    for rows in kernels.MOE_TILE_ROWS:
        for later in (False, True):
            y = torch.full((tokens * top, hidden), float("nan"), dtype=torch.float32, device=DEV)
            scratch = torch.zeros(2 * tokens * top + 3 * kernels.moe_max_tiles(tokens * top, experts, rows) + 1, dtype=torch.int32,
                                  device=DEV)
            act.fill_(float("nan"))
            out.zero_()
            kernels.moe_grouped(x, gate, up, down, idx, weight, act, y, None if later else out, scratch, rows,
                                activation="clamped_swish", limit=limit)
            if later:
                kernels.residual_norms(out, [], experts=(y, idx, weight, experts))
            assert torch.allclose(out.cpu().to(F64), want, **loose), (rows, later, float((out.cpu().to(F64) - want).abs().max()))


@pytest.mark.parametrize("values", [1, 1000, 5 * 32000])
def test_scaled_values(values):
    from pulse_infer_amd.ops import kernels

    x = rnd(values, seed=1)
    y = x.to(DEV)
    kernels.scale_values(y, -1.7)
    assert torch.allclose(y.cpu(), x * -1.7, rtol=1e-6, atol=0)


CHUNK_CASES = [
    # single tokens stand at a chunk's first, second and last position, at page borders and away from them
    dict(nq=6, nkv=2, d=32, bs=16, chunk=24, cap=7.0, lens=[150, 1, 24, 25, 48, 49, 72, 73, 74, 71], portion=70),
    dict(nq=4, nkv=4, d=48, bs=16, chunk=7, cap=0.0, lens=[90, 33, 17, 21, 22], portion=40),
    dict(nq=8, nkv=2, d=128, bs=32, chunk=64, cap=30.0, lens=[257, 100, 64, 65, 130], portion=129),
    dict(nq=8, nkv=1, d=64, bs=16, chunk=300, cap=20.0, lens=[700, 260, 17, 600, 601, 602, 899], portion=300),
    dict(nq=3, nkv=1, d=96, bs=16, chunk=41, cap=8.0, lens=[207, 41, 42, 5, 82, 83], portion=5),
    dict(nq=16, nkv=16, d=64, bs=16, chunk=96, cap=15.0, lens=[199, 96, 97], portion=14),
    dict(nq=4, nkv=2, d=128, bs=16, chunk=1, cap=5.0, lens=[130, 9, 1], portion=80),
    dict(nq=2, nkv=1, d=20, bs=4, chunk=5, cap=3.0, lens=[45, 9, 5, 6], portion=11),
]


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("case", CHUNK_CASES)
@pytest.mark.parametrize("needle", [None, "inside", "outside"])
def test_attention_inside_chunks(case, dtype, needle):
    """A portion of request 0 (over several chunks) beside single tokens of the others, with capped scores and one added to
    the softmax's sum, through every attention kernel and with one split and with several.  Pages that lie wholly before
    what a step can still see are gone from the block table, everything not stored is NaN.  With a needle, the key at the
    first position of the last token's chunk (or the one before it) is many times the query, so that it takes all the weight
    that the cap lets it take if it is seen."""
    from pulse_infer_amd.ops import attention_mfma as M
    from pulse_infer_amd.ops import kernels

    nq, nkv, d, bs, chunk, cap, lens, portion = (case[x] for x in ("nq", "nkv", "d", "bs", "chunk", "cap", "lens", "portion"))
    scale, share = 0.3, nq // nkv
    per = [(n + bs - 1) // bs for n in lens]
    perm = torch.randperm(sum(per) + 2, generator=torch.Generator().manual_seed(3)).tolist()
    kc = torch.full((len(perm), nkv, bs, d), float("nan"), dtype=dtype, device=DEV)
    vc = torch.full((len(perm), nkv, d, bs), float("nan"), dtype=dtype, device=DEV)
    table = torch.full((len(lens), max(per)), -1, dtype=torch.int32)
    firsts = [lens[0] - portion] + [n - 1 for n in lens[1:]]
    wants, qs, at = [], [], 0
    for r, n in enumerate(lens):
        q, qref = stored(rnd(n - firsts[r], nq, d, seed=10 + r), dtype)
        k, kref = stored(rnd(n, nkv, d, seed=40 + r), dtype)
        v, vref = stored(rnd(n, nkv, d, seed=70 + r), dtype)
        start = (n - 1) // chunk * chunk
        j = start if needle == "inside" else start - 1
        if needle and 0 <= j < n - 1:
            for g in range(nkv):
                k[j, g], kref[j, g] = stored(20.0 * qref[-1, g * share].float(), dtype)
        low = firsts[r] // chunk * chunk
        for i in range(per[r]):
            if (i + 1) * bs <= low:
                continue
            table[r, i] = perm[at + i]
            here = slice(i * bs, min(n, (i + 1) * bs))
            kc[perm[at + i], :, :here.stop - here.start] = k[here].transpose(0, 1)
            vc[perm[at + i], :, :, :here.stop - here.start] = v[here].permute(1, 2, 0)
        at += per[r]
        scores = torch.zeros(nq, n, n, dtype=F64)
        for h in range(nq):
            scores[h, firsts[r]:] = qref[:, h] @ kref[:, h // share].T * scale
        if cap:
            scores = cap * torch.tanh(scores / cap)
        a = P.softmax_weights(scores, P.same_chunk(n, chunk), extra=True)[:, firsts[r]:]
        wants.append(torch.stack([a[h] @ vref[:, h // share] for h in range(nq)], dim=1))
        qs.append(q)
        if needle == "inside" and cap == 0.0 and 0 <= j < n - 1:
            assert float(a[0, -1, j]) > 0.9
    q, want = torch.cat(qs).view(-1, nq * d).contiguous(), torch.cat(wants)
    positions = ints([p for r, n in enumerate(lens) for p in range(firsts[r], n)])
    entry = ints([r for r, n in enumerate(lens) for _ in range(firsts[r], n)])
    out = torch.zeros(q.shape[0], nq * d, dtype=dtype, device=DEV)
    extra = dict(sink=torch.zeros(nq, device=DEV), softcap=cap, chunk=chunk)
    paths = ["generic"]
    if M.supported(d, bs, dtype, dtype):
        paths += ["matrix", "matrix in splits", "matrix in the fewest keys' splits"]

    class E:
        def __init__(self, first_row, count):
            self.first_row, self.count = first_row, count

    for path in paths:
        out.fill_(float("nan"))
        if path == "generic":
            kernels.attn_generic(q, out, nq, nkv, d, kc, vc, positions, entry, table.to(DEV), scale, **extra)
        else:
            splits = 1 if path == "matrix" else 3
            numbered = list(enumerate([E(0, portion)] + [E(portion + i, 1) for i in range(len(lens) - 1)]))
            rows = q.shape[0] * nq * splits
            part_o = torch.full((rows, d), float("nan"), dtype=torch.float32, device=DEV) if splits > 1 else None
            part_ml = torch.full((rows, 2), float("nan"), dtype=torch.float32, device=DEV) if splits > 1 else None
            small = numbered
            if portion >= M.PORTION_MIN_TOKENS:
                small = numbered[1:]
                cut = splits if d in M.PREFILL_SPLIT_HEAD_DIMS else 1
                size = (lens[0] + cut * 64 - 1) // (cut * 64) * 64 if cut > 1 else 0
                M.attn_prefill(q, out, nq, nkv, d, kc, vc, positions, table.to(DEV), ints(M.build_items(numbered[:1], M.portion_tokens(share, d))),
                               scale, 0, size, cut, part_o if cut > 1 else None, part_ml if cut > 1 else None, **extra)
            items = ints(M.build_items(small, M.tokens_per_item(share)))
            span = max(lens) if path == "matrix in splits" else M.split_span(max(lens), chunk)
            split = (span + splits * 32 - 1) // (splits * 32) * 32
            M.attn_mfma(q, out, nq, nkv, d, kc, vc, positions, table.to(DEV), items, scale, 0, split, splits, max(lens), part_o, part_ml,
                        **extra)
        near(out.view(-1, nq, d), want, dtype, path)


@pytest.mark.parametrize("nq,nkv,d,dims,chunk,splits", [(8, 2, 128, 128, 48, 1), (8, 2, 128, 64, 300, 3), (4, 4, 64, 64, 33, 2),
                                                        (16, 1, 64, 0, 64, 1)])
def test_decoded_tokens_inside_chunks_from_the_projection_on(nq, nkv, d, dims, chunk, splits):
    """The kernel that turns q and the token's own key itself and stores key and value: tokens at every place of a chunk,
    also a chunk's first (which sees itself alone, and the one that is added)."""
    from pulse_infer_amd.ops import attention_mfma as M

    dtype, bs, scale, cap, share = torch.bfloat16, 16, 0.3, 6.0, nq // nkv
    lens = [1, 2, chunk, chunk + 1, chunk + 2, 2 * chunk, 2 * chunk + 1, 2 * chunk + 17, 3 * chunk - 1]
    r = rot(1e4, dims, scaling(4.0, 128, 8.0, 1.0)) if dims else None
    assert M.decode_takes(d, dims, 1)
    per = [(n + bs - 1) // bs for n in lens]
    perm = torch.randperm(sum(per) + 1, generator=torch.Generator().manual_seed(3)).tolist()
    kc = torch.full((len(perm), nkv, bs, d), float("nan"), dtype=dtype, device=DEV)
    vc = torch.full((len(perm), nkv, d, bs), float("nan"), dtype=dtype, device=DEV)
    table = torch.full((len(lens), max(per)), -1, dtype=torch.int32)
    raws, wants, at = [], [], 0
    for i, n in enumerate(lens):
        raw, ref = stored(rnd(1, (nq + 2 * nkv) * d, seed=i), dtype)
        k, kref = stored(rnd(n, nkv, d, seed=20 + i), dtype)
        v, vref = stored(rnd(n, nkv, d, seed=40 + i), dtype)
        q = P.turn(ref[:, :nq * d].view(1, nq, d), [n - 1], r, adjacent=False)[0]
        kref[n - 1] = P.turn(ref[:, nq * d:(nq + nkv) * d].view(1, nkv, d), [n - 1], r, adjacent=False)[0]
        vref[n - 1] = ref[0, (nq + nkv) * d:].view(nkv, d)
        for j in range((n - 1) // chunk * chunk // bs, per[i]):
            table[i, j] = perm[at + j]
            here = slice(j * bs, min(n - 1, (j + 1) * bs))
            if here.stop > here.start:
                kc[perm[at + j], :, :here.stop - here.start] = k[here].transpose(0, 1)
                vc[perm[at + j], :, :, :here.stop - here.start] = v[here].permute(1, 2, 0)
        at += per[i]
        s = torch.stack([kref[:, h // share] @ q[h] for h in range(nq)]) * scale
        full = torch.zeros(nq, n, n, dtype=F64)
        full[:, -1] = cap * torch.tanh(s / cap)
        a = P.softmax_weights(full, P.same_chunk(n, chunk), extra=True)[:, -1]
        wants.append(torch.stack([a[h] @ vref[:, h // share] for h in range(nq)]))
        raws.append(raw)
    cos = sin = None
    if dims:
        basis = torch.zeros(len(lens), 1, dims, dtype=F64)
        basis[..., :dims // 2] = 1.0
        cs = torch.cat([P.turn(basis[i:i + 1], [n - 1], r, adjacent=False)[:, 0] for i, n in enumerate(lens)])
        cos, sin = cs[:, :dims // 2].float().to(DEV).contiguous(), cs[:, dims // 2:].float().to(DEV).contiguous()
    out = torch.full((len(lens), nq * d), float("nan"), dtype=dtype, device=DEV)
    rows = len(lens) * nq * splits
    part_o = torch.full((rows, d), float("nan"), dtype=torch.float32, device=DEV) if splits > 1 else None
    part_ml = torch.full((rows, 2), float("nan"), dtype=torch.float32, device=DEV) if splits > 1 else None
    span = M.split_span(max(lens), chunk)
    M.attn_decode(torch.cat(raws).contiguous(), out, nq, nkv, d, kc, vc, ints([n - 1 for n in lens]), table.to(DEV), None, scale, 0,
                  (span + splits * 32 - 1) // (splits * 32) * 32, splits, max(lens), part_o, part_ml, None, None, 0.0, cos, sin, dims, 1,
                  True, sink=torch.zeros(nq, device=DEV), softcap=cap, chunk=chunk)
    near(out.view(-1, nq, d), torch.stack(wants), dtype)


def test_blended_rotation_tables_of_both_pairings():
    from types import SimpleNamespace

    from pulse_infer_amd.ops import kernels
    from pulse_infer_amd.parts.rope import RotaryEmbedding

    positions = [0, 1, 5, 63, 64, 2047, 100000]
    for r, pairing in ((rot(1e4, 64, scaling(8.0, 4096)), "half"), (rot(500.0, 8), "interleaved"), (rot(1e5, 48, scaling(16.0, 32, 4.0, 2.0)), "half"),
                       (rot(1e5, 16, scaling(2.0, 100)), "interleaved")):
        part = RotaryEmbedding({"theta": r["base"], "rotary_dim": r["dims"], "pairing": pairing, "yarn": r.get("scaling")},
                               SimpleNamespace(device=DEV))
        cos, sin = (torch.empty(len(positions), r["dims"] // 2, dtype=torch.float32, device=DEV) for _ in range(2))
        kernels.rope_table(ints(positions), part.inv_freq, cos, sin, part.magnitude)
        adjacent = pairing == "interleaved"
        first = slice(0, None, 2) if adjacent else slice(0, r["dims"] // 2)
        second = slice(1, None, 2) if adjacent else slice(r["dims"] // 2, None)
        x = torch.zeros(len(positions), 1, r["dims"], dtype=F64)
        x[..., first] = 1.0
        want = P.turn(x, positions, r, adjacent)[:, 0]
        assert torch.allclose(cos.cpu().to(F64), want[:, first], atol=1e-6, rtol=0)
        assert torch.allclose(sin.cpu().to(F64), want[:, second], atol=1e-6, rtol=0)


# ------------------------------------------------------------------------------------------------ what stands out
def edited_folder(cfg, folder, seed, edit):
    """A model folder whose random weights ``edit(tensors)`` has changed."""
    from safetensors.torch import load_file

    from pulse_infer_amd.config import SosuvikConfig
    from pulse_infer_amd.weights import write_model_folder
    from pulse_infer_amd.weights.safetensors_io import write_safetensors

    write_model_folder(SosuvikConfig.from_dict(cfg), folder, seed=seed)
    path = os.path.join(folder, "model.safetensors")
    tensors = load_file(path)
    edit(tensors)
    write_safetensors(path, {k: v.contiguous() for k, v in tensors.items()})
    return folder


@pytest.mark.parametrize("page", [4, 16])
@pytest.mark.parametrize("chunk,times", [(9, 0), (16, 0), (21, 2), (1, 2), (64, 0)])
def test_what_a_token_reaches_at_a_chunks_edge(tmp_path, chunk, times, page):
    """One layer of chunked attention, alone or run twice: a position's logits depend on exactly the earlier tokens of its
    own chunk.  Changing a token moves every later position of its chunk and none of the next one, in prompts and decoded
    (the edge then lies at every place of a page)."""
    from pulse_infer_amd.config import SosuvikConfig
    from pulse_infer_amd.weights import write_model_folder

    cfg = config(97, 64, 1e-5, 1.3, (0, 1, times) if times else None,
                 [layer(attention(4, 2, 16, 16, chunk, rot(500.0, 8, SLOW), 0.3, 5.0), None)])
    folder = write_model_folder(SosuvikConfig.from_dict(cfg), str(tmp_path / "m"), seed=5)
    oracle = P.PlainSosuvik.from_folder(folder)
    runner = new_runner(folder, "float32", page, 192)
    n = 70
    ids = token_ids(97, n, seed=3)
    ways = (("prompt", [n]), ("decoded", [20] + [1] * (n - 20)))
    base = {kind: run_alone(runner, ids, cuts) for kind, cuts in ways}
    for got in base.values():
        close(got, oracle.logits(ids), "float32", "base", TOL)
    for j in (0, 3, 8, 9, 15, 16, 20, 21, 31, 32, 41, 42, 63, 64):
        changed = list(ids)
        changed[j] = (ids[j] + 41) % 97
        want = oracle.logits(changed)
        end = min(n, (j // chunk + 1) * chunk)
        for kind, cuts in ways:
            got = run_alone(runner, changed, cuts)
            close(got, want, "float32", f"{kind}, token {j} changed", TOL)
            moved = (got - base[kind]).abs().max(dim=1).values.cpu()
            assert float(moved[j:end].min()) > 1e-5, (kind, j, moved[j:end])
            outside = torch.cat([moved[:j], moved[end:]])
            assert float(outside.max()) < 1e-6 * float(want.abs().max()) + 1e-6, (kind, j, float(outside.max()))


def asks_and_answers(kind, width=96):
    """A one-layer model in which a token's key is its query with the sign turned, and the tokens' embeddings 125 and 126 are
    each other's with the sign turned: where 125 asks, 126 stands out among the keys."""
    if kind == "attention":
        mixer = attention(4, 2, 32, 32, 128, rot(1e6, 8), 2.0, 40.0)
    else:
        mixer = latent(4, 32, 8, 32, 32, 1e6, 2.0)
    cfg = config(131, width, 1e-5, 1.0, None, [layer(mixer, None)])

    def edit(t):
        if kind == "attention":
            q = t["l0.mix.q"].view(2, 2, 32, width)
            t["l0.mix.k"] = -q[:, 0].reshape(64, width)
            t["l0.mix.q"] = torch.stack([q[:, 0], q[:, 0]], dim=1).reshape(128, width)
        else:
            q = t["l0.mix.q"].view(4, 40, width).clone()
            q[:, :32] = q[0, :32] * 1.5
            q[:, 32:] *= 0.2
            t["l0.mix.q"] = q.reshape(160, width)
            t["l0.mix.dkv"][:32] = q[0, :32]
            t["l0.mix.dkv.norm"] = torch.ones_like(t["l0.mix.dkv.norm"])
            t["l0.mix.uk"] = -torch.eye(32, dtype=q.dtype).repeat(4, 1)
        t["l0.mix.o"] *= 4.0
        t["embed"][126] = -t["embed"][125]
    return cfg, edit


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_far_token_stands_out_in_latent_attention(tmp_path, dtype):
    cfg, edit = asks_and_answers("latent_attention")
    folder = edited_folder(cfg, str(tmp_path / "m"), 7, edit)
    oracle = P.PlainSosuvik.from_folder(folder)
    runner = new_runner(folder, dtype, 16, 512)
    n = 330
    for far in (0, 1, 2, 15, 16, 31, 32, 300, n - 3):
        ids = token_ids(120, n, seed=9)
        other = list(ids)
        ids[far] = 126
        ids[-1] = other[-1] = 125
        want, without = oracle.logits(ids), oracle.logits(other)
        assert float((want[-1] - without[-1]).abs().max()) > 0.1 * float(want[-1].abs().max()), far
        for cuts in ([n], [n - 1, 1], [100, n - 102, 2], [n - 20] + [1] * 20):
            got = run_alone(runner, ids, cuts)
            close(got[-1:], want[-1:], dtype, f"far token at {far}, {cuts}", TOL)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_token_of_the_same_chunk_stands_out_and_one_before_it_does_not(tmp_path, dtype):
    cfg, edit = asks_and_answers("attention")
    folder = edited_folder(cfg, str(tmp_path / "m"), 7, edit)
    oracle = P.PlainSosuvik.from_folder(folder)
    runner = new_runner(folder, dtype, 16, 512)
    n = 330          # the last token's chunk starts at 256
    for far in (0, 240, 254, 255, 256, 257, 271, 272, n - 3):
        ids = token_ids(120, n, seed=9)
        other = list(ids)
        ids[far] = 126
        ids[-1] = other[-1] = 125
        want, without = oracle.logits(ids), oracle.logits(other)
        shift = float((want[-1] - without[-1]).abs().max()) / float(want[-1].abs().max())
        assert shift > 0.1 if far >= 256 else shift < 1e-12, (far, shift)
        for cuts in ([n], [n - 1, 1], [100, n - 102, 2], [255, 2, n - 257], [n - 80] + [1] * 80):
            got = run_alone(runner, ids, cuts)
            close(got[-1:], want[-1:], dtype, f"token at {far}, {cuts}", TOL)


def test_every_constant_counts(tmp_path):
    """What the engine must not leave out: the one added to the softmax's sum, the cap, the chunks counted from position 0,
    the blended rotation, the groups, the correction, the router's factor, the clamp, the embedding's output brought back in,
    the passes' vectors.  Each changes the plain implementation's logits visibly, and the engine gives the right ones."""
    cfg = config(97, 64, 1e-5, 1.4, (0, 2, 2), [
        layer(attention(4, 2, 16, 16, 13, rot(500.0, 16, SLOW), 1.5, 2.5), moe(8, (4, 2), 3, 40, 0.4, 2.0)),
        layer(latent(4, 16, 8, 16, 24, 500.0, 2.0), None)])

    def edit(t):
        t["l0.mlp.router"] *= 1.5
        t["l0.mlp.correction"] = torch.tensor([.3, -.2, .1, -.4, .5, -.1, .2, 0.], dtype=t["l0.mlp.correction"].dtype)
        t["loop.step"] = torch.randn(2, 64, generator=torch.Generator().manual_seed(1)).to(t["loop.step"].dtype)
        t["l0.mlp.e0.gate"] *= 2.0
    folder = edited_folder(cfg, str(tmp_path / "m"), 11, edit)
    oracle = P.PlainSosuvik.from_folder(folder)
    ids = clear_ids(oracle, 97, 60, seed=4)
    want = oracle.logits(ids)

    def changed(path, value):
        c = json.loads(json.dumps(cfg))
        at = c
        for key in path[:-1]:
            at = at[key]
        if value is None:
            del at[path[-1]]
        else:
            at[path[-1]] = value
        return P.forward(c, oracle.w, ids)

    l0 = ("layers", 0)
    others = {
        "cap": changed(l0 + ("mixer", "softcap"), 1e9), "chunk": changed(l0 + ("mixer", "mask", "size"), 14),
        "blend": changed(l0 + ("mixer", "rot", "scaling"), None), "slow": changed(l0 + ("mixer", "rot", "scaling", "slow"), 0.25),
        "groups": changed(l0 + ("mlp", "router", "groups"), None), "factor": changed(l0 + ("mlp", "router", "scale"), 1.0),
        "limit": changed(l0 + ("mlp", "expert", "limit"), 4.0), "logit_scale": changed(("logit_scale",), 1.0),
        "scale": changed(("layers", 1, "mixer", "scale"), 0.7), "times": changed(("loop", "times"), 1)}
    w = dict(oracle.w)
    for name, make in (("l0.mlp.correction", torch.zeros_like), ("loop.step", lambda t: t.flip(0)),
                       ("loop.in", lambda t: torch.cat([t[:, :64], torch.zeros_like(t[:, 64:])], dim=1))):
        others[name] = P.forward(cfg, dict(w, **{name: make(w[name])}), ids)
    real = P.softmax_weights
    try:
        P.softmax_weights = lambda scores, mask, extra=False: real(scores, mask, False)
        others["one in the sum"] = oracle.logits(ids)
    finally:
        P.softmax_weights = real
    for what, logits in others.items():
        assert float((logits - want).abs().max()) > 1e-2 * float(want.abs().max()), what
    calls = close_calls(oracle, ids)
    for dtype in ("float32", "bfloat16"):
        runner = new_runner(folder, dtype, 16, 128)
        agree(run_alone(runner, ids, [60]), want, dtype, "whole", calls)
        agree(run_alone(runner, ids, [9, 2, 29] + [1] * 20), want, dtype, "cut", calls)


# ------------------------------------------------------------------------------------------------ whole models
LENGTH = {"mixed": 130, "equal": 110, "straight": 120, "wide": 150}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name,page", [("mixed", 16), ("mixed", 4), ("equal", 16), ("equal", 64), ("straight", 16), ("wide", 16)])
def test_whole_tail_and_portions(runners, plain, name, page, dtype):
    ids = plain.ids(name, LENGTH[name], 3)
    want, calls = plain(name, ids), plain.close_calls(name, ids)
    runner = runners(name, dtype, page)
    n = len(ids)
    whole = run_alone(runner, ids, [n])
    agree(whole, want, dtype, f"{name} whole", calls)
    tail = run_alone(runner, ids, [n - 40] + [1] * 40)               # prefill against token-by-token decoding
    agree(tail, want, dtype, f"{name} tail", calls)
    agree(tail, whole, dtype, f"{name} tail against whole", calls, tol=SPLIT_TOL if dtype == "float32" else TOL)
    for cuts in ([2, 3, 31, 2, 17, n - 57, 2], [1, 1, 1, 31, n - 34], [n - 2, 2], [7] * (n // 7) + [n % 7 or 7][:n % 7 > 0]):
        cuts = [c for c in cuts if c]
        portions = run_alone(runner, ids, cuts)
        agree(portions, want, dtype, f"{name} portions {cuts}", calls)
        agree(portions, whole, dtype, f"{name} portions against whole", calls, tol=SPLIT_TOL if dtype == "float32" else TOL)
    first = run_alone(runner, ids[:3], [1, 1, 1])                     # the first tokens of a sequence
    agree(first, want[:3], dtype, f"{name} first tokens", calls)


@pytest.mark.parametrize("name", ["mixed", "equal", "straight"])
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
    assert len(seen) == len(want) == {"mixed": 9, "equal": 2, "straight": 3}[name]
    for i, (got, ref) in enumerate(zip(seen, want)):
        close(got, ref, "float32", f"{name} after layer run {i}", TOL)


def clear_trace(plain, name, seed):
    """``mixed_trace`` with tokens that leave no router a close call."""
    ids, steps = mixed_trace(CONFIGS[name]["vocab"], seed=seed, sizes=(2, 3, 5, 8, 13, 21, 34))
    ids = {k: plain.ids(name, len(v), 200 + i) for i, (k, v) in enumerate(ids.items())}
    fed = {k: 0 for k in ids}
    for step in steps:
        for e in step["entries"]:
            k, n = e["id"], len(e["tokens"])
            e["tokens"] = ids[k][fed[k]:fed[k] + n]
            fed[k] += n
    return ids, steps


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name,page", [("mixed", 16), ("equal", 32), ("straight", 16), ("wide", 16)])
def test_mixed_batches_with_pages_used_again(runners, plain, name, page, dtype):
    """Up to four live requests over a pool of 256 tokens, portions of some beside single tokens of others: every request's
    logits are what it gets alone, whoever held its pages before."""
    ids, steps = clear_trace(plain, name, seed=6)
    runner = runners(name, dtype, page, tokens=256)
    got, pages_seen, most_live = run_mixed(runner, steps)
    assert most_live == 4 and pages_were_used_again(pages_seen)
    for k, mine in got.items():
        agree(mine, plain(name, ids[k]), dtype, f"{name} mixed request {k}", plain.close_calls(name, ids[k]))


def test_pages_are_used_again_by_requests_of_other_lengths(runners, plain):
    from pulse_infer_amd.engine.runner import StepEntry

    name = "mixed"
    runner = runners(name, "float32", 16, tokens=160)
    for g in runner.cache.groups:                     # whatever a page held before must not show
        for t in g.spec.tensors(g.storage):
            t.fill_(float("nan"))
    lengths = [70, 3, 64, 17, 1, 80, 33, 16, 65, 48, 24, 25, 7, 8]
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
def test_a_long_prompt_over_many_chunks(runners, plain, dtype):
    """400 tokens through chunks of 7 to 50 positions (whose pages go back to the pool while the request runs) and through
    latent attention that sees all of them: whole, and with the last 60 tokens decoded; afterwards a chunk group holds no
    more pages than its live chunk."""
    from pulse_infer_amd.engine.runner import StepEntry

    name = "mixed"
    ids = plain.ids(name, 400, 21)
    want, calls = plain(name, ids), plain.close_calls(name, ids)
    runner = runners(name, dtype, 16, tokens=512)
    agree(run_alone(runner, ids, [400]), want, dtype, "whole", calls)
    agree(run_alone(runner, ids, [150, 190] + [1] * 60), want, dtype, "decoded tail", calls)
    runner.add_request("r")
    runner.reserve("r", 400)
    runner.step([StepEntry("r", ids, [])])
    seen = set()
    for g in runner.cache.groups:
        live = sum(p >= 0 for p in runner.cache.table(g.index, "r"))
        chunk = getattr(g.spec, "chunk", None)
        seen.add(chunk)
        assert live == 25 if not chunk else live == 25 - 400 // chunk * chunk // 16, (chunk, live)
    assert seen == {None, 7, 24, 50}
    runner.free_request("r")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_portions_beside_single_tokens(runners, plain, dtype):
    """Steps that hold portions of 64 tokens and more (over several chunks; the latent layers expand their rows to every
    head) beside short portions and single tokens of other requests, and a step of two long portions."""
    from pulse_infer_amd.engine.runner import StepEntry

    name = "wide"
    lengths = {"a": 420, "b": 90, "c": 300}
    ids = {k: plain.ids(name, n, 30 + i) for i, (k, n) in enumerate(lengths.items())}
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
        calls = plain.close_calls(name, ids[k])
        agree(torch.cat(got[k]), plain(name, ids[k]), dtype, f"request {k}", calls)
        agree(run_alone(runner, ids[k], [lengths[k]]), plain(name, ids[k]), dtype, f"request {k} whole", calls)


# ------------------------------------------------------------------------------------ seeded random configurations
def random_config(rng):
    """Layers drawn one by one, in any order: head sizes that are no multiples of 16 or of 4, keys wider or narrower than
    values, any grouping of heads, chunks from one token on, latent rows that are no multiples of 8, rotations on a part of a
    head and on all of it, with and without blended frequencies, experts in any number of groups, and any loop or none."""
    width = rng.choice([64, 96, 160, 256])
    layers = []
    n = rng.choice([2, 3, 4])
    for i in range(n):
        if rng.random() < 0.5:
            groups, dim = rng.choice([1, 2, 3]), rng.choice([16, 20, 24, 32, 64, 80, 128])
            dims = rng.choice([x for x in (2, 8, 16, dim) if x <= dim])
            s = rng.choice([None, scaling(rng.choice([1.0, 4.0, 16.0]), rng.choice([32, 256, 4096]), rng.choice([8.0, 32.0]), 1.0)])
            mixer = attention(groups * rng.choice([1, 2, 3, 4, 18]), groups, dim, rng.choice([8, 20, dim, dim, 64]),
                              rng.choice([1, 5, 16, 33, 100, 500]), rot(rng.choice([100.0, 1e4, 5e5]), dims, s),
                              rng.choice([0.1, dim ** -0.5, 0.3]), rng.choice([1.5, 10.0, 50.0]))
        else:
            mixer = latent(rng.choice([1, 2, 4, 20]), rng.choice([8, 16, 24, 40]), rng.choice([2, 8, 16, 32]), rng.choice([8, 20, 48, 64]),
                           rng.choice([12, 24, 32, 64, 100, 192]), rng.choice([100.0, 1e4, 5e5]), rng.choice([0.1, 0.3]))
        mlp = None
        if rng.random() < 0.75:
            count, size = rng.choice([1, 2, 3, 4]), rng.choice([1, 2, 3, 4])
            keep = rng.randint(1, count)
            mlp = moe(count * size, rng.choice([None, (count, keep)]), rng.randint(1, keep * size), rng.choice([32, 50, 96]),
                      rng.choice([0.5, 1.5, 7.0]), rng.choice([1.0, 0.6, 2.5]))
        layers.append(layer(mixer, mlp))
    start = rng.randint(0, n - 1)
    loop = rng.choice([None, (start, rng.randint(start + 1, n), rng.choice([1, 2, 3]))])
    return config(rng.choice([257, 300, 1000]), width, rng.choice([1e-6, 1e-5]), rng.choice([1.0, 0.3, 2.0]), loop, layers)


@pytest.mark.parametrize("seed", range(14))
def test_random_configurations(tmp_path, seed):
    """Whole, with the last 20 tokens one by one, and in portions of 2 to 70 tokens, in 32-bit and in bfloat16."""
    if not torch.cuda.is_available():
        pytest.skip("no GPU visible")
    from pulse_infer_amd.config import SosuvikConfig
    from pulse_infer_amd.weights import write_model_folder

    rng = random.Random(5100 + seed)
    cfg = random_config(rng)
    length = rng.choice([90, 150])
    folder = write_model_folder(SosuvikConfig.from_dict(cfg), str(tmp_path / "m"), seed=seed)
    oracle = P.PlainSosuvik.from_folder(folder)
    ids = clear_ids(oracle, cfg["vocab"], length, seed=seed, rounds=40)
    want, calls = oracle.logits(ids), close_calls(oracle, ids)
    what = f"{cfg} length {length}"
    print(what, flush=True)
    for dtype in ("float32", "bfloat16"):
        runner = new_runner(folder, dtype, 16, 256)
        whole = run_alone(runner, ids, [length])
        agree(whole, want, dtype, f"whole: {what}", calls)
        tail = run_alone(runner, ids, [length - 20] + [1] * 20)
        agree(tail, want, dtype, f"tail: {what}", calls)
        cuts, left_over, sizes = [], length, [40, 2, 17, 3, 70, 5, 19]
        while left_over:
            n = min(sizes[len(cuts) % len(sizes)], left_over)
            cuts.append(n)
            left_over -= n
        portions = run_alone(runner, ids, cuts)
        agree(portions, want, dtype, f"portions {cuts}: {what}", calls)
        del runner
    torch.cuda.empty_cache()


# ------------------------------------------------------------------------------------------------ long decoding
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["mixed", "wide"])
def test_long_decoding_of_three_requests(runners, plain, name, dtype, monkeypatch):
    """Three requests of unequal prompts decode 100 tokens together, over page and chunk borders; in bfloat16 the steps are
    recorded and replayed, and heads whose projection output needs no preparation go through the kernel that starts from it."""
    from pulse_infer_amd.engine.runner import StepEntry
    from pulse_infer_amd.ops import attention_mfma

    from_raw, real = [], attention_mfma.attn_decode

    def counted(*args, **kw):
        from_raw.append(kw.get("chunk"))
        return real(*args, **kw)

    monkeypatch.setattr(attention_mfma, "attn_decode", counted)
    new = 100
    runner = new_runner(plain.folders[name], dtype, 16, 704)
    prompt = {"d0": 1, "d1": 30, "d2": 47}
    ids = {k: plain.ids(name, n + new, 60 + i) for i, (k, n) in enumerate(prompt.items())}
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
            got[k].append(logits[row:row + 1].clone())
    assert (runner.graph_replays > replays) == (dtype == "bfloat16")
    assert bool(from_raw) == (dtype == "bfloat16" and name == "wide")
    for k in ids:
        runner.free_request(k)
        agree(torch.cat(got[k]), plain(name, ids[k])[prompt[k] - 1:], dtype, f"{name} decoding request {k}",
              plain.close_calls(name, ids[k]), first=prompt[k] - 1)


# --------------------------------------------------------------------------- generation through the scheduler
@pytest.mark.parametrize("name", ["mixed", "straight"])
def test_greedy_generation_through_the_engine(folders, plain, name):
    """In 32-bit the greedy choice does not depend on the batch: requests generated together, in small portions and
    with a pool so tight that some are preempted and recomputed, give what each gives alone and what the plain
    implementation chooses."""
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
    """Every token that the bfloat16 engine chooses is, for the plain implementation, within rounding of the best one
    (up to the first position at which a router's choice is a close call)."""
    from pulse_infer_amd import LLM

    name, new = "wide", 10
    prompts = [plain.ids(name, n, 90 + i) for i, n in enumerate((3, 21))]
    llm = LLM.from_pretrained(folders[name], dtype="bfloat16", max_batch_size=2, chunk_size=8, page_size=16, num_pages=32)
    judged = 0
    for prompt, out in zip(prompts, llm.generate(prompts, max_new_tokens=new, ignore_eos=True)):
        assert len(out) == new
        for t, token in enumerate(out):
            ids = prompt + out[:t]
            if plain.close_calls(name, ids):
                break
            row = plain(name, ids)[-1]
            assert float(row[token]) >= float(row.max()) - TOL["bfloat16"] * float(row.abs().max())
            judged += 1
    assert judged >= 2


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
    a, b = plain.ids(name, 70, 1), plain.ids(name, 21, 2)
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
    calls = {id(la): plain.close_calls(name, a), id(lb): plain.close_calls(name, b)}
    read = lambda i: torch.from_numpy(np.fromfile(out / f"{i}.f32", dtype="<f4").reshape(-1, vocab).copy())
    judged = 0
    for step, rows in ((0, [(la, 0), (la, 49)]), (1, [(lb, 19)]), (2, [(lb, 20), (la, 69)])):
        got = read(step)
        assert got.shape[0] == len(rows) and torch.isfinite(got).all()
        for i, (want, at) in enumerate(rows):
            if dtype == "bfloat16" and any(c <= at for c in calls[id(want)]):
                continue
            close(got[i:i + 1], want[at:at + 1], dtype, f"step {step} row {i}", TOL)
            judged += 1
    assert judged >= 3
