"""A plain, slow Sosuvik decoder: whole sequences, no cache, one function per mechanism, float64 on the CPU.
It shares no code with ``pulse_infer_amd``: it reads a model folder with ``json`` and the ``safetensors`` package
(or takes a dictionary of tensors) and is written from the design's equations.  Tests compare the engine with it.

Notation: x [T, W] the stream, p the position of a token (from 0 in each sequence), W_foo a weight stored [out, in].
"""
from __future__ import annotations

import json
import math
import os
from typing import Any, Dict, List, Optional, Tuple

import torch

DT = torch.float64


def rms_norm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    """x / sqrt(mean(x^2) + eps) * w over the last axis."""
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps) * w


# ------------------------------------------------------------------ rotation
def frequencies(rot: Dict[str, Any]) -> List[float]:
    """base^(-2i/dims), blended with its 1/factor by a ramp over i where ``scaling`` is given."""
    dims, base = rot["dims"], rot["base"]
    plain = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    s = rot.get("scaling")
    if not s:
        return plain

    def place(turns: float) -> float:      # the (real) index whose wavelength fits ``turns`` times into the original length
        return dims * math.log(s["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

    low = max(math.floor(place(s["fast"])), 0)
    high = min(math.ceil(place(s["slow"])), dims - 1)
    ramp = [min(max((i - low) / max(high - low, 0.001), 0.0), 1.0) for i in range(dims // 2)]
    return [f / s["factor"] * r + f * (1.0 - r) for f, r in zip(plain, ramp)]


def magnitude(rot: Dict[str, Any]) -> float:
    s = rot.get("scaling")
    return 0.1 * math.log(s["factor"]) + 1.0 if s else 1.0


def turn(x: torch.Tensor, positions: List[int], rot: Optional[Dict[str, Any]], adjacent: bool) -> torch.Tensor:
    """The first ``dims`` channels of every head turned by position * frequency: channel i with i + dims / 2, or
    (``adjacent``) 2i with 2i + 1; x [T, heads, d]."""
    if not rot or not rot["dims"]:
        return x
    n = rot["dims"]
    first, second = (slice(0, n, 2), slice(1, n, 2)) if adjacent else (slice(0, n // 2), slice(n // 2, n))
    angle = torch.tensor(positions, dtype=torch.float64).view(-1, 1, 1) * torch.tensor(frequencies(rot), dtype=torch.float64)
    c, s = (torch.cos(angle) * magnitude(rot)).to(x.dtype), (torch.sin(angle) * magnitude(rot)).to(x.dtype)
    out = x.clone()
    u, v = x[..., first], x[..., second]
    out[..., first] = u * c - v * s
    out[..., second] = v * c + u * s
    return out


# ------------------------------------------------------------------ softmax attention
def same_chunk(t: int, size: Optional[int]) -> torch.Tensor:
    """[T, T] bool: i sees j <= i of its own chunk of ``size`` positions counted from 0 (no size: every j <= i)."""
    i = torch.arange(t).view(-1, 1)
    j = torch.arange(t).view(1, -1)
    return (j <= i) & ((i // size == j // size) if size else True)


def softmax_weights(scores: torch.Tensor, mask: torch.Tensor, extra: bool = False) -> torch.Tensor:
    """Softmax over the visible keys of scores [H, T, T]; ``extra``: the denominator holds exp(0) once more."""
    s = scores.masked_fill(~mask.unsqueeze(0), float("-inf"))
    top = s.max(dim=-1, keepdim=True).values
    if extra:
        top = top.clamp(min=0.0)
    e = torch.exp(s - top)
    den = e.sum(dim=-1, keepdim=True) + (torch.exp(-top) if extra else 0.0)
    return e / den


def chunked_attention(x, w, p: str, m: Dict[str, Any], positions: List[int]) -> torch.Tensor:
    """Grouped attention inside chunks, capped scores, one more term of 1 in the softmax's denominator."""
    t, heads, groups, d, dv = x.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = turn((x @ w[p + ".q"].T).view(t, heads, d), positions, m.get("rot"), adjacent=False)
    k = turn((x @ w[p + ".k"].T).view(t, groups, d), positions, m.get("rot"), adjacent=False)
    v = (x @ w[p + ".v"].T).view(t, groups, dv)
    per = heads // groups
    scores = torch.stack([q[:, h] @ k[:, h // per].T for h in range(heads)]) * m["scale"]
    if m.get("softcap"):
        scores = m["softcap"] * torch.tanh(scores / m["softcap"])
    a = softmax_weights(scores, same_chunk(t, (m.get("mask") or {}).get("size")), extra=True)
    o = torch.stack([a[h] @ v[:, h // per] for h in range(heads)], dim=1)
    return o.reshape(t, heads * dv) @ w[p + ".o"].T


def latent_attention(x, w, p: str, m: Dict[str, Any], positions: List[int], eps: float) -> torch.Tensor:
    """Keys and values from one normed latent row a token and one turned key part for all heads; every j <= i seen."""
    t, heads, d, dv, rank = x.shape[0], m["heads"], m["dim"], m["vdim"], m["kv_rank"]
    q = (x @ w[p + ".q"].T).view(t, heads, d + m["rot_dim"])
    down = x @ w[p + ".dkv"].T
    c = rms_norm(down[:, :rank], w[p + ".dkv.norm"], eps)
    k_turned = turn(down[:, rank:].unsqueeze(1), positions, m["rot"], adjacent=True)[:, 0]
    q_turned = turn(q[:, :, d:], positions, m["rot"], adjacent=True)
    k_plain = (c @ w[p + ".uk"].T).view(t, heads, d)
    v = (c @ w[p + ".uv"].T).view(t, heads, dv)
    scores = torch.stack([q[:, h, :d] @ k_plain[:, h].T + q_turned[:, h] @ k_turned.T for h in range(heads)]) * m["scale"]
    a = softmax_weights(scores, same_chunk(t, None))
    o = torch.stack([a[h] @ v[:, h] for h in range(heads)], dim=1)
    return o.reshape(t, heads * dv) @ w[p + ".o"].T


# ------------------------------------------------------------------ routed experts
def choice_scores(x, w, p: str, router: Dict[str, Any]) -> Tuple[torch.Tensor, torch.Tensor, torch.Tensor]:
    """(scores, choice scores, choice scores with the outputs of the groups that are left out at -inf)."""
    s = torch.sigmoid(x @ w[p + ".router"].T)
    c = s + w[p + ".correction"]
    groups = router.get("groups")
    if not groups:
        return s, c, c
    t, n = c.shape
    count, keep, size = groups["count"], groups["keep"], n // groups["count"]
    marks = c.view(t, count, size).sort(dim=-1, descending=True).values[..., :2].sum(-1)
    order = marks.sort(dim=-1, descending=True, stable=True).indices
    allowed = torch.zeros(t, count, dtype=torch.bool).scatter(1, order[:, :keep], True)
    return s, c, c.masked_fill(~allowed.repeat_interleave(size, dim=1), float("-inf"))


def expert(h, w, p: str, limit: float) -> torch.Tensor:
    g = torch.clamp(h @ w[p + ".gate"].T, max=limit)
    u = torch.clamp(h @ w[p + ".up"].T, min=-limit, max=limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1.0)) @ w[p + ".down"].T


def routed_experts(x, w, p: str, m: Dict[str, Any]) -> torch.Tensor:
    router = m["router"]
    s, _, c = choice_scores(x, w, p, router)
    chosen = c.sort(dim=-1, descending=True, stable=True).indices[:, :router["top"]]
    weights = torch.gather(s, 1, chosen)
    weights = weights / (weights.sum(dim=-1, keepdim=True) + 1e-20) * router.get("scale", 1.0)
    out = torch.zeros_like(x)
    for e in range(c.shape[1]):
        token, place = (chosen == e).nonzero(as_tuple=True)
        if token.numel():
            out[token] += weights[token, place].view(-1, 1) * expert(x[token], w, f"{p}.e{e}", m["expert"]["limit"])
    return out


def router_margin(x, w, p: str, m: Dict[str, Any]) -> torch.Tensor:
    """Per token, how far the closest call of the router is from going the other way: between the last choice and the
    first one left out, and between the last group kept and the first one dropped."""
    router = m["router"]
    _, c, left = choice_scores(x, w, p, router)
    ranked = left.sort(dim=-1, descending=True).values
    top = router["top"]
    margin = torch.full((x.shape[0],), float("inf"), dtype=torch.float64)
    if top < ranked.shape[1]:
        margin = torch.minimum(margin, (ranked[:, top - 1] - ranked[:, top]).to(torch.float64))
    groups = router.get("groups")
    if groups and groups["keep"] < groups["count"]:
        size = c.shape[1] // groups["count"]
        marks = c.view(-1, groups["count"], size).topk(min(2, size), dim=-1).values.sum(-1).sort(dim=-1, descending=True).values
        margin = torch.minimum(margin, (marks[:, groups["keep"] - 1] - marks[:, groups["keep"]]).to(torch.float64))
    return margin


# ------------------------------------------------------------------ the model
def run_order(cfg: Dict[str, Any]) -> List[Tuple[int, Optional[int]]]:
    """(layer, the pass that starts with it or None) in the order of running."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    order: List[Tuple[int, Optional[int]]] = [(i, None) for i in range(loop["start"])]
    for t in range(loop["times"]):
        order += [(i, t if i == loop["start"] else None) for i in range(loop["start"], loop["stop"])]
    return order + [(i, None) for i in range(loop["stop"], n)]


def forward(cfg: Dict[str, Any], w: Dict[str, torch.Tensor], tokens: List[int], residuals: Optional[list] = None,
            margins: Optional[list] = None) -> torch.Tensor:
    """Logits [T, vocab] of one sequence; ``residuals`` collects the stream after every layer run, ``margins`` the
    routers' margins."""
    w = {k: v.to(DT) for k, v in w.items()}
    eps = cfg["norm"]["eps"]
    positions = list(range(len(tokens)))
    x0 = w["embed"][torch.tensor(tokens)]
    x = x0
    for layer, start_of in run_order(cfg):
        if start_of is not None:
            x = torch.cat([x, x0], dim=-1) @ w["loop.in"].T + w["loop.step"][start_of]
        spec, p = cfg["layers"][layer], f"l{layer}"
        m = spec["mixer"]
        n = rms_norm(x, w[p + ".norm1"], eps)
        if spec["type"] == "attention":
            y = chunked_attention(n, w, p + ".mix", m, positions)
        elif spec["type"] == "latent_attention":
            y = latent_attention(n, w, p + ".mix", m, positions, eps)
        else:
            raise ValueError(spec["type"])
        if spec.get("mlp"):
            n = rms_norm(x, w[p + ".norm2"], eps)
            if margins is not None:
                margins.append(router_margin(n, w, p + ".mlp", spec["mlp"]))
            y = y + routed_experts(n, w, p + ".mlp", spec["mlp"])
        x = x + y
        if residuals is not None:
            residuals.append(x.clone())
    return rms_norm(x, w["final.norm"], eps) @ w["head"].T * cfg.get("logit_scale", 1.0)


def load_folder(path: str):
    from safetensors.torch import load_file

    with open(os.path.join(path, "config.json")) as f:
        cfg = json.load(f)
    w: Dict[str, torch.Tensor] = {}
    for name in sorted(os.listdir(path)):
        if name.endswith(".safetensors"):
            w.update(load_file(os.path.join(path, name)))
    return cfg, w


class PlainSosuvik:
    """The functions above behind the few calls the tests make."""

    def __init__(self, cfg: Dict[str, Any], weights: Dict[str, torch.Tensor]):
        self.cfg = cfg
        self.w = {k: v.to(DT) for k, v in weights.items()}

    @classmethod
    def from_folder(cls, path: str) -> "PlainSosuvik":
        return cls(*load_folder(path))

    def logits(self, ids: List[int]) -> torch.Tensor:
        return forward(self.cfg, self.w, list(ids))

    def residuals(self, ids: List[int]) -> List[torch.Tensor]:
        out: List[torch.Tensor] = []
        forward(self.cfg, self.w, list(ids), residuals=out)
        return out

    def router_margins(self, ids: List[int]) -> torch.Tensor:
        """Per position the smallest margin of a router's choice over all layer runs."""
        out: List[torch.Tensor] = []
        forward(self.cfg, self.w, list(ids), margins=out)
        return torch.stack(out).min(dim=0).values if out else torch.full((len(ids),), float("inf"), dtype=torch.float64)

    def greedy(self, prompt: List[int], new: int) -> List[int]:
        ids, out = list(prompt), []
        for _ in range(new):
            token = int(self.logits(ids)[-1].argmax())
            out.append(token)
            ids.append(token)
        return out
