"""A plain, slow Makezen decoder: whole sequences, no cache, one function per mechanism, float64 on the CPU.
It shares no code with ``pulse_infer_amd``: it reads a model folder with ``json`` and the ``safetensors`` package
(or takes a dictionary of tensors) and is written from the design's equations.  Tests compare the engine with it.

Notation: x [T, W] the stream, p the position of a token (from 0 in each sequence), W_foo a weight stored [out, in].
"""
from __future__ import annotations

import json
import math
import os
from typing import Any, Dict, List, Optional

import torch

DT = torch.float64


def unit_rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    """x / sqrt(mean(x^2) + eps) over the last axis, eps inside the root."""
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def layer_norm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    """(x - mean) / sqrt(mean((x - mean)^2) + eps) * w."""
    c = x - x.mean(dim=-1, keepdim=True)
    return c / torch.sqrt((c * c).mean(dim=-1, keepdim=True) + eps) * w


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def softplus(z: torch.Tensor) -> torch.Tensor:
    return torch.log1p(torch.exp(-z.abs())) + torch.clamp(z, min=0.0)


def gelu_tanh(z: torch.Tensor) -> torch.Tensor:
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


# ------------------------------------------------------------------ rotation
def frequencies(rot: Dict[str, Any]) -> List[float]:
    """base^(-2i/dims), blended with its 1/factor by a ramp over i where ``scaling`` is given."""
    dims, base = rot["dims"], rot["base"]
    plain = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    s = rot.get("scaling")
    if not s:
        return plain

    def index_of(turns: float) -> float:      # the (real) index whose wavelength fits ``turns`` times into the original length
        return dims * math.log(s["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

    lo = max(math.floor(index_of(s["fast"])), 0)
    hi = min(math.ceil(index_of(s["slow"])), dims - 1)
    out = []
    for i, f in enumerate(plain):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(f / s["factor"] * ramp + f * (1.0 - ramp))
    return out


def magnitude(rot: Dict[str, Any]) -> float:
    s = rot.get("scaling")
    return 0.1 * math.log(s["factor"]) + 1.0 if s else 1.0


def turn(x: torch.Tensor, positions: List[int], rot: Dict[str, Any]) -> torch.Tensor:
    """The first ``dims`` channels of every head turned, channel i with i + dims / 2; x [T, heads, d]."""
    half = rot["dims"] // 2
    out = x.clone()
    angle = torch.tensor(positions, dtype=torch.float64).view(-1, 1, 1) * torch.tensor(frequencies(rot), dtype=torch.float64)
    c, s = (torch.cos(angle) * magnitude(rot)).to(x.dtype), (torch.sin(angle) * magnitude(rot)).to(x.dtype)
    u, v = x[..., :half], x[..., half:2 * half]
    out[..., :half] = u * c - v * s
    out[..., half:2 * half] = v * c + u * s
    return out


# ------------------------------------------------------------------ softmax attention
def visible(t: int, size: Optional[int]) -> torch.Tensor:
    """[T, T] bool: i sees j if 0 <= i - j < size (no size: every j <= i)."""
    i = torch.arange(t).view(-1, 1)
    j = torch.arange(t).view(1, -1)
    return (j <= i) & ((i - j < size) if size is not None else True)


def softmax_weights(scores: torch.Tensor, mask: torch.Tensor, sink: Optional[torch.Tensor] = None) -> torch.Tensor:
    """Softmax over the visible keys of scores [H, T, T]; with a sink the denominator holds exp(sink_h) once more."""
    s = scores.masked_fill(~mask.unsqueeze(0), float("-inf"))
    top = s.max(dim=-1, keepdim=True).values
    if sink is not None:
        top = torch.maximum(top, sink.view(-1, 1, 1))
    e = torch.exp(s - top)
    den = e.sum(dim=-1, keepdim=True)
    if sink is not None:
        den = den + torch.exp(sink.view(-1, 1, 1) - top)
    return e / den


def capped_attention(x, w, p: str, m: Dict[str, Any], positions: List[int], eps: float) -> torch.Tensor:
    """Grouped attention with biases, a weighted norm of every q and k head, a rotation and capped scores."""
    t, heads, groups, d, dv = x.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = (x @ w[p + ".q"].T + w[p + ".q.b"]).view(t, heads, d)
    k = (x @ w[p + ".k"].T + w[p + ".k.b"]).view(t, groups, d)
    v = (x @ w[p + ".v"].T + w[p + ".v.b"]).view(t, groups, dv)
    q = turn(unit_rms(q, eps) * w[p + ".q.norm"], positions, m["rot"])
    k = turn(unit_rms(k, eps) * w[p + ".k.norm"], positions, m["rot"])
    per = heads // groups
    scores = torch.stack([q[:, h] @ k[:, h // per].T for h in range(heads)]) * m["scale"]
    scores = m["softcap"] * torch.tanh(scores / m["softcap"])
    a = softmax_weights(scores, visible(t, None))
    o = torch.stack([a[h] @ v[:, h // per] for h in range(heads)], dim=1)
    return o.reshape(t, heads * dv) @ w[p + ".o"].T


def latent_row(x, w, p: str, m: Dict[str, Any], positions: List[int], eps: float):
    """What a token keeps: the normed latent row and the turned key part shared by all heads."""
    down, rank = x @ w[p + ".dkv"].T, m["kv_rank"]
    c = unit_rms(down[:, :rank], eps) * w[p + ".dkv.norm"]
    return c, turn(down[:, rank:].unsqueeze(1), positions, m["rot"])[:, 0]


def latent_attention(x, w, p: str, m: Dict[str, Any], positions: List[int], eps: float, kept) -> torch.Tensor:
    """Attention over the latent rows ``kept`` = (c, turned part) with this layer's own up projections and queries."""
    t, heads, d, dv = x.shape[0], m["heads"], m["dim"], m["vdim"]
    c, k_turned = kept
    q = ((unit_rms(x @ w[p + ".dq"].T, eps) * w[p + ".dq.norm"]) @ w[p + ".uq"].T).view(t, heads, d + m["rot_dim"])
    q_turned = turn(q[:, :, d:], positions, m["rot"])
    k_plain = (c @ w[p + ".uk"].T).view(t, heads, d)
    v = (c @ w[p + ".uv"].T).view(t, heads, dv)
    scores = torch.stack([q[:, h, :d] @ k_plain[:, h].T + q_turned[:, h] @ k_turned.T for h in range(heads)]) * m["scale"]
    a = softmax_weights(scores, visible(t, (m.get("mask") or {}).get("size")), w[p + ".sink"])
    o = torch.stack([a[h] @ v[:, h] for h in range(heads)], dim=1)
    o = o * torch.sigmoid(x @ w[p + ".g"].T).unsqueeze(-1)
    return o.reshape(t, heads * dv) @ w[p + ".o"].T


# ------------------------------------------------------------------ gated delta rule
def short_conv(x: torch.Tensor, taps: torch.Tensor) -> torch.Tensor:
    """y[t, c] = sum_j taps[c, j] x[t - (n - 1) + j, c], zeros before the start."""
    n = taps.shape[1]
    padded = torch.cat([x.new_zeros(n - 1, x.shape[1]), x])
    return sum(padded[j:j + x.shape[0]] * taps[:, j] for j in range(n))


def unit_vector(x: torch.Tensor) -> torch.Tensor:
    return x / torch.sqrt((x * x).sum(dim=-1, keepdim=True) + 1e-6)


def delta_walk(q, k, v, beta, log_decay) -> torch.Tensor:
    """Per head, token by token: D = e^a S; r = v - D^T k; S = D + beta k r^T; o = S^T q.  q, k [T, H, d],
    v [T, H, dv], beta and log_decay [T, H]."""
    t, heads, d = q.shape
    out = torch.zeros(t, heads, v.shape[2], dtype=q.dtype)
    for h in range(heads):
        s = torch.zeros(d, v.shape[2], dtype=q.dtype)
        for i in range(t):
            s = torch.exp(log_decay[i, h]) * s
            u = beta[i, h] * (v[i, h] - s.T @ k[i, h])
            s = s + torch.outer(k[i, h], u)
            out[i, h] = s.T @ q[i, h]
    return out


def delta_mixer(x, w, p: str, m: Dict[str, Any], eps: float) -> torch.Tensor:
    t, heads, groups, d, dv = x.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (silu(short_conv(x @ w[f"{p}.{n}"].T, w[f"{p}.{n}.conv"])) for n in "qkv")
    q = unit_vector(q.view(t, groups, d)) * d ** -0.5
    k = unit_vector(k.view(t, groups, d))
    q, k = (z.repeat_interleave(heads // groups, dim=1) for z in (q, k))
    beta = torch.sigmoid(x @ w[p + ".b"].T)
    log_decay = -torch.exp(w[p + ".A_log"]) * softplus(x @ w[p + ".a"].T + w[p + ".dt_bias"])
    o = delta_walk(q, k, v.view(t, heads, dv), beta, log_decay)
    o = unit_rms(o, eps) * w[p + ".norm"] * silu(x @ w[p + ".g"].T).view(t, heads, dv)
    return o.reshape(t, heads * dv) @ w[p + ".o"].T


def parallel_mixer(x, w, p: str, m: Dict[str, Any], positions: List[int], eps: float) -> torch.Tensor:
    left = capped_attention(x, w, p + ".left", m["left"], positions, eps)
    right = delta_mixer(x, w, p + ".right", m["right"], eps)
    return 0.5 * (unit_rms(left, eps) * w[p + ".left.out"] + unit_rms(right, eps) * w[p + ".right.out"])


def feed_forward(x, w, p: str) -> torch.Tensor:
    return gelu_tanh(x @ w[p + ".up"].T) @ w[p + ".down"].T


# ------------------------------------------------------------------ the model
def forward(cfg: Dict[str, Any], w: Dict[str, torch.Tensor], tokens: List[int],
            residuals: Optional[list] = None) -> torch.Tensor:
    """Logits [T, vocab] of one sequence; ``residuals`` collects the stream after every layer."""
    w = {k: v.to(DT) for k, v in w.items()}
    eps = cfg["norm"]["eps"]
    positions = list(range(len(tokens)))
    x = layer_norm(w["embed"][torch.tensor(tokens)], w["embed.norm"], eps)
    rows: Dict[int, Any] = {}
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}", layer["mixer"]
        n = layer_norm(x, w[p + ".norm1"], eps)
        if layer["type"] == "delta":
            y = delta_mixer(n, w, p + ".mix", m, eps)
        elif layer["type"] == "parallel":
            y = parallel_mixer(n, w, p + ".mix", m, positions, eps)
        elif layer["type"] == "latent_attention":
            source = m.get("kv_from")
            if source is None:
                rows[i] = latent_row(n, w, p + ".mix", m, positions, eps)
            y = latent_attention(n, w, p + ".mix", m, positions, eps, rows[i if source is None else source])
        else:
            raise ValueError(layer["type"])
        x = x + layer_norm(y, w[p + ".norm1b"], eps)
        if layer.get("mlp"):
            y = feed_forward(layer_norm(x, w[p + ".norm2"], eps), w, p + ".mlp")
            x = x + layer_norm(y, w[p + ".norm2b"], eps)
        if residuals is not None:
            residuals.append(x.clone())
    return layer_norm(x, w["final.norm"], eps) @ w["embed"].T


def fragile_positions(cfg: Dict[str, Any], w: Dict[str, torch.Tensor], tokens: List[int], above: float = 4.0) -> set:
    """Positions whose logits hang on cancellations: where these same equations evaluated in float32 stray from their
    float64 values ``above`` times further than at the median position.  (A delta head's output is divided by its own
    root mean square; where that output is small by chance, the division multiplies whatever rounding left in it,
    in any arithmetic, and no bound that holds elsewhere says anything there.)"""
    global DT
    exact = forward(cfg, w, tokens)
    DT = torch.float32
    try:
        rough = forward(cfg, w, tokens).to(torch.float64)
    finally:
        DT = torch.float64
    err = (rough - exact).abs().max(dim=1).values
    return set((err > above * err.median()).nonzero().flatten().tolist())


def load_folder(path: str):
    from safetensors.torch import load_file

    with open(os.path.join(path, "config.json")) as f:
        cfg = json.load(f)
    w: Dict[str, torch.Tensor] = {}
    for name in sorted(os.listdir(path)):
        if name.endswith(".safetensors"):
            w.update(load_file(os.path.join(path, name)))
    return cfg, w


class PlainMakezen:
    """The functions above behind the few calls the tests make."""

    def __init__(self, cfg: Dict[str, Any], weights: Dict[str, torch.Tensor]):
        self.cfg = cfg
        self.w = {k: v.to(DT) for k, v in weights.items()}

    @classmethod
    def from_folder(cls, path: str) -> "PlainMakezen":
        return cls(*load_folder(path))

    def logits(self, ids: List[int]) -> torch.Tensor:
        return forward(self.cfg, self.w, list(ids))

    def residuals(self, ids: List[int]) -> List[torch.Tensor]:
        out: List[torch.Tensor] = []
        forward(self.cfg, self.w, list(ids), residuals=out)
        return out

    def fragile_positions(self, ids: List[int]) -> set:
        return fragile_positions(self.cfg, self.w, list(ids))

    def greedy(self, prompt: List[int], new: int) -> List[int]:
        ids, out = list(prompt), []
        for _ in range(new):
            token = int(self.logits(ids)[-1].argmax())
            out.append(token)
            ids.append(token)
        return out
