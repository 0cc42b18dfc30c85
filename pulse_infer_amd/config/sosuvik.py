"""Sosuvik: a decoder whose layers run mixer and feed-forward side by side and some of whose layers run several times.

config.json holds ``architecture``, ``vocab``, ``width``, ``norm.eps``, ``logit_scale``, ``loop`` (``start``, ``stop``,
``times``) and ``layers``: for each layer its ``type`` (the mixer), the mixer's sizes and constants (``mixer``) and its
feed-forward (``mlp``, or null for none).  Every size and constant is taken from there.  Tensors: ``embed``, ``loop.in``
[width, 2 width], ``loop.step`` [times, width], ``l<i>.norm1`` / ``norm2``, ``l<i>.mix.*``, ``l<i>.mlp.*``, ``final.norm``,
``head``.

The model: x = x0 = embed[token]; per layer x <- x + (mixer(norm1(x)) + ff(norm2(x))), both of the same x, with RMSNorms
with plain weights.  The stretch of layers from ``start`` up to ``stop`` is gone through ``times`` times over (weights
shared, caches not); pass t begins with x <- loop.in [x; x0] + loop.step[t].  logits = logit_scale * head final.norm(x).

Mixers.  ``attention``: softmax attention with grouped key/value heads (``heads``, ``kv_heads``, ``dim``, ``vdim``), a
rotation of the first ``rot.dims`` channels of every head in pairs (i, i + dims / 2), its frequencies blended by
``rot.scaling`` (``factor``, ``original``, ``fast``, ``slow``), ``scale`` and ``softcap`` on the scores, one added to the
softmax's sum, and chunks: a token sees the earlier tokens of its own chunk of ``mask.size`` positions only.
``latent_attention``: keys and values from one normed latent row a token (``kv_rank``) and one turned key part (``rot_dim``
channels, adjacent pairs) shared by all heads; every earlier token is visible.

Feed-forward.  ``moe``: ``router.experts`` gated experts of width ``expert.ff`` with an activation clamped at
``expert.limit``; scores are sigmoids, choices go by score + correction inside the best ``router.groups.keep`` of
``router.groups.count`` groups, weights are the chosen scores divided by their sum, times ``router.scale``.

All of that is said to the engine as parameters of registered parts (``model_spec``); there is no model class.
"""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Any, Dict, List, Optional

from .base import ConfigError, JsonReader, ModelConfig, require_positive
from .makezen import Rotation
from ..models.spec import LayerSpec, ModelSpec, PartSpec, RunSpec

ARCHITECTURE = "Sosuvik"
MIXER_TYPES = ("attention", "latent_attention")
MLP_KINDS = ("moe",)
MAX_ROUTER_OUTPUTS = 1024
MAX_CHOICES = 64
MAX_GROUPS = 64


def _object(value: Any, where: str, what: str) -> Dict[str, Any]:
    if not isinstance(value, dict):
        raise ConfigError(f"'{where}': key '{what}' must be an object")
    return value


@dataclass
class AttentionSizes:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    softcap: float              # 0: none
    chunk: Optional[int]        # None: config.json names no mask, every earlier token is visible
    rot: Rotation

    @classmethod
    def read(cls, data: Dict[str, Any], where: str) -> "AttentionSizes":
        r = JsonReader(data, where)
        heads, dim = r.integer("heads"), r.integer("dim")
        chunk = None
        if r.raw("mask") is not None:
            chunk = JsonReader(_object(r.raw("mask"), where, "mask"), f"{where}.mask").integer("size")
        return cls(heads=heads, kv_heads=r.integer("kv_heads", heads), dim=dim, vdim=r.integer("vdim", dim),
                   scale=r.number("scale"), softcap=r.number("softcap", 0.0), chunk=chunk, rot=Rotation.read(r.raw("rot"), where))

    def check(self, where: str) -> None:
        require_positive(where, heads=self.heads, kv_heads=self.kv_heads, dim=self.dim, vdim=self.vdim)
        if self.chunk is not None:
            require_positive(where, size=self.chunk)
        if self.softcap < 0.0:
            raise ConfigError(f"'{where}': softcap ({self.softcap}) must not be negative")
        if self.softcap > 0.0 and not self.scale > 0.0:
            raise ConfigError(f"'{where}': a softcap needs a positive scale, got {self.scale}")
        if self.heads % self.kv_heads:
            raise ConfigError(f"'{where}': {self.heads} query heads cannot be shared out evenly over {self.kv_heads} "
                              "key/value heads")
        self.rot.check(where, self.dim)

    def to_dict(self) -> Dict[str, Any]:
        out: Dict[str, Any] = {"dim": self.dim, "heads": self.heads, "kv_heads": self.kv_heads, "scale": self.scale,
                               "softcap": self.softcap, "vdim": self.vdim}
        if self.chunk is not None:
            out["mask"] = {"size": self.chunk}
        if self.rot.dims:
            out["rot"] = self.rot.to_dict()
        return out


@dataclass
class LatentSizes:
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    kv_rank: int
    scale: float
    rot: Rotation

    @classmethod
    def read(cls, data: Dict[str, Any], where: str) -> "LatentSizes":
        r = JsonReader(data, where)
        return cls(heads=r.integer("heads"), dim=r.integer("dim"), rot_dim=r.integer("rot_dim"), vdim=r.integer("vdim"),
                   kv_rank=r.integer("kv_rank"), scale=r.number("scale"), rot=Rotation.read(r.raw("rot"), where))

    def check(self, where: str) -> None:
        require_positive(where, heads=self.heads, dim=self.dim, rot_dim=self.rot_dim, vdim=self.vdim, kv_rank=self.kv_rank)
        self.rot.check(where, self.rot_dim)
        if self.rot.dims != self.rot_dim:
            raise ConfigError(f"'{where}': rot.dims ({self.rot.dims}) must be rot_dim ({self.rot_dim}): the turned part "
                              "is turned as a whole")

    def to_dict(self) -> Dict[str, Any]:
        return {"dim": self.dim, "heads": self.heads, "kv_rank": self.kv_rank, "rot": self.rot.to_dict(),
                "rot_dim": self.rot_dim, "scale": self.scale, "vdim": self.vdim}


@dataclass
class SosuvikMLP:
    kind: str
    ff: int                     # an expert's inner width
    limit: float
    experts: int
    top: int
    scale: float = 1.0
    groups: int = 1             # 1: config.json names no groups (one group of all experts is the same)
    keep: int = 1

    @classmethod
    def read(cls, data: Dict[str, Any], where: str) -> "SosuvikMLP":
        r = JsonReader(data, where)
        kind = r.string("kind")
        if kind not in MLP_KINDS:
            raise ConfigError(f"'{where}': there is no feed-forward '{kind}' (known: {', '.join(MLP_KINDS)})")
        router = JsonReader(_object(r.raw("router"), where, "router"), f"{where}.router")
        expert = JsonReader(_object(r.raw("expert"), where, "expert"), f"{where}.expert")
        groups = keep = 1
        if router.raw("groups") is not None:
            g = JsonReader(_object(router.raw("groups"), f"{where}.router", "groups"), f"{where}.router.groups")
            groups, keep = g.integer("count"), g.integer("keep")
        return cls(kind=kind, ff=expert.integer("ff"), limit=expert.number("limit"), experts=router.integer("experts"),
                   top=router.integer("top"), scale=router.number("scale", 1.0), groups=groups, keep=keep)

    def check(self, where: str) -> None:
        require_positive(where, ff=self.ff, limit=self.limit, experts=self.experts, top=self.top, count=self.groups,
                         keep=self.keep)
        if self.experts > MAX_ROUTER_OUTPUTS or self.top > MAX_CHOICES or self.groups > MAX_GROUPS:
            raise ConfigError(f"'{where}': the router's kernel takes at most {MAX_ROUTER_OUTPUTS} experts in {MAX_GROUPS} "
                              f"groups and {MAX_CHOICES} choices a token")
        if self.experts % self.groups:
            raise ConfigError(f"'{where}': {self.experts} experts do not form {self.groups} equal groups")
        if self.keep > self.groups:
            raise ConfigError(f"'{where}': {self.keep} of {self.groups} groups cannot be kept")
        if self.top > self.keep * (self.experts // self.groups):
            raise ConfigError(f"'{where}': {self.top} experts cannot be chosen from {self.keep} groups of "
                              f"{self.experts // self.groups}")

    def to_dict(self) -> Dict[str, Any]:
        return {"expert": {"ff": self.ff, "limit": self.limit}, "kind": self.kind,
                "router": {"experts": self.experts, "groups": {"count": self.groups, "keep": self.keep},
                           "scale": self.scale, "top": self.top}}


@dataclass
class SosuvikLayer:
    type: str
    attention: Optional[AttentionSizes] = None
    latent: Optional[LatentSizes] = None
    mlp: Optional[SosuvikMLP] = None

    @property
    def sizes(self) -> Any:
        return self.attention if self.attention is not None else self.latent

    def to_dict(self) -> Dict[str, Any]:
        return {"mixer": self.sizes.to_dict(), "mlp": None if self.mlp is None else self.mlp.to_dict(), "type": self.type}


@dataclass
class SosuvikConfig(ModelConfig):
    vocab_size: int
    width: int
    norm_eps: float
    logit_scale: float = 1.0
    loop_start: int = 0
    loop_stop: int = 0
    loop_times: int = 1             # 1 with start == stop: config.json names no loop
    has_loop: bool = False
    layers: List[SosuvikLayer] = field(default_factory=list)
    eos_token_ids: List[int] = field(default_factory=list)
    temperature: float = 0.0
    top_k: int = 0
    top_p: float = 0.0
    # An option of the engine, not a key of config.json: the most positions a request may reach.
    max_positions: int = 1 << 20
    architecture: str = ARCHITECTURE

    engine_options = {
        "max_positions": {"type": int, "help": "the most positions a request may reach (the design sets no limit)"}}

    # ------------------------------------------------------------------ reading
    @classmethod
    def from_dict(cls, data: Dict[str, Any], origin: str = "<dict>", generation: Optional[Dict[str, Any]] = None,
                  generation_origin: str = "<dict>") -> "SosuvikConfig":
        r = JsonReader(data, origin)
        norm = JsonReader(_object(r.raw("norm"), origin, "norm"), f"{origin}: norm")
        listed = r.raw("layers")
        if not isinstance(listed, list) or not listed:
            raise ConfigError(f"'{origin}': key 'layers' must be a list with at least one layer")
        start = stop = 0
        times, has_loop = 1, False
        if r.raw("loop") is not None:
            loop = JsonReader(_object(r.raw("loop"), origin, "loop"), f"{origin}: loop")
            start, stop, times, has_loop = loop.integer("start"), loop.integer("stop"), loop.integer("times"), True
        cfg = cls(vocab_size=r.integer("vocab"), width=r.integer("width"), norm_eps=norm.number("eps"),
                  logit_scale=r.number("logit_scale", 1.0), loop_start=start, loop_stop=stop, loop_times=times,
                  has_loop=has_loop,
                  layers=[cls._read_layer(entry, f"{origin}: layers[{i}]") for i, entry in enumerate(listed)],
                  eos_token_ids=r.int_or_int_list("eos_token_id"))
        cfg.read_generation_defaults(generation, generation_origin)
        cfg.validate(origin)
        return cfg

    @staticmethod
    def _read_layer(entry: Any, origin: str) -> SosuvikLayer:
        if not isinstance(entry, dict):
            raise ConfigError(f"'{origin}' must be an object")
        r = JsonReader(entry, origin)
        kind = r.string("type")
        if kind not in MIXER_TYPES:
            raise ConfigError(f"'{origin}': there is no mixer '{kind}' (known: {', '.join(MIXER_TYPES)})")
        mixer = _object(r.raw("mixer"), origin, "mixer")
        layer = SosuvikLayer(type=kind)
        if kind == "attention":
            layer.attention = AttentionSizes.read(mixer, f"{origin}.mixer")
        else:
            layer.latent = LatentSizes.read(mixer, f"{origin}.mixer")
        mlp = r.raw("mlp")
        if mlp is not None:
            layer.mlp = SosuvikMLP.read(_object(mlp, origin, "mlp"), f"{origin}.mlp")
        return layer

    # --------------------------------------------------------------- validation
    def validate(self, origin: str = "<config>") -> None:
        require_positive(origin, vocab=self.vocab_size, width=self.width, max_positions=self.max_positions)
        if not self.norm_eps >= 0.0:
            raise ConfigError(f"'{origin}': norm.eps ({self.norm_eps}) must not be negative")
        if not self.layers:
            raise ConfigError(f"'{origin}': a model needs at least one layer")
        if self.has_loop:
            if not 0 <= self.loop_start <= self.loop_stop <= len(self.layers):
                raise ConfigError(f"'{origin}': loop {self.loop_start} .. {self.loop_stop} does not lie inside the "
                                  f"{len(self.layers)} layers")
            if self.loop_times < 1:
                raise ConfigError(f"'{origin}': loop.times ({self.loop_times}) must be at least 1")
        for i, layer in enumerate(self.layers):
            where = f"{origin}: layers[{i}]"
            layer.sizes.check(f"{where}.mixer")
            if layer.mlp is not None:
                layer.mlp.check(f"{where}.mlp")

    # ------------------------------------------------------------------ writing
    def to_dict(self) -> Dict[str, Any]:
        out: Dict[str, Any] = {
            "architecture": self.architecture,
            "layers": [layer.to_dict() for layer in self.layers],
            "logit_scale": self.logit_scale,
            "norm": {"eps": self.norm_eps},
            "vocab": self.vocab_size,
            "width": self.width,
        }
        if self.has_loop:
            out["loop"] = {"start": self.loop_start, "stop": self.loop_stop, "times": self.loop_times}
        if self.eos_token_ids:
            out["eos_token_id"] = self.eos_token_ids[0] if len(self.eos_token_ids) == 1 else list(self.eos_token_ids)
        return out

    # ------------------------------------------------------------ the model
    def _mixer(self, layer: SosuvikLayer, positions: Dict[str, PartSpec]) -> PartSpec:
        if layer.type == "latent_attention":
            m = layer.latent
            return PartSpec("latent_attention", {
                "hidden_size": self.width, "num_heads": m.heads, "head_dim": m.dim, "rotary_dim": m.rot_dim,
                "value_dim": m.vdim, "latent_dim": m.kv_rank, "scale": m.scale, "norm_eps": self.norm_eps,
                "position": m.rot.position(m.rot_dim, positions, "interleaved"), "prefix": "mix"})
        m = layer.attention
        return PartSpec("attention_rows", {
            "hidden_size": self.width, "num_heads": m.heads, "num_kv_heads": m.kv_heads, "head_dim": m.dim,
            "value_dim": m.vdim, "scale": m.scale, "score_cap": m.softcap, "chunk": m.chunk, "fixed_sink": 0.0,
            "position": m.rot.position(m.dim, positions), "prefix": "mix"})

    def _ffn(self, layer: SosuvikLayer) -> Optional[PartSpec]:
        m = layer.mlp
        if m is None:
            return None
        return PartSpec("routed_experts", {
            "hidden_size": self.width, "expert_size": m.ff, "num_experts": m.experts, "top": m.top, "correction": True,
            "score": "sigmoid", "renormalize": True, "weight_scale": m.scale,
            "groups": {"count": m.groups, "keep": m.keep} if m.groups > 1 else None,
            "expert_activation": "clamped_swish", "limit": m.limit, "prefix": "mlp"})

    def run_order(self) -> List[RunSpec]:
        """The layers in the order of running: those of the loop ``times`` times; the first layer of every pass brings the
        embedding's output back in and is marked by the pass's row of ``loop.step``."""
        n = len(self.layers)
        if not self.has_loop:
            return [RunSpec(layer=i) for i in range(n)]
        order = [RunSpec(layer=i) for i in range(self.loop_start)]
        for t in range(self.loop_times):
            for i in range(self.loop_start, self.loop_stop):
                first = i == self.loop_start
                order.append(RunSpec(layer=i, offset=("loop.step", t) if first else None, rejoin="loop.in" if first else None))
        return order + [RunSpec(layer=i) for i in range(self.loop_stop, n)]

    def model_spec(self) -> ModelSpec:
        norm = PartSpec("rmsnorm", {"size": self.width, "eps": self.norm_eps, "tensor": ""})
        positions: Dict[str, PartSpec] = {}
        layers = []
        for i, layer in enumerate(self.layers):
            layers.append(LayerSpec(prefix=f"l{i}", mixer=self._mixer(layer, positions), ffn=self._ffn(layer),
                                    norms={"mixer_norm": norm, "ffn_norm": norm},
                                    block=PartSpec("parallel_pair", {"mixer_norm": "norm1", "ffn_norm": "norm2"})))
        looped = self.has_loop and self.loop_stop > self.loop_start
        spec = ModelSpec(
            architecture=self.architecture,
            vocab_size=self.vocab_size,
            hidden_size=self.width,
            max_positions=self.max_positions,
            embedding=PartSpec("embedding", {"vocab_size": self.vocab_size, "hidden_size": self.width, "name": "embed"}),
            layers=layers,
            order=self.run_order(),
            final_norm=norm,
            final_norm_prefix="final.norm",
            head=PartSpec("lm_head", {"vocab_size": self.vocab_size, "hidden_size": self.width, "name": "head",
                                      "scale": self.logit_scale}),
            positions=positions,
            offsets={"loop.step": self.loop_times} if looped else {},
            rejoins=["loop.in"] if looped else [],
        )
        spec.validate()
        return spec
