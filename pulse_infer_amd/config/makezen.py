"""Makezen: a decoder with a norm before and after every sublayer, whose mixers are the gated delta rule, capped attention
beside the gated delta rule, and windowed attention over latent rows that layers may share.

config.json holds ``architecture``, ``vocab``, ``width``, ``norm.eps`` and ``layers``: for each layer its ``type`` (the
mixer), the mixer's sizes and constants (``mixer``) and its feed-forward (``mlp``, or null for none).  Every size and
constant is taken from there.  Tensors: ``embed``, ``embed.norm``, ``l<i>.norm1`` / ``norm1b`` / ``norm2`` / ``norm2b``,
``l<i>.mix.*``, ``l<i>.mlp.up`` / ``down``, ``final.norm``; the logits are a product with ``embed``.

The model: the token's row of ``embed`` through ``embed.norm``; every sublayer f (a layer's mixer, then its
feed-forward) adds post(f(pre(x))), with ``norm1`` and ``norm1b`` around the mixer, ``norm2`` and ``norm2b`` around the
feed-forward; all these norms are layer norms with a weight and no bias.  logits = embed final.norm(x).

Mixers.  ``delta``: the gated delta rule behind convolutions of ``conv`` taps (``heads`` x ``dim`` x ``vdim`` states,
``kv_heads`` heads of q and k).  ``parallel``: half the sum of two mixers on the same input, each result divided by its
root mean square and multiplied by a weight.  Left: softmax attention with biases, grouped key/value heads (``heads``,
``kv_heads``, ``dim``, ``vdim``), a weighted norm of every q and k head, a rotation (``rot``), ``scale`` and ``softcap``
on the scores.  Right: a gated delta rule.  ``latent_attention``: queries from a latent of ``q_rank`` values, keys and
values from one normed latent row a token (``kv_rank``) and one turned key part (``rot_dim`` channels) shared by all heads;
a window of ``mask.size`` tokens; sinks; an output gate a head.  With ``kv_from`` = j a layer reads the rows that layer j
caches.  Rotations turn the first ``rot.dims`` channels in pairs (i, i + dims / 2), their frequencies blended by
``rot.scaling`` (``factor``, ``original``, ``fast``, ``slow``).

Feed-forward.  ``dense``: down(gelu(up x)) with the tanh form of gelu, ``ff`` wide.

All of that is said to the engine as parameters of registered parts (``model_spec``); there is no model class.
"""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Any, Dict, List, Optional

from .base import ConfigError, JsonReader, ModelConfig, require_positive
from ..models.spec import LayerSpec, ModelSpec, PartSpec, RunSpec

ARCHITECTURE = "Makezen"
MIXER_TYPES = ("delta", "parallel", "latent_attention")
MLP_KINDS = ("dense",)
SCALING_KEYS = ("factor", "original", "fast", "slow")


def _object(value: Any, where: str, what: str) -> Dict[str, Any]:
    if not isinstance(value, dict):
        raise ConfigError(f"'{where}': key '{what}' must be an object")
    return value


def _window(r: JsonReader, where: str) -> Optional[int]:
    if r.raw("mask") is None:
        return None
    return JsonReader(_object(r.raw("mask"), where, "mask"), f"{where}.mask").integer("size")


@dataclass
class Rotation:
    base: float = 1.0
    dims: int = 0                                  # 0: config.json names no rotation
    scaling: Optional[Dict[str, float]] = None     # the numbers of SCALING_KEYS

    @classmethod
    def read(cls, value: Any, where: str) -> "Rotation":
        if value is None:
            return cls()
        r = JsonReader(_object(value, where, "rot"), f"{where}.rot")
        scaling = None
        if r.raw("scaling") is not None:
            s = JsonReader(_object(r.raw("scaling"), f"{where}.rot", "scaling"), f"{where}.rot.scaling")
            scaling = {key: s.number(key) for key in SCALING_KEYS}
        return cls(base=r.number("base"), dims=r.integer("dims"), scaling=scaling)

    def check(self, where: str, most: int) -> None:
        if self.dims < 0 or self.dims % 2 or self.dims > most:
            raise ConfigError(f"'{where}': rot.dims ({self.dims}) must be even and at most {most}")
        if self.dims and not self.base > 0:
            raise ConfigError(f"'{where}': rot.base must be positive, got {self.base}")
        if self.scaling is not None:
            if self.base == 1.0:
                raise ConfigError(f"'{where}': rot.scaling has no meaning for a rot.base of 1")
            require_positive(f"{where}.rot.scaling", **self.scaling)

    def to_dict(self) -> Optional[Dict[str, Any]]:
        if not self.dims:
            return None
        out: Dict[str, Any] = {"base": self.base, "dims": self.dims}
        if self.scaling is not None:
            out["scaling"] = dict(self.scaling)
        return out

    def position(self, head_dim: int, positions: Dict[str, PartSpec], pairing: str = "half") -> Optional[str]:
        """The name under which the model lists this rotation (listed on the way); None without one."""
        if not self.dims:
            return None
        scaled = "" if self.scaling is None else ":" + ":".join(repr(self.scaling[key]) for key in SCALING_KEYS)
        name = f"rope:{self.base!r}:{self.dims}{scaled}" + ("" if pairing == "half" else f":{pairing}")
        params: Dict[str, Any] = {"theta": self.base, "rotary_dim": self.dims, "head_dim": max(head_dim, self.dims), "pairing": pairing}
        if self.scaling is not None:
            params["yarn"] = dict(self.scaling)
        positions.setdefault(name, PartSpec("rope", params))
        return name


@dataclass
class DeltaSizes:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int

    @classmethod
    def read(cls, data: Dict[str, Any], where: str) -> "DeltaSizes":
        r = JsonReader(data, where)
        heads, dim = r.integer("heads"), r.integer("dim")
        return cls(heads=heads, kv_heads=r.integer("kv_heads", heads), dim=dim, vdim=r.integer("vdim", dim),
                   conv=r.integer("conv"))

    def check(self, where: str) -> None:
        require_positive(where, heads=self.heads, kv_heads=self.kv_heads, dim=self.dim, vdim=self.vdim, conv=self.conv)
        if self.heads % self.kv_heads:
            raise ConfigError(f"'{where}': {self.heads} heads cannot be shared out evenly over {self.kv_heads} heads of q and k")
        if self.dim > 256:
            raise ConfigError(f"'{where}': the state's kernels take at most 256 key channels a head, dim is {self.dim}")
        if self.conv > 16:
            raise ConfigError(f"'{where}': the convolution's kernels take at most 16 taps, conv is {self.conv}")

    def to_dict(self) -> Dict[str, Any]:
        return {"conv": self.conv, "dim": self.dim, "heads": self.heads, "kv_heads": self.kv_heads, "vdim": self.vdim}

    def part(self, width: int, eps: float, prefix: str) -> PartSpec:
        return PartSpec("gated_delta", {"hidden_size": width, "num_heads": self.heads, "num_groups": self.kv_heads,
                                        "head_dim": self.dim, "value_dim": self.vdim, "conv": self.conv, "norm_eps": eps,
                                        "prefix": prefix})


@dataclass
class LeftSizes:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    softcap: float              # 0: none
    rot: Rotation

    @classmethod
    def read(cls, data: Dict[str, Any], where: str) -> "LeftSizes":
        r = JsonReader(data, where)
        heads, dim = r.integer("heads"), r.integer("dim")
        return cls(heads=heads, kv_heads=r.integer("kv_heads", heads), dim=dim, vdim=r.integer("vdim", dim),
                   scale=r.number("scale"), softcap=r.number("softcap", 0.0), rot=Rotation.read(r.raw("rot"), where))

    def check(self, where: str) -> None:
        require_positive(where, heads=self.heads, kv_heads=self.kv_heads, dim=self.dim, vdim=self.vdim)
        if self.softcap < 0.0:
            raise ConfigError(f"'{where}': softcap ({self.softcap}) must not be negative")
        if self.heads % self.kv_heads:
            raise ConfigError(f"'{where}': {self.heads} query heads cannot be shared out evenly over {self.kv_heads} "
                              "key/value heads")
        self.rot.check(where, self.dim)

    def to_dict(self) -> Dict[str, Any]:
        out: Dict[str, Any] = {"dim": self.dim, "heads": self.heads, "kv_heads": self.kv_heads, "scale": self.scale,
                               "softcap": self.softcap, "vdim": self.vdim}
        if self.rot.dims:
            out["rot"] = self.rot.to_dict()
        return out


@dataclass
class LatentSizes:
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    q_rank: int
    kv_rank: int
    scale: float
    window: Optional[int]
    rot: Rotation
    kv_from: Optional[int] = None

    @classmethod
    def read(cls, data: Dict[str, Any], where: str) -> "LatentSizes":
        r = JsonReader(data, where)
        return cls(heads=r.integer("heads"), dim=r.integer("dim"), rot_dim=r.integer("rot_dim"), vdim=r.integer("vdim"),
                   q_rank=r.integer("q_rank"), kv_rank=r.integer("kv_rank"), scale=r.number("scale"), window=_window(r, where),
                   rot=Rotation.read(r.raw("rot"), where), kv_from=r.integer("kv_from", None))

    def check(self, where: str) -> None:
        require_positive(where, heads=self.heads, dim=self.dim, rot_dim=self.rot_dim, vdim=self.vdim, q_rank=self.q_rank,
                         kv_rank=self.kv_rank)
        if self.window is not None:
            require_positive(where, size=self.window)
        self.rot.check(where, self.rot_dim)
        if self.rot.dims != self.rot_dim:
            raise ConfigError(f"'{where}': rot.dims ({self.rot.dims}) must be rot_dim ({self.rot_dim}): the turned part "
                              "is turned as a whole")

    def to_dict(self) -> Dict[str, Any]:
        out = {"dim": self.dim, "heads": self.heads, "kv_rank": self.kv_rank, "q_rank": self.q_rank, "rot": self.rot.to_dict(),
               "rot_dim": self.rot_dim, "scale": self.scale, "vdim": self.vdim}
        if self.window is not None:
            out["mask"] = {"size": self.window}
        if self.kv_from is not None:
            out["kv_from"] = self.kv_from
        return out


@dataclass
class MakezenMLP:
    kind: str
    ff: int

    @classmethod
    def read(cls, data: Dict[str, Any], where: str) -> "MakezenMLP":
        r = JsonReader(data, where)
        kind = r.string("kind")
        if kind not in MLP_KINDS:
            raise ConfigError(f"'{where}': there is no feed-forward '{kind}' (known: {', '.join(MLP_KINDS)})")
        return cls(kind=kind, ff=r.integer("ff"))

    def check(self, where: str) -> None:
        require_positive(where, ff=self.ff)

    def to_dict(self) -> Dict[str, Any]:
        return {"ff": self.ff, "kind": self.kind}


@dataclass
class MakezenLayer:
    type: str
    delta: Optional[DeltaSizes] = None      # of a delta layer, or the right side of a parallel one
    left: Optional[LeftSizes] = None
    latent: Optional[LatentSizes] = None
    mlp: Optional[MakezenMLP] = None

    def to_dict(self) -> Dict[str, Any]:
        if self.type == "parallel":
            mixer: Dict[str, Any] = {"left": self.left.to_dict(), "right": self.delta.to_dict()}
        else:
            mixer = (self.delta if self.type == "delta" else self.latent).to_dict()
        return {"mixer": mixer, "mlp": None if self.mlp is None else self.mlp.to_dict(), "type": self.type}


@dataclass
class MakezenConfig(ModelConfig):
    vocab_size: int
    width: int
    norm_eps: float
    layers: List[MakezenLayer] = field(default_factory=list)
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
                  generation_origin: str = "<dict>") -> "MakezenConfig":
        r = JsonReader(data, origin)
        norm = JsonReader(_object(r.raw("norm"), origin, "norm"), f"{origin}: norm")
        listed = r.raw("layers")
        if not isinstance(listed, list) or not listed:
            raise ConfigError(f"'{origin}': key 'layers' must be a list with at least one layer")
        cfg = cls(vocab_size=r.integer("vocab"), width=r.integer("width"), norm_eps=norm.number("eps"),
                  layers=[cls._read_layer(entry, f"{origin}: layers[{i}]") for i, entry in enumerate(listed)],
                  eos_token_ids=r.int_or_int_list("eos_token_id"))
        cfg.read_generation_defaults(generation, generation_origin)
        cfg.validate(origin)
        return cfg

    @staticmethod
    def _read_layer(entry: Any, origin: str) -> MakezenLayer:
        if not isinstance(entry, dict):
            raise ConfigError(f"'{origin}' must be an object")
        r = JsonReader(entry, origin)
        kind = r.string("type")
        if kind not in MIXER_TYPES:
            raise ConfigError(f"'{origin}': there is no mixer '{kind}' (known: {', '.join(MIXER_TYPES)})")
        mixer = _object(r.raw("mixer"), origin, "mixer")
        layer = MakezenLayer(type=kind)
        if kind == "delta":
            layer.delta = DeltaSizes.read(mixer, f"{origin}.mixer")
        elif kind == "parallel":
            m = JsonReader(mixer, f"{origin}.mixer")
            layer.left = LeftSizes.read(_object(m.raw("left"), f"{origin}.mixer", "left"), f"{origin}.mixer.left")
            layer.delta = DeltaSizes.read(_object(m.raw("right"), f"{origin}.mixer", "right"), f"{origin}.mixer.right")
        else:
            layer.latent = LatentSizes.read(mixer, f"{origin}.mixer")
        mlp = r.raw("mlp")
        if mlp is not None:
            layer.mlp = MakezenMLP.read(_object(mlp, origin, "mlp"), f"{origin}.mlp")
        return layer

    # --------------------------------------------------------------- validation
    def validate(self, origin: str = "<config>") -> None:
        require_positive(origin, vocab=self.vocab_size, width=self.width, max_positions=self.max_positions)
        if not self.norm_eps >= 0.0:
            raise ConfigError(f"'{origin}': norm.eps ({self.norm_eps}) must not be negative")
        if not self.layers:
            raise ConfigError(f"'{origin}': a model needs at least one layer")
        for i, layer in enumerate(self.layers):
            where = f"{origin}: layers[{i}]"
            if layer.left is not None:
                layer.left.check(f"{where}.mixer.left")
            if layer.delta is not None:
                layer.delta.check(f"{where}.mixer{'.right' if layer.left is not None else ''}")
            if layer.latent is not None:
                layer.latent.check(f"{where}.mixer")
                self._check_source(i, where)
            if layer.mlp is not None:
                layer.mlp.check(f"{where}.mlp")

    def _check_source(self, index: int, where: str) -> None:
        """A layer that reads another layer's rows: that layer comes before it, caches rows, and they are of its form."""
        m = self.layers[index].latent
        if m.kv_from is None:
            return
        source = self.layers[m.kv_from].latent if 0 <= m.kv_from < index else None
        if source is None or source.kv_from is not None:
            raise ConfigError(f"'{where}': kv_from ({m.kv_from}) must name an earlier latent_attention layer with rows of its own")
        if (source.kv_rank, source.rot_dim, source.rot) != (m.kv_rank, m.rot_dim, m.rot):
            raise ConfigError(f"'{where}': kv_rank, rot_dim and rot must be those of layer {m.kv_from}, whose rows it reads")

    # ------------------------------------------------------------------ writing
    def to_dict(self) -> Dict[str, Any]:
        out: Dict[str, Any] = {
            "architecture": self.architecture,
            "layers": [layer.to_dict() for layer in self.layers],
            "norm": {"eps": self.norm_eps},
            "vocab": self.vocab_size,
            "width": self.width,
        }
        if self.eos_token_ids:
            out["eos_token_id"] = self.eos_token_ids[0] if len(self.eos_token_ids) == 1 else list(self.eos_token_ids)
        return out

    # ------------------------------------------------------------ the model
    def rows_kept(self, index: int) -> int:
        """How far back the rows of latent layer ``index`` are read, by itself and by the layers that read them (0: to
        the start): what its cache must keep."""
        readers = [layer.latent for i, layer in enumerate(self.layers)
                   if layer.latent is not None and (i == index or layer.latent.kv_from == index)]
        return 0 if any(m.window is None for m in readers) else max(m.window for m in readers)

    def _mixer(self, index: int, layer: MakezenLayer, positions: Dict[str, PartSpec]) -> PartSpec:
        if layer.type == "delta":
            return layer.delta.part(self.width, self.norm_eps, "mix")
        if layer.type == "latent_attention":
            m = layer.latent
            return PartSpec("latent_attention", {
                "hidden_size": self.width, "num_heads": m.heads, "head_dim": m.dim, "rotary_dim": m.rot_dim,
                "value_dim": m.vdim, "latent_dim": m.kv_rank, "query_dim": m.q_rank, "scale": m.scale,
                "norm_eps": self.norm_eps, "position": m.rot.position(m.rot_dim, positions), "window": m.window,
                "cache_window": self.rows_kept(index) if m.kv_from is None else m.window,
                "reads_rows": m.kv_from is not None, "sink": True, "output_gate": "head", "prefix": "mix"})
        left = layer.left
        attention = {"hidden_size": self.width, "num_heads": left.heads, "num_kv_heads": left.kv_heads,
                     "head_dim": left.dim, "value_dim": left.vdim, "scale": left.scale, "score_cap": left.softcap,
                     "bias": True, "qk_norm": "head", "qk_norm_weights": True, "qk_norm_eps": self.norm_eps,
                     "position": left.rot.position(left.dim, positions), "prefix": "left"}
        return PartSpec("side_by_side", {
            "hidden_size": self.width, "prefix": "mix",
            "branch_norm": {"tensor": "out", "eps": self.norm_eps, "factor": 0.5},
            "branches": [{"kind": "attention_rows", "params": attention},
                         {"kind": "gated_delta", "params": layer.delta.part(self.width, self.norm_eps, "right").params}]})

    def _ffn(self, layer: MakezenLayer) -> Optional[PartSpec]:
        if layer.mlp is None:
            return None
        return PartSpec("mlp", {"hidden_size": self.width, "intermediate_size": layer.mlp.ff, "activation": "gelu_tanh",
                                "prefix": "mlp"})

    def model_spec(self) -> ModelSpec:
        norm = PartSpec("layernorm", {"size": self.width, "eps": self.norm_eps, "tensor": "", "bias": False})
        places = {"mixer_norm": "norm1", "mixer_post": "norm1b", "ffn_norm": "norm2", "ffn_post": "norm2b"}
        positions: Dict[str, PartSpec] = {}
        layers, order = [], []
        for i, layer in enumerate(self.layers):
            layers.append(LayerSpec(prefix=f"l{i}", mixer=self._mixer(i, layer, positions), ffn=self._ffn(layer),
                                    norms={place: norm for place in places}, block=PartSpec("sandwich", places)))
            order.append(RunSpec(layer=i, cache_of=layer.latent.kv_from if layer.latent is not None else None))
        spec = ModelSpec(
            architecture=self.architecture,
            vocab_size=self.vocab_size,
            hidden_size=self.width,
            max_positions=self.max_positions,
            embedding=PartSpec("embedding", {"vocab_size": self.vocab_size, "hidden_size": self.width, "name": "embed",
                                             "norm": {"kind": "layernorm", "tensor": "embed.norm", "eps": self.norm_eps}}),
            layers=layers,
            order=order,
            final_norm=norm,
            final_norm_prefix="final.norm",
            head=PartSpec("lm_head", {"vocab_size": self.vocab_size, "hidden_size": self.width, "name": "head", "tied": True}),
            positions=positions,
        )
        spec.validate()
        return spec
