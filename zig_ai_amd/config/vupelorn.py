"""Typed configuration of Vupelorn, a decoder whose layers mix tokens in one of three ways,
listed layer by layer in config.json:

  ``gla``                 gated linear attention: a matrix state a head whose rows decay by a
                          factor of their own, made from the token (``parts/recurrent.py``,
                          ``gated_linear``)
  ``latent_attention``    queries through a normed latent; keys and values of every head are
                          expansions of one normed latent a token, beside a rotated key part
                          that all heads share; rotary positions in halves, with frequencies
                          stretched for long contexts (``rope``, ``scaling`` of type ``yarn``)
  ``latent_attention_2``  the same with rotary positions in adjacent pairs; a layer with
                          ``kv_from: j`` makes no latent of its own and reads layer ``j``'s
                          cached rows (``parts/latent_attention.py``, ``latent_attention``)

Norms stand on the parts' outputs only: ``x <- x + norm1(mixer(x))``, ``x <- x +
norm2(ff(x))`` (``normed_output``).  The feed-forward (``mlp``, may be absent) is a set of
small bounded gated experts chosen by a router with sigmoid scores, a token's weight
multiplying the expert's input (``routed_experts``).  The embedding adds a row that the
token and its predecessor pick from a second table; the predecessor is part of a request's
state (``token_embedding`` with ``pair``).  The head is the embedding table.

config.json keys: ``architecture``, ``vocab``, ``width``, ``norm.eps``, ``embedding.bigram.{buckets,
mul_prev, mul_cur}``, ``layers[i] = {type, mixer, mlp}``; tensor names: ``embed``, ``bigram``,
``l<i>.norm1``, ``l<i>.norm2``, ``l<i>.mix.*``, ``l<i>.mlp.*``, ``final.norm``.  The rank of a
``gla`` layer's decay projection is given by its tensors (``with_shapes``).
"""

from __future__ import annotations

from dataclasses import dataclass, replace
from typing import Any, Callable, Dict, Mapping, Optional, Tuple

from .fields import read_float, read_int
from .spec import ConfigError, LayerCall, LayerSpec, ModelSpec, PartSpec

LAYER_TYPES = ("gla", "latent_attention", "latent_attention_2")
# constants of the design
ROTARY_PAIRING = {"latent_attention": "half", "latent_attention_2": "adjacent"}
GATE_SLOPE = 1.702                  # of the experts' sigmoid
UP_OFFSET = 1.0                     # added to the experts' bounded up projection
DEFAULT_DECAY_RANK = 16             # where neither config.json nor a tensor says


def _mapping(data: Mapping[str, Any], key: str, where: str) -> Mapping[str, Any]:
    value = data.get(key)
    if not isinstance(value, Mapping):
        raise ConfigError(f"{where} has no {key} object")
    return value


@dataclass(frozen=True)
class YarnSizes:
    factor: float
    original: float
    fast: float
    slow: float

    @classmethod
    def read(cls, data: Mapping[str, Any], where: str) -> "YarnSizes":
        if not isinstance(data, Mapping):
            raise ConfigError(f"{where} must be an object with factor, original, fast and slow")
        return cls(*(read_float(data, [k], positive=True)
                     for k in ("factor", "original", "fast", "slow")))

    def to_dict(self) -> dict:
        return {"factor": self.factor, "original": self.original, "fast": self.fast,
                "slow": self.slow}


@dataclass(frozen=True)
class LatentSizes:
    heads: int
    dim: int                         # unrotated query/key elements a head
    vdim: int
    kv_rank: int
    q_rank: int
    scale: float
    rot_dim: int                     # rotated query/key elements
    rot_dims: int                    # how many of them the rotation turns
    rot_base: float
    scaling: Optional[YarnSizes] = None
    kv_from: Optional[int] = None    # the layer whose cached rows this one reads

    @classmethod
    def read(cls, m: Mapping[str, Any], where: str) -> "LatentSizes":
        heads = read_int(m, ["heads"], minimum=1)
        dim = read_int(m, ["dim"], minimum=1)
        rot_dim = read_int(m, ["rot_dim"], minimum=2)
        rot = _mapping(m, "rot", where)
        rot_dims = read_int(rot, ["dims"], default=rot_dim, minimum=2)
        if rot_dims % 2 or rot_dims > rot_dim:
            raise ConfigError(f"{where}: rot.dims {rot_dims} must be even and at most rot_dim "
                              f"{rot_dim}")
        scaling = rot.get("scaling")
        if scaling is not None:
            scaling = YarnSizes.read(scaling, where + ".rot.scaling")
        source = m.get("kv_from")
        if source is not None:
            source = read_int(m, ["kv_from"], minimum=0)
        return cls(heads, dim, read_int(m, ["vdim"], default=dim, minimum=1),
                   read_int(m, ["kv_rank"], minimum=1), read_int(m, ["q_rank"], minimum=1),
                   read_float(m, ["scale"], default=(dim + rot_dim) ** -0.5),
                   rot_dim, rot_dims, read_float(rot, ["base"], positive=True), scaling, source)

    def rotation(self) -> tuple:
        return (self.rot_dim, self.rot_dims, self.rot_base, self.scaling)

    def to_dict(self) -> dict:
        rot: Dict[str, Any] = {"dims": self.rot_dims, "base": self.rot_base}
        if self.scaling is not None:
            rot["scaling"] = self.scaling.to_dict()
        out: Dict[str, Any] = {"heads": self.heads, "dim": self.dim, "vdim": self.vdim,
                               "kv_rank": self.kv_rank, "q_rank": self.q_rank,
                               "scale": self.scale, "rot_dim": self.rot_dim, "rot": rot}
        if self.kv_from is not None:
            out["kv_from"] = self.kv_from
        return out


@dataclass(frozen=True)
class GlaSizes:
    heads: int
    dim: int                         # key channels a head (rows of its state)
    vdim: int
    tau: float
    decay_rank: int = DEFAULT_DECAY_RANK

    @classmethod
    def read(cls, m: Mapping[str, Any]) -> "GlaSizes":
        dim = read_int(m, ["dim"], minimum=1)
        return cls(read_int(m, ["heads"], minimum=1), dim,
                   read_int(m, ["vdim"], default=dim, minimum=1),
                   read_float(m, ["tau"], positive=True),
                   read_int(m, ["decay_rank"], default=DEFAULT_DECAY_RANK, minimum=1))

    def to_dict(self) -> dict:
        return {"heads": self.heads, "dim": self.dim, "vdim": self.vdim, "tau": self.tau,
                "decay_rank": self.decay_rank}


@dataclass(frozen=True)
class ExpertSizes:
    experts: int
    top: int
    ff: int                          # width inside an expert
    limit: float

    @classmethod
    def read(cls, mlp: Mapping[str, Any], where: str) -> "ExpertSizes":
        router, expert = _mapping(mlp, "router", where), _mapping(mlp, "expert", where)
        experts = read_int(router, ["experts"], minimum=1)
        top = read_int(router, ["top"], minimum=1)
        if top > experts:
            raise ConfigError(f"{where}.router: top {top} of {experts} experts")
        return cls(experts, top, read_int(expert, ["ff"], minimum=1),
                   read_float(expert, ["limit"], positive=True))

    def to_dict(self) -> dict:
        return {"kind": "moe", "expert": {"ff": self.ff, "limit": self.limit},
                "router": {"experts": self.experts, "top": self.top}}


@dataclass(frozen=True)
class PairTable:
    buckets: int
    mul_prev: int
    mul_cur: int

    @classmethod
    def read(cls, data: Mapping[str, Any]) -> "PairTable":
        return cls(read_int(data, ["buckets"], minimum=1), read_int(data, ["mul_prev"], minimum=0),
                   read_int(data, ["mul_cur"], minimum=0))

    def to_dict(self) -> dict:
        return {"buckets": self.buckets, "mul_prev": self.mul_prev, "mul_cur": self.mul_cur}


@dataclass(frozen=True)
class VupelornLayer:
    type: str
    latent: Optional[LatentSizes] = None
    gla: Optional[GlaSizes] = None
    mlp: Optional[ExpertSizes] = None


@dataclass(frozen=True)
class VupelornConfig:
    architecture: str
    vocab_size: int
    hidden_size: int
    norm_eps: float
    layers: Tuple[VupelornLayer, ...]
    pair: Optional[PairTable] = None
    max_position_embeddings: int = 0
    eos_token_id: Optional[int] = None

    # ---------------------------------------------------------------- parsing
    @classmethod
    def from_dict(cls, data: Mapping[str, Any]) -> "VupelornConfig":
        entries = data.get("layers")
        if not isinstance(entries, (list, tuple)) or not entries:
            raise ConfigError("config.json has no layers list")
        layers = []
        for i, entry in enumerate(entries):
            where = f"layers[{i}]"
            if not isinstance(entry, Mapping) or entry.get("type") not in LAYER_TYPES:
                raise ConfigError(f"{where}.type must be one of {', '.join(LAYER_TYPES)}, got "
                                  f"{entry.get('type') if isinstance(entry, Mapping) else entry!r}")
            kind, m = entry["type"], _mapping(entry, "mixer", where)
            kw: Dict[str, Any] = {}
            if kind == "gla":
                kw["gla"] = GlaSizes.read(m)
            else:
                kw["latent"] = LatentSizes.read(m, where + ".mixer")
            mlp = entry.get("mlp")
            if mlp is not None:
                if not isinstance(mlp, Mapping) or mlp.get("kind") != "moe":
                    raise ConfigError(f"{where}.mlp must be null or of kind moe")
                kw["mlp"] = ExpertSizes.read(mlp, where + ".mlp")
            layers.append(VupelornLayer(kind, **kw))
            if kind != "gla" and layers[i].latent.kv_from is not None:
                cls._check_source(layers, i)
        embedding = data.get("embedding") or {}
        pair = embedding.get("bigram") if isinstance(embedding, Mapping) else None
        if not isinstance(embedding, Mapping) or (pair is not None and not isinstance(pair, Mapping)):
            raise ConfigError("embedding.bigram must be an object with buckets, mul_prev and mul_cur")
        eos = data.get("eos_token_id")
        return cls(
            architecture=str(data.get("architecture") or "Vupelorn"),
            vocab_size=read_int(data, ["vocab"], minimum=1),
            hidden_size=read_int(data, ["width"], minimum=1),
            norm_eps=read_float(_mapping(data, "norm", "config.json"), ["eps"], positive=True),
            layers=tuple(layers), pair=PairTable.read(pair) if pair is not None else None,
            max_position_embeddings=read_int(data, ["max_position_embeddings"], default=0, minimum=0),
            eos_token_id=eos if isinstance(eos, int) and not isinstance(eos, bool) else None)

    @staticmethod
    def _check_source(layers, i: int) -> None:
        """A layer may only read the cached rows of an earlier layer that makes its own, of
        the same width, turned by the same rotation."""
        mine, j = layers[i].latent, layers[i].latent.kv_from
        where = f"layers[{i}].mixer.kv_from: layer {j}"
        if j >= i or layers[j].latent is None:
            raise ConfigError(f"{where} is not an earlier latent attention layer")
        source = layers[j].latent
        if source.kv_from is not None:
            raise ConfigError(f"{where} has no latent of its own")
        if source.kv_rank != mine.kv_rank or source.rotation() != mine.rotation() \
                or ROTARY_PAIRING[layers[j].type] != ROTARY_PAIRING[layers[i].type]:
            raise ConfigError(f"{where} differs in kv_rank or rotation")

    def to_dict(self) -> dict:
        layers = [{"type": layer.type,
                   "mixer": (layer.gla if layer.type == "gla" else layer.latent).to_dict(),
                   "mlp": layer.mlp.to_dict() if layer.mlp is not None else None}
                  for layer in self.layers]
        out: Dict[str, Any] = {"architecture": self.architecture, "vocab": self.vocab_size,
                               "width": self.hidden_size, "norm": {"eps": self.norm_eps},
                               "layers": layers}
        if self.pair is not None:
            out["embedding"] = {"bigram": self.pair.to_dict()}
        if self.max_position_embeddings:
            out["max_position_embeddings"] = self.max_position_embeddings
        if self.eos_token_id is not None:
            out["eos_token_id"] = self.eos_token_id
        return out

    # ---------------------------------------------- sizes only the tensors give
    def with_shapes(self, shape_of: Callable[[str], Optional[Tuple[int, ...]]]) -> "VupelornConfig":
        """The configuration with the ranks of the decay projections taken from a
        checkpoint: ``shape_of(name)`` is a stored tensor's shape, or None."""
        layers = []
        for i, layer in enumerate(self.layers):
            shape = shape_of(f"l{i}.mix.a1") if layer.gla is not None else None
            if shape:
                layer = replace(layer, gla=replace(layer.gla, decay_rank=int(shape[0])))
            layers.append(layer)
        return replace(self, layers=tuple(layers))

    # ------------------------------------------------------------ translation
    def _norm_spec(self, name: str) -> PartSpec:
        return PartSpec("rms_norm", {"width": self.hidden_size, "eps": self.norm_eps},
                        {"weight": (name,)})

    def _gla_spec(self, s: GlaSizes, p: str) -> PartSpec:
        return PartSpec(
            "gated_linear",
            {"hidden_size": self.hidden_size, "num_heads": s.heads, "head_dim": s.dim,
             "value_dim": s.vdim, "decay_rank": s.decay_rank, "decay_root": s.tau,
             "norm_eps": self.norm_eps, "gate": "silu"},
            {"q_proj.weight": (p + "q",), "k_proj.weight": (p + "k",), "v_proj.weight": (p + "v",),
             "gate_proj.weight": (p + "g",), "decay_down.weight": (p + "a1",),
             "decay_up.weight": (p + "a2",), "decay_up.bias": (p + "a2.b",),
             "norm.weight": (p + "norm",), "out_proj.weight": (p + "o",)})

    def _latent_spec(self, kind: str, s: LatentSizes, p: str) -> PartSpec:
        rope: Dict[str, Any] = {"head_dim": s.rot_dim, "rotary_dim": s.rot_dims, "theta": s.rot_base,
                                "pairing": ROTARY_PAIRING[kind]}
        if s.scaling is not None:
            rope["scaling"] = dict(s.scaling.to_dict(), type="yarn")
        own = s.kv_from is None
        names = {"q_down.weight": (p + "dq",), "q_norm.weight": (p + "dq.norm",),
                 "q_up.weight": (p + "uq",), "k_up.weight": (p + "uk",), "v_up.weight": (p + "uv",),
                 "out_proj.weight": (p + "o",)}
        if own:
            names.update({"kv_down.weight": (p + "dkv",), "kv_norm.weight": (p + "dkv.norm",)})
        return PartSpec(
            "latent_attention",
            {"hidden_size": self.hidden_size, "num_heads": s.heads, "head_dim": s.dim,
             "rotated_dim": s.rot_dim, "value_dim": s.vdim, "kv_rank": s.kv_rank,
             "q_rank": s.q_rank, "softmax_scale": s.scale, "norm_eps": self.norm_eps,
             "sink": False, "gate": None, "makes_rows": own, "position": PartSpec("rope", rope)},
            names)

    def _mlp_spec(self, s: ExpertSizes, p: str) -> PartSpec:
        names = {"router.weight": (p + "router",)}
        for e in range(s.experts):
            for w in ("gate", "up", "down"):
                names[f"experts.{e}.{w}.weight"] = (f"{p}e{e}.{w}",)
        return PartSpec(
            "routed_experts",
            {"hidden_size": self.hidden_size, "intermediate_size": s.ff, "experts": s.experts,
             "top": s.top, "scores": "sigmoid", "renormalize": False, "weight_on": "input",
             "activation": "bounded_glu", "bound": s.limit, "gate_slope": GATE_SLOPE,
             "up_offset": UP_OFFSET}, names)

    def run_order(self) -> Tuple[LayerCall, ...]:
        """Every layer once; one with ``kv_from`` reads that layer's cache and writes none."""
        calls = []
        for i, layer in enumerate(self.layers):
            source = layer.latent.kv_from if layer.latent is not None else None
            calls.append(LayerCall(i, cache=i) if source is None
                         else LayerCall(i, cache=source, writes_cache=False))
        return tuple(calls)

    def to_spec(self) -> ModelSpec:
        H = self.hidden_size
        layers = []
        for i, layer in enumerate(self.layers):
            p = f"l{i}."
            mixer = self._gla_spec(layer.gla, p + "mix.") if layer.type == "gla" \
                else self._latent_spec(layer.type, layer.latent, p + "mix.")
            parts: Dict[str, PartSpec] = {"mixer": mixer, "mixer_norm": self._norm_spec(p + "norm1")}
            kind = "normed_output_no_ff"
            if layer.mlp is not None:
                parts["feed_forward"] = self._mlp_spec(layer.mlp, p + "mlp.")
                parts["feed_forward_norm"] = self._norm_spec(p + "norm2")
                kind = "normed_output"
            layers.append(LayerSpec(parts, kind))
        params: Dict[str, Any] = {"vocab_size": self.vocab_size, "hidden_size": H}
        names = {"weight": ("embed",)}
        if self.pair is not None:
            params["pair"] = self.pair.to_dict()
            names["pair.weight"] = ("bigram",)
        lm_head = PartSpec("linear_head", {"vocab_size": self.vocab_size, "hidden_size": H,
                                           "tied": True})
        # a layer without a feed-forward may still carry its second norm; it is not read
        ignored = tuple(f"l{i}.norm2" for i, layer in enumerate(self.layers) if layer.mlp is None)
        return ModelSpec(self.architecture, H, self.vocab_size,
                         PartSpec("token_embedding", params, names), tuple(layers),
                         self.run_order(), self._norm_spec("final.norm"), lm_head,
                         self.max_position_embeddings, ignored)
