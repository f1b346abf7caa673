"""Typed configuration of Torisun, a decoder whose layers all mix tokens by attention, listed
layer by layer in config.json:

  ``attention``   grouped-query attention with values of a width of their own: one RMS norm over
                  all of a token's queries and one over all of its keys, rotary positions in
                  halves on the first ``rot.dims`` elements of a head (frequencies stretched
                  for long contexts and a factor on the rotation: ``scaling``), a sliding
                  window beside which the first ``mask.keep_first`` tokens stay visible, and a
                  learned sink a head in the softmax.  A layer with ``kv_from: j`` makes no keys
                  and values; it reads layer ``j``'s, with queries, window and sink of its own
                  (``gqa_attention`` with ``qk_norm="row"``, ``keep_first``, ``sink``,
                  ``makes_kv``)

Norms stand on the parts' outputs only: ``x <- x + norm1(mixer(x))``, ``x <- x + norm2(ff(x))``
(``normed_output``).  The feed-forward (``mlp``, may be absent) is dense with bounded gate and
up projections (``clamped_glu``), or a set of small gated experts chosen by a router with
sigmoid scores, their weights divided by their sum, beside a shared expert that runs for every
token (``routed_experts``).  The embedding's rows are normed; the head is the embedding table.

config.json keys: ``architecture``, ``vocab``, ``width``, ``norm.eps``, ``layers[i] = {type, mixer,
mlp}``; tensor names: ``embed``, ``embed.norm``, ``l<i>.norm1``, ``l<i>.norm2``, ``l<i>.mix.*``,
``l<i>.mlp.*``, ``final.norm``.
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Dict, List, Mapping, Optional, Tuple

from .fields import read_float, read_int
from .spec import ConfigError, LayerCall, LayerSpec, ModelSpec, PartSpec
from .vupelorn import YarnSizes

LAYER_TYPES = ("attention",)
# constants of the design
GATE_SLOPE = 1.702                  # of the dense feed-forward's sigmoid
UP_OFFSET = 1.0                     # added to its bounded up projection
EXPERT_ACTIVATION = "silu"          # on the gate inside an expert


def _mapping(data: Mapping[str, Any], key: str, where: str) -> Mapping[str, Any]:
    value = data.get(key)
    if not isinstance(value, Mapping):
        raise ConfigError(f"{where} has no {key} object")
    return value


@dataclass(frozen=True)
class AttentionSizes:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot_dims: int = 0                # elements of a head that turn (0: no positions)
    rot_base: float = 10000.0
    scaling: Optional[YarnSizes] = None
    window: int = 0                  # mask.size (0: every earlier key)
    keep_first: int = 0
    kv_from: Optional[int] = None    # the layer whose keys and values this one reads

    @classmethod
    def read(cls, m: Mapping[str, Any], where: str) -> "AttentionSizes":
        heads = read_int(m, ["heads"], minimum=1)
        kv = read_int(m, ["kv_heads"], default=heads, minimum=1)
        if heads % kv:
            raise ConfigError(f"{where}: {heads} heads do not divide into {kv} kv_heads")
        dim = read_int(m, ["dim"], minimum=1)
        kw: Dict[str, Any] = {}
        if m.get("rot") is not None:
            rot = _mapping(m, "rot", where)
            dims = read_int(rot, ["dims"], default=dim, minimum=0)
            if dims % 2 or dims > dim:
                raise ConfigError(f"{where}: rot.dims {dims} must be even and at most dim {dim}")
            if dims:
                kw.update(rot_dims=dims, rot_base=read_float(rot, ["base"], positive=True))
                if rot.get("scaling") is not None:
                    kw["scaling"] = YarnSizes.read(rot["scaling"], where + ".rot.scaling")
        if m.get("mask") is not None:
            mask = _mapping(m, "mask", where)
            kw["window"] = read_int(mask, ["size"], minimum=1)
            kw["keep_first"] = read_int(mask, ["keep_first"], default=0, minimum=0)
        if m.get("kv_from") is not None:
            kw["kv_from"] = read_int(m, ["kv_from"], minimum=0)
        return cls(heads, kv, dim, read_int(m, ["vdim"], default=dim, minimum=1),
                   read_float(m, ["scale"], default=dim ** -0.5, positive=True), **kw)

    def shares_with(self) -> tuple:
        """What a layer and the layer whose keys and values it reads have in common."""
        return (self.heads, self.kv_heads, self.dim, self.vdim, self.rot_dims, self.rot_base,
                self.scaling)

    def to_dict(self) -> dict:
        out: Dict[str, Any] = {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim,
                               "vdim": self.vdim, "scale": self.scale}
        if self.rot_dims:
            out["rot"] = {"dims": self.rot_dims, "base": self.rot_base}
            if self.scaling is not None:
                out["rot"]["scaling"] = self.scaling.to_dict()
        if self.window:
            out["mask"] = {"size": self.window, "keep_first": self.keep_first}
        if self.kv_from is not None:
            out["kv_from"] = self.kv_from
        return out


@dataclass(frozen=True)
class FeedForwardSizes:
    kind: str                        # "dense" or "moe"
    ff: int                          # of the dense feed-forward, or of one expert
    limit: float = 0.0               # dense: the bound (0: none)
    experts: int = 0
    top: int = 0
    route_scale: float = 1.0
    shared_ff: int = 0               # width of the shared expert (0: there is none)

    @classmethod
    def read(cls, mlp: Any, where: str) -> "FeedForwardSizes":
        if not isinstance(mlp, Mapping) or mlp.get("kind") not in ("dense", "moe"):
            raise ConfigError(f"{where} must be null, or of kind dense or moe")
        if mlp["kind"] == "dense":
            return cls("dense", read_int(mlp, ["ff"], minimum=1),
                       read_float(mlp, ["limit"], default=0.0))
        router, expert = _mapping(mlp, "router", where), _mapping(mlp, "expert", where)
        experts = read_int(router, ["experts"], minimum=1)
        top = read_int(router, ["top"], minimum=1)
        if top > experts:
            raise ConfigError(f"{where}.router: top {top} of {experts} experts")
        shared = 0
        if mlp.get("shared") is not None:
            shared = read_int(_mapping(mlp, "shared", where), ["ff"], minimum=1)
        return cls("moe", read_int(expert, ["ff"], minimum=1), 0.0, experts, top,
                   read_float(router, ["scale"], default=1.0), shared)

    def to_dict(self) -> dict:
        if self.kind == "dense":
            out: Dict[str, Any] = {"kind": "dense", "ff": self.ff}
            if self.limit:
                out["limit"] = self.limit
            return out
        out = {"kind": "moe", "expert": {"ff": self.ff},
               "router": {"experts": self.experts, "top": self.top, "scale": self.route_scale}}
        if self.shared_ff:
            out["shared"] = {"ff": self.shared_ff}
        return out


@dataclass(frozen=True)
class TorisunLayer:
    attention: AttentionSizes
    mlp: Optional[FeedForwardSizes] = None
    type: str = "attention"


@dataclass(frozen=True)
class TorisunConfig:
    architecture: str
    vocab_size: int
    hidden_size: int
    norm_eps: float
    layers: Tuple[TorisunLayer, ...]
    max_position_embeddings: int = 0
    eos_token_id: Optional[int] = None

    # ---------------------------------------------------------------- parsing
    @classmethod
    def from_dict(cls, data: Mapping[str, Any]) -> "TorisunConfig":
        entries = data.get("layers")
        if not isinstance(entries, (list, tuple)) or not entries:
            raise ConfigError("config.json has no layers list")
        layers: List[TorisunLayer] = []
        for i, entry in enumerate(entries):
            where = f"layers[{i}]"
            if not isinstance(entry, Mapping) or entry.get("type") not in LAYER_TYPES:
                raise ConfigError(f"{where}.type must be one of {', '.join(LAYER_TYPES)}, got "
                                  f"{entry.get('type') if isinstance(entry, Mapping) else entry!r}")
            sizes = AttentionSizes.read(_mapping(entry, "mixer", where), where + ".mixer")
            if sizes.kv_from is not None:
                cls._check_source(layers, i, sizes)
            mlp = entry.get("mlp")
            layers.append(TorisunLayer(
                sizes, None if mlp is None else FeedForwardSizes.read(mlp, where + ".mlp"),
                entry["type"]))
        eos = data.get("eos_token_id")
        return cls(
            architecture=str(data.get("architecture") or "Torisun"),
            vocab_size=read_int(data, ["vocab"], minimum=1),
            hidden_size=read_int(data, ["width"], minimum=1),
            norm_eps=read_float(_mapping(data, "norm", "config.json"), ["eps"], positive=True),
            layers=tuple(layers),
            max_position_embeddings=read_int(data, ["max_position_embeddings"], default=0, minimum=0),
            eos_token_id=eos if isinstance(eos, int) and not isinstance(eos, bool) else None)

    @staticmethod
    def _check_source(layers: List[TorisunLayer], i: int, mine: AttentionSizes) -> None:
        """A layer may only read the keys and values of an earlier layer that makes its own,
        with the same heads and rotation."""
        j = mine.kv_from
        where = f"layers[{i}].mixer.kv_from: layer {j}"
        if j >= len(layers):
            raise ConfigError(f"{where} is not an earlier layer")
        source = layers[j].attention
        if source.kv_from is not None:
            raise ConfigError(f"{where} has no keys and values of its own")
        if source.shares_with() != mine.shares_with():
            raise ConfigError(f"{where} differs in heads, widths or rotation")

    def to_dict(self) -> dict:
        out: Dict[str, Any] = {
            "architecture": self.architecture, "vocab": self.vocab_size, "width": self.hidden_size,
            "norm": {"eps": self.norm_eps},
            "layers": [{"type": layer.type, "mixer": layer.attention.to_dict(),
                        "mlp": layer.mlp.to_dict() if layer.mlp is not None else None}
                       for layer in self.layers]}
        if self.max_position_embeddings:
            out["max_position_embeddings"] = self.max_position_embeddings
        if self.eos_token_id is not None:
            out["eos_token_id"] = self.eos_token_id
        return out

    # ------------------------------------------------------------ translation
    def _source_of(self, i: int) -> int:
        j = self.layers[i].attention.kv_from
        return i if j is None else j

    def _held(self, i: int) -> Tuple[int, int]:
        """(window, kept first tokens) of layer ``i``'s keys and values in the cache: what the
        layer that makes them and all layers that read them need together."""
        users = [layer.attention for k, layer in enumerate(self.layers)
                 if self._source_of(k) == self._source_of(i)]
        if any(s.window == 0 for s in users):
            return 0, 0
        return max(s.window for s in users), max(s.keep_first for s in users)

    def _norm_spec(self, name: str) -> PartSpec:
        return PartSpec("rms_norm", {"width": self.hidden_size, "eps": self.norm_eps},
                        {"weight": (name,)})

    def _attention_spec(self, i: int) -> PartSpec:
        s, p = self.layers[i].attention, f"l{i}.mix."
        position = None
        if s.rot_dims:
            rope: Dict[str, Any] = {"head_dim": s.dim, "rotary_dim": s.rot_dims, "theta": s.rot_base,
                                    "pairing": "half"}
            if s.scaling is not None:
                rope["scaling"] = dict(s.scaling.to_dict(), type="yarn")
            position = PartSpec("rope", rope)
        held_window, held_first = self._held(i)
        own = s.kv_from is None
        names = {"q_proj.weight": (p + "q",), "q_norm.weight": (p + "q.norm",), "sink": (p + "sink",),
                 "out_proj.weight": (p + "o",)}
        if own:
            names.update({"k_proj.weight": (p + "k",), "k_norm.weight": (p + "k.norm",),
                          "v_proj.weight": (p + "v",)})
        return PartSpec(
            "gqa_attention",
            {"hidden_size": self.hidden_size, "num_heads": s.heads, "num_kv_heads": s.kv_heads,
             "head_dim": s.dim, "value_dim": s.vdim, "norm_eps": self.norm_eps,
             "softmax_scale": s.scale, "qk_norm": "row", "window": s.window,
             "keep_first": s.keep_first, "cache_window": held_window,
             "cache_keep_first": held_first, "sink": True, "makes_kv": own,
             "position": position}, names)

    def _mlp_spec(self, s: FeedForwardSizes, p: str) -> PartSpec:
        H = self.hidden_size
        if s.kind == "dense":
            return PartSpec("clamped_glu",
                            {"hidden_size": H, "intermediate_size": s.ff, "limit": s.limit,
                             "alpha": GATE_SLOPE, "up_offset": UP_OFFSET,
                             "unit_in_product": True},
                            {f"{w}.weight": (p + w,) for w in ("gate", "up", "down")})
        names = {"router.weight": (p + "router",)}
        for e in range(s.experts):
            for w in ("gate", "up", "down"):
                names[f"experts.{e}.{w}.weight"] = (f"{p}e{e}.{w}",)
        if s.shared_ff:
            for w in ("gate", "up", "down"):
                names[f"shared.{w}.weight"] = (f"{p}shared.{w}",)
        return PartSpec(
            "routed_experts",
            {"hidden_size": H, "intermediate_size": s.ff, "experts": s.experts, "top": s.top,
             "scores": "sigmoid", "renormalize": True, "route_scale": s.route_scale,
             "activation": EXPERT_ACTIVATION, "shared_size": s.shared_ff}, names)

    def run_order(self) -> Tuple[LayerCall, ...]:
        """Every layer once; one with ``kv_from`` reads that layer's cache and writes none."""
        return tuple(LayerCall(i, cache=self._source_of(i), writes_cache=self._source_of(i) == i)
                     for i in range(len(self.layers)))

    def to_spec(self) -> ModelSpec:
        H = self.hidden_size
        layers = []
        for i, layer in enumerate(self.layers):
            p = f"l{i}."
            parts: Dict[str, PartSpec] = {"mixer": self._attention_spec(i),
                                          "mixer_norm": self._norm_spec(p + "norm1")}
            kind = "normed_output_no_ff"
            if layer.mlp is not None:
                parts["feed_forward"] = self._mlp_spec(layer.mlp, p + "mlp.")
                parts["feed_forward_norm"] = self._norm_spec(p + "norm2")
                kind = "normed_output"
            layers.append(LayerSpec(parts, kind))
        embedding = PartSpec("token_embedding",
                             {"vocab_size": self.vocab_size, "hidden_size": H, "norm": True,
                              "norm_eps": self.norm_eps},
                             {"weight": ("embed",), "norm.weight": ("embed.norm",)})
        lm_head = PartSpec("linear_head", {"vocab_size": self.vocab_size, "hidden_size": H,
                                           "tied": True})
        # a layer without a feed-forward may still carry its second norm; it is not read
        ignored = tuple(f"l{i}.norm2" for i, layer in enumerate(self.layers) if layer.mlp is None)
        return ModelSpec(self.architecture, H, self.vocab_size, embedding, tuple(layers),
                         self.run_order(), self._norm_spec("final.norm"), lm_head,
                         self.max_position_embeddings, ignored)
