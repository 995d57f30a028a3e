"""Configuration of the Pagonex design: a list of layers, each a mixer (the gated delta rule, or latent
attention through a query latent) and, optionally, a routed feed-forward, with layer norms on the branches'
outputs and a short convolution over the residual sum in front of each branch.

``config.json`` of this design is nested: ``vocab``, ``width``, ``norm.eps``, ``canon.taps`` (the convolutions in front of
the branches), ``embedding.bigram`` (buckets, mul_prev, mul_cur), ``logit_scale`` and ``layers`` (one object per layer: ``type``
"channel_delta" or "latent_attention", the mixer's sizes in ``mixer``, the feed-forward in ``mlp`` or null).  Every size and
constant is read here and nowhere else; a key this reader does not know is refused with its name.  What the
file leaves out is off: no ``mask``, every earlier key visible; no ``rot``, no rotation; no ``rot.scaling``, frequencies
as they are; no ``shared``, no shared expert; no ``logit_scale``, logits as they are.

Two sizes are in no key of the file: the narrow middles of a delta layer's decay and gate projections.  They are the
first dimensions of ``l<i>.mix.a1`` and ``l<i>.mix.g1`` and are taken from there when a model folder is opened
(``with_tensor_shapes``); a configuration made by hand may give them as ``decay_rank`` and ``gate_rank``
(random-weights mode falls back to DEFAULT_RANK).
"""
from __future__ import annotations

import math
from dataclasses import dataclass, replace
from typing import Any, Dict, Optional, Tuple, Union

from .base import ConfigError, ModelConfig, special_tokens_from
from .fovosun import _obj
from .kuvonex import _num, _only
from .pazatar import YARN_KEYS, RotConfig

LAYER_TYPES = ("channel_delta", "latent_attention")
MLP_KINDS = ("moe",)
DEFAULT_RANK = 16


@dataclass(frozen=True)
class DeltaMixerConfig:
    """The gated delta rule: ``heads`` states of ``dim`` key and ``vdim`` value channels over ``kv_heads`` query/key heads."""

    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int                   # taps of the convolutions behind q, k and v
    decay_rank: Optional[int] = None
    gate_rank: Optional[int] = None

    @classmethod
    def from_dict(cls, d: Dict[str, Any], where: str) -> "DeltaMixerConfig":
        _only(d, ("heads", "kv_heads", "dim", "vdim", "conv", "decay_rank", "gate_rank"), where)
        heads, dim = _num(d, "heads", where), _num(d, "dim", where)
        return cls(heads=heads, kv_heads=_num(d, "kv_heads", where, int, heads), dim=dim, vdim=_num(d, "vdim", where, int, dim),
                   conv=_num(d, "conv", where), decay_rank=None if d.get("decay_rank") is None else _num(d, "decay_rank", where),
                   gate_rank=None if d.get("gate_rank") is None else _num(d, "gate_rank", where))

    def to_dict(self) -> Dict[str, Any]:
        out: Dict[str, Any] = {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim, "conv": self.conv}
        if self.decay_rank is not None:
            out["decay_rank"] = self.decay_rank
        if self.gate_rank is not None:
            out["gate_rank"] = self.gate_rank
        return out


@dataclass(frozen=True)
class QueryLatentMixerConfig:
    """Latent attention whose queries come through a latent of their own."""

    heads: int
    dim: int                    # unrotated width of a query / key head
    rot_dim: int                # rotated width
    vdim: int                   # width of a value head
    q_rank: int                 # width of the queries' latent
    kv_rank: int                # width of the keys' and values' latent
    scale: float                # of the scores
    window: Optional[int] = None         # mask.size: a query sees itself and the window - 1 tokens before it
    rot: Optional[RotConfig] = None
    kv_from: Optional[int] = None        # the layer whose latent and rotated key part this one attends over

    @classmethod
    def from_dict(cls, d: Dict[str, Any], where: str) -> "QueryLatentMixerConfig":
        _only(d, ("heads", "dim", "rot_dim", "vdim", "q_rank", "kv_rank", "scale", "mask", "rot", "kv_from"), where)
        rot, mask = _obj(d, "rot", where), _obj(d, "mask", where)
        if mask is not None:
            _only(mask, ("size",), where + ".mask")
        dim, rot_dim = _num(d, "dim", where), _num(d, "rot_dim", where)
        if rot is not None and "dims" not in rot:
            rot = {**rot, "dims": rot_dim}
        return cls(heads=_num(d, "heads", where), dim=dim, rot_dim=rot_dim, vdim=_num(d, "vdim", where, int, dim),
                   q_rank=_num(d, "q_rank", where), kv_rank=_num(d, "kv_rank", where),
                   scale=_num(d, "scale", where, float, 1.0 / math.sqrt(dim + rot_dim)),
                   window=None if mask is None else _num(mask, "size", where + ".mask"),
                   rot=None if rot is None else RotConfig.from_dict(rot, where + ".rot", YARN_KEYS),
                   kv_from=None if d.get("kv_from") is None else _num(d, "kv_from", where))

    def to_dict(self) -> Dict[str, Any]:
        out: Dict[str, Any] = {"heads": self.heads, "dim": self.dim, "rot_dim": self.rot_dim, "vdim": self.vdim, "q_rank": self.q_rank,
                               "kv_rank": self.kv_rank, "scale": self.scale}
        if self.window is not None:
            out["mask"] = {"size": self.window}
        if self.rot is not None:
            out["rot"] = self.rot.to_dict()
        if self.kv_from is not None:
            out["kv_from"] = self.kv_from
        return out


@dataclass(frozen=True)
class ScaledMoeConfig:
    """``experts`` clamped gated units of which a token uses ``top``, their weights times ``scale``, and a shared one
    (``shared_ff`` wide, ``shared_limit``; 0: none) that every token uses."""

    experts: int
    top: int
    ff: int
    limit: float
    scale: float = 1.0
    shared_ff: int = 0
    shared_limit: float = 0.0

    @classmethod
    def from_dict(cls, d: Dict[str, Any], where: str) -> "ScaledMoeConfig":
        if d.get("kind") not in MLP_KINDS:
            raise ConfigError(f"{where}: kind {d.get('kind')!r} is not known ({', '.join(MLP_KINDS)})")
        _only(d, ("kind", "expert", "router", "shared"), where)
        ex, ro, sh = _obj(d, "expert", where, True), _obj(d, "router", where, True), _obj(d, "shared", where)
        _only(ex, ("ff", "limit"), where + ".expert")
        _only(ro, ("experts", "top", "scale"), where + ".router")
        if sh is not None:
            _only(sh, ("ff", "limit"), where + ".shared")
        return cls(experts=_num(ro, "experts", where + ".router"), top=_num(ro, "top", where + ".router"),
                   ff=_num(ex, "ff", where + ".expert"), limit=_num(ex, "limit", where + ".expert", float),
                   scale=_num(ro, "scale", where + ".router", float, 1.0),
                   shared_ff=0 if sh is None else _num(sh, "ff", where + ".shared"),
                   shared_limit=0.0 if sh is None else _num(sh, "limit", where + ".shared", float))

    def to_dict(self) -> Dict[str, Any]:
        out: Dict[str, Any] = {"kind": "moe", "expert": {"ff": self.ff, "limit": self.limit},
                               "router": {"experts": self.experts, "top": self.top, "scale": self.scale}}
        if self.shared_ff:
            out["shared"] = {"ff": self.shared_ff, "limit": self.shared_limit}
        return out


@dataclass(frozen=True)
class PagonexLayerConfig:
    type: str
    mixer: Union[DeltaMixerConfig, QueryLatentMixerConfig]
    mlp: Optional[ScaledMoeConfig] = None

    @classmethod
    def from_dict(cls, d: Dict[str, Any], where: str) -> "PagonexLayerConfig":
        if not isinstance(d, dict):
            raise ConfigError(f"{where} must be an object")
        _only(d, ("type", "mixer", "mlp"), where)
        kind = d.get("type")
        if kind not in LAYER_TYPES:
            raise ConfigError(f"{where}: type {kind!r} is not known ({', '.join(LAYER_TYPES)})")
        m, mlp = _obj(d, "mixer", where, True), _obj(d, "mlp", where)
        mixer = (DeltaMixerConfig if kind == "channel_delta" else QueryLatentMixerConfig).from_dict(m, where + ".mixer")
        return cls(type=kind, mixer=mixer, mlp=None if mlp is None else ScaledMoeConfig.from_dict(mlp, where + ".mlp"))

    def to_dict(self) -> Dict[str, Any]:
        return {"type": self.type, "mixer": self.mixer.to_dict(), "mlp": None if self.mlp is None else self.mlp.to_dict()}


@dataclass(frozen=True)
class BigramConfig:
    buckets: int
    mul_prev: int
    mul_cur: int


@dataclass
class PagonexConfig(ModelConfig):
    vocab_size: int = 0
    width: int = 0
    norm_eps: float = 1e-5
    canon_taps: int = 1
    bigram: Optional[BigramConfig] = None
    logit_scale: float = 1.0
    layers: Tuple[PagonexLayerConfig, ...] = ()

    @classmethod
    def from_dict(cls, d: Dict[str, Any]) -> "PagonexConfig":
        _only(d, ("architecture", "architectures", "canon", "embedding", "layers", "logit_scale", "norm", "vocab", "width",
                  "eos_token_id", "bos_token_id"), "config.json")
        norm, canon, emb = _obj(d, "norm", "config.json", True), _obj(d, "canon", "config.json", True), _obj(d, "embedding", "config.json")
        _only(norm, ("eps",), "norm")
        _only(canon, ("taps",), "canon")
        bigram = None
        if emb is not None:
            _only(emb, ("bigram",), "embedding")
            big = _obj(emb, "bigram", "embedding")
            if big is not None:
                _only(big, ("buckets", "mul_prev", "mul_cur"), "embedding.bigram")
                bigram = BigramConfig(*(_num(big, k, "embedding.bigram") for k in ("buckets", "mul_prev", "mul_cur")))
        layers = d.get("layers")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("config.json: 'layers' must be a list of layers")
        from .base import architecture_name

        return cls(architecture=architecture_name(d), vocab_size=_num(d, "vocab", "config.json"), width=_num(d, "width", "config.json"),
                   norm_eps=_num(norm, "eps", "norm", float), canon_taps=_num(canon, "taps", "canon"), bigram=bigram,
                   logit_scale=_num(d, "logit_scale", "config.json", float, 1.0),
                   layers=tuple(PagonexLayerConfig.from_dict(x, f"layers[{i}]") for i, x in enumerate(layers)),
                   **special_tokens_from(d))

    def to_dict(self) -> Dict[str, Any]:
        out: Dict[str, Any] = {"architecture": self.architecture or "Pagonex", "vocab": self.vocab_size, "width": self.width,
                               "norm": {"eps": self.norm_eps}, "canon": {"taps": self.canon_taps}, "logit_scale": self.logit_scale,
                               "layers": [x.to_dict() for x in self.layers]}
        if self.bigram is not None:
            b = self.bigram
            out["embedding"] = {"bigram": {"buckets": b.buckets, "mul_prev": b.mul_prev, "mul_cur": b.mul_cur}}
        out.update(self.special_tokens_dict())
        return out

    def with_tensor_shapes(self, available: Dict[str, tuple]) -> "PagonexConfig":
        layers = []
        for i, layer in enumerate(self.layers):
            if layer.type == "channel_delta":
                ranks = {}
                for key, name in (("decay_rank", "a1"), ("gate_rank", "g1")):
                    found = available.get(f"l{i}.mix.{name}")
                    if found is not None and len(found[0]) == 2:
                        ranks[key] = int(found[0][0])
                layer = replace(layer, mixer=replace(layer.mixer, **ranks))
            layers.append(layer)
        return self.replace(layers=tuple(layers))

    def validate(self) -> None:
        if self.vocab_size < 1 or self.width < 1 or not self.norm_eps > 0 or self.canon_taps < 1:
            raise ConfigError("vocab, width and canon.taps must be positive and norm.eps above zero")
        if self.bigram is not None and self.bigram.buckets < 1:
            raise ConfigError("embedding.bigram: buckets must be positive")
        for i, layer in enumerate(self.layers):
            where, m = f"layers[{i}].mixer", layer.mixer
            if layer.type == "channel_delta":
                if min(m.heads, m.kv_heads, m.dim, m.vdim, m.conv) < 1 or min(m.decay_rank or 1, m.gate_rank or 1) < 1 or m.heads % m.kv_heads:
                    raise ConfigError(f"{where}: heads, kv_heads, dim, vdim and conv must be positive and kv_heads divide heads")
            else:
                if min(m.heads, m.dim, m.rot_dim, m.vdim, m.q_rank, m.kv_rank) < 1:
                    raise ConfigError(f"{where}: heads, dim, rot_dim, vdim, q_rank and kv_rank must be positive")
                if m.window is not None and m.window < 1:
                    raise ConfigError(f"{where}.mask: size must be positive")
                if m.rot is not None:
                    if m.rot.dims % 2 or not 2 <= m.rot.dims <= m.rot_dim or not m.rot.base > 1:
                        raise ConfigError(f"{where}.rot: dims must be even and lie in 2..rot_dim {m.rot_dim}, base above 1")
                    if m.rot.scaling is not None and not all(v > 0 for v in m.rot.scaling_dict().values()):
                        raise ConfigError(f"{where}.rot.scaling: {', '.join(YARN_KEYS)} must be positive")
                if m.kv_from is not None:
                    if not 0 <= m.kv_from < i or self.layers[m.kv_from].type != "latent_attention":
                        raise ConfigError(f"{where}: kv_from {m.kv_from} must name an earlier latent attention layer")
                    src = self.layers[m.kv_from].mixer
                    if src.kv_from is not None:
                        raise ConfigError(f"{where}: kv_from names layer {m.kv_from}, which keeps no latent of its own")
                    if (src.kv_rank, src.rot_dim, src.rot) != (m.kv_rank, m.rot_dim, m.rot):
                        raise ConfigError(f"{where}: kv_rank, rot_dim and rot must equal those of layer {m.kv_from}")
            f = layer.mlp
            if f is not None:
                where = f"layers[{i}].mlp"
                if f.ff < 1 or not f.limit > 0 or not 1 <= f.top <= f.experts:
                    raise ConfigError(f"{where}: expert.ff and expert.limit must be positive and 1 <= top <= experts")
                if f.shared_ff < 0 or (f.shared_ff and not f.shared_limit > 0):
                    raise ConfigError(f"{where}.shared: ff and limit must be positive")
