"""Configuration of the Rigodra design: a list of layers, each a mixer (grouped-query attention or latent attention)
and, optionally, a feed-forward without a gate (dense or routed), with a layer norm of the whole sum behind each branch.

``config.json`` of this design is nested: ``vocab``, ``width``, ``norm.eps``, ``postln_alpha`` (what the residual sum is
multiplied by before a branch is added) and ``layers`` (one object per layer: ``type`` "attention" or "latent_attention",
the mixer's sizes in ``mixer``, the feed-forward in ``mlp`` or null).  Every size and constant is read here and nowhere
else; a key this reader does not know is refused with its name.  What the file leaves out is off: no ``mask``, every
earlier key visible; no ``mask.keep_first``, no kept tokens; no ``rot``, no rotation; no ``v_mix``, values as projected; no
``shared``, no shared expert; no ``router.groups`` and no ``router.identity``, none.
"""
from __future__ import annotations

import math
from dataclasses import dataclass
from typing import Any, Dict, Optional, Tuple, Union

from .base import ConfigError, ModelConfig, architecture_name, special_tokens_from
from .fovosun import _obj
from .kuvonex import _num, _only
from .pagonex import QueryLatentMixerConfig
from .pazatar import RotConfig

LAYER_TYPES = ("attention", "latent_attention")
MLP_KINDS = ("dense", "moe")


@dataclass(frozen=True)
class SharedValueMixerConfig:
    """Grouped-query attention behind a window that may keep the sequence's first tokens in sight."""

    heads: int
    kv_heads: int
    dim: int                    # width of a query / key head
    vdim: int                   # width of a value head
    scale: float                # of the scores
    window: Optional[int] = None         # mask.size: a query sees itself and the window - 1 tokens before it
    keep_first: int = 0                  # mask.keep_first: and the sequence's first so many
    rot: Optional[RotConfig] = None
    v_mix: bool = False                  # values mixed with those of the first layer that says so

    @classmethod
    def from_dict(cls, d: Dict[str, Any], where: str) -> "SharedValueMixerConfig":
        _only(d, ("heads", "kv_heads", "dim", "vdim", "scale", "mask", "rot", "v_mix"), where)
        rot, mask = _obj(d, "rot", where), _obj(d, "mask", where)
        if mask is not None:
            _only(mask, ("size", "keep_first"), where + ".mask")
        if not isinstance(d.get("v_mix", False), (bool, type(None))):
            raise ConfigError(f"{where}: 'v_mix' must be true or false (got {d['v_mix']!r})")
        heads, dim = _num(d, "heads", where), _num(d, "dim", where)
        if rot is not None and "dims" not in rot:
            rot = {**rot, "dims": dim}
        return cls(heads=heads, kv_heads=_num(d, "kv_heads", where, int, heads), dim=dim, vdim=_num(d, "vdim", where, int, dim),
                   scale=_num(d, "scale", where, float, 1.0 / math.sqrt(dim)),
                   window=None if mask is None else _num(mask, "size", where + ".mask"),
                   keep_first=0 if mask is None or mask.get("keep_first") is None else _num(mask, "keep_first", where + ".mask"),
                   rot=None if rot is None else RotConfig.from_dict(rot, where + ".rot", ()), v_mix=bool(d.get("v_mix")))

    def to_dict(self) -> Dict[str, Any]:
        out: Dict[str, Any] = {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim, "scale": self.scale}
        if self.window is not None:
            out["mask"] = {"size": self.window}
            if self.keep_first:
                out["mask"]["keep_first"] = self.keep_first
        if self.rot is not None:
            out["rot"] = self.rot.to_dict()
        if self.v_mix:
            out["v_mix"] = True
        return out


@dataclass(frozen=True)
class UngatedMlpConfig:
    """A feed-forward without a gate: dense (``ff`` wide), or ``experts`` of them of which a token uses ``top``, beside
    ``identity`` experts that return the input, chosen from the ``keep`` best of ``groups`` groups, and a shared one."""

    kind: str
    ff: int
    experts: int = 0
    top: int = 0
    groups: int = 1
    keep: int = 1
    identity: int = 0
    shared_ff: int = 0          # 0: no shared expert

    @classmethod
    def from_dict(cls, d: Dict[str, Any], where: str) -> "UngatedMlpConfig":
        kind = d.get("kind")
        if kind not in MLP_KINDS:
            raise ConfigError(f"{where}: kind {kind!r} is not known ({', '.join(MLP_KINDS)})")
        if kind == "dense":
            _only(d, ("kind", "ff"), where)
            return cls(kind=kind, ff=_num(d, "ff", where))
        _only(d, ("kind", "expert", "router", "shared"), where)
        ex, ro, sh = _obj(d, "expert", where, True), _obj(d, "router", where, True), _obj(d, "shared", where)
        _only(ex, ("ff",), where + ".expert")
        _only(ro, ("experts", "top", "groups", "identity"), where + ".router")
        gr = _obj(ro, "groups", where + ".router")
        if gr is not None:
            _only(gr, ("count", "keep"), where + ".router.groups")
        if sh is not None:
            _only(sh, ("ff",), where + ".shared")
        return cls(kind=kind, ff=_num(ex, "ff", where + ".expert"), experts=_num(ro, "experts", where + ".router"),
                   top=_num(ro, "top", where + ".router"), groups=1 if gr is None else _num(gr, "count", where + ".router.groups"),
                   keep=1 if gr is None else _num(gr, "keep", where + ".router.groups"),
                   identity=0 if ro.get("identity") is None else _num(ro, "identity", where + ".router"),
                   shared_ff=0 if sh is None else _num(sh, "ff", where + ".shared"))

    def to_dict(self) -> Dict[str, Any]:
        if self.kind == "dense":
            return {"kind": "dense", "ff": self.ff}
        router: Dict[str, Any] = {"experts": self.experts, "top": self.top}
        if (self.groups, self.keep) != (1, 1):
            router["groups"] = {"count": self.groups, "keep": self.keep}
        if self.identity:
            router["identity"] = self.identity
        out: Dict[str, Any] = {"kind": "moe", "expert": {"ff": self.ff}, "router": router}
        if self.shared_ff:
            out["shared"] = {"ff": self.shared_ff}
        return out


@dataclass(frozen=True)
class RigodraLayerConfig:
    type: str
    mixer: Union[SharedValueMixerConfig, QueryLatentMixerConfig]
    mlp: Optional[UngatedMlpConfig] = None

    @classmethod
    def from_dict(cls, d: Dict[str, Any], where: str) -> "RigodraLayerConfig":
        if not isinstance(d, dict):
            raise ConfigError(f"{where} must be an object")
        _only(d, ("type", "mixer", "mlp"), where)
        kind = d.get("type")
        if kind not in LAYER_TYPES:
            raise ConfigError(f"{where}: type {kind!r} is not known ({', '.join(LAYER_TYPES)})")
        m, mlp = _obj(d, "mixer", where, True), _obj(d, "mlp", where)
        if kind == "latent_attention":
            for key, inner in (("kv_from", m), ("scaling", m.get("rot") if isinstance(m.get("rot"), dict) else {})):
                if inner.get(key) is not None:
                    raise ConfigError(f"{where}.mixer: unknown key(s) {key}")
        mixer = (SharedValueMixerConfig if kind == "attention" else QueryLatentMixerConfig).from_dict(m, where + ".mixer")
        return cls(type=kind, mixer=mixer, mlp=None if mlp is None else UngatedMlpConfig.from_dict(mlp, where + ".mlp"))

    def to_dict(self) -> Dict[str, Any]:
        return {"type": self.type, "mixer": self.mixer.to_dict(), "mlp": None if self.mlp is None else self.mlp.to_dict()}


@dataclass
class RigodraConfig(ModelConfig):
    vocab_size: int = 0
    width: int = 0
    norm_eps: float = 1e-5
    alpha: float = 1.0
    layers: Tuple[RigodraLayerConfig, ...] = ()

    @classmethod
    def from_dict(cls, d: Dict[str, Any]) -> "RigodraConfig":
        _only(d, ("architecture", "architectures", "layers", "norm", "postln_alpha", "vocab", "width", "eos_token_id", "bos_token_id"),
              "config.json")
        norm = _obj(d, "norm", "config.json", True)
        _only(norm, ("eps",), "norm")
        layers = d.get("layers")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("config.json: 'layers' must be a list of layers")
        return cls(architecture=architecture_name(d), vocab_size=_num(d, "vocab", "config.json"), width=_num(d, "width", "config.json"),
                   norm_eps=_num(norm, "eps", "norm", float), alpha=_num(d, "postln_alpha", "config.json", float),
                   layers=tuple(RigodraLayerConfig.from_dict(x, f"layers[{i}]") for i, x in enumerate(layers)), **special_tokens_from(d))

    def to_dict(self) -> Dict[str, Any]:
        out: Dict[str, Any] = {"architecture": self.architecture or "Rigodra", "vocab": self.vocab_size, "width": self.width,
                               "norm": {"eps": self.norm_eps}, "postln_alpha": self.alpha, "layers": [x.to_dict() for x in self.layers]}
        out.update(self.special_tokens_dict())
        return out

    def validate(self) -> None:
        if self.vocab_size < 1 or self.width < 1 or not self.norm_eps > 0 or not math.isfinite(self.alpha):
            raise ConfigError("vocab and width must be positive, norm.eps above zero and postln_alpha a finite number")
        shared_values = None            # (layer, heads, width) of the values that later layers mix in
        for i, layer in enumerate(self.layers):
            where, m = f"layers[{i}].mixer", layer.mixer
            if layer.type == "attention":
                if min(m.heads, m.kv_heads, m.dim, m.vdim) < 1 or m.heads % m.kv_heads or m.dim % 2:
                    raise ConfigError(f"{where}: heads, kv_heads, dim and vdim must be positive, kv_heads divide heads and dim be even")
                if m.keep_first < 0 or (m.keep_first and m.window is None):
                    raise ConfigError(f"{where}.mask: keep_first must not be negative and comes with a size")
                widest = m.dim
                if m.v_mix:
                    if shared_values is None:
                        shared_values = (i, m.kv_heads, m.vdim)
                    elif shared_values[1:] != (m.kv_heads, m.vdim):
                        raise ConfigError(f"{where}: kv_heads and vdim must equal those of layer {shared_values[0]}, whose values it mixes in")
            else:
                if min(m.heads, m.dim, m.rot_dim, m.vdim, m.q_rank, m.kv_rank) < 1:
                    raise ConfigError(f"{where}: heads, dim, rot_dim, vdim, q_rank and kv_rank must be positive")
                widest = m.rot_dim
            if m.window is not None and m.window < 1:
                raise ConfigError(f"{where}.mask: size must be positive")
            if m.rot is not None and (m.rot.dims % 2 or not 2 <= m.rot.dims <= widest or not m.rot.base > 0):
                raise ConfigError(f"{where}.rot: dims must be even and lie in 2..{widest}, base above 0")
            f = layer.mlp
            if f is None:
                continue
            where = f"layers[{i}].mlp"
            if f.ff < 1 or f.shared_ff < 0:
                raise ConfigError(f"{where}: ff must be positive")
            if f.kind == "moe":
                scored = f.experts + f.identity
                if f.experts < 1 or f.identity < 0 or not 1 <= f.keep <= f.groups or scored % f.groups:
                    raise ConfigError(f"{where}: {f.groups} groups (keep {f.keep}) do not divide {f.experts} experts and {f.identity} identity experts")
                if not 1 <= f.top <= f.keep * (scored // f.groups):
                    raise ConfigError(f"{where}: top {f.top} must lie in 1..{f.keep * (scored // f.groups)}, the experts of the kept groups")
