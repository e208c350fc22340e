"""Typed configuration of the Zikupel decoder, read from config.json.

The file lists the layers one by one; every size and every constant that can differ between
models comes from it:

    {"architecture": "Zikupel", "vocab": V, "width": H, "norm": {"eps": e},
     "layers": [{"type": "attention",
                 "mixer": {"heads": h, "kv_heads": g, "dim": d, "vdim": d, "scale": s, "softcap": c,
                           "rot": {"base": t, "dims": r,
                                   "scaling": {"factor": f, "original": n, "fast": a, "slow": b}}},
                 "mlp": {"kind": "dense", "ff": F}
                      | {"kind": "moe", "expert": {"ff": F}, "router": {"experts": E, "top": k},
                         "shared": {"ff": S}}
                      | null},
                {"type": "lightning",
                 "mixer": {"heads": h, "dim": d, "vdim": v, "decay": [one number a head]},
                 "mlp": ...}, ...]}

A missing ``rot`` means that nothing is rotated, a missing ``rot.scaling`` the plain frequencies, a
missing ``softcap`` that scores are not capped, a missing ``shared`` that no expert is shared.  An
attention layer's values are its keys, so its ``vdim`` (which may be left out) equals its ``dim``.
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Mapping

from .model_config import ConfigError, _require


def _mapping(d: Mapping[str, Any], key: str, where: str) -> Mapping[str, Any]:
    value = d.get(key)
    if not isinstance(value, Mapping):
        raise ConfigError(f"config.json: {where}{key!r} must be an object")
    return value


@dataclass(frozen=True)
class YarnConfig:
    factor: float
    original: float
    fast: float
    slow: float

    @classmethod
    def from_dict(cls, d: Mapping[str, Any], where: str) -> "YarnConfig":
        out = cls(*(_require(d, k, float) for k in ("factor", "original", "fast", "slow")))
        if min(out.factor, out.original, out.fast, out.slow) <= 0:
            raise ConfigError(f"config.json: {where}factor, original, fast and slow must be positive, got {dict(d)}")
        return out

    def as_scaling(self) -> dict:
        return {"rope_type": "yarn", "factor": self.factor, "original": self.original, "fast": self.fast,
                "slow": self.slow}


@dataclass(frozen=True)
class KeyValueAttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    scale: float
    softcap: float  # 0: none
    rot_dims: int  # 0: nothing is rotated
    rot_base: float
    yarn: YarnConfig | None

    @classmethod
    def from_dict(cls, d: Mapping[str, Any], where: str) -> "KeyValueAttentionConfig":
        heads, kv, dim = _require(d, "heads", int), _require(d, "kv_heads", int), _require(d, "dim", int)
        if min(heads, kv, dim) <= 0 or heads % kv:
            raise ConfigError(f"config.json: {where}sizes must be positive and heads a multiple of kv_heads "
                              f"(heads {heads}, kv_heads {kv}, dim {dim})")
        if d.get("vdim") is not None and _require(d, "vdim", int) != dim:
            raise ConfigError(f"config.json: {where}vdim: the values are the keys, so vdim must equal dim "
                              f"({dim}), got {d['vdim']}")
        dims, base, yarn = 0, 1.0, None
        if d.get("rot") is not None:
            rot = _mapping(d, "rot", where)
            dims, base = _require(rot, "dims", int), _require(rot, "base", float)
            if dims < 0 or dims % 2 or dims > dim or base <= 0:
                raise ConfigError(f"config.json: {where}rot.dims must be even and at most dim ({dim}), rot.base "
                                  f"positive, got {dict(rot)}")
            if rot.get("scaling") is not None:
                yarn = YarnConfig.from_dict(_mapping(rot, "scaling", where + "rot."), where + "rot.scaling.")
                if base == 1.0:
                    raise ConfigError(f"config.json: {where}rot.scaling needs a rot.base other than one")
        softcap = 0.0 if d.get("softcap") is None else _require(d, "softcap", float)
        if softcap < 0 or (d.get("softcap") is not None and softcap == 0):
            raise ConfigError(f"config.json: {where}softcap must be positive when given")
        return cls(heads, kv, dim, _require(d, "scale", float), softcap, dims, base, yarn)


@dataclass(frozen=True)
class LightningConfig:
    heads: int
    dim: int
    vdim: int
    decay: tuple[float, ...]

    @classmethod
    def from_dict(cls, d: Mapping[str, Any], where: str) -> "LightningConfig":
        heads, dim, vdim = (_require(d, k, int) for k in ("heads", "dim", "vdim"))
        if min(heads, dim, vdim) <= 0:
            raise ConfigError(f"config.json: {where}heads, dim and vdim must be positive")
        decay = d.get("decay")
        if not isinstance(decay, (list, tuple)) or len(decay) != heads \
                or not all(isinstance(v, (int, float)) and not isinstance(v, bool) for v in decay):
            raise ConfigError(f"config.json: {where}decay must be a list of one number a head ({heads})")
        return cls(heads, dim, vdim, tuple(float(v) for v in decay))


@dataclass(frozen=True)
class DenseConfig:
    ff: int


@dataclass(frozen=True)
class SquaredExpertsConfig:
    ff: int
    experts: int
    top: int
    shared_ff: int  # 0: no shared expert


def _feed_forward(d: Mapping[str, Any], where: str) -> DenseConfig | SquaredExpertsConfig:
    kind = d.get("kind")
    if kind == "dense":
        ff = _require(d, "ff", int)
        if ff <= 0:
            raise ConfigError(f"config.json: {where}ff must be positive")
        return DenseConfig(ff)
    if kind == "moe":
        ff = _require(_mapping(d, "expert", where), "ff", int)
        router = _mapping(d, "router", where)
        experts, top = _require(router, "experts", int), _require(router, "top", int)
        shared = 0
        if d.get("shared") is not None:
            shared = _require(_mapping(d, "shared", where), "ff", int)
            if shared <= 0:
                raise ConfigError(f"config.json: {where}shared.ff must be positive")
        if ff <= 0 or experts <= 0 or not 0 < top <= experts:
            raise ConfigError(f"config.json: {where}{top} of {experts} experts of {ff} units: sizes do not fit")
        return SquaredExpertsConfig(ff, experts, top, shared)
    raise ConfigError(f"config.json: {where}kind {kind!r} is not supported (supported: 'dense', 'moe')")


MIXERS = {"attention": KeyValueAttentionConfig, "lightning": LightningConfig}


@dataclass(frozen=True)
class ZikupelLayerConfig:
    mixer: KeyValueAttentionConfig | LightningConfig
    mlp: DenseConfig | SquaredExpertsConfig | None


@dataclass(frozen=True)
class ZikupelConfig:
    vocab: int
    width: int
    eps: float
    layers: tuple[ZikupelLayerConfig, ...]
    max_position_embeddings: int
    eos_token_ids: tuple[int, ...] = ()

    @classmethod
    def from_dict(cls, d: Mapping[str, Any]) -> "ZikupelConfig":
        vocab, width = _require(d, "vocab", int), _require(d, "width", int)
        if vocab <= 0 or width <= 0:
            raise ConfigError("config.json: vocab and width must be positive")
        eps = _require(_mapping(d, "norm", ""), "eps", float)
        raw_layers = d.get("layers")
        if not isinstance(raw_layers, list) or not raw_layers:
            raise ConfigError("config.json: 'layers' must be a list of at least one layer")
        layers: list[ZikupelLayerConfig] = []
        for i, raw in enumerate(raw_layers):
            where = f"layers[{i}]."
            if not isinstance(raw, Mapping):
                raise ConfigError(f"config.json: layers[{i}] must be an object")
            kind = MIXERS.get(raw.get("type"))
            if kind is None:
                raise ConfigError(f"config.json: {where}type {raw.get('type')!r} is not supported "
                                  f"(supported: {sorted(MIXERS)})")
            mixer = kind.from_dict(_mapping(raw, "mixer", where), where + "mixer.")
            mlp = None if raw.get("mlp") is None else _feed_forward(_mapping(raw, "mlp", where), where + "mlp.")
            layers.append(ZikupelLayerConfig(mixer, mlp))
        eos = d.get("eos_token_id")
        eos_ids = () if eos is None else tuple(int(e) for e in (eos if isinstance(eos, (list, tuple)) else [eos]))
        return cls(vocab, width, eps, tuple(layers), int(d.get("max_position_embeddings") or 131072), eos_ids)
