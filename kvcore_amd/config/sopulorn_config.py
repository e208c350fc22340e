"""Typed configuration of the Sopulorn decoder, read from config.json.

The file lists the layers one by one; every size and every constant that can differ between
models comes from it:

    {"architecture": "Sopulorn", "vocab": V, "width": H, "norm": {"eps": e},
     "embedding": {"bigram": {"buckets": n, "mul_prev": a, "mul_cur": b}},
     "layers": [{"type": "attention",
                 "mixer": {"heads": h, "kv_heads": g, "dim": d, "vdim": v, "scale": s,
                           "rot": {"base": t, "dims": r}, "kv_from": j},
                 "mlp": {"kind": "dense", "ff": F, "limit": c}
                      | {"kind": "moe", "expert": {"ff": F}, "router": {"experts": E, "top": k},
                         "shared": {"ff": S}}
                      | null}, ...]}

A missing ``rot`` means that nothing is rotated, a missing ``kv_from`` that the layer has keys and
values of its own (with it the layer reads those of the earlier layer ``j``, whose sizes must equal
its own), a missing ``shared`` that no expert is shared, a missing ``bigram`` that tokens alone are
embedded.
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
class SharedCacheAttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot_dims: int  # 0: nothing is rotated
    rot_base: float
    kv_from: int | None  # the layer whose keys and values this one reads

    @classmethod
    def from_dict(cls, d: Mapping[str, Any], where: str) -> "SharedCacheAttentionConfig":
        heads, kv, dim = _require(d, "heads", int), _require(d, "kv_heads", int), _require(d, "dim", int)
        vdim = _require(d, "vdim", int)
        if min(heads, kv, dim, vdim) <= 0 or heads % kv:
            raise ConfigError(f"config.json: {where}sizes must be positive and heads a multiple of kv_heads "
                              f"(heads {heads}, kv_heads {kv}, dim {dim}, vdim {vdim})")
        dims, base = 0, 1.0
        if d.get("rot") is not None:
            rot = _mapping(d, "rot", where)
            dims, base = _require(rot, "dims", int), _require(rot, "base", float)
            if dims < 0 or dims % 2 or dims > dim or base <= 0:
                raise ConfigError(f"config.json: {where}rot.dims must be even and at most dim ({dim}), rot.base "
                                  f"positive, got {dict(rot)}")
        return cls(heads, kv, dim, vdim, _require(d, "scale", float), dims, base,
                   None if d.get("kv_from") is None else _require(d, "kv_from", int))


@dataclass(frozen=True)
class ClampedFeedForwardConfig:
    ff: int
    limit: float


@dataclass(frozen=True)
class GatedExpertsConfig:
    ff: int
    experts: int
    top: int
    shared_ff: int  # 0: no shared expert


def _feed_forward(d: Mapping[str, Any], where: str) -> ClampedFeedForwardConfig | GatedExpertsConfig:
    kind = d.get("kind")
    if kind == "dense":
        ff, limit = _require(d, "ff", int), _require(d, "limit", float)
        if ff <= 0 or not limit > 0:
            raise ConfigError(f"config.json: {where}ff and limit must be positive")
        return ClampedFeedForwardConfig(ff, limit)
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
        return GatedExpertsConfig(ff, experts, top, shared)
    raise ConfigError(f"config.json: {where}kind {kind!r} is not supported (supported: 'dense', 'moe')")


@dataclass(frozen=True)
class BigramConfig:
    buckets: int
    mul_prev: int
    mul_cur: int


@dataclass(frozen=True)
class SopulornLayerConfig:
    mixer: SharedCacheAttentionConfig
    mlp: ClampedFeedForwardConfig | GatedExpertsConfig | None


@dataclass(frozen=True)
class SopulornConfig:
    vocab: int
    width: int
    eps: float
    bigram: BigramConfig | None
    layers: tuple[SopulornLayerConfig, ...]
    max_position_embeddings: int
    eos_token_ids: tuple[int, ...] = ()

    @classmethod
    def from_dict(cls, d: Mapping[str, Any]) -> "SopulornConfig":
        vocab, width = _require(d, "vocab", int), _require(d, "width", int)
        if vocab <= 0 or width <= 0:
            raise ConfigError("config.json: vocab and width must be positive")
        eps = _require(_mapping(d, "norm", ""), "eps", float)
        bigram = None
        if d.get("embedding") is not None and _mapping(d, "embedding", "").get("bigram") is not None:
            raw = _mapping(d["embedding"], "bigram", "embedding.")
            bigram = BigramConfig(*(_require(raw, k, int) for k in ("buckets", "mul_prev", "mul_cur")))
            if bigram.buckets < 1 or min(bigram.mul_prev, bigram.mul_cur) < 0:
                raise ConfigError(f"config.json: embedding.bigram needs a positive number of buckets and multipliers "
                                  f"that are not negative, got {dict(raw)}")
        raw_layers = d.get("layers")
        if not isinstance(raw_layers, list) or not raw_layers:
            raise ConfigError("config.json: 'layers' must be a list of at least one layer")
        layers: list[SopulornLayerConfig] = []
        for i, raw in enumerate(raw_layers):
            where = f"layers[{i}]."
            if not isinstance(raw, Mapping):
                raise ConfigError(f"config.json: layers[{i}] must be an object")
            if raw.get("type") != "attention":
                raise ConfigError(f"config.json: {where}type {raw.get('type')!r} is not supported "
                                  f"(supported: 'attention')")
            mixer = SharedCacheAttentionConfig.from_dict(_mapping(raw, "mixer", where), where + "mixer.")
            if mixer.kv_from is not None:
                if not 0 <= mixer.kv_from < i or layers[mixer.kv_from].mixer.kv_from is not None:
                    raise ConfigError(f"config.json: {where}mixer.kv_from must name an earlier layer with keys and "
                                      f"values of its own, got {mixer.kv_from}")
                owner = layers[mixer.kv_from].mixer
                if (owner.kv_heads, owner.dim, owner.vdim) != (mixer.kv_heads, mixer.dim, mixer.vdim):
                    raise ConfigError(f"config.json: {where}mixer.kv_from: layer {mixer.kv_from} keeps keys and values "
                                      f"of other sizes")
            mlp = None if raw.get("mlp") is None else _feed_forward(_mapping(raw, "mlp", where), where + "mlp.")
            layers.append(SopulornLayerConfig(mixer, mlp))
        eos = d.get("eos_token_id")
        eos_ids = () if eos is None else tuple(int(e) for e in (eos if isinstance(eos, (list, tuple)) else [eos]))
        return cls(vocab, width, eps, bigram, tuple(layers), int(d.get("max_position_embeddings") or 131072), eos_ids)
