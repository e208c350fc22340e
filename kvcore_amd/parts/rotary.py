"""Rotary position encoding: a frequency table, optionally rescaled, and per-step
cos/sin tables computed once in float32 and shared by every layer.

Reference: kvcore/model/layer/rotary_embedding.py:52-98: ``inv_freq[j] = base **
(-2j/d)``, angles ``position * inv_freq`` in float32, element ``j`` paired with
``j + d/2``.  The reference rounds cos and sin to the model dtype before the multiply
(:95-96); here the rotation itself is float32 and only its result is rounded.  The
``llama3`` frequency rescaling has no counterpart in the reference.
"""

from __future__ import annotations

import math

import torch

from kvcore_amd.ops import library as ops

from .base import PositionEncoding, RotaryTables, register_position_encoding


def yarn_ramp(rot_dim: int, theta: float, original: float, fast: float, slow: float) -> torch.Tensor:
    """float64 ``[rot_dim / 2]``: 0 for the pairs that turn ``fast`` times or more over ``original`` positions
    (their frequency stays), 1 for those that turn ``slow`` times or less, rising linearly over the pairs
    between."""
    def pair(turns: float) -> float:
        return rot_dim * math.log(original / (2.0 * math.pi * turns)) / (2.0 * math.log(theta))

    low = max(math.floor(pair(fast)), 0)
    high = min(math.ceil(pair(slow)), rot_dim - 1)
    index = torch.arange(rot_dim // 2, dtype=torch.float64)
    return ((index - low) / max(high - low, 0.001)).clamp(0.0, 1.0)


def rotary_table_scale(scaling: dict | None) -> float:
    """What cosine and sine are multiplied by: ``0.1 ln(factor) + 1`` under YaRN, else one."""
    if scaling and scaling.get("rope_type") == "yarn":
        return 0.1 * math.log(float(scaling["factor"])) + 1.0
    return 1.0


def rotary_inv_freq(rot_dim: int, theta: float, scaling: dict | None = None) -> torch.Tensor:
    """float32 ``[rot_dim / 2]``.  ``scaling`` None or ``{"rope_type": "default"}`` is the
    plain table; ``{"rope_type": "llama3", factor, low_freq_factor, high_freq_factor,
    original_max_position_embeddings}`` divides long wavelengths by ``factor``, keeps
    short ones and blends linearly (in original_length / wavelength) between the two;
    ``{"rope_type": "yarn", factor, original, fast, slow}`` divides the frequencies by ``factor``
    as far as ``yarn_ramp`` says."""
    exponents = torch.arange(0, rot_dim, 2, dtype=torch.float64) / rot_dim
    inv_freq = 1.0 / (torch.tensor(float(theta), dtype=torch.float64) ** exponents)
    rope_type = "default" if not scaling else scaling.get("rope_type", "default")
    if rope_type == "llama3":
        factor = float(scaling["factor"])
        low = float(scaling["low_freq_factor"])
        high = float(scaling["high_freq_factor"])
        orig = float(scaling["original_max_position_embeddings"])
        wavelen = 2.0 * math.pi / inv_freq
        smooth = ((orig / wavelen - low) / (high - low)).clamp(0.0, 1.0)
        blended = (1.0 - smooth) * inv_freq / factor + smooth * inv_freq
        inv_freq = torch.where(wavelen < orig / high, inv_freq,
                               torch.where(wavelen > orig / low, inv_freq / factor, blended))
    elif rope_type == "yarn":
        missing = [k for k in ("factor", "original", "fast", "slow") if k not in scaling]
        if missing:
            raise ValueError(f"rope_type 'yarn' needs {missing}")
        ramp = yarn_ramp(rot_dim, float(theta), *(float(scaling[k]) for k in ("original", "fast", "slow")))
        inv_freq = inv_freq / float(scaling["factor"]) * ramp + inv_freq * (1.0 - ramp)
    elif rope_type != "default":
        raise ValueError(f"unsupported rope_type {rope_type!r}")
    return inv_freq.to(torch.float32)


class RotaryEncoding(PositionEncoding):
    def __init__(self, *, rot_dim: int, theta: float, scaling: dict | None = None,
                 interleaved: bool = False) -> None:
        if rot_dim <= 0 or rot_dim % 2:
            raise ValueError(f"rotary dimension must be positive and even, got {rot_dim}")
        self.rot_dim = rot_dim
        self.theta = theta
        self.scaling = scaling
        self.interleaved = interleaved
        self.table_scale = rotary_table_scale(scaling)
        self._key = ("rotary", id(self))

    def setup(self, runtime) -> None:
        super().setup(runtime)
        self.inv_freq = rotary_inv_freq(self.rot_dim, self.theta, self.scaling).to(runtime.device)

    def prepare(self, ctx) -> None:
        half = self.rot_dim // 2
        cos = ctx.buf(f"rope_cos_{id(self)}", half, torch.float32)
        sin = ctx.buf(f"rope_sin_{id(self)}", half, torch.float32)
        ops.rope_table(cos, sin, ctx.positions, self.inv_freq, self.table_scale)
        ctx.scratch[self._key] = RotaryTables(cos, sin, self.rot_dim, self.interleaved)

    def rotary(self, ctx) -> RotaryTables:
        return ctx.scratch[self._key]


class NoPositionEncoding(PositionEncoding):
    """Nothing is rotated and nothing is added."""


register_position_encoding("rotary", RotaryEncoding)
register_position_encoding("none", NoPositionEncoding)
