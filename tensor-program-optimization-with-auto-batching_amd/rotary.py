"""Rotation tables: frequencies, optional YaRN scaling, interleaved pairs."""
from __future__ import annotations

import dataclasses
import math
from typing import Optional

import numpy as np


@dataclasses.dataclass(frozen=True)
class YarnScaling:
    factor: float
    original: float      # context length of the unscaled model
    fast: float          # turns over that length above which a frequency stays as it is ...
    slow: float          # ... and below which it is divided by the factor


@dataclasses.dataclass(frozen=True)
class Rotation:
    base: float
    dims: int                                  # leading dimensions that turn, in pairs (2 i, 2 i + 1)
    scaling: Optional[YarnScaling] = None

    @classmethod
    def from_config(cls, c: dict) -> "Rotation":
        sc = c.get("scaling")
        if sc is not None:
            sc = YarnScaling(float(sc["factor"]), float(sc["original"]), float(sc["fast"]), float(sc["slow"]))
        return cls(float(c["base"]), int(c["dims"]), sc)

    def frequencies(self) -> np.ndarray:
        n = self.dims
        f = self.base ** (-2.0 * np.arange(n // 2, dtype=np.float64) / n)
        if self.scaling is None:
            return f
        s = self.scaling
        index_of = lambda turns: n * math.log(s.original / (2.0 * math.pi * turns)) / (2.0 * math.log(self.base))
        lo = max(math.floor(index_of(s.fast)), 0)
        hi = min(math.ceil(index_of(s.slow)), n - 1)
        ramp = np.clip((np.arange(n // 2, dtype=np.float64) - lo) / max(hi - lo, 0.001), 0.0, 1.0)
        return f / s.factor * ramp + f * (1.0 - ramp)

    @property
    def magnitude(self) -> float:
        """Factor on cos and sin."""
        return 1.0 if self.scaling is None else 0.1 * math.log(self.scaling.factor) + 1.0

    def tables(self, width: int, max_pos: int):
        """cos, sin [max_pos, width / 2] float32 for vectors of `width` dimensions (float64 math, rounded once); pairs past
        `dims` pass unchanged."""
        if self.dims % 2 or width % 2 or self.dims > width:
            raise ValueError(f"rotation of {self.dims} of {width} dimensions")
        ang = np.arange(max_pos, dtype=np.float64)[:, None] * self.frequencies()[None, :]
        cos, sin = np.ones((max_pos, width // 2), np.float32), np.zeros((max_pos, width // 2), np.float32)
        cos[:, : self.dims // 2] = self.magnitude * np.cos(ang)
        sin[:, : self.dims // 2] = self.magnitude * np.sin(ang)
        return cos, sin
