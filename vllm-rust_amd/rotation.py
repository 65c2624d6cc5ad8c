"""Rotary position code of a head as configurations describe it (plain or stretched steps); the library makes the step table
(`vmx_rotation_steps`)."""
from __future__ import annotations

import dataclasses

from ._lib import Rotation


@dataclasses.dataclass
class RotationSpec:
    dims: int = 0                # rotated coordinates per head (0: none)
    base: float = 10000.0
    scaling: dict | None = None  # {factor, original, fast, slow}: slow pairs turn `factor` times slower

    @staticmethod
    def from_config(rot: dict | None) -> "RotationSpec":
        if not rot or not rot.get("dims"):
            return RotationSpec()
        sc = rot.get("scaling")
        return RotationSpec(int(rot["dims"]), float(rot["base"]),
                            {k: float(sc[k]) for k in ("factor", "original", "fast", "slow")} if sc else None)

    def to_config(self) -> dict | None:
        if not self.dims:
            return None
        d = {"base": self.base, "dims": self.dims}
        if self.scaling:
            d["scaling"] = dict(self.scaling)
        return d

    def to_struct(self) -> Rotation:
        sc = self.scaling or {}
        return Rotation(self.dims, self.base, sc.get("factor", 0.0), sc.get("original", 0.0), sc.get("fast", 0.0), sc.get("slow", 0.0))
