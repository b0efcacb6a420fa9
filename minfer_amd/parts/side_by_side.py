"""Two mixers on one input, their results scaled and summed:
y = left_scale left(x) + right_scale right(x).

Either side is any registered mixer that takes an `out_scale` (applied to its result before its last
product, so the sum costs no pass of its own: the second side's product adds onto the first's).  A cache entry
holds what both sides ask for: pages for the one that attends, a fixed-size state for the one that recurs
(at most one of each kind).

Or both results RMS-normed over the model's width first, each with a gain of its own, and then summed:
y = scale (norm(left(x)) + norm(right(x))).  The sides then leave their results in rows of their own and one kernel
norms and sums them.
"""
from __future__ import annotations

import torch

from ..cache.paged import split_request
from ..kernels import ops
from ..weights.loader import TensorSpec
from .base import MIXERS, Mixer, make_part, register_mixer
from .spec import PartSpec


@register_mixer("side_by_side")
class SideBySide(Mixer):
    """params: left, right (PartSpecs of mixers), left_scale, right_scale, left_prefix, right_prefix (put
    before the sides' tensor names)."""

    takes_normed = True
    can_overwrite = True

    def __init__(self, spec, rt):
        super().__init__(spec, rt)
        p = spec.params
        self.sides = [(p.get(side + "_prefix", side + "."), self._side(side, p, rt)) for side in ("left", "right")]
        kinds = [split_request(part.cache_request()) for _, part in self.sides]
        if sum(kv is not None for kv, _ in kinds) > 1 or sum(st is not None for _, st in kinds) > 1:
            raise ValueError("side_by_side: both sides ask the cache for the same kind of storage")

    def _side(self, side: str, p, rt):
        inner = p[side]
        scaled = PartSpec(inner.kind, dict(inner.params, out_scale=float(p.get(side + "_scale", 1.0))))
        part = make_part(MIXERS, scaled, rt, "mixer")
        if not getattr(part, "can_overwrite", False) or not hasattr(part, "out_scale"):
            raise ValueError(f"side_by_side: the mixer {inner.kind!r} takes no out_scale")
        return part

    def tensor_specs(self):
        return {prefix + name: ts for prefix, part in self.sides for name, ts in part.tensor_specs().items()}

    def load(self, get):
        for prefix, part in self.sides:
            part.load(lambda name, p=prefix: get(p + name))

    def cache_request(self):
        asked = []
        for _, part in self.sides:
            asked += [r for r in split_request(part.cache_request()) if r is not None]
        return tuple(asked) if len(asked) > 1 else (asked[0] if asked else None)

    def decode_copies(self, make: bool, min_row_length: int = 0) -> int:
        return sum(part.decode_copies(make, min_row_length) for _, part in self.sides)

    def prepare(self, max_len: int) -> None:
        for _, part in self.sides:
            part.prepare(max_len)

    def forward(self, x, h, ctx, entry: int, writes_cache: bool, accumulate: bool = True) -> None:
        for i, (_, part) in enumerate(self.sides):
            part.forward(x, h, ctx, entry, writes_cache, accumulate=accumulate or i > 0)


@register_mixer("side_by_side_normed")
class SideBySideNormed(SideBySide):
    """params: hidden_size, left, right (PartSpecs of mixers that can overwrite), left_prefix, right_prefix, left_norm,
    right_norm (tensor names of the gains), eps, scale (of the sum)."""

    def __init__(self, spec, rt):
        super().__init__(spec, rt)
        p = spec.params
        self.hidden, self.eps, self.scale = int(p["hidden_size"]), float(p["eps"]), float(p.get("scale", 1.0))
        self.gain_names = (p["left_norm"], p["right_norm"])
        self.gains = None
        self.takes_normed = all(getattr(part, "takes_normed", False) for _, part in self.sides)

    def _side(self, side: str, p, rt):
        part = make_part(MIXERS, p[side], rt, "mixer")
        if not getattr(part, "can_overwrite", False):
            raise ValueError(f"side_by_side_normed: the mixer {p[side].kind!r} cannot leave its result in rows of its own")
        return part

    def tensor_specs(self):
        return dict(super().tensor_specs(), **{name: TensorSpec((self.hidden,), init="ones") for name in self.gain_names})

    def load(self, get):
        super().load(get)
        self.gains = [get(name).to(torch.float32).contiguous() for name in self.gain_names]

    def forward(self, x, h, ctx, entry: int, writes_cache: bool, accumulate: bool = True) -> None:
        rows = []
        for _, part in self.sides:
            y = torch.empty(h.shape, dtype=torch.float32, device=h.device)
            part.forward(x, y, ctx, entry, writes_cache, accumulate=False)
            rows.append(y)
        ops.rmsnorm_pair(rows[0], self.gains[0], rows[1], self.gains[1], self.eps, self.scale, h, accumulate=accumulate)
