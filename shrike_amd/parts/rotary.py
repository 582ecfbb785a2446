"""Rotary position encoding with the half-split pairing (i, i + rot_dim/2), its rates by the base
alone or stretched for longer contexts (YaRN), and with neighbouring pairs."""

from __future__ import annotations

import math

import torch

from .base import PositionEncoding, register_position


def yarn_rates(theta: float, dims: int, factor: float, original: float, fast: float, slow: float):
    """(rates [dims / 2], magnitude) in double precision.  A pair i that makes t full turns within
    `original` positions has 2 i = dims * ln(original / (2 pi t)) / ln theta; the pairs from the one of
    `fast` turns (rounded down) to the one of `slow` turns (rounded up) pass linearly from theta ** (-2i /
    dims) to that rate over `factor`."""

    def pair_of(turns: float) -> float:
        return dims * math.log(original / (2.0 * math.pi * turns)) / (2.0 * math.log(theta))

    lo = max(math.floor(pair_of(fast)), 0)
    hi = min(math.ceil(pair_of(slow)), dims - 1)
    rates = []
    for i in range(dims // 2):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        rate = theta ** (-2.0 * i / dims)
        rates.append(rate / factor * ramp + rate * (1.0 - ramp))
    return rates, 0.1 * math.log(factor) + 1.0


class RotaryHalf(PositionEncoding):
    """inv_freq[i] = theta ** (-2i / rot_dim), formed in float32 exactly as the
    reference does (shrike/models/qwen.py:80); the angle of position p is
    float32(p) * inv_freq[i] (:86).  The rotation itself runs inside the
    cache-write kernel."""

    launches_follow_shape = True
    adjacent_pairs = False  # pairs are (i, i + rot_dim / 2)
    magnitude = 1.0  # what cosine and sine are multiplied by

    def load(self, tensors, runtime):
        d = int(self.spec.rotary_dim)
        scaling = getattr(self.spec, "scaling", None)
        if scaling is not None:
            rates, self.magnitude = yarn_rates(float(self.spec.theta), d, *scaling)
            inv_freq = torch.tensor(rates, dtype=torch.float64).to(torch.float32)
        else:
            inv_freq = 1.0 / (float(self.spec.theta) ** (torch.arange(0, d, 2).float() / d))
        self.inv_freq = inv_freq.to(runtime.device)
        self.rot_dim = d

    def rotary_table(self):
        return self.inv_freq, self.rot_dim


register_position("rotary_half", RotaryHalf)


class RotaryAdjacent(PositionEncoding):
    """The same rotation on neighbouring elements: pair i of a head is (2i, 2i + 1),
    i < rot_dim / 2, and turns by position * theta ** (-2i / rot_dim); elements
    from rot_dim on pass unchanged.  The rates are formed in float64 and rounded
    once; the cache-write kernel forms the angle as a float32 product."""

    launches_follow_shape = True
    adjacent_pairs = True
    magnitude = 1.0

    def load(self, tensors, runtime):
        d = int(self.spec.rotary_dim)
        inv_freq = float(self.spec.theta) ** (-torch.arange(0, d, 2, dtype=torch.float64) / d)
        self.inv_freq = inv_freq.to(torch.float32).to(runtime.device)
        self.rot_dim = d

    def rotary_table(self):
        return self.inv_freq, self.rot_dim


register_position("rotary_adjacent", RotaryAdjacent)
