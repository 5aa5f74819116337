"""Rotary tables from a RotarySpec (host-side, 64-bit, stored as floats)."""
import math

import torch

from .configs import RotarySpec


def frequencies(spec: RotarySpec):
    """-> (angle per position of every pair, factor on cos and sin).

    With scaling (YaRN), pairs that turn more than `fast` times over the
    original context keep their frequency, pairs that turn less than `slow`
    times are stretched by `factor`, with a linear ramp over the pair index
    in between.
    """
    half = spec.dims // 2
    i = torch.arange(half, dtype=torch.float64)
    f = spec.base ** (-2.0 * i / spec.dims)
    if spec.factor is None:
        return f, 1.0

    def pair_of(turns):
        return spec.dims * math.log(
            spec.original / (2 * math.pi * turns)) / (2 * math.log(spec.base))
    lo = max(math.floor(pair_of(spec.fast)), 0)
    hi = min(math.ceil(pair_of(spec.slow)), spec.dims - 1)
    ramp = ((i - lo) / max(hi - lo, 0.001)).clamp(0.0, 1.0)
    return f / spec.factor * ramp + f * (1 - ramp), \
        0.1 * math.log(spec.factor) + 1.0


def table(spec: RotarySpec, max_pos: int, device) -> torch.Tensor:
    """[max_pos, dims / 2, 2] cos and sin, scaled."""
    f, amp = frequencies(spec)
    a = torch.outer(torch.arange(max_pos, dtype=torch.float64), f)
    return (torch.stack([a.cos(), a.sin()], -1) * amp).float().contiguous() \
        .to(device)
