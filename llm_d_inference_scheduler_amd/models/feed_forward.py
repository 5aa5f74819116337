"""Feed-forwards of the layer-listed designs: a gated MLP, and experts.

Called with the normed stream of a batch's rows; -> (y, rows): the output is
y [T, width] (None if everything is in rows) plus, for every token, the sum of
its `top` rows [T * top, width]. The stream update adds both.
"""
from typing import Callable, Optional, Tuple

import torch

from ..ops import layered as ops
from ..ops.layered import linear
from .configs import ExpertsSpec, FeedForwardSpec, GatedSpec

Output = Tuple[Optional[torch.Tensor], Optional[torch.Tensor]]


class GatedMLP:
    def __init__(self, spec: GatedSpec, take: Callable, dtype: torch.dtype):
        self.spec = spec
        self.gate_up = torch.cat([take("gate"), take("up")]).to(dtype)
        self.down = take("down").to(dtype)

    def __call__(self, h: torch.Tensor) -> Output:
        return linear(ops.gated_act(linear(h, self.gate_up), self.spec.act),
                      self.down), None


class Experts:
    """Tokens sorted by expert, then one grouped product for all experts'
    inner layers and one for their outputs."""

    def __init__(self, spec: ExpertsSpec, take: Callable,
                 dtype: torch.dtype):
        self.spec = spec

        def stack(leaf):
            first = take(f"e0.{leaf}").to(dtype)
            out = torch.empty((spec.experts,) + first.shape, dtype=dtype,
                              device=first.device)
            out[0] = first
            for e in range(1, spec.experts):
                out[e] = take(f"e{e}.{leaf}")
            return out
        self.router = take("router").to(dtype)
        self.up, self.down = stack("up"), stack("down")
        self.shared_up = self.shared_down = None
        if spec.shared_ff:
            self.shared_up = take("shared.up").to(dtype)
            self.shared_down = take("shared.down").to(dtype)

    def __call__(self, h: torch.Tensor) -> Output:
        s = self.spec
        ids, weights = ops.route(h, self.router, s.top)
        rows = ops.experts(h, ids, weights, self.up, self.down, s.act)
        if self.shared_up is None:
            return None, rows
        return linear(ops.activate(linear(h, self.shared_up), s.act),
                      self.shared_down), rows


def build(spec: FeedForwardSpec, take: Callable, dtype: torch.dtype):
    kind = GatedMLP if isinstance(spec, GatedSpec) else Experts
    return kind(spec, take, dtype)
