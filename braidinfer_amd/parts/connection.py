"""Connections of a layer's halves to a residual kept as several streams.

`hyper_connection`: the half reads u = sum_s in[s] x_s and its output y goes back as
x_t <- sum_s mix[s, t] x_s + out[t] y, all streams at once from the old ones (mix is indexed [from, to]), with learnt
vectors in, out [streams] and a matrix mix [streams, streams]; all of it float.  The reference has one residual row a
token."""
from __future__ import annotations

from typing import Dict, List, Sequence

import torch

from .. import kernels as K
from ..errors import ConfigError
from ..weights import TensorSpec
from .base import Connection, Runtime, register_part

MAX_STREAMS = 16      # the kernels' limit


class HyperConnection(Connection):
    graph_safe = True

    def __init__(self, hidden_size: int, streams: int, branch_scales: Sequence[float] = (1.0,)):
        """`branch_scales`: what the outputs of the half's parts (one, or two side by side) are multiplied by in their sum."""
        self.width, self.streams = int(hidden_size), int(streams)
        self.branch_scales = [float(v) for v in branch_scales]
        if not 1 <= self.streams <= MAX_STREAMS or not 1 <= len(self.branch_scales) <= 2:
            raise ConfigError(f"hyper connection: 1 to {MAX_STREAMS} streams and one or two branches, got {streams} and {len(branch_scales)}")
        self.coef = None

    def weight_specs(self, prefix: str) -> List[TensorSpec]:
        S = self.streams
        return [TensorSpec(prefix + "in", (S,), kind="vector", init="ones"), TensorSpec(prefix + "out", (S,), kind="vector", init="ones"),
                TensorSpec(prefix + "mix", (S, S), kind="vector", init="normal")]

    def load(self, tensors: Dict[str, torch.Tensor], prefix: str, rt: Runtime) -> None:
        self.rt = rt
        self.coef = rt.own(torch.cat([tensors[prefix + n].to(torch.float32).reshape(-1) for n in ("in", "out", "mix")]))

    @staticmethod
    def _point(norm):
        """(whether a kernel can apply the norm in passing, its arguments)."""
        if norm is None:
            return True, None
        args = norm.point_args()
        return args is not None, args

    def open(self, X, norm, h, ws) -> None:
        fused, args = self._point(norm)
        if fused:
            K.streams_open(X, h, self.streams, self.coef, args)
            return
        u = ws.get("connection_u", (X.shape[0], self.width), torch.float32)
        K.streams_open(X, u, self.streams, self.coef)
        norm.forward(u, h)

    def join(self, X, branches, then, then_norm, then_h) -> bool:
        scaled = [(y, bias, scale) for (y, bias), scale in zip(branches, self.branch_scales, strict=True)]
        fused, args = self._point(then_norm)
        if then_h is None or not fused or not isinstance(then, HyperConnection):
            K.streams_join(X, self.coef, scaled, self.streams)
            return False
        K.streams_join(X, self.coef, scaled, self.streams, then_h, then.coef, args)
        return True


register_part("connection", "hyper_connection", HyperConnection, replace=True)
