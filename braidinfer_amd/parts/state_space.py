"""Mamba-2 (state-space duality): an outer-product state with one decay and one step size per head and token.

One projection of the mixer's input n gives [z | x | B | C | dt]: a gate z and inputs x (H heads of e channels), B and C
(G groups of N channels; head h reads group h // (H / G)), a step size per head.  x, B and C pass a short causal
convolution over time per channel with a bias (`taps` numbers a channel, the last one the current token's, zeros before
the sequence's start) and silu.  With s = softplus(dt + dt_bias), per head

    S <- exp(-exp(A_log) s) S + s B x^T;   y = S^T C + D x

(the read-out sees the token's own write).  The heads are concatenated, multiplied by silu(z), divided in `norm_groups`
equal parts by each part's root mean square, multiplied by a weight and projected by W_o.

What a sequence keeps is fixed in size and float in both precisions, in its slot of the cache's state area (`StateNeed`):
S per head (zero at first, laid out as the scan kernel's lanes hold it) and, for the convolution, the last taps - 1 inputs
of every channel behind it.  The projection leaves float sums, so everything up to the norm works on unrounded numbers.
Long prompts that would leave the chip idle are cut into pieces that are walked side by side, twice.  The reference has
no recurrent mixer.
"""
from __future__ import annotations

from typing import Dict, List, Optional

import torch

from .. import kernels as K
from ..cache import StateNeed
from ..errors import ConfigError, StepError
from ..weights import TensorSpec
from .base import Mixer, MixerContext, Runtime, register_part
from .delta_rule import state_floats
from .gated_recurrence import HGRN2, pieces_for
from .linear import linear, padded_rows, stream_layout


class StateSpace(Mixer):
    graph_safe = True
    through_linear_only = True

    NAMES = {"in": "in", "conv": "conv", "conv_bias": "conv.b", "dt_bias": "dt_bias", "A_log": "A_log", "D": "D", "norm": "norm", "o": "o"}
    MIN_PIECE = 128          # tokens: shorter pieces do not pay for the second walk

    def __init__(self, hidden_size: int, num_heads: int, value_dim: int, state_dim: int, groups: int, norm_groups: int, taps: int,
                 norm_eps: float, out_scale: float = 1.0, names: Optional[Dict[str, str]] = None):
        if num_heads <= 0 or groups <= 0 or num_heads % groups:
            raise ConfigError(f"state space: {num_heads} heads are not a multiple of {groups} groups")
        if not 0 < state_dim <= 512 or not 0 < value_dim <= 512 or not 1 <= int(taps) <= 16:
            raise ConfigError(f"state space: {state_dim} state channels and heads of {value_dim} with {taps} taps (widths 1..512, 1..16 taps)")
        if norm_groups <= 0 or (num_heads * value_dim) % norm_groups:
            raise ConfigError(f"state space: {num_heads * value_dim} channels do not divide into {norm_groups} normed parts")
        self.H, self.nh, self.e, self.n, self.ng = int(hidden_size), int(num_heads), int(value_dim), int(state_dim), int(groups)
        self.parts, self.taps, self.eps, self.out_scale = int(norm_groups), int(taps), float(norm_eps), float(out_scale)
        self.names = dict(self.NAMES, **(names or {}))
        self.inner = self.nh * self.e
        self.C = self.inner + 2 * self.ng * self.n          # convolved channels: x | B | C
        self.state_floats = state_floats(self.nh, self.n, self.e)
        self.w_in = self.w_o = self.conv_t = self.conv_b = self.a_log = self.dt_bias = self.skip = self.norm_w = None

    def weight_specs(self, prefix: str) -> List[TensorSpec]:
        n = self.names
        vec = lambda what, shape, init="normal": TensorSpec(prefix + n[what], shape, kind="vector", init=init)
        return [TensorSpec(prefix + n["in"], (self.inner + self.C + self.nh, self.H)), vec("conv", (self.C, self.taps)), vec("conv_bias", (self.C,)),
                vec("dt_bias", (self.nh,)), vec("A_log", (self.nh,)), vec("D", (self.nh,), "ones"), vec("norm", (self.inner,), "ones"),
                TensorSpec(prefix + n["o"], (self.H, self.inner))]

    def load(self, tensors: Dict[str, torch.Tensor], prefix: str, rt: Runtime) -> None:
        self.rt = rt
        n = self.names
        self.w_in = stream_layout(tensors[prefix + n["in"]], rt)
        self.w_o = stream_layout(tensors[prefix + n["o"]], rt)
        flat = lambda what: tensors[prefix + n[what]].to(torch.float32).reshape(-1)
        self.conv_t = rt.own(flat("conv").reshape(self.C, self.taps).t().contiguous())          # [taps, channels]
        self.conv_b, self.a_log, self.dt_bias, self.skip = (rt.own(flat(x)) for x in ("conv_bias", "A_log", "dt_bias", "D"))
        self.norm_w = rt.own(flat("norm") * self.out_scale)

    def state_need(self) -> StateNeed:
        # the heads' states as the scan keeps them, then the convolution's last inputs [taps - 1][channels]
        return StateNeed((self.state_floats + (self.taps - 1) * self.C,), torch.float32)

    def forward(self, h, x, step, ctx: MixerContext) -> None:
        T, nh, e, n, ng, inner, C = step.n_tokens, self.nh, self.e, self.n, self.ng, self.inner, self.C
        if ctx.state is None:
            raise StepError("state space: the cache gave this mixer no state")
        rows = padded_rows(step.ws, "ssm_rows", T, inner + C + nh)
        linear(h, self.w_in, rows, step.ws)
        xbc = step.ws.get("ssm_xbc", (T, C), torch.float32)
        gb = step.ws.get("ssm_gb", (T, 2 * nh), torch.float32)
        kept = ctx.state[:, self.state_floats:] if self.taps > 1 else None
        K.ssm_prepare(rows[:, inner:inner + C], self.conv_t, self.conv_b, kept, rows[:, inner + C:], self.a_log, self.dt_bias,
                      step.seq_of_token, step.cu_seqlens, step.slots, xbc, gb, step.n_seqs, single_tokens=step.is_decode)
        y = step.ws.get("ssm_y", (T, inner), torch.float32)
        shape = tuple(K.glr_state_shape(nh, n, e))
        S = ctx.state[:, :self.state_floats].view((-1,) + shape)
        keys, queries, values = xbc[:, inner:inner + ng * n], xbc[:, inner + ng * n:], xbc[:, :inner]
        pieces = pieces_for(step, nh * -(-e // 16), self.MIN_PIECE)
        if pieces > 1:
            cu, numbers = HGRN2._piece_arrays(step, pieces)
            piece_state = step.ws.get("ssm_piece_state", (step.n_seqs * pieces,) + shape, torch.float32)
            piece_decay = step.ws.get("ssm_piece_decay", (step.n_seqs * pieces, nh), torch.float32)
            K.dr_scan_pieces(queries, keys, values, None, y, S, step.slots, cu, numbers, piece_state, step.n_seqs, pieces, nh, n, e, G=ng,
                             gb=gb, skip=self.skip, piece_decay=piece_decay)
        else:
            K.dr_scan(queries, keys, values, gb, None, y, S, step.cu_seqlens, step.slots, step.n_seqs, nh, ng, n, e, weighted=True, skip=self.skip)
        out = step.ws.get("ssm_out", (T, inner), self.rt.dtype)
        K.head_norm_gate(y, self.norm_w, rows[:, :inner], out, self.parts, inner // self.parts, self.eps, gate_first=True)
        linear(out, self.w_o, x, step.ws, accumulate=True)


register_part("mixer", "state_space", StateSpace, replace=True)
