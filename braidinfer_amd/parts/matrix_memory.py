"""Matrix memory with exponential gates (the mLSTM of xLSTM): an outer-product state and a normaliser, both kept relative
to a running maximum of the gates' logarithms.

With n the mixer's input: q = W_q n d^-1/2 and k = W_k n (H heads of d channels), v = W_v n (H of e).  Per head the log
input gate i = cap tanh((W_i n + b_i) / cap) and the log forget gate f = log sigmoid(cap tanh((W_f n + b_f) / cap)).  With
m starting at 0, m' = max(f + m, i),

    S <- exp(f + m - m') S + exp(i - m') k v^T;   c <- the same with k alone;   m <- m'
    o = S^T q / (max(|c . q|, exp(-m)) + 1e-6)

Every head's o is divided by its root mean square, the heads are concatenated, multiplied by a weight and by sigmoid(W_g n)
and projected by W_o.

What a sequence keeps is fixed in size and float in both precisions, in its slot of the cache's state area (`StateNeed`):
S per head with c as one column more (its value is 1 for every token), laid out as the scan kernel's lanes hold it, and m
behind it.  All projections of the input are one product that leaves float sums.  The gates of a step's tokens are made
first (`exp_gates`); the memory is then a sum with a decay and a weight per token and walked like the other recurrences,
long prompts in pieces side by side.  The reference has no recurrent mixer.
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
from .linear import fused_layout, linear, padded_rows, stream_layout


class MatrixMemory(Mixer):
    graph_safe = True
    through_linear_only = True

    NAMES = {"q": "q", "k": "k", "v": "v", "g": "g", "i": "i", "f": "f", "i_bias": "i.b", "f_bias": "f.b", "norm": "norm", "o": "o"}
    MIN_PIECE = 128          # tokens: shorter pieces do not pay for the second walk

    def __init__(self, hidden_size: int, num_heads: int, key_dim: int, value_dim: int, gate_cap: float, norm_eps: float,
                 out_scale: float = 1.0, names: Optional[Dict[str, str]] = None):
        if num_heads <= 0 or not 0 < key_dim <= 512 or not 0 < value_dim <= 512 or not float(gate_cap) > 0:
            raise ConfigError(f"matrix memory: {num_heads} heads of {key_dim} key and {value_dim} value channels with gates bounded by "
                              f"{gate_cap} (all positive, widths at most 512)")
        self.H, self.nh, self.d, self.e = int(hidden_size), int(num_heads), int(key_dim), int(value_dim)
        self.cap, self.eps, self.out_scale = float(gate_cap), float(norm_eps), float(out_scale)
        self.names = dict(self.NAMES, **(names or {}))
        self.state_floats = state_floats(self.nh, self.d, self.e + 1)
        self.w_in = self.w_o = self.b_i = self.b_f = self.norm_w = None

    def weight_specs(self, prefix: str) -> List[TensorSpec]:
        n, hd, he = self.names, self.nh * self.d, self.nh * self.e
        return [TensorSpec(prefix + n["q"], (hd, self.H)), TensorSpec(prefix + n["k"], (hd, self.H)), TensorSpec(prefix + n["v"], (he, self.H)),
                TensorSpec(prefix + n["g"], (he, self.H)), TensorSpec(prefix + n["o"], (self.H, he)),
                TensorSpec(prefix + n["norm"], (he,), kind="vector", init="ones"),
                TensorSpec(prefix + n["i"], (self.nh, self.H)), TensorSpec(prefix + n["i_bias"], (self.nh,), kind="vector", init="normal"),
                TensorSpec(prefix + n["f"], (self.nh, self.H)), TensorSpec(prefix + n["f_bias"], (self.nh,), kind="vector", init="normal")]

    def load(self, tensors: Dict[str, torch.Tensor], prefix: str, rt: Runtime) -> None:
        self.rt = rt
        n = self.names
        self.w_in = fused_layout([tensors[prefix + n[x]] for x in ("q", "k", "v", "g", "i", "f")], rt)
        self.w_o = stream_layout(tensors[prefix + n["o"]], rt)
        self.b_i, self.b_f = (rt.own(tensors[prefix + n[x]].to(torch.float32).reshape(-1)) for x in ("i_bias", "f_bias"))
        self.norm_w = rt.own(tensors[prefix + n["norm"]].to(torch.float32).reshape(-1) * self.out_scale)

    def state_need(self) -> StateNeed:
        # the heads' memories and normalisers as the scan keeps them, then the running maxima
        return StateNeed((self.state_floats + self.nh,), torch.float32)

    def forward(self, h, x, step, ctx: MixerContext) -> None:
        T, nh, d, e = step.n_tokens, self.nh, self.d, self.e
        if ctx.state is None:
            raise StepError("matrix memory: the cache gave this mixer no state")
        hd, he = nh * d, nh * e
        g0, i0 = 2 * hd + he, 2 * hd + 2 * he
        rows = padded_rows(step.ws, "mm_rows", T, i0 + 2 * nh)
        linear(h, self.w_in, rows, step.ws)
        gb = step.ws.get("mm_gb", (T, 2 * nh), torch.float32)
        m = step.ws.get("mm_m", (T, nh), torch.float32)
        K.exp_gates(rows[:, i0:i0 + nh], rows[:, i0 + nh:], self.b_i, self.b_f, self.cap, ctx.state[:, self.state_floats:], step.cu_seqlens,
                    step.slots, gb, m, step.n_seqs, single_tokens=step.is_decode)
        o = step.ws.get("mm_o", (T, he), torch.float32)
        c_out = step.ws.get("mm_c", (T, nh), torch.float32)
        shape = tuple(K.glr_state_shape(nh, d, e + 1))
        S = ctx.state[:, :self.state_floats].view((-1,) + shape)
        q, k, v = rows[:, :hd], rows[:, hd:2 * hd], rows[:, 2 * hd:g0]
        pieces = pieces_for(step, nh * -(-(e + 1) // 16), self.MIN_PIECE)
        if pieces > 1:
            cu, numbers = HGRN2._piece_arrays(step, pieces)
            piece_state = step.ws.get("mm_piece_state", (step.n_seqs * pieces,) + shape, torch.float32)
            piece_decay = step.ws.get("mm_piece_decay", (step.n_seqs * pieces, nh), torch.float32)
            K.dr_scan_pieces(q, k, v, None, o, S, step.slots, cu, numbers, piece_state, step.n_seqs, pieces, nh, d, e, gb=gb, n_out=c_out,
                             piece_decay=piece_decay)
        else:
            K.dr_scan(q, k, v, gb, None, o, S, step.cu_seqlens, step.slots, step.n_seqs, nh, nh, d, e, weighted=True, n_out=c_out)
        y = step.ws.get("mm_y", (T, he), self.rt.dtype)
        K.head_norm_gate(o, self.norm_w, rows[:, g0:i0], y, nh, e, self.eps, gate_sigmoid=True, normaliser=(c_out, m, d ** -0.5))
        linear(y, self.w_o, x, step.ws, accumulate=True)


register_part("mixer", "matrix_memory", MatrixMemory, replace=True)
