"""A recurrent mixer whose memory is a vector (`GatedRecurrenceSpec`): a real-gated linear recurrent unit behind a short causal
filter, beside a second branch that multiplies its state.

    [y | x] = W_in h                    one product over the two branches' rows
    u = filter(x + b_x) + bias;  r = sigmoid(R u + b_r), i = sigmoid(I u + b_i) in each of `blocks` equal parts
    S_t = a S_(t-1) + sqrt(1 - a^2) i u,  a = exp(-factor r softplus(lam));      delta = W_o (S * gelu_tanh(y + b_y))

Everything between the two products runs in float32 under either precision, the parts' matrix products included (bfloat16
matrices are exact in it); S and the filter's last inputs are float32 in the request's slot.  A prompt portion is four
launches (filter, ring, gates, walk in token order); a step of single tokens on bfloat16 matrices is one.
"""
from __future__ import annotations

import torch

from ..cache.needs import StateNeed
from .base import ParamSpec, register
from .matrix_memory import _stack_rows


@register("mixer", "gated_recurrence")
class GatedRecurrence:
    graph_safe = True   # forward launches kernels only: no host reads, no data-dependent launches
    takes_scaled_rows = True

    def __init__(self, spec, runtime):
        self.spec = spec
        self.rt = runtime
        self.w_in = self.w_o = self.w_gates = None

    @staticmethod
    def _names(spec):
        return dict(zip(("y", "y_b", "x", "x_b", "conv", "conv_b", "r", "r_b", "i", "i_b", "lam", "o"), spec.names))

    @classmethod
    def params(cls, spec):
        n, s = cls._names(spec), spec
        size = s.width // s.blocks
        return {
            n["y"]: ParamSpec((s.width, s.hidden_size)), n["y_b"]: ParamSpec((s.width,), "float", ("normal", 0.1)),
            n["x"]: ParamSpec((s.width, s.hidden_size)), n["x_b"]: ParamSpec((s.width,), "float", ("normal", 0.1)),
            n["conv"]: ParamSpec((s.width, s.conv_taps), "float", ("normal", 0.5)), n["conv_b"]: ParamSpec((s.width,), "float", ("normal", 0.1)),
            n["r"]: ParamSpec((s.blocks, size, size), "float", ("normal", 0.1)), n["r_b"]: ParamSpec((s.blocks, size), "float", ("normal", 0.5)),
            n["i"]: ParamSpec((s.blocks, size, size), "float", ("normal", 0.1)), n["i_b"]: ParamSpec((s.blocks, size), "float", ("normal", 0.5)),
            n["lam"]: ParamSpec((s.width,), "float", ("normal", 1.0)), n["o"]: ParamSpec((s.hidden_size, s.width)),
        }

    @classmethod
    def placement(cls, spec):
        n = cls._names(spec)
        return {n[k]: "float32" for k in ("y_b", "x_b", "conv", "conv_b", "r_b", "i_b", "lam")}

    @staticmethod
    def variants(spec, dtype):
        return [("gated_recurrence", None)]

    def load(self, tensors):
        n, s = self._names(self.spec), self.spec
        self.w_in = _stack_rows(self.rt, [tensors[n["y"]], tensors[n["x"]]])
        self.w_o = self.rt.weight(tensors[n["o"]])
        self.y_b, self.x_b, self.conv_b = tensors[n["y_b"]], tensors[n["x_b"]], tensors[n["conv_b"]]
        self.conv = tensors[n["conv"]].t().contiguous()                     # [taps, width]
        r, i = tensors[n["r"]], tensors[n["i"]]
        if r.dtype != i.dtype:
            r, i = r.float(), i.float()
        self.mfma = self.rt.ops.recurrence_mfma_ok(r.dtype, s.width // s.blocks)
        if self.mfma:
            self.w_gates = torch.stack([r, i], dim=1).contiguous()          # [blocks, 2, out, in]
        else:
            self.w_gates = torch.cat([r, i], dim=1).transpose(1, 2).contiguous()     # [blocks, in, 2 out]
        self.r_b, self.i_b = tensors[n["r_b"]].reshape(-1).contiguous(), tensors[n["i_b"]].reshape(-1).contiguous()
        self.decay = (float(s.factor) * torch.nn.functional.softplus(tensors[n["lam"]].double())).float().contiguous()

    def cache_need(self):
        return None

    def state_need(self):
        return StateNeed((self.rt.ops.recurrence_state_size(self.spec.width, self.spec.conv_taps),), "float32")

    def forward(self, x, batch, cache, state):
        s, rt, ops = self.spec, self.rt, self.rt.ops
        n, width = x.shape[0], s.width
        proj = rt.linear(x, self.w_in)                    # float32 [n, y | x]
        out = rt.empty((n, width), rt.act_dtype)
        if self.mfma and batch.n_portions == 0:
            ops.recurrence_step(proj, 0, width, self.y_b, self.x_b, self.conv, self.conv_b, self.w_gates, self.r_b, self.i_b, self.decay,
                                state, batch.positions, batch.seq_of_token, batch.slots, out)
        else:
            u = ops.recurrence_filter(proj, width, self.x_b, self.conv, self.conv_b, state, batch.positions, batch.seq_of_token, batch.q_start,
                                      batch.q_len, batch.slots, rt.empty((n, width), torch.float32))
            terms = ops.recurrence_gates(u, self.w_gates, self.r_b, self.i_b, self.decay, rt.empty((n, width, 2), torch.float32), self.mfma)
            ops.recurrence_scan(terms, proj, 0, self.y_b, state, batch.q_start, batch.q_len, batch.slots, out)
        return rt.linear(out, self.w_o, slabs=True, defer=True)
