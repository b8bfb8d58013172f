"""The gated delta rule: a matrix state per head and request that forgets by a scalar per token and corrects what it
holds for the token's key.

One product gives gate, q, k and v (a caller with another product of the same input may take it along), a small one in
float32 the logits of the step sizes and decays. One kernel runs the short convolutions with their activations from the
row's last inputs, makes q and k unit vectors and takes the gates; one walks each sequence's tokens of the step from the
row's float32 state; the head norms and the gate are the kernel that serves the other recurrent mixers.
"""

from __future__ import annotations

import torch

from ..config.specs import GatedDeltaSpec
from .registry import RowState, TensorDecl, register_part


def _state_layout(spec: GatedDeltaSpec):
    """(where the matrix state starts, elements of a row's state): the convolutions' last inputs lie in front of it; both
    are multiples of four, so that the state is read 16 bytes at a time."""
    start = ((spec.conv_taps - 1) * spec.conv_channels + 3) // 4 * 4
    return start, (start + spec.n_heads * spec.head_dim * spec.v_dim + 3) // 4 * 4


class GatedDelta:
    takes_out_dtype = True      # forward(..., out_dtype=): the dtype of its last product
    takes_partial = True
    takes_first = True          # forward(..., first=): (rows, column) of ``w_first``'s product, taken by the caller

    @staticmethod
    def tensors(spec: GatedDeltaSpec):
        H, G, D, Dv, d, n = spec.n_heads, spec.n_kv_heads, spec.head_dim, spec.v_dim, spec.hidden, spec.conv_taps
        return {"q": TensorDecl((G * D, d)), "k": TensorDecl((G * D, d)), "v": TensorDecl((H * Dv, d)),
                "q.conv": TensorDecl((G * D, n), "vector"), "k.conv": TensorDecl((G * D, n), "vector"),
                "v.conv": TensorDecl((H * Dv, n), "vector"), "b": TensorDecl((H, d)), "a": TensorDecl((H, d)),
                "A_log": TensorDecl((H,), "vector"), "dt_bias": TensorDecl((H,), "vector"),
                "norm": TensorDecl((Dv,), "vector"), "g": TensorDecl((H * Dv, d)), "o": TensorDecl((d, H * Dv))}

    @staticmethod
    def cache_need(spec: GatedDeltaSpec):
        # [the convolutions' last taps - 1 inputs, by tap and channel | the state, heads x value channels x key channels]
        return RowState((_state_layout(spec)[1],))

    def __init__(self, spec: GatedDeltaSpec, tensors, ops):
        self.spec, self.ops = spec, ops
        self.w_first = torch.cat([tensors[k] for k in ("g", "q", "k", "v")], dim=0).contiguous()
        # what enters the recurrence besides q, k and v: float32 sums
        self.w_gates = torch.cat([tensors["b"], tensors["a"]], dim=0).contiguous()
        self.taps = torch.cat([tensors[k + ".conv"] for k in "qkv"], dim=0).to(torch.float32).contiguous()
        self.a_log, self.dt_bias = (tensors[k].to(torch.float32).contiguous() for k in ("A_log", "dt_bias"))
        self.gain = tensors["norm"].to(torch.float32).repeat(spec.n_heads).contiguous()
        self.w_o = tensors["o"]
        self.state_at = _state_layout(spec)[0]

    def forward(self, x, ctx, slot, write=True, out_dtype=None, first=None, partial=False):
        """``first``: see ``takes_first``; ``partial``: the result may come as float32 partial sums [S, N, hidden]."""
        s, ops = self.spec, self.ops
        H, inner = s.n_heads, s.n_heads * s.v_dim
        if not write:
            raise ValueError("a recurrence writes the state it reads")
        first, at = first if first is not None else (ops.linear(x, self.w_first), 0)
        z = ops.linear(x, self.w_gates, out_dtype=torch.float32)
        raw = ops.delta_rule(first, at + inner, s.n_kv_heads, H, s.head_dim, s.v_dim, self.taps, float(s.head_dim) ** -0.5,
                             s.unit_eps, z, self.a_log, self.dt_bias, slot.state, 0, self.state_at, ctx)
        o = ops.gated_group_norm(raw, first[:, at:at + inner], self.gain, H, s.eps, gate_first=False)
        return ops.linear(o, self.w_o, out_dtype=out_dtype, **({"allow_partial": True} if partial else {}))


register_part(GatedDeltaSpec, GatedDelta)
