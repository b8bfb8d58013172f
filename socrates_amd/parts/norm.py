"""RMSNorm: y = x / sqrt(mean(x^2) + eps) * w  (model/qwen/qwen_kv_cont.py:45-53).

eps sits inside the square root and the gain is the plain weight, as in the
reference. Statistics are taken in float32 whatever the compute dtype.
``LayerNorm`` takes the mean off first and adds a bias.
"""

from __future__ import annotations

import torch

from ..config.specs import LayerNormSpec, RMSNormSpec, ScalarRMSNormSpec
from .registry import TensorDecl, register_part


class RMSNorm:
    @staticmethod
    def tensors(spec: RMSNormSpec):
        return {spec.tensor: TensorDecl((spec.dim,), "vector")}

    def __init__(self, spec: RMSNormSpec, tensors, ops):
        self.spec, self.ops = spec, ops
        self.weight = tensors[spec.tensor]

    free_layout = True      # add_norm takes ``by_tile``

    def add_norm(self, residual, delta, rows=None, by_tile=False):
        """residual (fp32, [N, dim]) += delta; return norm(residual) in the compute dtype.

        With ``rows`` (int32 indices) only those rows are summed and normed, into a
        new [len(rows), dim] tensor, and ``residual`` is left unchanged. ``by_tile``: the
        result goes to one product of the kernel set and nowhere else, so the kernel set may
        lay it out as that product reads it best.
        """
        if by_tile and getattr(self.ops, "rows_by_tile", None):
            return self.ops.add_rmsnorm(residual, delta, self.weight, self.spec.eps, rows, by_tile=True)
        return self.ops.add_rmsnorm(residual, delta, self.weight, self.spec.eps, rows)

    def fusable(self):
        """(gain, eps): all a kernel set needs to compute this norm inside the products
        around it (``HipKernels.linear_add_norm``)."""
        return self.weight, self.spec.eps

    def terms(self):
        """(gain, bias or None, eps, whether the mean is taken off): what the kernel for copies of the stream needs."""
        return self.weight, None, self.spec.eps, False

    def __call__(self, x):
        """Plain norm over the last dimension of ``x`` (any leading shape)."""
        return self.ops.rmsnorm(x, self.weight, self.spec.eps)


class ScalarRMSNorm(RMSNorm):
    """RMSNorm whose gain is one stored number (a tensor without dimensions that carries the
    norm's own name). The kernels take a gain per element: the number is spread once here."""

    @staticmethod
    def tensors(spec: ScalarRMSNormSpec):
        return {"": TensorDecl((), "vector")}

    def __init__(self, spec: ScalarRMSNormSpec, tensors, ops):
        self.spec, self.ops = spec, ops
        self.weight = tensors[""].to(torch.float32).reshape(1).expand(spec.dim).contiguous()


class LayerNorm:
    """y = (x - mean) / sqrt(variance + eps) * w + b, the variance being the mean of the squared deviations."""

    @staticmethod
    def tensors(spec: LayerNormSpec):
        return {"": TensorDecl((spec.dim,), "vector"), "b": TensorDecl((spec.dim,), "vector")}

    def __init__(self, spec: LayerNormSpec, tensors, ops):
        self.spec, self.ops = spec, ops
        self.weight, self.bias = (tensors[k].to(torch.float32).contiguous() for k in ("", "b"))

    def terms(self):
        return self.weight, self.bias, self.spec.eps, True

    def add_norm(self, residual, delta, rows=None):
        """As ``RMSNorm.add_norm``; with ``rows`` and a ``delta`` only the rows' sum is taken, and the stream is left
        as it is."""
        N, d = residual.shape
        if delta is not None and rows is not None:
            residual = residual[rows.long()].contiguous()
            delta = delta.index_select(delta.dim() - 2, rows.long()).contiguous()
            rows = None
        view = residual.view(residual.shape[0], 1, d)
        if delta is None:
            return self.ops.streams_norm(view, None, self.terms(), rows)
        return self.ops.streams_update(view, [(delta, 1.0)], None, None, None, self.terms())


register_part(RMSNormSpec, RMSNorm)
register_part(LayerNormSpec, LayerNorm)
register_part(ScalarRMSNormSpec, ScalarRMSNorm)
