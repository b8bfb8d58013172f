"""Wrappers of the kernels in ``csrc/delta.hip``: what prepares the gated delta rule and the recurrence itself. The
library is compiled and loaded when a model first asks for it."""

from __future__ import annotations

from ctypes import c_float, c_int

import torch

from .build import load_library
from .common import _DELTA_SIGNATURES, KernelError, _check, _declare, _ptr


class Delta:
    def _delta(self):
        lib = getattr(self, "_delta_lib", None)
        if lib is None:
            lib = self._delta_lib = load_library("delta")
            _declare(lib, _DELTA_SIGNATURES)
        return lib

    def delta_rule(self, x, col, G, H, D, Dv, taps_w, q_scale, unit_eps, z, a_log, dt_bias, state, conv_offset, offset, ctx):
        """x [N, ld] holds q (G heads of D), k (G of D) and v (H of Dv) from column ``col`` on. Every channel passes a causal
        convolution (``taps_w`` float32 [channels, taps], the last tap the current token's; earlier inputs from the row's
        state, [taps - 1, channels] from ``conv_offset``) and silu; q and k become unit vectors, x / sqrt(sum(x^2) +
        unit_eps), q also times ``q_scale``. z float32 [N, 2 H]: logits of beta = sigmoid(z) and, behind them, of
        g = exp(-exp(a_log) softplus(z + dt_bias)). Per head, from and into the row's state ([H, Dv, D] from ``offset``):
        S <- g S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q. float32 [N, H * Dv]."""
        N, ld = x.shape
        self._want(x, "x", self.dtype)
        if G < 1 or H < 1 or H % G or not 1 <= D <= 256 or Dv < 1:
            raise KernelError(f"gated delta rule: {H} heads over {G} key heads of {D} (at most 256), values of {Dv}")
        C, taps = 2 * G * D + H * Dv, taps_w.shape[1]
        if col < 0 or col + C > ld or not 1 <= taps <= 33:
            raise KernelError(f"gated delta rule: columns {col}..{col + C} of {ld}, {taps} taps (at most 33)")
        self._want(taps_w, "taps", torch.float32, (C, taps))
        self._want(z, "gate logits", torch.float32, (N, 2 * H))
        self._want(a_log, "A_log", torch.float32, (H,))
        self._want(dt_bias, "dt bias", torch.float32, (H,))
        stride = self._state(state, offset, H * D * Dv, ctx)
        self._state(state, conv_offset, (taps - 1) * C, ctx)
        if D % 4 == 0 and (offset % 4 or state.shape[1] % 4):
            raise KernelError("gated delta rule: a row's matrix state starts on 16 bytes")
        Dp = (D + 63) // 64 * 64
        qk = torch.empty((N, 2, G, Dp), dtype=torch.float32, device=self.device)
        v = torch.empty((N, H * Dv), dtype=self.dtype, device=self.device)
        gates = torch.empty((N, H, 2), dtype=torch.float32, device=self.device)
        out = torch.empty((N, H * Dv), dtype=torch.float32, device=self.device)
        lib = self._delta()
        _check(lib.soc_delta_prepare(
            _ptr(x), c_int(ld), c_int(col), c_int(G), c_int(H), c_int(D), c_int(Dv), c_int(Dp), _ptr(taps_w), c_int(taps),
            c_float(q_scale), c_float(unit_eps), _ptr(z), _ptr(a_log), _ptr(dt_bias), _ptr(state), stride, c_int(conv_offset),
            _ptr(ctx.seq_qstart), _ptr(ctx.seq_rows), _ptr(qk), _ptr(v), _ptr(gates), c_int(ctx.n_seqs),
            c_int(max(1, ctx.max_q_len)), c_int(self.code), self._stream()), "delta_prepare")
        _check(lib.soc_delta_walk(
            _ptr(qk), _ptr(v), _ptr(gates), c_int(G), c_int(H), c_int(D), c_int(Dv), c_int(Dp), _ptr(state), stride, c_int(offset),
            _ptr(ctx.seq_qstart), _ptr(ctx.seq_rows), _ptr(out), c_int(ctx.n_seqs), c_int(self.code), self._stream()), "delta_walk")
        return out
