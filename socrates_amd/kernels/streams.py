"""Wrappers of the kernels in ``csrc/streams.hip``: the embedding with learned positions spread over several copies of
the residual stream, and the step between two branches: results added up, new copies from the old ones, and the
combination that the next branch reads, normed. The library is compiled and loaded when a model first asks for one of them."""

from __future__ import annotations

from ctypes import c_float, c_int

import torch

from .build import load_library
from .common import _DTYPE_CODE, _STREAMS_SIGNATURES, KernelError, _check, _declare, _ptr
from .hybrid import ExpertSums

MAX_STREAMS = 16
MAX_STREAM_WIDTH = 16000


class Streams:
    def _streams(self):
        lib = getattr(self, "_streams_lib", None)
        if lib is None:
            lib = self._streams_lib = load_library("streams")
            _declare(lib, _STREAMS_SIGNATURES)
        return lib

    def embedding_streams(self, ids, table, scale, positions, position_table, n):
        """float32 [N, n, d]: every copy of token i is scale * table[ids[i]] + position_table[positions[i]]
        (``position_table`` None: without it)."""
        self._want(ids, "ids", torch.int32)
        self._want(table, "embedding table")
        N, (V, d) = ids.numel(), table.shape
        if not 1 <= n <= MAX_STREAMS or table.dtype not in _DTYPE_CODE:
            raise KernelError(f"{n} copies of rows in {table.dtype}")
        rows = 0
        if position_table is not None:
            self._want(positions, "positions", torch.int32, (N,))
            rows = position_table.shape[0]
            self._want(position_table, "position table", table.dtype, (rows, d))
        out = torch.empty((N, n, d), dtype=torch.float32, device=self.device)
        step = 65535
        for lo in range(0, N, step):
            m = min(step, N - lo)
            _check(self._streams().soc_embedding_streams(
                _ptr(ids[lo:]), _ptr(table), c_float(scale), _ptr(positions[lo:]) if position_table is not None else None,
                _ptr(position_table), c_int(rows), _ptr(out[lo:]), c_int(m), c_int(n), c_int(d), c_int(V),
                c_int(_DTYPE_CODE[table.dtype]), self._stream()), "embedding_streams")
        return out

    def _branch_args(self, branch, N, d):
        if branch is None:
            return [None, c_int(0), None, None, c_int(0), None, c_float(0.0)]
        y, scale = branch
        if isinstance(y, ExpertSums):
            top = y.weight.shape[1]
            self._want(y.y, "expert results", torch.float32, (N * top, d))
            self._want(y.weight, "expert weights", torch.float32, (N, top))
            if y.through is not None:
                self._want(y.through, "the experts' input", self.dtype, (N, d))
            return [_ptr(y.y), c_int(0), _ptr(y.runs.place), _ptr(y.weight), c_int(top), _ptr(y.through), c_float(scale)]
        parts = 0
        if y.dim() == 3:
            parts = y.shape[0]
            self._want(y, "partial sums", torch.float32, (parts, N, d))
        elif y.dtype == torch.float32:
            parts = 1
            self._want(y, "branch result", torch.float32, (N, d))
        else:
            self._want(y, "branch result", self.dtype, (N, d))
        return [_ptr(y), c_int(parts), None, None, c_int(0), None, c_float(scale)]

    def _run_streams(self, x, branches, mix, out_w, read, norm, rows):
        if x.dim() != 3 or not 1 <= x.shape[1] <= MAX_STREAMS or not 1 <= x.shape[2] <= MAX_STREAM_WIDTH:
            raise KernelError(f"copies of the stream {tuple(x.shape)}: [tokens, 1 to {MAX_STREAMS}, 1 to {MAX_STREAM_WIDTH}]")
        N, S, d = x.shape
        self._want(x, "copies of the stream", torch.float32)
        if (mix is None) != (out_w is None):
            raise KernelError("the copies' weights of each other and of the branch come together")
        for t, name, shape in ((mix, "mix", (S, S)), (out_w, "out", (S,)), (read, "in", (S,))):
            if t is not None:
                self._want(t, name, torch.float32, shape)
        gain, bias, eps, centred = norm if norm is not None else (None, None, 0.0, False)
        n_out = N
        if rows is not None:
            self._want(rows, "rows", torch.int32)
            n_out = rows.numel()
        out = None
        if gain is not None:
            self._want(gain, "norm gain", torch.float32, (d,))
            if bias is not None:
                self._want(bias, "norm bias", torch.float32, (d,))
            out = torch.empty((n_out, d), dtype=self.dtype, device=self.device)
        pair = list(branches) + [None] * (2 - len(branches))
        _check(self._streams().soc_streams(
            _ptr(x), c_int(S), *self._branch_args(pair[0], N, d), *self._branch_args(pair[1], N, d), _ptr(mix), _ptr(out_w), _ptr(read),
            _ptr(gain), _ptr(bias), c_float(eps), c_int(1 if centred else 0), _ptr(rows), _ptr(out), c_int(N), c_int(n_out), c_int(d),
            c_int(self.code), self._stream()), "streams")
        return out

    def streams_norm(self, x, read, norm, rows=None):
        """norm(sum over s of read[s] x[:, s]) in the compute dtype; x float32 [N, S, d], ``read`` float32 [S] (None: the plain
        sum), ``norm`` (gain, bias or None, eps, whether the mean is taken off); ``rows``: of these rows only."""
        return self._run_streams(x, [], None, None, read, norm, rows)

    def streams_update(self, x, branches, mix, out, read=None, norm=None):
        """x (float32 [N, S, d], in place): x_t <- sum over s of mix[s, t] x_s + out[t] y, all t from the old copies, with
        y = the sum of one or two branches (result, scale): a result [N, d] in the compute dtype or float32, float32
        partial sums [P, N, d], or an ``ExpertSums``. ``mix`` and ``out`` None: x_t <- x_t + y. With ``norm``: returns what
        ``streams_norm`` would of the new copies; else None."""
        if not 1 <= len(branches) <= 2:
            raise KernelError(f"{len(branches)} branches in one sum")
        return self._run_streams(x, branches, mix, out, read, norm, None)
