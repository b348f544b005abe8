"""Python faces of csrc/streams.hip: several residual streams in place of one - spreading the
embedded rows, the weighted sum that a sublayer reads (normed), and the step that moves all
streams by a sublayer's result.  Shape checks on the host, then the launch."""
import ctypes
from typing import Optional

import torch

from .library import KernelError, check, library, ptr, require_contiguous, require_device, stream_handle

_i, _f = ctypes.c_int, ctypes.c_float

MAX_STREAMS = 16


def _check_streams(X, what):
    if X.dtype != torch.float32 or X.dim() != 3 or not 1 <= X.shape[1] <= MAX_STREAMS:
        raise KernelError(f"{what}: the streams must be float32 [N, 1..{MAX_STREAMS}, D], are "
                          f"{tuple(X.shape)} {X.dtype}")


def _check_vector(t, n, what):
    if t.dtype != torch.float32 or t.numel() != n:
        raise KernelError(f"{what} must be float32 with {n} elements")


def spread(x: torch.Tensor, streams: int) -> torch.Tensor:
    """float32 [N, S, D]: every stream a copy of x float32 [N, D]."""
    require_device(x)
    require_contiguous(x=x)
    if x.dtype != torch.float32 or x.dim() != 2 or not 1 <= streams <= MAX_STREAMS:
        raise KernelError(f"streams: x must be float32 [N, D], streams 1..{MAX_STREAMS}")
    X = torch.empty((x.shape[0], streams, x.shape[1]), dtype=torch.float32, device=x.device)
    check(library("streams").gfa_streams_spread(ptr(x), ptr(X), _i(x.shape[0]), _i(streams),
                                                _i(x.shape[1]), stream_handle()), "streams_spread")
    return X


def read(X: torch.Tensor, w_in: torch.Tensor, weight: torch.Tensor, eps: float, out_dtype: torch.dtype,
         rows: Optional[torch.Tensor] = None) -> torch.Tensor:
    """[n, D] in ``out_dtype``: the RMS norm (``eps`` inside the root, weight float32 [D]) of
    ``sum_s w_in[s] X[:, s]``; ``rows`` int32: only these tokens, in this order."""
    require_device(X, w_in, weight, rows)
    require_contiguous(X=X, w_in=w_in, weight=weight, rows=rows)
    _check_streams(X, "streams.read")
    N, S, D = X.shape
    _check_vector(w_in, S, "streams.read: w_in")
    _check_vector(weight, D, "streams.read: the norm weight")
    if rows is not None and rows.dtype != torch.int32:
        raise KernelError("streams.read: rows must be int32")
    if out_dtype not in (torch.float32, torch.bfloat16):
        raise KernelError("streams.read: float32 or bfloat16")
    n = N if rows is None else rows.numel()
    out = torch.empty((n, D), dtype=out_dtype, device=X.device)
    check(library("streams").gfa_streams_read(
        ptr(X), ptr(w_in), ptr(weight), _f(eps), ptr(rows), ptr(out), _i(int(out_dtype == torch.bfloat16)),
        _i(n), _i(S), _i(D), stream_handle()), "streams_read")
    return out


def join(X: torch.Tensor, y: torch.Tensor, mix: torch.Tensor, w_out: torch.Tensor,
         next_in: Optional[torch.Tensor] = None, next_weight: Optional[torch.Tensor] = None,
         next_eps: float = 0.0, out_dtype: Optional[torch.dtype] = None) -> Optional[torch.Tensor]:
    """In place, all streams from the old ones: ``X_t <- sum_s mix[s, t] X_s + w_out[t] y``.  With
    ``next_in`` also returns what :func:`read` makes of the new streams with ``next_in``,
    ``next_weight``, ``next_eps``, from the same pass.  y: float32 or bfloat16 [N, D], or float32
    [P, N, D], partial sums that are added in order."""
    require_device(X, y, mix, w_out, next_in, next_weight)
    require_contiguous(X=X, y=y, mix=mix, w_out=w_out, next_in=next_in, next_weight=next_weight)
    _check_streams(X, "streams.join")
    N, S, D = X.shape
    if tuple(y.shape[-2:]) != (N, D) or y.dim() not in (2, 3) or y.dtype not in (torch.float32, torch.bfloat16) \
            or (y.dim() == 3 and (y.dtype != torch.float32 or y.shape[0] < 1)):
        raise KernelError(f"streams.join: y {tuple(y.shape)} {y.dtype} does not fit streams {tuple(X.shape)}")
    _check_vector(mix, S * S, "streams.join: mix")
    _check_vector(w_out, S, "streams.join: w_out")
    out = None
    if next_in is not None:
        _check_vector(next_in, S, "streams.join: next_in")
        if next_weight is None or out_dtype not in (torch.float32, torch.bfloat16):
            raise KernelError("streams.join: the next read needs its norm weight and output type")
        _check_vector(next_weight, D, "streams.join: the next norm's weight")
        out = torch.empty((N, D), dtype=out_dtype, device=X.device)
    check(library("streams").gfa_streams_join(
        ptr(X), ptr(y), _i(int(y.dtype == torch.bfloat16)), _i(y.shape[0] if y.dim() == 3 else 1), ptr(mix),
        ptr(w_out), ptr(next_in), ptr(next_weight), _f(next_eps), ptr(out),
        _i(int(out is not None and out.dtype == torch.bfloat16)), _i(N), _i(S), _i(D), stream_handle()),
        "streams_join")
    return out
