"""Python face of csrc/short_conv.hip: short causal convolutions over time with their tails.
Shape checks on the host, then the launch."""
import ctypes
from typing import Optional

import torch

from .library import KernelError, check, library, ptr, require_contiguous, require_device, stream_handle

_i, _sz = ctypes.c_int, ctypes.c_size_t

MAX_TAPS = 16


def short_conv(proj: torch.Tensor, taps: torch.Tensor, state: torch.Tensor, tail_offset: int, tok_seq,
               q_start, slots, n_seqs: int, bias: Optional[torch.Tensor] = None, column: int = 0,
               max_q_len: int = 0) -> torch.Tensor:
    """silu of the causal convolution of C columns of proj (float32 [N, W], from ``column`` on)
    over each sequence's tokens, float32 [N, C]; taps float32 [C, K], the last column the
    current token's; bias float32 [C] or None.  ``state`` [slots, size] holds every sequence's
    last K - 1 inputs at ``tail_offset`` ([K - 1, C], oldest first; zero for a new sequence) and
    is left holding the step's.  ``max_q_len`` 1 says that no sequence brings more than one
    token (0: not known)."""
    require_device(proj, taps, bias, state, tok_seq, q_start, slots)
    require_contiguous(proj=proj, taps=taps, bias=bias, state=state, tok_seq=tok_seq, q_start=q_start,
                       slots=slots)
    for name, t in (("proj", proj), ("taps", taps), ("bias", bias), ("state", state)):
        if t is not None and t.dtype != torch.float32:
            raise KernelError(f"short_conv: {name} must be float32, is {t.dtype}")
    for name, t in (("tok_seq", tok_seq), ("q_start", q_start), ("slots", slots)):
        if t.dtype != torch.int32:
            raise KernelError(f"short_conv: {name} must be int32")
    if taps.dim() != 2 or not 1 <= taps.shape[1] <= MAX_TAPS:
        raise KernelError(f"short_conv: taps must be [C, 1..{MAX_TAPS}], are {tuple(taps.shape)}")
    C, K = taps.shape
    if proj.dim() != 2 or column < 0 or column + C > proj.shape[1]:
        raise KernelError(f"short_conv: {C} channels from column {column} of rows {tuple(proj.shape)}")
    if bias is not None and bias.numel() != C:
        raise KernelError(f"short_conv: bias must have {C} elements")
    if state.dim() != 2 or tail_offset < 0 or tail_offset + (K - 1) * C > state.shape[1]:
        raise KernelError("short_conv: the tails do not fit the state")
    if tok_seq.numel() < proj.shape[0] or q_start.numel() < n_seqs + 1 or slots.numel() < n_seqs:
        raise KernelError("short_conv: tok_seq / q_start / slots are shorter than the batch")
    y = torch.empty((proj.shape[0], C), dtype=torch.float32, device=proj.device)
    check(library("short_conv").gfa_short_conv(
        ptr(proj), _i(proj.shape[1]), _i(column), ptr(taps), ptr(bias), _i(K), _i(C), ptr(state),
        _sz(state.stride(0)), _sz(tail_offset), ptr(tok_seq), ptr(q_start), ptr(slots), ptr(y),
        _i(proj.shape[0]), _i(n_seqs), _i(max_q_len), stream_handle()), "short_conv")
    return y
