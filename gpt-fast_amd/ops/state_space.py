"""Python faces of the state-space cell's kernels (csrc/state_space.hip), token by token and a
chunk of tokens at a time.  Shape checks on the host, then the launch."""
import ctypes
from dataclasses import dataclass

import torch

from .library import KernelError, check, library, ptr, require_contiguous, require_device, stream_handle

_i, _sz = ctypes.c_int, ctypes.c_size_t

MAX_STATE = 512              # rows of S a workgroup's threads hold in registers


@dataclass(frozen=True)
class RowLayout:
    """Where a token's values lie in a row of the fused projection (column offsets, in
    elements): the gate z (at ``g``), then the ``conv`` convolved channels x, B, C (from
    ``conv_at`` on), then one step size per head (``dt``)."""
    width: int
    g: int
    conv_at: int
    conv: int
    dt: int

    @staticmethod
    def fused(n_heads: int, value_dim: int, n_groups: int, state: int) -> "RowLayout":
        inner = n_heads * value_dim
        conv = inner + 2 * n_groups * state
        return RowLayout(inner + conv + n_heads, 0, inner, conv, inner + conv)


def state_size(n_heads: int, value_dim: int, n_groups: int, state: int, taps: int) -> int:
    """float32 elements of one sequence's state: S [H, N, dv], then the convolution's last
    ``taps - 1`` inputs [taps - 1, C]."""
    return n_heads * state * value_dim + (taps - 1) * (n_heads * value_dim + 2 * n_groups * state)


CHUNKS_FROM_TOKENS = 16      # runs shorter than this go token by token


def chunks_available(state: int, value_dim: int) -> bool:
    return bool(library("state_space").gfa_state_space_chunks_take(_i(state), _i(value_dim)))


def cell(conv, proj, layout, A_log, dt_bias, skip, state, q_start, slots, n_seqs, max_q_len, n_heads,
         n_groups, n_state, value_dim) -> torch.Tensor:
    """Which kernel runs the cell: token by token for short runs (single-token steps), a chunk
    of tokens at a time where some sequence brings many."""
    chunked = max_q_len >= CHUNKS_FROM_TOKENS and chunks_available(n_state, value_dim)
    return scan(conv, proj, layout, A_log, dt_bias, skip, state, q_start, slots, n_seqs, n_heads,
                n_groups, n_state, value_dim, chunked=chunked, max_q_len=max_q_len)


def scan(conv: torch.Tensor, proj: torch.Tensor, layout: RowLayout, A_log: torch.Tensor,
         dt_bias: torch.Tensor, skip: torch.Tensor, state: torch.Tensor, q_start, slots, n_seqs: int,
         n_heads: int, n_groups: int, n_state: int, value_dim: int, chunked: bool = False,
         max_q_len: int = 64) -> torch.Tensor:
    """The cell over every sequence's new tokens in order; ``state`` [slots, size] holds S
    [H, N, dv] at its start and is read and left updated.  conv float32 [N, C]: x, B, C after the
    convolution; proj float32 [N, layout.width] holds the step sizes' pre-activations; A_log,
    dt_bias, skip float32 [H].  Returns y float32 [N, H * dv] with the skip ``D x`` added.
    ``chunked``: the kernel that takes a chunk of tokens at a time (chunks of 64 tokens if
    ``max_q_len``, the longest run of new tokens, is beyond 32, else of 32)."""
    require_device(conv, proj, A_log, dt_bias, skip, state, q_start, slots)
    require_contiguous(conv=conv, proj=proj, A_log=A_log, dt_bias=dt_bias, skip=skip, state=state,
                       q_start=q_start, slots=slots)
    for name, t in (("conv", conv), ("proj", proj), ("state", state), ("A_log", A_log),
                    ("dt_bias", dt_bias), ("skip", skip)):
        if t.dtype != torch.float32:
            raise KernelError(f"state space: {name} must be float32, is {t.dtype}")
    for name, t in (("q_start", q_start), ("slots", slots)):
        if t.dtype != torch.int32:
            raise KernelError(f"state space: {name} must be int32")
    C = n_heads * value_dim + 2 * n_groups * n_state
    if proj.dim() != 2 or proj.shape[1] != layout.width or layout.dt + n_heads > layout.width:
        raise KernelError(f"state space: rows are {tuple(proj.shape)}, expected [N, {layout.width}]")
    if tuple(conv.shape) != (proj.shape[0], C) or layout.conv != C:
        raise KernelError(f"state space: the convolved rows must be float32 [N, {C}]")
    for name, t in (("A_log", A_log), ("dt_bias", dt_bias), ("skip", skip)):
        if t.numel() != n_heads:
            raise KernelError(f"state space: {name} must have {n_heads} elements")
    if n_groups < 1 or n_heads % n_groups or not 1 <= n_state <= MAX_STATE:
        raise KernelError(f"state space: {n_heads} heads over {n_groups} groups of {n_state} states "
                          f"(up to {MAX_STATE})")
    if state.dim() != 2 or state.shape[1] < n_heads * n_state * value_dim:
        raise KernelError("state space: the state is smaller than S [H, N, dv]")
    if q_start.numel() < n_seqs + 1 or slots.numel() < n_seqs:
        raise KernelError("state space: q_start / slots are shorter than the batch")
    out = torch.empty((proj.shape[0], n_heads * value_dim), dtype=torch.float32, device=proj.device)
    lib = library("state_space")
    if chunked and not chunks_available(n_state, value_dim):
        raise KernelError("state space: the chunked kernel does not take these sizes")
    head = (ptr(conv), _i(C), ptr(proj), _i(layout.width), _i(layout.dt), ptr(A_log), ptr(dt_bias),
            ptr(skip), ptr(state), _sz(state.stride(0)), ptr(q_start), ptr(slots), ptr(out), _i(n_seqs))
    tail = (_i(n_heads), _i(n_groups), _i(n_state), _i(value_dim), stream_handle())
    if chunked:
        check(lib.gfa_state_space_chunks(*head, _i(int(max_q_len)), *tail), "state_space_chunks")
    else:
        check(lib.gfa_state_space_scan(*head, *tail), "state_space_scan")
    return out
