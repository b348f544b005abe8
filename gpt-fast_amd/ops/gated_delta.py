"""Python faces of the gated-delta-rule kernels of csrc/gated_delta.hip and csrc/delta_chunks.hip: the
cell behind the short causal convolutions (ops/short_conv.py), token by token, a chunk of tokens at
a time in one kernel, and all chunks at once with one small kernel that walks them.  Shape checks on
the host, then the launch."""
import ctypes
from dataclasses import dataclass
from typing import Optional

import torch

from .library import KernelError, check, library, ptr, require_contiguous, require_device, stream_handle

_i, _f, _sz = ctypes.c_int, ctypes.c_float, ctypes.c_size_t

MAX_KEY_DIM = 512            # rows of S a workgroup's threads hold in registers


@dataclass(frozen=True)
class RowLayout:
    """Where a token's values lie in a row of the fused projection (column offsets, in
    elements): the convolved channels q, k, v first (``conv`` of them), then the
    pre-activations of beta and of the decay (one per head each), then the output gate.  Where
    the decay or the gate is a product of two matrices, ``a`` or ``g`` is the place of the first
    one's ``a_rank`` or ``g_rank`` sums, padded to a multiple of eight."""
    width: int
    conv: int
    b: int
    a: int
    g: int
    a_rank: int = 0
    g_rank: int = 0

    @staticmethod
    def fused(n_heads: int, n_kv_heads: int, key_dim: int, value_dim: int) -> "RowLayout":
        conv = 2 * n_kv_heads * key_dim + n_heads * value_dim
        b = conv
        a = b + n_heads
        g = a + n_heads
        return RowLayout(g + n_heads * value_dim, conv, b, a, g)

    @staticmethod
    def low_rank(n_heads: int, n_kv_heads: int, key_dim: int, value_dim: int, a_rank: int,
                 g_rank: int) -> "RowLayout":
        """Decay and gate (each: a rank, or 0 for none) through two matrices; every part behind the
        convolved channels starts at a multiple of eight, and the two first products lie side by
        side at the row's end."""
        up = lambda n: (n + 7) // 8 * 8
        conv = 2 * n_kv_heads * key_dim + n_heads * value_dim
        b = up(conv)
        a = b + n_heads                            # one per head,
        g = up(a + (0 if a_rank else n_heads))     # or a gate as wide as the values
        first = up(g + (0 if g_rank else n_heads * value_dim))
        return RowLayout(first + up(a_rank) + up(g_rank), conv, b, first if a_rank else a,
                         first + up(a_rank) if g_rank else g, up(a_rank), up(g_rank))

    def shifted(self, column: int, width: int) -> "RowLayout":
        """The same row as part of a wider one, from ``column`` on (``conv`` stays a count)."""
        return RowLayout(width, self.conv, self.b + column, self.a + column, self.g + column, self.a_rank,
                         self.g_rank)


def state_size(n_heads: int, n_kv_heads: int, key_dim: int, value_dim: int, taps: int) -> int:
    """float32 elements of one sequence's state: S [H, dk, dv], then the convolutions' last
    ``taps - 1`` inputs [taps - 1, C]."""
    conv = 2 * n_kv_heads * key_dim + n_heads * value_dim
    return n_heads * key_dim * value_dim + (taps - 1) * conv


def _check_step(proj, layout, state, q_start, slots, n_seqs):
    for name, t in (("proj", proj), ("state", state)):
        if t.dtype != torch.float32:
            raise KernelError(f"gated delta: {name} must be float32, is {t.dtype}")
    for name, t in (("q_start", q_start), ("slots", slots)):
        if t.dtype != torch.int32:
            raise KernelError(f"gated delta: {name} must be int32")
    if proj.dim() != 2 or proj.shape[1] != layout.width:
        raise KernelError(f"gated delta: rows are {tuple(proj.shape)}, expected [N, {layout.width}]")
    if q_start.numel() < n_seqs + 1 or slots.numel() < n_seqs:
        raise KernelError("gated delta: q_start / slots are shorter than the batch")


CHUNKS_FROM_TOKENS = 16      # runs shorter than this go token by token


def chunks_available(key_dim: int, value_dim: int) -> bool:
    return bool(library("gated_delta").gfa_gated_delta_chunks_take(_i(key_dim), _i(value_dim)))


PARALLEL_CHUNK = 64          # tokens per chunk of csrc/delta_chunks.hip
# (sequence, chunk, head) triples whose intermediate matrices are in memory at once (0.2 MB each for
# 128 x 128 heads); longer prompts go through in several rounds
PARALLEL_TRIPLES = 8192


def parallel_chunks_available(key_dim: int, value_dim: int) -> bool:
    return bool(library("delta_chunks").gfa_delta_chunks_take(_i(key_dim), _i(value_dim)))


def cell(conv, proj, layout, A_log, dt_bias, state, q_start, slots, n_seqs, max_q_len, n_heads,
         n_kv_heads, key_dim, value_dim, q_scale, unit_eps, decays=None) -> torch.Tensor:
    """Which kernels run the cell: token by token for short runs (single-token steps), chunks of
    tokens where some sequence brings many."""
    chunked = False
    if max_q_len >= CHUNKS_FROM_TOKENS:
        if parallel_chunks_available(key_dim, value_dim):
            return parallel_chunks(conv, proj, layout, A_log, dt_bias, state, q_start, slots, n_seqs,
                                   max_q_len, n_heads, n_kv_heads, key_dim, value_dim, q_scale, unit_eps,
                                   decays=decays)
        chunked = decays is None and chunks_available(key_dim, value_dim)
    return scan(conv, proj, layout, A_log, dt_bias, state, q_start, slots, n_seqs, n_heads, n_kv_heads,
                key_dim, value_dim, q_scale, unit_eps, chunked=chunked, max_q_len=max_q_len, decays=decays)


def scan(conv: torch.Tensor, proj: torch.Tensor, layout: RowLayout, A_log: torch.Tensor,
         dt_bias: torch.Tensor, state: torch.Tensor, q_start, slots, n_seqs: int, n_heads: int,
         n_kv_heads: int, key_dim: int, value_dim: int, q_scale: float, unit_eps: float,
         chunked: bool = False, max_q_len: int = 64, decays: Optional[torch.Tensor] = None) -> torch.Tensor:
    """The cell over every sequence's new tokens in order; ``state`` [slots, size] holds S
    [H, dk, dv] at its start and is read and left updated.  conv float32 [N, C]: q, k, v after
    their convolutions; proj float32 [N, layout.width] holds the pre-activations of beta and
    of the decay; A_log, dt_bias float32 [H].  Returns o float32 [N, H * dv].  ``chunked``:
    the kernel that takes a chunk of tokens at a time (the same arithmetic written out; chunks
    of 64 tokens if ``max_q_len``, the longest run of new tokens, is beyond 32, else of 32).
    ``decays`` float32 [N, >= H * dk] (unit stride along a row): a decay per head and key channel
    with these pre-activations; dt_bias is then float32 [H * dk]."""
    C, out = _check_cell(conv, proj, layout, A_log, dt_bias, state, q_start, slots, n_seqs, n_heads, n_kv_heads,
                         key_dim, value_dim, decays)
    lib = library("gated_delta")
    if chunked and (decays is not None or not chunks_available(key_dim, value_dim)):
        raise KernelError("gated delta: the chunked kernel does not take these sizes")
    head = (ptr(conv), _i(C), ptr(proj), _i(layout.width), _i(layout.b), _i(layout.a))
    if not chunked:
        head += (ptr(decays), _i(0 if decays is None else decays.stride(0)))
    head += (ptr(A_log), ptr(dt_bias), ptr(state), _sz(state.stride(0)), ptr(q_start), ptr(slots), ptr(out),
             _i(n_seqs))
    tail = (_i(n_heads), _i(n_kv_heads), _i(key_dim), _i(value_dim), _f(q_scale), _f(unit_eps),
            stream_handle())
    if chunked:
        check(lib.gfa_gated_delta_chunks(*head, _i(int(max_q_len)), *tail), "gated_delta_chunks")
    else:
        check(lib.gfa_gated_delta_scan(*head, *tail), "gated_delta_scan")
    return out


def parallel_chunks(conv, proj, layout: RowLayout, A_log, dt_bias, state, q_start, slots, n_seqs: int,
                    max_q_len: int, n_heads: int, n_kv_heads: int, key_dim: int, value_dim: int,
                    q_scale: float, unit_eps: float, decays: Optional[torch.Tensor] = None,
                    chunks_at_once: Optional[int] = None) -> torch.Tensor:
    """:func:`scan` over chunks of 64 tokens: what a chunk does to the state, whatever the state is,
    is worked out for all chunks at once, and a small kernel walks them (csrc/delta_chunks.hip).
    ``max_q_len``: the longest run of new tokens; ``chunks_at_once``: chunks of each sequence per
    round (None: by PARALLEL_TRIPLES)."""
    C, out = _check_cell(conv, proj, layout, A_log, dt_bias, state, q_start, slots, n_seqs, n_heads, n_kv_heads,
                         key_dim, value_dim, decays)
    if not parallel_chunks_available(key_dim, value_dim):
        raise KernelError("gated delta: the parallel chunks' kernels do not take these sizes")
    lib = library("delta_chunks")
    chunks = (int(max_q_len) + PARALLEL_CHUNK - 1) // PARALLEL_CHUNK
    seg = chunks_at_once or max(1, PARALLEL_TRIPLES // (n_seqs * n_heads))
    seg = min(seg, chunks)
    sizes = [ctypes.c_int() for _ in range(4)]
    lib.gfa_delta_chunks_floats(_i(key_dim), _i(value_dim), *(ctypes.byref(n) for n in sizes))
    triples = n_seqs * seg * n_heads
    room = torch.empty(triples * sum(n.value for n in sizes), dtype=torch.float32, device=proj.device)
    parts, at = [], 0
    for n in sizes:                                # every size is a multiple of 256 floats
        parts.append(room[at:])
        at += triples * n.value
    check(lib.gfa_delta_chunks(
        ptr(conv), _i(C), ptr(proj), _i(layout.width), _i(layout.b), _i(layout.a), ptr(decays),
        _i(0 if decays is None else decays.stride(0)), ptr(A_log), ptr(dt_bias), ptr(state),
        _sz(state.stride(0)), ptr(q_start), ptr(slots), ptr(out), *(ptr(p) for p in parts), _i(n_seqs),
        _i(int(max_q_len)), _i(seg), _i(n_heads), _i(n_kv_heads), _i(key_dim), _i(value_dim), _f(q_scale),
        _f(unit_eps), stream_handle()), "delta_chunks")
    return out


def _check_cell(conv, proj, layout, A_log, dt_bias, state, q_start, slots, n_seqs, n_heads, n_kv_heads, key_dim,
                value_dim, decays):
    """Shape checks of the cell's arguments: (convolved channels, a new tensor for the result)."""
    require_device(conv, proj, A_log, dt_bias, state, q_start, slots, decays)
    require_contiguous(conv=conv, proj=proj, A_log=A_log, dt_bias=dt_bias, state=state,
                       q_start=q_start, slots=slots)
    if decays is not None and (decays.dtype != torch.float32 or decays.dim() != 2 or decays.stride(1) != 1
                               or decays.shape[0] != proj.shape[0] or decays.shape[1] < n_heads * key_dim):
        raise KernelError(f"gated delta: decays must be float32 [N, >= {n_heads * key_dim}]")
    _check_step(proj, layout, state, q_start, slots, n_seqs)
    C = 2 * n_kv_heads * key_dim + n_heads * value_dim
    if conv.dtype != torch.float32 or tuple(conv.shape) != (proj.shape[0], C) or layout.conv != C:
        raise KernelError(f"gated delta: the convolved rows must be float32 [N, {C}]")
    for name, t, count in (("A_log", A_log, n_heads),
                           ("dt_bias", dt_bias, n_heads * (1 if decays is None else key_dim))):
        if t.dtype != torch.float32 or t.numel() != count:
            raise KernelError(f"gated delta: {name} must be float32 [{count}]")
    if n_heads % n_kv_heads or key_dim > MAX_KEY_DIM:
        raise KernelError(f"gated delta: {n_heads} heads over {n_kv_heads} key heads of {key_dim}")
    if state.dim() != 2 or state.shape[1] < n_heads * key_dim * value_dim:
        raise KernelError("gated delta: the state is smaller than S [H, dk, dv]")
    out = torch.empty((proj.shape[0], n_heads * value_dim), dtype=torch.float32, device=proj.device)
    return C, out
