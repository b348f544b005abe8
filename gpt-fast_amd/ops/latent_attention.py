"""Python face of csrc/latent_attention.hip: many query heads over one cached key / value head.
Rows and sizes the matrix-core kernels do not take go to the general kernels
(``ops.scored_attention``)."""
import ctypes
from typing import Optional

import torch

from . import linear as L
from . import scored_attention as SA
from .kernels import PAGE
from .library import KernelError, check, library, ptr, require_contiguous, require_device, stream_handle

_i, _f, _ll = ctypes.c_int, ctypes.c_float, ctypes.c_longlong

BLOCK = 32                   # keys a workgroup has in shared memory at a time (two such blocks)
MAX_PARTS = 64


def parts(n_heads: int, n_seqs: int, pages: int, window: int, units: int) -> int:
    """Parts that a single-token step's keys are cut into over workgroups, from the shapes alone
    (a recorded step serves every length its tables have room for): enough to give every
    compute unit a workgroup, as long as a part has two blocks of keys."""
    blocks = pages * PAGE // BLOCK
    if window:
        blocks = min(blocks, (window + BLOCK - 2) // BLOCK + 1)
    groups = (n_heads + 63) // 64 * n_seqs
    return max(1, min(units // max(groups, 1), (blocks + 1) // 2, MAX_PARTS))


def attention(q: torch.Tensor, k_pages: torch.Tensor, v_pages: torch.Tensor, tok_seq, tok_pos, table,
              scale: float, step, *, window: int = 0, gate: Optional[torch.Tensor] = None,
              n_parts: Optional[int] = None) -> torch.Tensor:
    """q [H, N, hd] head by head, k_pages [pages, 1, 64, hd], v_pages [pages, 1, vd, 64] -> [H, N, vd];
    ``step`` = (q_start int32 [B + 1], start_pos int32 [B], B, longest run of new tokens); gate
    float32 [N, >= H] (a view allowed): head h of token n times ``sigmoid(gate[n, h])``.
    ``n_parts``: parts of the keys in a single-token step (None: :func:`parts`)."""
    H, n, hd = q.shape
    vd = v_pages.shape[2]
    # the library is asked for only where its kernels could run: a float32 engine has no use for it
    if q.dtype != torch.bfloat16 or q.data_ptr() % 16 or q.stride(0) % 8 or q.stride(1) % 8 or q.stride(2) != 1 \
            or not library("latent_attention").gfa_latent_attention_takes(_i(H), _i(hd), _i(vd)):
        return SA.attention(q, k_pages, v_pages, tok_seq, tok_pos, table, scale, window=window,
                            head_major=True, gate=gate, step=step)
    q_start, start_pos, n_seqs, max_q_len = step
    require_device(q, k_pages, v_pages, table, q_start, start_pos, gate)
    require_contiguous(table=table, q_start=q_start, start_pos=start_pos)
    SA._check_pages(k_pages, v_pages, 1, hd, vd, q.dtype)
    for name, t, count in (("q_start", q_start, n_seqs + 1), ("start_pos", start_pos, n_seqs), ("table", table, 0)):
        if t.dtype != torch.int32 or t.numel() < count:
            raise KernelError(f"latent attention: {name} must be int32 and cover the batch")
    if table.dim() != 2 or table.shape[0] < n_seqs:
        raise KernelError("latent attention: the table must have a row per sequence")
    if gate is not None and (gate.dtype != torch.float32 or gate.dim() != 2 or gate.shape[0] != n
                             or gate.shape[1] < H or (H > 1 and gate.stride(1) != 1)):
        raise KernelError("latent attention: gate must be float32 [N, >= H] with unit stride along a row")
    out = torch.empty((H, n, vd), dtype=q.dtype, device=q.device)
    P, ml, po = 1, None, None
    if max_q_len == 1:
        P = n_parts or parts(H, n_seqs, table.shape[1], window, L._compute_units(q.device))
        if P > 1:
            ml = torch.empty((n_seqs, H, P, 2), dtype=torch.float32, device=q.device)
            po = torch.empty((n_seqs, H, P, vd), dtype=torch.float32, device=q.device)
    check(library("latent_attention").gfa_latent_attention(
        ptr(q), ptr(k_pages), ptr(v_pages), ptr(q_start), ptr(start_pos), ptr(table), _i(table.shape[1]),
        ptr(out), ptr(ml), ptr(po), _i(P), _i(n_seqs), _i(max_q_len), _i(H), _i(hd), _i(vd),
        _ll(q.stride(1)), _ll(q.stride(0)), _ll(out.stride(1)), _ll(out.stride(0)), _f(scale), _i(window or 0),
        ptr(gate), _ll(0 if gate is None else gate.stride(0)), stream_handle()), "latent_attention")
    return out
