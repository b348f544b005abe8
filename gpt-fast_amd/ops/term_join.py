"""Python face of csrc/term_join.hip: several results join the residual stream in one pass.  Shape
checks on the host, then the launch."""
import ctypes
from typing import Optional, Sequence, Tuple

import torch

from .library import KernelError, check, library, ptr, require_contiguous, require_device, stream_handle

_i, _f = ctypes.c_int, ctypes.c_float

MAX_TERMS = 4
NORMS = {None: 0, "plain": 0, "layer": 1, "rms": 2}


def join(residual: torch.Tensor, terms: Sequence[Tuple[torch.Tensor, float]], norm: Optional[str] = None,
         weight: Optional[torch.Tensor] = None, bias: Optional[torch.Tensor] = None, eps: float = 0.0,
         out_dtype: Optional[torch.dtype] = None) -> Optional[torch.Tensor]:
    """residual (float32 [N, D], in place) += sum of ``factor * y`` over ``terms`` = (y, factor), y
    float32 or bfloat16 [N, D] or float32 [S, N, D] (partial sums, added in order).  With ``norm``
    also returns, from the same pass and in ``out_dtype``, the new rows ("plain"), their layer norm
    ("layer", with ``weight``, ``bias`` or None, ``eps``) or their RMS norm ("rms", ``weight``, ``eps``)."""
    require_device(residual, weight, bias, *(y for y, _ in terms))
    require_contiguous(residual=residual, weight=weight, bias=bias,
                       **{f"term {i}": y for i, (y, _) in enumerate(terms)})
    if residual.dim() != 2 or residual.dtype != torch.float32:
        raise KernelError("term_join: the stream must be float32 [N, D]")
    if not 1 <= len(terms) <= MAX_TERMS or norm not in NORMS:
        raise KernelError(f"term_join: 1..{MAX_TERMS} terms, norm in {list(NORMS)}")
    N, D = residual.shape
    mask = 0
    for i, (y, _) in enumerate(terms):
        if tuple(y.shape[-2:]) != (N, D) or y.dim() not in (2, 3) \
                or y.dtype not in (torch.float32, torch.bfloat16) \
                or (y.dim() == 3 and (y.dtype != torch.float32 or y.shape[0] < 1)):
            raise KernelError(f"term_join: term {tuple(y.shape)} {y.dtype} does not fit {tuple(residual.shape)}")
        mask |= int(y.dtype == torch.bfloat16) << i
    for name, t in (("weight", weight), ("bias", bias)):
        if t is not None and (t.dtype != torch.float32 or t.numel() != D):
            raise KernelError(f"term_join: {name} must be float32 [{D}]")
    if norm in ("layer", "rms") and weight is None or (bias is not None and norm != "layer"):
        raise KernelError("term_join: a norm needs its weight, and only a layer norm takes a bias")
    out = None
    if norm is not None:
        if out_dtype not in (torch.float32, torch.bfloat16):
            raise KernelError("term_join: float32 or bfloat16")
        out = torch.empty((N, D), dtype=out_dtype, device=residual.device)
    ys = [y for y, _ in terms] + [None] * (MAX_TERMS - len(terms))
    check(library("term_join").gfa_term_join(
        ptr(residual), *(ptr(y) for y in ys), _i(len(terms)), _i(mask),
        *(_i(y.shape[0] if y is not None and y.dim() == 3 else 1) for y in ys),
        *(_f(float(terms[i][1]) if i < len(terms) else 0.0) for i in range(MAX_TERMS)),
        _i(NORMS[norm]), ptr(weight), ptr(bias), _f(eps), ptr(out),
        _i(int(out is not None and out.dtype == torch.bfloat16)), _i(N), _i(D), stream_handle()), "term_join")
    return out
