"""Recurrent mixer: a state-space cell with a decay per token behind a short causal convolution
(Mamba-2)."""
import dataclasses

import torch

from ..cache.store import StateNeed
from ..config.spec import StateSpaceSpec
from ..ops import decayed_memory as DM
from ..ops import linear as L
from ..ops import short_conv as SC
from ..ops import state_space as SS
from .base import Param, Part, Runtime, add_late, check_bound, register_mixer


class StateSpace(Part):
    """Per head a state ``S [N, dv]``, float32, zero at a sequence's start, kept in the cache's
    state slot of the sequence together with the convolution's last inputs:

        z, xBC, dt' = w_in h                       x, B, C = silu(conv(xBC) + conv_bias)
        dt = softplus(dt' + dt_bias)               (per head; B and C per group of heads)
        S <- exp(-exp(A_log) dt) S + dt B x^T      y = S^T C + skip x

    then all heads' y times silu(z), then every one of ``norm_groups`` parts over its root mean
    square, times ``norm``, then ``wo``.  The input projection keeps its float32 sums: the
    convolution, the step sizes, the state and everything up to the operand of ``wo`` are float32
    whatever the engine's type."""

    replayable = True
    libraries = ("state_space", "short_conv", "decayed_memory")
    defers_sum = True              # ``residual`` may be a parts.base.ResidualStream

    def __init__(self, spec: StateSpaceSpec, runtime: Runtime):
        s = spec
        if s.n_heads % s.n_groups or (s.n_heads * s.value_dim) % s.norm_groups:
            raise ValueError(f"state space: {s.n_heads} heads of {s.value_dim} in {s.n_groups} groups, "
                             f"{s.norm_groups} norm groups")
        if not 1 <= s.state <= SS.MAX_STATE or not 1 <= s.conv_taps <= SC.MAX_TAPS:
            raise ValueError(f"state space: {s.state} states (up to {SS.MAX_STATE}), "
                             f"{s.conv_taps} taps (1..{SC.MAX_TAPS})")
        self.spec = spec
        self.rt = runtime
        rows = SS.RowLayout.fused(s.n_heads, s.value_dim, s.n_groups, s.state)
        self.in_rows = rows.width                       # rows of w_in as it is stored
        self.rows = dataclasses.replace(rows, width=(rows.width + 7) // 8 * 8)
        self.tail_offset = s.n_heads * s.state * s.value_dim
        self.w_in = self.wo = self.taps = self.conv_bias = self.norm = None
        self.A_log = self.dt_bias = self.skip = None

    def parameters(self):
        s = self.spec
        inner = s.n_heads * s.value_dim
        return {"w_in": Param((self.in_rows, s.dim)),
                "taps": Param((self.rows.conv, s.conv_taps), role="vector", init="unit"),
                "conv_bias": Param((self.rows.conv,), role="vector", init="around_zero"),
                "A_log": Param((s.n_heads,), role="vector", init="around_zero"),
                "dt_bias": Param((s.n_heads,), role="vector", init="around_zero"),
                "skip": Param((s.n_heads,), role="vector", init="norm"),
                "norm": Param((inner,), role="vector", init="norm"),
                "wo": Param((s.dim, inner))}

    def bind(self, tensors):
        check_bound("StateSpace", self.parameters(), tensors)
        # zero rows up to a multiple of eight: the products' kernels store whole groups
        self.w_in, self.wo = L.pad_rows(tensors["w_in"], 8), tensors["wo"]
        for name in ("taps", "conv_bias", "A_log", "dt_bias", "skip", "norm"):
            setattr(self, name, tensors[name].to(torch.float32).contiguous())

    def cache_need(self):
        s = self.spec
        # (a multiple of four floats: slots that start where 16-byte loads may)
        size = SS.state_size(s.n_heads, s.value_dim, s.n_groups, s.state, s.conv_taps)
        return StateNeed(((size + 3) // 4 * 4,), "float32")

    def step_flops(self, q_lens, starts) -> float:
        s = self.spec
        n = sum(q_lens)
        cell = 2.0 * 2.0 * s.n_heads * s.state * s.value_dim            # update and read of S
        return n * (2.0 * (self.in_rows + s.n_heads * s.value_dim) * s.dim + cell
                    + 2.0 * self.rows.conv * s.conv_taps)

    def _gated(self, x, batch, entry):
        s = self.spec
        proj = L.linear(x, self.w_in, out_dtype=torch.float32)
        conv = SC.short_conv(proj, self.taps, entry.state, self.tail_offset, batch.tok_seq, batch.q_start,
                             batch.slots, batch.n_seqs, bias=self.conv_bias, column=self.rows.conv_at,
                             max_q_len=batch.max_q_len)
        y = SS.cell(conv, proj, self.rows, self.A_log, self.dt_bias, self.skip, entry.state,
                    batch.q_start, batch.slots, batch.n_seqs, batch.max_q_len, s.n_heads, s.n_groups,
                    s.state, s.value_dim)
        return DM.row_norm_gate(y, self.norm, proj, self.rows, s.eps, self.rt.dtype,
                                groups=s.norm_groups, gate="silu", gate_first=True)

    def forward(self, x, batch, entry, residual):
        y = self._gated(x, batch, entry)
        add_late(residual, lambda rows, then_norm, takes_halves: L.linear_into(
            y, self.wo, rows, then_norm, takes_halves))

    def forward_last(self, x, batch, entry):
        """The operand and the matrix of the last product, which the block runs."""
        return self._gated(x, batch, entry), self.wo

    def forward_rows(self, x, batch, entry):
        """The mixer's output alone: the output projection's float32 sums."""
        return L.linear(self._gated(x, batch, entry), self.wo, out_dtype=torch.float32)


register_mixer("state_space", StateSpace)
