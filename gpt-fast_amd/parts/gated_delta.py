"""Recurrent mixer with the gated delta rule behind short causal convolutions."""
import dataclasses

import torch

from ..cache.store import StateNeed
from ..config.spec import GatedDeltaSpec
from ..ops import decayed_memory as DM
from ..ops import gated_delta as GD
from ..ops import kernels as K
from ..ops import linear as L
from ..ops import short_conv as SC
from .base import Param, Part, Runtime, add_late, check_bound, register_mixer


class GatedDelta(Part):
    """Per head a state ``S [dk, dv]``, float32, zero at a sequence's start, kept in the cache's
    state slot of the sequence together with the convolutions' last inputs:

        q, k, v = silu(conv(w x))                         (a causal convolution per channel)
        q = q / |q| * dk^-1/2     k = k / |k|             (per head; |.| with unit_eps inside)
        beta = sigmoid(w_b x)     g = exp(-exp(A_log) softplus(w_a x + dt_bias))
        S <- g S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q

    then each head's o over its root mean square, times ``norm`` (shared by the heads), times
    silu (or, as the spec says, sigmoid) of w_g x, then ``wo``.  The input projections are one matrix
    ``w_in`` (rows of q, k, v, beta, the decay, the gate) whose product keeps its float32 sums: the
    convolutions, the gates, the state and everything up to the operand of ``wo`` are float32
    whatever the engine's type.

    With ``decay_rank`` the decay is a number per head and key channel, ``g = exp(-exp(A_log_h)
    softplus(w_a2 (w_a1 x) + dt_bias))`` on the rows of S, and with ``gate_rank`` the gate's projection
    is ``w_g2 (w_g1 x)``: w_a1 and w_g1 are the last rows of ``w_in``, and one further product with
    both second matrices (zeros between them) takes their sums to the channels."""

    replayable = True
    libraries = ("gated_delta", "delta_chunks", "short_conv", "decayed_memory")
    defers_sum = True              # ``residual`` may be a parts.base.ResidualStream

    def __init__(self, spec: GatedDeltaSpec, runtime: Runtime):
        s = spec
        if s.n_heads % s.n_kv_heads:
            raise ValueError(f"gated delta: {s.n_heads} heads do not divide into {s.n_kv_heads} key heads")
        if s.key_dim > GD.MAX_KEY_DIM or not 1 <= s.conv_taps <= SC.MAX_TAPS:
            raise ValueError(f"gated delta: key_dim {s.key_dim} (up to {GD.MAX_KEY_DIM}), "
                             f"{s.conv_taps} taps (1..{SC.MAX_TAPS})")
        self.spec = spec
        self.rt = runtime
        if s.gate not in ("silu", "sigmoid") or min(s.decay_rank or 1, s.gate_rank or 1) < 1:
            raise ValueError(f"gated delta: gate '{s.gate}' (silu or sigmoid), ranks {s.decay_rank}, {s.gate_rank}")
        self.ra, self.rg = s.decay_rank or 0, s.gate_rank or 0
        if self.ra or self.rg:
            self.rows = GD.RowLayout.low_rank(s.n_heads, s.n_kv_heads, s.key_dim, s.value_dim, self.ra, self.rg)
        else:
            rows = GD.RowLayout.fused(s.n_heads, s.n_kv_heads, s.key_dim, s.value_dim)
            self.rows = dataclasses.replace(rows, width=(rows.width + 7) // 8 * 8)
        # rows of w_in as it is stored, part by part, and where each part lies in a row of sums
        r, H = self.rows, s.n_heads
        self.in_parts = [(r.conv, 0), (H, r.b)]
        if not self.ra:
            self.in_parts.append((H, r.a))
        if not self.rg:
            self.in_parts.append((H * s.value_dim, r.g))
        self.in_parts += [(n, at) for n, at in ((self.ra, r.a), (self.rg, r.g)) if n]
        self.in_rows = sum(n for n, _ in self.in_parts)
        self.tail_offset = s.n_heads * s.key_dim * s.value_dim
        self.w_in = self.wo = self.taps = self.norm = self.A_log = self.dt_bias = self.w_second = None
        self._scaled_norms = {}

    def parameters(self):
        s = self.spec
        decays = s.n_heads * (s.key_dim if self.ra else 1)
        p = {"w_in": Param((self.in_rows, s.dim)),
             "taps": Param((self.rows.conv, s.conv_taps), role="vector", init="unit"),
             "A_log": Param((s.n_heads,), role="vector", init="around_zero"),
             "dt_bias": Param((decays,), role="vector", init="around_zero"),
             "norm": Param((s.value_dim,), role="vector", init="norm"),
             "wo": Param((s.dim, s.n_heads * s.value_dim))}
        if self.ra:
            p["w_a2"] = Param((decays, self.ra))
        if self.rg:
            p["w_g2"] = Param((s.n_heads * s.value_dim, self.rg))
        return p

    def bind(self, tensors):
        check_bound("GatedDelta", self.parameters(), tensors)
        # zero rows between the parts and up to a multiple of eight: the products' kernels store
        # whole groups
        w = tensors["w_in"]
        if self.rows.width != self.in_rows:
            w = w.new_zeros((self.rows.width, w.shape[1]))
            at = 0
            for n, place in self.in_parts:
                w[place:place + n] = tensors["w_in"][at:at + n]
                at += n
        self.w_in, self.wo = w, tensors["wo"]
        if self.ra or self.rg:
            s, r = self.spec, self.rows
            decays = s.n_heads * s.key_dim if self.ra else 0
            gates = s.n_heads * s.value_dim if self.rg else 0
            second = w.new_zeros(((decays + gates + 7) // 8 * 8, r.a_rank + r.g_rank))
            if self.ra:
                second[:decays, :self.ra] = tensors["w_a2"]
            if self.rg:
                second[decays:decays + gates, r.a_rank:r.a_rank + self.rg] = tensors["w_g2"]
            self.w_second = second
            self.second_rows = dataclasses.replace(r, width=second.shape[0], g=decays)
        f32 = lambda name: tensors[name].to(torch.float32).contiguous()
        self.taps, self.norm, self.A_log, self.dt_bias = f32("taps"), f32("norm"), f32("A_log"), f32("dt_bias")

    def cache_need(self):
        s = self.spec
        return StateNeed((GD.state_size(s.n_heads, s.n_kv_heads, s.key_dim, s.value_dim, s.conv_taps),),
                         "float32")

    def step_flops(self, q_lens, starts) -> float:
        s = self.spec
        n = sum(q_lens)
        cell = 2.0 * 3.0 * s.n_heads * s.key_dim * s.value_dim          # two reads and the update of S
        second = s.n_heads * (self.ra * s.key_dim + self.rg * s.value_dim)
        return n * (2.0 * (self.in_rows + s.n_heads * s.value_dim) * s.dim + 2.0 * second + cell
                    + 2.0 * self.rows.conv * s.conv_taps)

    def gated(self, proj, column, batch, entry, out=None, factor: float = 1.0):
        """The normed, gated heads side by side, [N, H * dv] (into ``out``, a view of wider rows),
        times ``factor``, from the float32 sums of the input projection, which lie in proj from
        ``column`` on."""
        s = self.spec
        rows = self.rows if proj.shape[1] == self.rows.width else self.rows.shifted(column, proj.shape[1])
        conv = SC.short_conv(proj, self.taps, entry.state, self.tail_offset, batch.tok_seq,
                             batch.q_start, batch.slots, batch.n_seqs, column=column, max_q_len=batch.max_q_len)
        second, decays, gates, gate_rows = None, None, proj, rows
        if self.w_second is not None:
            first = rows.a if self.ra else rows.g
            second = L.linear(K.cast_columns(proj, first, rows.a_rank + rows.g_rank, self.rt.dtype),
                              self.w_second, out_dtype=torch.float32)
            decays = second[:, :s.n_heads * s.key_dim] if self.ra else None
            if self.rg:
                gates, gate_rows = second, self.second_rows
        o = GD.cell(conv, proj, rows, self.A_log, self.dt_bias, entry.state, batch.q_start,
                    batch.slots, batch.n_seqs, batch.max_q_len, s.n_heads, s.n_kv_heads, s.key_dim,
                    s.value_dim, s.key_dim ** -0.5, s.unit_eps, decays=decays)
        norm = self.norm
        if factor != 1.0:
            norm = self._scaled_norms.get(factor)
            if norm is None:
                norm = self._scaled_norms[factor] = self.norm * factor
        return DM.row_norm_gate(o, norm, gates, gate_rows, s.eps, self.rt.dtype,
                                groups=s.n_heads, gate=s.gate, out=out)

    def _gated(self, x, batch, entry):
        return self.gated(L.linear(x, self.w_in, out_dtype=torch.float32), 0, batch, entry)

    # for a block or mixer that joins this part's first and last product with others': the rows it
    # reads, the row its results take in the last product's operand, and that product's matrix
    def joint_input(self):
        return self.w_in

    def joint_output(self):
        return self.wo

    def release_joint(self):
        """The joined matrices stand in for this part's own, which only its own forward needs."""
        self.w_in = self.wo = None

    def forward_joint(self, proj, column, batch, entry, out, factor):
        self.gated(proj, column, batch, entry, out, factor)

    def forward(self, x, batch, entry, residual):
        y = self._gated(x, batch, entry)
        add_late(residual, lambda rows, then_norm, takes_halves: L.linear_into(
            y, self.wo, rows, then_norm, takes_halves))

    def forward_rows(self, x, batch, entry):
        """The mixer's output alone: the output projection's float32 sums."""
        return L.linear(self._gated(x, batch, entry), self.wo, out_dtype=torch.float32)


register_mixer("gated_delta", GatedDelta)
