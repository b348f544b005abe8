"""Attention whose keys and values are expanded from one cached latent per token."""
import torch

from ..cache.store import KVNeed
from ..config.spec import LatentAttentionSpec
from ..ops import kernels as K
from ..ops import latent_attention as LA
from ..ops import linear as L
from ..ops import scored_attention as SA
from .base import Param, Part, Runtime, add_late, check_bound, register_mixer
from .position import RotaryPosition, frequencies_and_trig_scale


class LatentAttention(Part):
    """``cq = norm(w_dq x)``, ``q = w_uq cq`` (per head ``d`` plain and ``dr`` rotated
    elements); ``[c', kr'] = w_dkv x``, ``c = norm(c')`` the token's latent, ``kr`` = kr'
    rotated by position, one key part for all heads.  A head's plain key is ``w_uk[h] c`` and
    its value ``w_uv[h] c``, so

        score_h(i, j) = (q_plain_h(i) . w_uk[h] c_j + q_rot_h(i) . kr_j) * scale
                      = ([w_uk[h]^T q_plain_h(i), q_rot_h(i)] . [c_j, kr_j]) * scale
        out_h(i) = w_uv[h] sum_j softmax_j(score_h)(i, j) c_j

    that is attention with one kv head whose key is ``[c, kr]`` and whose value is ``c``: the
    query is carried into the latent's space by ``w_uk`` before and the result out of it by
    ``w_uv`` after, one small product per head each.  The cache holds the latent (once in the
    order the kernels read keys in, once in the order they read values in) and the rotated
    part.  The rotated parts take either pair layout and a ladder whose cos and sin carry a
    factor.  Keys at distance < ``window`` are seen.  The down projections keep their float32
    sums until the norms; the query's up projection keeps them until the rotation.

    With ``head_gate`` head h's result is multiplied by ``sigmoid(w_g x)_h``: the gates are more
    rows of the down projection, and the attention kernel applies them to the latents it writes
    (a factor per head passes through ``w_uv``).

    Without a query latent (``q_rank`` None) ``q = w_q x``: the kv down projection and ``w_q``
    are then one matrix over x, whose float32 sums serve both."""

    @staticmethod
    def libraries(runtime):
        return ("scored_attention",) if runtime.is_float32 else ("scored_attention", "latent_attention")

    replayable = True
    defers_sum = True              # ``residual`` may be a parts.base.ResidualStream

    def __init__(self, spec: LatentAttentionSpec, runtime: Runtime):
        self.spec = spec
        self.rt = runtime
        self.rotary_dim, self.freqs, self.layout, self.trig = 0, None, 0, 1.0
        if spec.position.kind == "rope":
            freqs, self.trig = frequencies_and_trig_scale(spec.position)
            self.rotary_dim, self.freqs = spec.position.rotary_dim, freqs.to(runtime.device)
            self.layout = RotaryPosition.LAYOUTS[spec.position.layout]
        elif spec.position.kind != "none":
            raise ValueError(f"latent attention: position kind '{spec.position.kind}'")
        if self.rotary_dim > spec.rot_dim:
            raise ValueError(f"latent attention: {self.rotary_dim} rotated elements of {spec.rot_dim}")
        self.window = 0 if spec.window is None else int(spec.window)
        self.q_rank = int(spec.q_rank or 0)
        self.q_rows = spec.n_heads * (spec.head_dim + spec.rot_dim)
        # rows over x: [query latent | kv latent | rotated key part | q, if it has no latent | gates]
        self.gate_at = self.q_rank + spec.kv_rank + spec.rot_dim + (0 if self.q_rank else self.q_rows)
        self.down_rows = self.gate_at + (spec.n_heads if spec.head_gate else 0)
        self.w_down = self.w_uq = self.w_uk = self.w_uv = self.wo = None
        self.q_norm = self.kv_norm = None

    def parameters(self):
        s = self.spec
        p = {"w_down": Param((self.down_rows, s.dim)),
             "kv_norm": Param((s.kv_rank,), role="vector", init="norm"),
             "w_uk": Param((s.n_heads * s.head_dim, s.kv_rank)),
             "w_uv": Param((s.n_heads * s.value_dim, s.kv_rank)),
             "wo": Param((s.dim, s.n_heads * s.value_dim))}
        if self.q_rank:
            p["q_norm"] = Param((s.q_rank,), role="vector", init="norm")
            p["w_uq"] = Param((self.q_rows, s.q_rank))
        return p

    def bind(self, tensors):
        check_bound("LatentAttention", self.parameters(), tensors)
        s = self.spec
        # zero rows up to a multiple of eight: the products' kernels store whole groups
        self.w_down = L.pad_rows(tensors["w_down"], 8)
        self.w_uq = L.pad_rows(tensors["w_uq"], 8) if self.q_rank else None
        self.wo = tensors["wo"]
        # per head: [d, R] carries a plain query into the latent's space, [R, dv] a result out;
        # both lie so that the batched products take them as they are, not transposed
        self.w_uk = tensors["w_uk"].view(s.n_heads, s.head_dim, s.kv_rank)
        self.w_uv = tensors["w_uv"].view(s.n_heads, s.value_dim, s.kv_rank).transpose(1, 2).contiguous()
        self.q_norm = tensors["q_norm"].to(torch.float32).contiguous() if self.q_rank else None
        self.kv_norm = tensors["kv_norm"].to(torch.float32).contiguous()

    def cache_need(self):
        s = self.spec
        return KVNeed(1, s.kv_rank + s.rot_dim, s.window, s.kv_rank)

    def step_flops(self, q_lens, starts) -> float:
        s = self.spec
        n = sum(q_lens)
        per_token = (self.down_rows * s.dim + self.q_rows * self.q_rank
                     + s.n_heads * (s.head_dim + s.value_dim) * s.kv_rank
                     + s.n_heads * s.value_dim * s.dim)
        flops = 2.0 * n * per_token
        for q, start in zip(q_lens, starts):
            keys = q * start + q * (q + 1) / 2.0
            if s.window is not None:
                keys = min(keys, q * float(s.window))
            flops += 2.0 * s.n_heads * (2 * s.kv_rank + s.rot_dim) * keys
        return flops

    def _per_head(self, a, w, out):
        """out[h] = a[h] w[h] for every head: a [H, N, K], w [H, K, M], out [H, N, M] (a view)."""
        if a.dtype == torch.float32:
            return K.gemm_f32_batched(a, w.transpose(1, 2), out)
        return torch.bmm(a, w, out=out)                        # the vendor library, as for prompts

    def _heads(self, x, batch, entry):
        s = self.spec
        n = x.shape[0]
        R = s.kv_rank
        down = L.linear(x, self.w_down, out_dtype=torch.float32)
        write = entry is not None and entry.writes
        table = batch.table(entry.group_id)
        cq = SA.latent_store(down, self.q_rank, R, s.rot_dim, self.q_norm, self.kv_norm, s.eps,
                             self.freqs, self.rotary_dim, batch.tok_seq, batch.tok_pos, table,
                             entry.k_pages if write else None, entry.v_pages if write else None,
                             self.rt.dtype, layout=self.layout, trig_scale=self.trig)
        if self.q_rank:
            q = L.linear(cq, self.w_uq, out_dtype=torch.float32)[:, :self.q_rows]
        else:
            q = down[:, R + s.rot_dim:R + s.rot_dim + self.q_rows]       # a view of the wider rows
        plain, full = SA.latent_query(q, self.freqs, self.rotary_dim, batch.tok_pos, s.n_heads,
                                      s.head_dim, s.rot_dim, R, self.rt.dtype, layout=self.layout,
                                      trig_scale=self.trig)
        self._per_head(plain, self.w_uk, full[:, :, :R])
        latent = LA.attention(full, entry.k_pages, entry.v_pages, batch.tok_seq, batch.tok_pos, table,
                              s.scale, (batch.q_start, batch.start_pos, batch.n_seqs, batch.max_q_len),
                              window=self.window,
                              gate=down[:, self.gate_at:self.down_rows] if s.head_gate else None)
        y = torch.empty((n, s.n_heads, s.value_dim), dtype=self.rt.dtype, device=x.device)
        self._per_head(latent, self.w_uv, y.permute(1, 0, 2))
        return y.view(n, s.n_heads * s.value_dim)

    def forward(self, x, batch, entry, residual):
        y = self._heads(x, batch, entry)
        add_late(residual, lambda rows, then_norm, takes_halves: L.linear_into(
            y, self.wo, rows, then_norm, takes_halves))

    def forward_last(self, x, batch, entry):
        """The operand and the matrix of the last product, which the block runs."""
        return self._heads(x, batch, entry), self.wo

    def forward_rows(self, x, batch, entry):
        """The mixer's output alone: the output projection's float32 sums."""
        return L.linear(self._heads(x, batch, entry), self.wo, out_dtype=torch.float32)


register_mixer("latent_attention", LatentAttention)
