"""Pitenex on the GPU against the plain float64 implementation of tests/plain_pitenex.py: each
mechanism's kernels alone (the layer norm with its bias, the joining kernel in every form, clamped and
identity experts, chunked attention with sinks and keys that stand out at its edges, the delta rule
with a decay per channel token by token and in chunks, with carried state and with decays from none to
total), the block and the joined mixer with parts of every kind, whole prompts with the stream after
every layer, prompts in portions, token-by-token decoding, unequal batches, slots and pages that come
back, keys just inside and outside a chunk, state that lasts, long decoding, and greedy generation
through the library's generation loop, command line and trace replay."""
import os

import pytest
import torch

import plain_pitenex as P
import util
from pitenex_cases import CASES, make_folder, random_case, write_model
from util import TOL_BF16, rel_err

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
F = torch.float64
# float32 engine against float64 over a few hundred tokens and several norms
TOL_F32_LONG = 1e-4


def row_errors(got, want):
    """Per row: root mean square of the difference over that of all of ``want``."""
    got, want = got.double().cpu(), want.double().cpu()
    return (got - want).pow(2).mean(-1).sqrt() / want.pow(2).mean().sqrt()


def close(got, want, dtype, tol):
    """float32: the largest difference.  bfloat16: a router of these small random models now and
    then takes another expert after a rounding, which changes one position and a little of those
    behind it, so the typical row is held to the tolerance and all but one in ten (at least one) to a
    bound that a wrong key, a lost state or a missing term, which touch most rows, would break; the
    float32 engine is the sharp test."""
    if dtype == "float32":
        return rel_err(got, want) < tol
    e = row_errors(got, want).sort().values
    rest = e[:max(1, e.numel() - max(1, e.numel() // 10))]
    return float(rest.max()) < 0.3 and float(e.median()) < 1.5 * TOL_BF16


def _engine(folder, dtype, **kw):
    import gpt_fast_amd as gfa
    kw.setdefault("max_tokens", 4096)
    return gfa.Engine.from_folder(folder, dtype=dtype, device=DEV, **kw)


def _steps(eng, toks, cuts):
    """Feed ``toks`` as one sequence in portions that end at ``cuts``; logits of every token."""
    import gpt_fast_amd as gfa
    slot = eng.start_sequence()
    out, lo = [], 0
    for hi in list(cuts) + [len(toks)]:
        if hi <= lo:
            continue
        out.append(eng.step([gfa.Entry(slot, toks[lo:hi], want=list(range(hi - lo)))]).cpu())
        lo = hi
    eng.end_sequence(slot)
    return torch.cat(out)


def _ints(values):
    return torch.tensor(values, dtype=torch.int32, device=DEV)


def _f32(t):
    return t.to(torch.float32).to(DEV).contiguous()


# --------------------------------------------------------------------------- norm and join
@pytest.mark.parametrize("dim", [50, 96, 1030, 4096, 8200])
def test_layer_norm_with_a_bias(dim):
    from gpt_fast_amd.ops import kernels as K
    g = torch.Generator().manual_seed(dim)
    x = torch.randn(6, dim, generator=g, dtype=F) * 3 + 50.0             # a mean far from zero
    w, b = torch.rand(dim, generator=g, dtype=F) + 0.5, torch.randn(dim, generator=g, dtype=F)
    want = P.layer_norm(x.float().double(), w, b, 1e-3)
    assert rel_err(K.layer_norm(_f32(x), _f32(w), 1e-3, torch.float32, bias=_f32(b)), want) < 2e-5
    assert rel_err(K.layer_norm(_f32(x), _f32(w), 1e-3, torch.bfloat16, bias=_f32(b)), want) < 1e-2
    rows = _ints([5, 0, 5])
    assert rel_err(K.layer_norm(_f32(x), _f32(w), 1e-3, torch.float32, rows=rows, bias=_f32(b)), want[[5, 0, 5]]) < 2e-5


@pytest.mark.parametrize("dim", [50, 96, 1030, 4096, 8200])
def test_results_of_every_form_join_the_stream_and_are_normed(dim):
    from gpt_fast_amd.ops import term_join as TJ
    g = torch.Generator().manual_seed(dim)
    n, eps = 5, 1e-3
    res = torch.randn(n, dim, generator=g, dtype=F)
    plain, half = torch.randn(n, dim, generator=g, dtype=F), torch.randn(n, dim, generator=g, dtype=F).bfloat16()
    slices = torch.randn(3, n, dim, generator=g, dtype=F)
    w, b = torch.rand(dim, generator=g, dtype=F) + 0.5, torch.randn(dim, generator=g, dtype=F)
    forms = [(_f32(plain), 0.7, plain), (half.to(DEV), -1.3, half.double()), (_f32(slices), 0.4, slices.sum(0))]
    norms = {None: None, "plain": lambda x: x, "layer": lambda x: P.layer_norm(x, w, b, eps),
             "rms": lambda x: P.over_rms(x, eps) * w}
    for pick in ([0], [1], [2], [0, 1], [2, 1], [0, 1, 2], [2, 2, 0, 1]):
        want = res + sum(forms[i][1] * forms[i][2] for i in pick)
        for norm, f in norms.items():
            for dtype, tol in ((torch.float32, 2e-5), (torch.bfloat16, 1e-2)):
                new = _f32(res)
                out = TJ.join(new, [forms[i][:2] for i in pick], norm, _f32(w) if norm in ("layer", "rms") else None,
                              _f32(b) if norm == "layer" else None, eps, dtype)
                assert rel_err(new, want) < 1e-5
                assert out is None if norm is None else rel_err(out, f(want)) < tol


@pytest.mark.parametrize("dtype,tol", [("float32", 1e-5), ("bfloat16", 2e-2)])
def test_the_block_with_parts_that_offer_less_and_other_norms(dtype, tol):
    """A mixer that only adds into the stream beside each feed-forward; an RMS norm, a layer norm
    without a bias, none; the block called with the plain tensor and before a norm it knows."""
    import gpt_fast_amd as gfa
    from gpt_fast_amd.config.spec import DenseFeedForwardSpec, GatedFeedForwardSpec, LayerSpec, NormSpec
    from gpt_fast_amd.parts.base import BLOCKS, NORMS, ResidualStream, Runtime
    from gpt_fast_amd.parts.model import _Arranged

    class Doubling:
        kind = "doubling_for_a_test"

    class DoublingMixer:
        def __init__(self, spec, runtime):
            pass

        def parameters(self):
            return {}

        def bind(self, tensors):
            pass

        def cache_need(self):
            return None

        def forward(self, x, batch, entry, residual):
            residual += 2.0 * x.float()
    gfa.register_mixer("doubling_for_a_test", DoublingMixer)
    rt = Runtime(torch.float32 if dtype == "float32" else torch.bfloat16, DEV)
    D, H, m = 72, 136, 0.35
    for kind, bias in (("rms", False), ("layer", False), ("layer", True), ("none", False)):
        for ff in (GatedFeedForwardSpec(D, H, "gelu_tanh"), GatedFeedForwardSpec(D, H, "clamped_swish", 0.9),
                   DenseFeedForwardSpec(D, H, "silu"), None):
            norm = NormSpec(D, 1e-5, kind=kind, bias=bias)
            layer = LayerSpec(name="l", arrangement="parallel", result_scale=m, mixer=Doubling(), mixer_norm=norm,
                              feed_forward=ff)
            block, after = BLOCKS.build(_Arranged(layer), rt), NORMS.build(norm, rt)
            torch.manual_seed(8)
            t = {}
            for name, p in block.parameters().items():
                scale = 0.3 if p.role == "matrix" else 1.0
                t[name] = (torch.randn(p.shape, device=DEV) * scale).to(rt.dtype if p.role == "matrix" else torch.float32)
            block.bind(t)
            after.bind({k[len("mixer_norm."):]: v for k, v in t.items() if k.startswith("mixer_norm.")})
            d = {k: v.double().cpu() for k, v in t.items()}

            def normed(x):
                if kind == "none":
                    return x
                w = d["mixer_norm.weight"]
                return P.over_rms(x, 1e-5) * w if kind == "rms" else \
                    P.layer_norm(x, w, d["mixer_norm.bias"] if bias else 0.0, 1e-5)
            for rows in (2, 40, 130):
                X = torch.randn(rows, D, device=DEV)
                x = X.double().cpu()
                h = normed(x)
                y = 2.0 * h
                if ff is not None and ff.kind == "gated":
                    gu = h @ d["feed_forward.w13"].T
                    a, u = gu[:, :H], gu[:, H:]
                    if ff.activation == "gelu_tanh":
                        inner = P.gelu_tanh(a) * u
                    else:
                        a, u = a.clamp(max=0.9), u.clamp(-0.9, 0.9)
                        inner = a * torch.sigmoid(1.702 * a) * (u + 1)
                    y = y + inner @ d["feed_forward.w2"].T
                elif ff is not None:
                    y = y + P.silu(h @ d["feed_forward.w_up"].T) @ d["feed_forward.w_down"].T
                want = x + m * y
                stream = ResidualStream(X.clone())
                block.forward(stream, None, None)
                assert rel_err(stream.normed(after), normed(want)) < 3 * tol, (kind, bias, ff, rows)
                assert rel_err(stream.tensor, want) < tol
                block.forward(X, None, None)
                assert rel_err(X, want) < tol


# --------------------------------------------------------------------------- experts
def _mixture(E, I, top, D, Fh, limit, shared, dtype):
    from gpt_fast_amd.config.spec import RoutedExpertsSpec
    from gpt_fast_amd.parts.base import FEED_FORWARDS, Runtime
    rt = Runtime(torch.float32 if dtype == "float32" else torch.bfloat16, DEV)
    part = FEED_FORWARDS.build(RoutedExpertsSpec(
        dim=D, n_experts=E, top=top, hidden=Fh, shared_hidden=shared[0] if shared else 0,
        activation="clamped_swish", choice_correction=True, gated=True, identity=I, limit=limit,
        shared_limit=shared[1] if shared else None), rt)
    g = torch.Generator().manual_seed(E * 7 + D)
    t = {n: torch.randn(p.shape, generator=g) * (0.1 if n == "correction" else 0.4) for n, p in part.parameters().items()}
    t = {n: v.to(torch.float32 if n == "correction" else rt.dtype).to(DEV) for n, v in t.items()}
    part.bind(t)
    d = {n: v.double().cpu() for n, v in t.items()}
    w = {"router": d["w_router"], "correction": d["correction"]}
    for e in range(E):
        w[f"e{e}.gate"], w[f"e{e}.up"], w[f"e{e}.down"] = d["w_up"][e, :Fh], d["w_up"][e, Fh:], d["w_down"][e]
    if shared:
        n = shared[0]
        w["shared.gate"], w["shared.up"], w["shared.down"] = d["shared_up"][:n], d["shared_up"][n:], d["shared_down"]
    mlp = {"kind": "moe", "expert": {"ff": Fh, "limit": limit}, "router": {"experts": E, "identity": I, "top": top},
           "shared": {"ff": shared[0], "limit": shared[1]} if shared else None}
    return part, rt, w, mlp


@pytest.mark.parametrize("dtype,tol", [("float32", 2e-5), ("bfloat16", 2e-2)])
@pytest.mark.parametrize("E,I,top,D,Fh,shared", [(7, 3, 3, 96, 40, (56, 0.7)), (4, 0, 4, 104, 24, None),
                                                 (1, 1, 1, 128, 48, (32, 2.0)), (5, 2, 2, 50, 18, (22, 1.1)),
                                                 (6, 10, 4, 64, 32, None), (20, 5, 6, 192, 72, (88, 0.5))])
def test_clamped_experts_and_identity_experts(dtype, tol, E, I, top, D, Fh, shared):
    """Few rows, a decoding step, prompts whose experts' shares are alike and prompts in which one
    expert has them all; the choice goes by score plus correction, the weights by score."""
    part, rt, w, mlp = _mixture(E, I, top, D, Fh, 0.8, shared, dtype)

    class Step:
        is_decode = False
    g = torch.Generator().manual_seed(2)
    named = False
    for rows in (1, 3, 16, 17, 90, 400):
        for skewed in (False, True):
            x = torch.randn(rows, D, generator=g)
            if skewed:
                x = x * 0.05 + torch.randn(1, D, generator=g)
            x = x.to(rt.dtype)
            for decode in (False, True):
                Step.is_decode = decode
                got = part.forward_rows(x.to(DEV), Step)
                want = P.mixture(w, "", mlp, x.double())
                named = named or bool((part.last_chosen >= E).any())
                e = row_errors(got, want)
                # a choice that two scores nearly share may fall the other way
                if dtype == "float32":
                    assert rel_err(got, want) < tol, (rows, skewed, decode)
                else:
                    assert float(e.sort().values[:max(1, int(rows * 0.9))].max()) < tol, (rows, skewed, decode)
    assert named or not I                                  # or the test shows nothing of them


@pytest.mark.parametrize("E,D,Fh,counts", [(5, 72, 40, [128, 0, 129, 1, 60]), (3, 256, 64, [0, 300, 0]),
                                           (4, 136, 200, [1, 127, 128, 257]), (2, 64, 10, [40, 90]),
                                           (40, 96, 24, [3] * 39 + [200])])
def test_tiles_of_the_experts_rows(E, D, Fh, counts):
    """Shares of no row, one row, a tile's 128 and one more; inner sizes that end inside a piece of K
    and a tile of columns; every gate and activation; identity pairs behind the experts' are not
    written."""
    from gpt_fast_amd.ops import routed_experts as RE
    g = torch.Generator().manual_seed(D)
    top, n = 3, (sum(counts) + 7 + 2) // 3
    pairs = n * top
    ids = torch.tensor([e for e, c in enumerate(counts) for _ in range(c)] + [E] * (pairs - sum(counts)), dtype=torch.int32)
    chosen = ids[torch.randperm(pairs, generator=g)].view(n, top).to(DEV)
    offsets, order, place = RE.expert_order(chosen, E + 1)
    assert offsets[:E + 1].tolist() == [sum(counts[:e]) for e in range(E + 1)]
    tiles = RE.expert_tiles(offsets, E, pairs)
    listed = [t for t in tiles.tolist() if t[0] >= 0]
    assert listed == [[e, sum(counts[:e]) + i] for e, c in enumerate(counts) for i in range(0, c, 128)]
    x = torch.randn(n, D, generator=g).bfloat16()
    w = (torch.randn(E, 2 * Fh, D, generator=g) * 0.3).bfloat16()
    xs = x.double()[(order.cpu() // top).long()]
    args = (x.to(DEV), order, top)
    for act, gated, limit in ((None, False, None), ("silu", False, None), ("gelu", False, None), ("silu", True, None),
                              ("gelu_tanh", True, None), ("clamped_swish", True, 0.9)):
        got = RE.expert_tile_product(*args, w.to(DEV), offsets, tiles, pairs, act, gated, limit).double().cpu()
        for e, c in enumerate(counts):
            lo = sum(counts[:e])
            z = xs[lo:lo + c] @ w[e].double().T
            f = {None: lambda v: v, "silu": P.silu, "gelu": torch.nn.functional.gelu, "gelu_tanh": P.gelu_tanh}
            if act == "clamped_swish":
                a, u = z[:, :Fh].clamp(max=limit), z[:, Fh:].clamp(-limit, limit)
                z = a * torch.sigmoid(1.702 * a) * (u + 1)
            else:
                z = f[act](z[:, :Fh]) * z[:, Fh:] if gated else f[act](z)
            if c:
                assert rel_err(got[lo:lo + c], z) < 1e-2, (act, gated, e)
    # rows in their own order (a second product)
    rows = torch.randn(pairs, D, generator=g).bfloat16()
    got = RE.expert_tile_product(rows.to(DEV), None, 1, w.to(DEV), offsets, tiles, pairs).double().cpu()
    for e, c in enumerate(counts):
        lo = sum(counts[:e])
        if c:
            assert rel_err(got[lo:lo + c], rows[lo:lo + c].double() @ w[e].double().T) < 1e-2


def test_the_correction_moves_the_choice_and_not_the_weights():
    part, rt, w, mlp = _mixture(4, 2, 2, 64, 32, 1.0, None, "float32")
    part.correction.copy_(torch.tensor([0.0, 0.0, 0.0, 0.0, 5.0, 5.0]))     # both identity experts, always
    x = torch.randn(9, 64, device=DEV)
    assert rel_err(part.forward_rows(x, None), x.double()) < 1e-6
    part.correction.copy_(torch.tensor([0.0, 5.0, 0.0, 0.0, 5.0, 0.0]))     # expert 1 and the first identity
    z = x.double().cpu() @ w["router"].T
    s = torch.softmax(z, -1)[:, [1, 4]]
    s = s / s.sum(-1, keepdim=True)
    want = s[:, :1] * P.clamped_expert(w, "e1.", 1.0, x.double().cpu()) + s[:, 1:] * x.double().cpu()
    assert rel_err(part.forward_rows(x, None), want) < 1e-5


# --------------------------------------------------------------------------- attention
@pytest.mark.parametrize("dtype,tol", [(torch.float32, 2e-5), (torch.bfloat16, 2e-2)])
@pytest.mark.parametrize("H,G,hd,vd", [(6, 2, 24, 32), (5, 1, 80, 48), (8, 8, 8, 24), (3, 3, 10, 6), (8, 2, 128, 128),
                                       (2, 1, 160, 200)])
def test_chunks_and_sinks_with_keys_that_stand_out_at_the_edges(dtype, tol, H, G, hd, vd):
    """The first key of the last token's chunk, and the one before it, are loud in turn; prompts,
    portions and single tokens, with the kernel that works token by token and the matrix-core
    kernels; pages before the chunk and the pool behind the ends hold no number."""
    from gpt_fast_amd.ops import scored_attention as SA
    for chunk in (1, 7, 31, 64, 100, 300):
        for lens, starts in (([150], [0]), ([9, 40], [120, 3]), ([1, 1, 1], [40, 127, 200]), ([2], [99])):
            for off in (0, -1):
                g = torch.Generator().manual_seed(chunk + H)
                total = [s + l for s, l in zip(starts, lens)]
                n_pages = sum((t + 63) // 64 for t in total)
                order, tables, at = list(range(n_pages))[::-1], [], 0
                for t in total:
                    n = (t + 63) // 64
                    tables.append(order[at:at + n])
                    at += n
                widest = max(len(t) for t in tables)
                table = _ints([t + [-1] * (widest - len(t)) for t in tables])
                ks = [torch.randn(t, G, hd, generator=g, dtype=F) for t in total]
                vs = [torch.randn(t, G, vd, generator=g, dtype=F) for t in total]
                qs = [torch.randn(l, H, hd, generator=g, dtype=F) for l in lens]
                sinks = torch.randn(H, generator=g, dtype=F) * 2 + 1
                for b, t in enumerate(total):
                    j = (t - 1) // chunk * chunk + off
                    qs[b][..., 0] = 3.0
                    ks[b][..., 0] = 0.0
                    if j >= 0:
                        ks[b][j, :, 0] = 12.0
                if dtype == torch.bfloat16:
                    ks, vs, qs = ([t.to(dtype).double() for t in ts] for ts in (ks, vs, qs))
                k_pages = torch.full((n_pages + 1, G, 64, hd), float("nan"), dtype=dtype, device=DEV)
                v_pages = torch.full((n_pages + 1, G, vd, 64), float("nan"), dtype=dtype, device=DEV)
                rows = torch.cat([torch.cat([torch.zeros(t, hd, dtype=F), k.reshape(t, -1), v.reshape(t, -1)], 1)
                                  for t, k, v in zip(total, ks, vs)])
                wide = torch.full((rows.shape[0], rows.shape[1] + 8), float("nan"))
                wide[:, 3:3 + rows.shape[1]] = rows                     # a view of wider rows
                SA.unit_heads_store(wide.to(DEV)[:, 3:], None, _ints([b for b, t in enumerate(total) for _ in range(t)]),
                                    _ints([i for t in total for i in range(t)]), table, k_pages, v_pages, 1, G, hd, vd,
                                    None, dtype)
                for b, s in enumerate(starts):              # pages nobody can see any more
                    for pg in range(s // chunk * chunk // 64):
                        k_pages[tables[b][pg]] = float("nan")
                        v_pages[tables[b][pg]] = float("nan")
                want = []
                for b, l in enumerate(lens):
                    for i in range(l):
                        p = starts[b] + i
                        lo = p // chunk * chunk
                        k, v = (t[b][lo:p + 1].repeat_interleave(H // G, 1) for t in (ks, vs))
                        s = torch.einsum("hd,jhd->hj", qs[b][i], k) * 0.25
                        a = P.softmax_with_sink(s[:, None], sinks)[:, 0]
                        want.append(torch.einsum("hj,jhe->he", a, v) * 0.8)
                want = torch.stack(want)
                q = torch.cat(qs).to(dtype).to(DEV)
                tok_seq = _ints([b for b, l in enumerate(lens) for _ in range(l)])
                tok_pos = _ints([s + i for s, l in zip(starts, lens) for i in range(l)])
                step = (_ints([sum(lens[:b]) for b in range(len(lens) + 1)]), _ints(starts), len(lens), max(lens))
                for how in (None, step):
                    out = torch.zeros(sum(lens), H * vd + 6, dtype=dtype, device=DEV)
                    got = SA.attention(q, k_pages, v_pages, tok_seq, tok_pos, table, 0.25, chunk=chunk, sink=True,
                                       sinks=_f32(sinks), out_factor=0.8, step=how)
                    assert rel_err(got, want) < tol, (chunk, lens, off, how is None)
                    SA.attention(q, k_pages, v_pages, tok_seq, tok_pos, table, 0.25, chunk=chunk, sink=True,
                                 sinks=_f32(sinks), out_factor=0.8, step=how,
                                 out=out[:, 2:2 + H * vd].view(-1, H, vd))
                    assert torch.equal(out[:, 2:2 + H * vd].reshape(-1, H, vd), got)
                    assert not out[:, :2].any() and not out[:, 2 + H * vd:].any()


def test_a_chunk_and_a_window_together_and_a_sink_that_takes_everything():
    from gpt_fast_amd.ops import scored_attention as SA
    H, hd, T = 2, 16, 130
    g = torch.Generator().manual_seed(3)
    k_pages = torch.zeros(3, H, 64, hd, device=DEV)
    v_pages = torch.zeros(3, H, hd, 64, device=DEV)
    rows = torch.randn(T, 3 * H * hd, generator=g, dtype=F)
    pos, seq, table = _ints(list(range(T))), _ints([0] * T), _ints([[2, 0, 1]])
    q = SA.unit_heads_store(_f32(rows), None, seq, pos, table, k_pages, v_pages, H, H, hd, hd, None, torch.float32)
    k, v = rows[:, H * hd:2 * H * hd].view(T, H, hd), rows[:, 2 * H * hd:].view(T, H, hd)
    i, j = torch.arange(T)[:, None], torch.arange(T)[None]
    mask = P.chunk_mask(T, 50) & (i - j < 20)
    s = torch.einsum("ihd,jhd->hij", rows[:, :H * hd].view(T, H, hd), k) * 0.2
    for sink in (0.3, 60.0):
        sinks = torch.full((H,), sink, dtype=F)
        a = P.softmax_with_sink(s.masked_fill(~mask, float("-inf")), sinks)
        got = SA.attention(q, k_pages, v_pages, seq, pos, table, 0.2, window=20, chunk=50, sink=True, sinks=_f32(sinks))
        want = torch.einsum("hij,jhe->ihe", a, v)
        assert rel_err(got, want) < 2e-5
        assert float(got.abs().max()) < (1e-20 if sink == 60.0 else 10)


# --------------------------------------------------------------------------- the delta rule
def _cell_case(H, G, dk, dv, lens, seed, channel=True, decay=None):
    from gpt_fast_amd.ops import gated_delta as GD
    g = torch.Generator().manual_seed(seed)
    layout = GD.RowLayout.low_rank(H, G, dk, dv, 8, 8) if channel else GD.RowLayout.fused(H, G, dk, dv)
    C = layout.conv
    case = {"layout": layout,
            "conv": [torch.randn(n, C, generator=g, dtype=F) for n in lens],
            "proj": [torch.randn(n, layout.width, generator=g, dtype=F) for n in lens],
            "z": [torch.randn(n, H * dk + 4, generator=g, dtype=F) * 2 for n in lens],
            "A_log": torch.rand(H, generator=g, dtype=F) * 5 - 4,
            "dt_bias": torch.randn(H * (dk if channel else 1), generator=g, dtype=F) - 1}
    if decay is not None:
        decay(case)
    return case


def _cell_want(case, b, H, G, dk, dv, T=None):
    layout = case["layout"]
    conv, proj, z = (case[n][b][:T] for n in ("conv", "proj", "z"))
    n = conv.shape[0]
    of = [h // (H // G) for h in range(H)]
    q = P.unit(conv[:, :G * dk].view(n, G, dk))[:, of] * dk ** -0.5
    k = P.unit(conv[:, G * dk:2 * G * dk].view(n, G, dk))[:, of]
    v = conv[:, 2 * G * dk:].view(n, H, dv)
    beta = torch.sigmoid(proj[:, layout.b:layout.b + H])
    if case["dt_bias"].numel() == H:
        z = (proj[:, layout.a:layout.a + H] + case["dt_bias"])[..., None].expand(n, H, dk)
    else:
        z = (z[:, :H * dk] + case["dt_bias"]).view(n, H, dk)
    gdec = torch.exp(-torch.exp(case["A_log"])[:, None] * P.softplus(z))
    return P.channel_delta_rule(q, k, v, beta, gdec).reshape(n, H * dv)


def _cell_got(case, H, G, dk, dv, portions, slots, kernel, **kw):
    from gpt_fast_amd.ops import gated_delta as GD
    channel = case["dt_bias"].numel() != H
    state = torch.zeros(7, H * dk * dv + 4, dtype=torch.float32, device=DEV)
    state[1].fill_(float("nan"))                                     # a slot nobody owns
    n_seq = len(case["conv"])
    fed, got = [0] * n_seq, [[] for _ in range(n_seq)]
    for portion in portions:
        live = [b for b in range(n_seq) if portion[b]]
        take = [portion[b] for b in live]
        cut = lambda rows: _f32(torch.cat([rows[b][fed[b]:fed[b] + n] for b, n in zip(live, take)]))
        q_start = _ints([sum(take[:i]) for i in range(len(take) + 1)])
        args = (cut(case["conv"]), cut(case["proj"]), case["layout"], _f32(case["A_log"]), _f32(case["dt_bias"]), state,
                q_start, _ints([slots[b] for b in live]), len(live))
        sizes = (H, G, dk, dv, dk ** -0.5, 1e-6)
        decays = cut(case["z"]) if channel else None
        if kernel == "tokens":
            y = GD.scan(*args, *sizes, decays=decays)
        elif kernel == "chunks":
            y = GD.parallel_chunks(*args, max(take), *sizes, decays=decays, **kw)
        else:
            y = GD.cell(*args, max(take), *sizes, decays=decays)
        at = 0
        for b, n in zip(live, take):
            got[b].append(y[at:at + n].double().cpu())
            at += n
            fed[b] += n
    assert torch.isnan(state[1]).all()
    return [torch.cat(g) for g in got]


SIZES = [(4, 2, 24, 16), (3, 3, 32, 48), (1, 1, 12, 40), (3, 1, 10, 14), (6, 3, 40, 24), (2, 1, 64, 64), (3, 3, 128, 144),
         (2, 1, 96, 100), (2, 2, 70, 33)]


@pytest.mark.parametrize("kernel", ["tokens", "chunks", "cell"])
@pytest.mark.parametrize("H,G,dk,dv", SIZES + [(2, 1, 144, 32)])
@pytest.mark.parametrize("channel", [True, False])
def test_the_cell_with_carried_state(H, G, dk, dv, kernel, channel):
    """Three sequences in scattered slots, fed in portions of unequal sizes (down to one and two
    tokens; a chunk's 64 and one more among them); the state travels from step to step."""
    from gpt_fast_amd.ops import gated_delta as GD
    if kernel == "chunks" and not GD.parallel_chunks_available(dk, dv):
        assert dk > 128
        return
    lens = [230, 9, 135]
    case = _cell_case(H, G, dk, dv, lens, H * 31 + dk, channel)
    portions = ([1, 2, 70], [2, 1, 64], [130, 1, 0], [65, 5, 0], [32, 0, 1])
    got = _cell_got(case, H, G, dk, dv, portions, [5, 0, 3], kernel)
    for b in range(3):
        assert rel_err(got[b], _cell_want(case, b, H, G, dk, dv)) < 1e-4, b


@pytest.mark.parametrize("at_once", [1, 2, 3])
def test_long_prompts_go_through_in_rounds(at_once):
    H, G, dk, dv = 2, 1, 24, 16
    case = _cell_case(H, G, dk, dv, [300, 1, 190], 5)
    got = _cell_got(case, H, G, dk, dv, ([300, 1, 190],), [2, 0, 6], "chunks", chunks_at_once=at_once)
    for b in range(3):
        assert rel_err(got[b], _cell_want(case, b, H, G, dk, dv)) < 1e-4, b


@pytest.mark.parametrize("kernel", ["tokens", "chunks"])
@pytest.mark.parametrize("kind", ["none", "total", "uneven", "one token", "single channels"])
def test_decays_from_none_to_total(kind, kernel):
    """A state that never forgets over 300 tokens, one that forgets at once, channels that decay by
    everything between side by side, one token in the middle that wipes the state (those behind it
    keep their digits), and single channels that lose e^-5 to e^-30 a token, whose sums inside a tile no
    factor could carry."""
    H, G, dk, dv, T = 2, 1, 32, 24, 300

    def decay(c):
        z, A = c["z"][0], c["A_log"]
        if kind == "none":
            A[:] = -14.0
        elif kind == "total":
            A[:], z[:] = 6.0, 3.0
        elif kind == "uneven":
            A[:] = 0.0
            c["dt_bias"][:] = torch.linspace(-9.0, 12.0, H * dk, dtype=F)
        elif kind == "one token":
            A[:], z[:], c["dt_bias"][:] = 0.0, -4.0, 0.0
            z[137] = 300.0
        else:
            A[:], z[:], c["dt_bias"][:] = 0.0, -4.0, 0.0
            z[:, ::7] = torch.rand(T, z[:, ::7].shape[1], generator=torch.Generator().manual_seed(1), dtype=F) * 25 + 5
    case = _cell_case(H, G, dk, dv, [T], 77, True, decay)
    want = _cell_want(case, 0, H, G, dk, dv)
    got = _cell_got(case, H, G, dk, dv, ([T],), [4], kernel)[0]
    assert torch.isfinite(got).all()
    assert rel_err(got, want) < 3e-5
    if kind == "one token":
        tail = slice(137, 200)
        assert rel_err(got[tail], want[tail]) < 2e-5


# --------------------------------------------------------------------------- whole models
@pytest.mark.parametrize("name", sorted(CASES))
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_whole_prompt_at_every_position_and_the_stream_after_every_layer(tmp_path, name, dtype):
    folder = make_folder(tmp_path, name, seed=11)
    cfg, w = P.load_folder(folder)
    toks = util.random_tokens(cfg["vocab"], 150, 3)
    outs = []
    want = P.forward(w, cfg, toks, outs)
    eng = _engine(folder, dtype)
    taps = []
    eng.model.tap = lambda n, x: taps.append(x.double().cpu())
    got = _steps(eng, toks, [])
    eng.model.tap = None
    assert close(got, want, dtype, TOL_F32_LONG)
    assert len(taps) == len(outs) == len(cfg["layers"])
    if dtype == "float32":
        for n, (a, b) in enumerate(zip(taps, outs)):
            assert rel_err(a, b) < TOL_F32_LONG, n
        # one token, and the first tokens of a sequence (fewer than the taps)
        assert rel_err(_steps(eng, toks[:1], []), want[:1]) < TOL_F32_LONG
        assert rel_err(_steps(eng, toks[:3], []), want[:3]) < TOL_F32_LONG
        assert rel_err(_steps(eng, toks[:3], [1, 2]), want[:3]) < TOL_F32_LONG


@pytest.mark.parametrize("name", sorted(CASES))
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_portions_and_token_by_token_equal_the_whole_prompt(tmp_path, name, dtype):
    folder = make_folder(tmp_path, name, seed=12)
    cfg, w = P.load_folder(folder)
    toks = util.random_tokens(cfg["vocab"], 210, 5)
    want = P.forward(w, cfg, toks)
    eng = _engine(folder, dtype)
    for cuts in ([], [2, 4, 5, 70, 128, 129], [39, 40, 41, 100, 192], [17, 150], list(range(150, 210)),
                 list(range(1, 80)), list(range(2, 210, 2))):
        assert close(_steps(eng, toks, cuts), want, dtype, TOL_F32_LONG), cuts
    eng.cache.check()


@pytest.mark.parametrize("name", ["A", "B", "C"])
@pytest.mark.parametrize("dtype,same", [("float32", 2e-5), ("bfloat16", TOL_BF16)])
def test_unequal_batches_equal_each_request_alone(tmp_path, name, dtype, same):
    import gpt_fast_amd as gfa
    folder = make_folder(tmp_path, name, seed=13)
    cfg, w = P.load_folder(folder)
    lens = [1, 5, 131, 64, 70]
    tail = 30
    seqs = [util.random_tokens(cfg["vocab"], n + tail, 40 + n) for n in lens]
    eng = _engine(folder, dtype, max_tokens=64 * 20, max_sequences=6)
    alone = [_steps(eng, s, [n] + list(range(n + 1, n + tail))) for s, n in zip(seqs, lens)]
    slots = [eng.start_sequence() for _ in seqs]
    got = [[] for _ in seqs]
    out = eng.step([gfa.Entry(sl, s[:n], want=list(range(n))) for sl, s, n in zip(slots, seqs, lens)]).cpu()
    at = 0
    for b, n in enumerate(lens):
        got[b].append(out[at:at + n])
        at += n
    live = list(range(len(seqs)))
    for t in range(tail):
        if t == 10:                                  # a shorter request ends earlier
            eng.end_sequence(slots[1])
            live.remove(1)
        out = eng.step([gfa.Entry(slots[b], [seqs[b][lens[b] + t]], want=[0]) for b in live]).cpu()
        for i, b in enumerate(live):
            got[b].append(out[i:i + 1])
    for b in live:
        eng.end_sequence(slots[b])
    eng.cache.check()
    for b, s in enumerate(seqs):
        g = torch.cat(got[b])
        assert close(g, alone[b][:g.shape[0]], dtype, same), b
        assert close(g, P.forward(w, cfg, s)[:g.shape[0]], dtype, TOL_F32_LONG), b


@pytest.mark.parametrize("name", ["A", "C"])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_step_that_mixes_single_tokens_a_portion_and_a_new_prompt(tmp_path, name, dtype):
    import gpt_fast_amd as gfa
    folder = make_folder(tmp_path, name, seed=21)
    cfg, w = P.load_folder(folder)
    _, before, mixed = util.mixed_step_case(cfg["vocab"])
    lens = {"d0": 9, "d1": 66, "d2": 130, "c": 112, "p": 131}
    seqs = {r: util.random_tokens(cfg["vocab"], n, 300 + n) for r, n in lens.items()}
    eng = _engine(folder, dtype, max_tokens=64 * 16, max_sequences=5)
    slots = {r: eng.start_sequence() for r in seqs}
    got = {r: [] for r in seqs}
    fed = {r: 0 for r in seqs}

    def step(order, portions):
        logits = eng.step([gfa.Entry(slots[r], seqs[r][fed[r]:fed[r] + portions[r]], want=list(range(portions[r])))
                           for r in order]).cpu()
        at = 0
        for r in order:
            got[r].append(logits[at:at + portions[r]])
            at += portions[r]
            fed[r] += portions[r]
    step(["d0", "d1", "d2", "c"], before)
    step(["d0", "c", "d1", "p", "d2"], mixed)
    for r in ("c", "p"):
        while fed[r] < len(seqs[r]):
            step([r], {r: 1})
    for r in seqs:
        eng.end_sequence(slots[r])
    eng.cache.check()
    assert eng.cache.slots.held == 0
    for r, toks in seqs.items():
        assert close(torch.cat(got[r]), P.forward(w, cfg, toks)[:fed[r]], dtype, TOL_F32_LONG), r


@pytest.mark.parametrize("batch", [12, 20, 40])
def test_wide_decoding_steps_take_the_larger_products_kernels(tmp_path, batch):
    """A dozen to forty requests decode together: the products' kernels change with the number
    of rows, the results do not."""
    import gpt_fast_amd as gfa
    folder = make_folder(tmp_path, "C", seed=27)
    cfg, w = P.load_folder(folder)
    seqs = [util.random_tokens(cfg["vocab"], 3 + b % 5 + 6, 500 + b) for b in range(batch)]
    eng = _engine(folder, "bfloat16", max_tokens=64 * batch, max_sequences=batch)
    slots = [eng.start_sequence() for _ in seqs]
    got = [[] for _ in seqs]
    eng.step([gfa.Entry(sl, s[:-6], want=[]) for sl, s in zip(slots, seqs)])
    for t in range(6):
        out = eng.step([gfa.Entry(sl, [s[len(s) - 6 + t]], want=[0]) for sl, s in zip(slots, seqs)]).cpu()
        for b in range(batch):
            got[b].append(out[b:b + 1])
    want = torch.cat([P.forward(w, cfg, s)[-6:] for s in seqs])
    assert close(torch.cat([torch.cat(g) for g in got]), want, "bfloat16", None)


def test_slots_and_pages_that_come_back_start_clean(tmp_path):
    """A cache of few pages and two slots: requests follow one another in the same slots and pages
    (the cell's state, the convolutions' tails and the previous token among their state), pages of
    chunks that have ended come back while a request runs, and every request equals the plain
    computation of itself alone."""
    import gpt_fast_amd as gfa
    folder = make_folder(tmp_path, "A", seed=14)
    cfg, w = P.load_folder(folder)
    eng = _engine(folder, "float32", max_tokens=64 * 7, max_sequences=2)
    for again in range(3):
        a = util.random_tokens(cfg["vocab"], 150 + 60, 60 + again)
        b = util.random_tokens(cfg["vocab"], 40 + 60, 70 + again)
        sa, sb = eng.start_sequence(), eng.start_sequence()
        assert {sa, sb} == {0, 1}
        got_a, got_b = [], []
        out = eng.step([gfa.Entry(sa, a[:150], want=[149]), gfa.Entry(sb, b[:40], want=[39])]).cpu()
        got_a.append(out[0:1])
        got_b.append(out[1:2])
        for t in range(59):
            out = eng.step([gfa.Entry(sa, [a[150 + t]], want=[0]), gfa.Entry(sb, [b[40 + t]], want=[0])]).cpu()
            got_a.append(out[0:1])
            got_b.append(out[1:2])
        eng.cache.check()
        eng.end_sequence(sb)
        eng.end_sequence(sa)
        assert rel_err(torch.cat(got_a), P.forward(w, cfg, a[:-1])[149:]) < TOL_F32_LONG
        assert rel_err(torch.cat(got_b), P.forward(w, cfg, b[:-1])[39:]) < TOL_F32_LONG
    for _, g in eng.cache.paged_groups:
        assert g.pages.held == 0


@pytest.mark.parametrize("chunk,edge", [(64, 128), (40, 120), (100, 200), (150, 150)])
def test_keys_just_inside_and_outside_a_chunk_in_a_whole_model(tmp_path, chunk, edge):
    """One layer whose attention scores are large and whose recurrence does not write: the token at
    the chunk's first position is replaced, and the logits behind it change until the chunk ends;
    the token before it is replaced, and they do not (beyond its own neighbour, which sees it as its
    previous token); whole, in portions and decoded."""
    import copy
    config = copy.deepcopy(CASES["A"])
    config["layers"] = [config["layers"][1]]
    config["layers"][0]["mixer"]["left"]["mask"]["size"] = chunk

    def patch(t):
        t["l0.mix.left.q"] = t["l0.mix.left.q"] * 10
        t["l0.mix.right.v"] = t["l0.mix.right.v"] * 0
    folder = write_model(os.path.join(str(tmp_path), f"edge{chunk}"), config, 40, patch=patch)
    cfg, w = P.load_folder(folder)
    T = edge + min(chunk, 60)
    toks = util.random_tokens(cfg["vocab"], T, 5)
    variants = [toks]
    for place in (edge, edge - 1):
        other = list(toks)
        other[place] = (other[place] + 7) % cfg["vocab"]
        variants.append(other)
    wants = [P.forward(w, cfg, s) for s in variants]
    assert float(row_errors(wants[1], wants[0])[edge + 5:].max()) > 0.03      # inside: it matters
    # outside: the neighbour's own row changes (its previous token), and what attends to the neighbour
    eng = _engine(folder, "float32", max_tokens=64 * 8, max_sequences=1)
    for s, want in zip(variants, wants):
        for cuts in ([], [edge], [edge - 1, edge + 1], [edge - 20] + list(range(edge - 19, T))):
            assert rel_err(_steps(eng, s, cuts), want) < 5 * TOL_F32_LONG, cuts
    eng = _engine(folder, "bfloat16", max_tokens=64 * 8, max_sequences=1)
    for s, want in zip(variants, wants):
        got = _steps(eng, s, [edge - 20] + list(range(edge - 19, T)))
        assert float(row_errors(got, want).median()) < 2 * TOL_BF16
    eng.cache.check()


def test_the_previous_token_reaches_a_portion_s_first_token(tmp_path):
    """With the same last token but another one before it, the first logits of the next portion
    differ by the pair's row alone (a model whose mixers are silent)."""
    def patch(t):
        for n in t:
            if n.endswith(".o"):
                t[n] = t[n] * 0
    folder = make_folder(tmp_path, "B", seed=9, patch=patch, tag="silent")
    cfg, w = P.load_folder(folder)
    eng = _engine(folder, "float32")
    toks = util.random_tokens(cfg["vocab"], 12, 1)
    for change in (4, 5):
        s = list(toks)
        s[change] = (s[change] + 3) % cfg["vocab"]
        assert rel_err(_steps(eng, s, [6]), P.forward(w, cfg, s)) < TOL_F32_LONG
        assert rel_err(_steps(eng, s, list(range(1, 12))), P.forward(w, cfg, s)) < TOL_F32_LONG


def test_state_that_lasts_hundreds_of_tokens_and_long_decoding(tmp_path):
    """Decays next to one: the first tokens decide the last logits five hundred tokens later,
    through a prompt and 130 tokens decoded one by one, long after every chunk of theirs ended."""
    def patch(t):
        for name in t:
            if name.endswith(".A_log"):
                t[name] = torch.full_like(t[name], -9.0)
    folder = make_folder(tmp_path, "A", seed=16, patch=patch, tag="lasting")
    cfg, w = P.load_folder(folder)
    toks = util.random_tokens(cfg["vocab"], 520, 21)
    want = P.forward(w, cfg, toks)
    # it matters: with other first tokens the last logits are others
    other = util.random_tokens(cfg["vocab"], 20, 22) + toks[20:]
    assert rel_err(P.forward(w, cfg, other)[-40:], want[-40:]) > 1e-2
    for dtype in ("float32", "bfloat16"):
        eng = _engine(folder, dtype, max_tokens=64 * 10, max_sequences=1)
        got = _steps(eng, toks, [390] + list(range(391, 520)))
        assert close(got, want, dtype, 3 * TOL_F32_LONG)
        eng.cache.check()


@pytest.mark.parametrize("seed", [1, 2, 3, 4, 5, 6, 7, 8])
def test_random_configurations_whole_and_in_a_batch_that_is_decoded_together(tmp_path, seed):
    """Sizes drawn at random (pitenex_cases.random_case): requests of 300, 130, 33 and 1 tokens,
    each whole, then their prompts in one batch and twenty tokens decoded together."""
    import gpt_fast_amd as gfa
    config = random_case(seed)
    folder = write_model(os.path.join(str(tmp_path), f"random{seed}"), config, 100 + seed, std=0.05)
    cfg, w = P.load_folder(folder)
    lens = [300, 130, 33, 1]
    seqs = [util.random_tokens(cfg["vocab"], n + 20, 7 * seed + n) for n in lens]
    want = [P.forward(w, cfg, s) for s in seqs]
    for dtype in ("float32", "bfloat16"):
        eng = _engine(folder, dtype, max_tokens=4096, max_sequences=4)
        for s, wanted in zip(seqs, want):
            assert close(_steps(eng, s, []), wanted, dtype, 3 * TOL_F32_LONG), (dtype, len(s))
        slots = [eng.start_sequence() for _ in seqs]
        got = [[] for _ in seqs]
        out = eng.step([gfa.Entry(sl, s[:n], want=list(range(n))) for sl, s, n in zip(slots, seqs, lens)]).cpu()
        at = 0
        for b, n in enumerate(lens):
            got[b].append(out[at:at + n])
            at += n
        for t in range(20):
            out = eng.step([gfa.Entry(slots[b], [seqs[b][lens[b] + t]], want=[0]) for b in range(len(seqs))]).cpu()
            for b in range(len(seqs)):
                got[b].append(out[b:b + 1])
        for sl in slots:
            eng.end_sequence(sl)
        eng.cache.check()
        for b in range(len(seqs)):
            assert close(torch.cat(got[b]), want[b], dtype, 3 * TOL_F32_LONG), (dtype, b)


# --------------------------------------------------------------------------- generation
@pytest.mark.parametrize("name", ["A", "C"])
def test_greedy_generation_through_the_loop_and_the_recorded_step(tmp_path, name):
    from gpt_fast_amd.engine.generate import generate
    folder = make_folder(tmp_path, name, seed=17)
    cfg, w = P.load_folder(folder)
    prompts = [util.random_tokens(cfg["vocab"], n, 80 + n) for n in (7, 1, 90, 30)]
    want = [P.greedy_generate(w, cfg, p, 12) for p in prompts]
    eng = _engine(folder, "float32", max_tokens=64 * 12, max_sequences=4)
    assert eng.model.replayable
    for use_graph in (False, True, True):                       # the recording is replayed
        got = generate(eng, prompts, max_new_tokens=12, temperature=0.0, use_graph=use_graph)
        assert got.tokens == want, use_graph
    # two at a time: slots and state come back between the batches
    got = generate(eng, prompts, max_new_tokens=12, temperature=0.0, batch_size=2)
    assert got.tokens == want
    eng.cache.check()
    # bfloat16 through the recorded step: the tokens of the step that is not recorded
    eng = _engine(folder, "bfloat16", max_tokens=64 * 12, max_sequences=4)
    plain_steps = generate(eng, prompts, max_new_tokens=12, temperature=0.0, use_graph=False).tokens
    for _ in range(2):
        assert generate(eng, prompts, max_new_tokens=12, temperature=0.0, use_graph=True).tokens == plain_steps


def test_command_line_entry_point(tmp_path):
    import gpt_fast_amd as gfa
    folder = make_folder(tmp_path, "B", seed=18)
    cfg, w = P.load_folder(folder)
    prompt = util.random_tokens(cfg["vocab"], 20, 1)
    lines = []
    res = gfa.main(prompt=prompt, num_samples=1, max_new_tokens=8, temperature=0.0, top_k=None,
                   checkpoint_path=folder, dtype="float32", device=DEV, out=lines.append)
    assert res["result"].tokens[0] == P.greedy_generate(w, cfg, prompt, 8)
    assert any("tokens/sec" in str(l) for l in lines)


def test_trace_replay_program(tmp_path):
    """bin/trace_run as a program on a Pitenex folder: two batches of unequal requests one after
    the other (the second takes the slots, state and pages the first gave back), logits wanted
    at some places only, steps in which nothing is wanted, a request that ends in the step that
    brings its prompt."""
    import json
    import subprocess

    import numpy as np
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    folder = make_folder(tmp_path, "A", seed=19)
    cfg, w = P.load_folder(folder)
    V = cfg["vocab"]
    reqs = {"a": util.random_tokens(V, 140, 1), "b": util.random_tokens(V, 9, 2), "c": util.random_tokens(V, 1, 3),
            "d": util.random_tokens(V, 150, 4), "e": util.random_tokens(V, 70, 5)}
    prompt = {"a": 120, "b": 3, "c": 1, "d": 130, "e": 64}
    steps, where = [], {r: [] for r in reqs}          # request -> (step, row in the file, position)
    n = 0
    for ids in (["a", "b", "c"], ["d", "e"]):
        live, t = list(ids), 0
        while live:
            entries, row = [], 0
            for r in live:
                lo, hi = (0, prompt[r]) if t == 0 else (prompt[r] + t - 1, prompt[r] + t)
                want = [i for i in range(hi - lo) if (lo + i) % 3 != 1]
                entries.append({"id": r, "tokens": reqs[r][lo:hi], "want": want})
                for i in want:
                    where[r].append((n, row, lo + i))
                    row += 1
            ends = [r for r in live if (prompt[r] + t if t else prompt[r]) >= len(reqs[r])]
            steps.append({"step": n, "entries": entries, "end": ends})
            live = [r for r in live if r not in ends]
            n += 1
            t += 1
    for dtype in ("float32", "bfloat16"):
        out_dir = os.path.join(str(tmp_path), "out_" + dtype)
        proc = subprocess.run(
            [os.path.join(root, "bin", "trace_run"), "--model", folder, "--dtype", dtype, "--out", out_dir,
             "--max-tokens", "400"],
            input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=600)
        assert proc.returncode == 0, proc.stderr[-2000:]
        assert [l for l in proc.stdout.splitlines() if l.startswith("done ")] == [f"done {i}" for i in range(n)]
        for r, toks in reqs.items():
            if not where[r]:
                continue
            got = torch.stack([torch.from_numpy(np.fromfile(os.path.join(out_dir, f"{s}.f32"), dtype="<f4")
                                                .reshape(-1, V)[row]) for s, row, _ in where[r]])
            want = P.forward(w, cfg, toks)[[p for _, _, p in where[r]]]
            assert close(got, want, dtype, TOL_F32_LONG), (dtype, r)
