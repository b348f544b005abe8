"""CPU tests of Pitenex: what fixes the plain implementation of tests/plain_pitenex.py beside its
equations (hand-made cases and identities of each mechanism), the configuration reader, the
checkpoint layout against the model's parameters, and the plan's cache needs."""
import copy
import math
import os

import pytest
import torch

import plain_pitenex as P
import util
from pitenex_cases import CASES, make_folder, random_case, split_ranks, write_model

F = torch.float64


# --------------------------------------------------------------------------- the plain implementation
def test_layer_norm_by_hand():
    x = torch.tensor([[1.0, 3.0]], dtype=F)               # mean 2, variance 1
    y = P.layer_norm(x, torch.tensor([2.0, 1.0], dtype=F), torch.tensor([10.0, -1.0], dtype=F), 3.0)
    assert y[0].tolist() == pytest.approx([10.0 - 2.0 / 2.0, -1.0 + 1.0 / 2.0])
    g = torch.Generator().manual_seed(1)
    x, w, b = (torch.randn(*s, generator=g, dtype=F) for s in ((4, 9), (9,), (9,)))
    assert util.rel_err(P.layer_norm(x, w, b, 1e-3), torch.nn.functional.layer_norm(x, (9,), w, b, 1e-3)) < 1e-12


def test_the_pair_embedding_by_hand():
    w = {"embed": torch.arange(4, dtype=F)[:, None] * 100, "bigram": torch.arange(6, dtype=F)[:, None]}
    cfg = {"embedding": {"bigram": {"buckets": 5, "mul_prev": 3, "mul_cur": 2}}}
    # first: row 5; then (2 * 3 + 1 * 2) % 5 = 3; then (1 * 3 + 3 * 2) % 5 = 4
    assert P.embed(w, cfg, [2, 1, 3]).flatten().tolist() == [205.0, 103.0, 304.0]


def test_rotation_pairs_sign_and_relative_positions():
    rot = {"dims": 6, "base": 100.0}
    x = torch.zeros(3, 1, 8, dtype=F)
    x[2, 0, 2] = 1.0                                       # pair 1 is (2, 3), position 2
    y = P.rotate_pairs(x, rot)
    a = 2.0 * 100.0 ** (-2.0 / 6.0)
    assert abs(float(y[2, 0, 2]) - math.cos(a)) < 1e-12 and abs(float(y[2, 0, 3]) - math.sin(a)) < 1e-12
    g = torch.Generator().manual_seed(1)
    q, k = (torch.randn(1, 1, 8, generator=g, dtype=F).expand(120, 1, 8) for _ in range(2))
    rq, rk = P.rotate_pairs(q, rot)[:, 0], P.rotate_pairs(k, rot)[:, 0]
    assert torch.equal(rq[:, 6:], q[:, 0, 6:])
    assert float(rq[17] @ rk[11]) == pytest.approx(float(rq[106] @ rk[100]), abs=1e-10)
    assert abs(float(rq[17] @ rk[11]) - float(rq[17] @ rk[12])) > 1e-3


def test_chunks_are_counted_from_the_start_and_a_sink_is_a_key_without_a_value():
    m = P.chunk_mask(7, 3)
    assert [int(r.sum()) for r in m] == [1, 2, 3, 1, 2, 3, 1] and bool(m[5, 3]) and not m[3, 2] and not m[3, 4]
    s = torch.tensor([[[1.0, 2.0]]], dtype=F)
    p = P.softmax_with_sink(s, torch.tensor([3.0], dtype=F))[0, 0]
    total = math.exp(1) + math.exp(2) + math.exp(3)
    assert p.tolist() == pytest.approx([math.exp(1) / total, math.exp(2) / total])
    # a very low sink is an ordinary softmax; a very high one leaves nothing and overflows nowhere
    assert util.rel_err(P.softmax_with_sink(s, torch.tensor([-1e3], dtype=F)), torch.softmax(s, -1)) < 1e-12
    assert float(P.softmax_with_sink(s, torch.tensor([1e3], dtype=F)).sum()) == 0.0


def test_short_convolution_against_the_library_s_convolution_and_by_hand():
    g = torch.Generator().manual_seed(2)
    x, taps = torch.randn(9, 5, generator=g, dtype=F), torch.randn(5, 4, generator=g, dtype=F)
    want = torch.nn.functional.conv1d(torch.nn.functional.pad(x.T[None], (3, 0)), taps[:, None], groups=5)[0].T
    assert util.rel_err(P.short_convolution(x, taps), want) < 1e-12
    assert util.rel_err(P.short_convolution(x[:2], taps), want[:2]) < 1e-12        # fewer tokens than taps
    y = P.short_convolution(torch.tensor([[1.0], [10.0]], dtype=F), torch.tensor([[3.0, 2.0]], dtype=F))
    assert y.flatten().tolist() == [2.0, 23.0]


def test_the_delta_rule_by_hand_and_in_its_written_out_form():
    """One channel, one value: S = 0 -> write -> decay, correct, write."""
    one = torch.ones(1, 1, 1, dtype=F)
    o = P.channel_delta_rule(torch.cat([one, one]), torch.cat([one, one]), torch.cat([2 * one, 5 * one]),
                             torch.full((2, 1), 0.5, dtype=F), torch.full((2, 1, 1), 0.25, dtype=F))
    # S = 0 + 0.5 * 2 = 1; then 0.25 + 0.5 * (5 - 0.25) = 2.625
    assert o.flatten().tolist() == [1.0, 2.625]
    # u = U0 - W S0 with the unit lower triangular system over all tokens, channels decaying apart
    g = torch.Generator().manual_seed(3)
    T, d, dv = 9, 4, 3
    q, k, v = (torch.randn(T, 1, n, generator=g, dtype=F) for n in (d, d, dv))
    k = P.unit(k)
    beta = torch.rand(T, 1, generator=g, dtype=F)
    dec = torch.rand(T, 1, d, generator=g, dtype=F) * 0.9 + 0.1
    G = torch.log(dec[:, 0]).cumsum(0)
    pair = torch.exp(G[:, None] - G[None])                              # [t, s, d]
    A = beta * torch.einsum("td,sd,tsd->ts", k[:, 0], k[:, 0], pair).tril(-1)
    U = torch.linalg.solve(torch.eye(T, dtype=F) + A, beta * v[:, 0])
    o = torch.einsum("td,sd,tsd->ts", q[:, 0], k[:, 0], pair).tril() @ U
    assert util.rel_err(P.channel_delta_rule(q, k, v, beta, dec)[:, 0], o) < 1e-10


def test_experts_clamp_and_the_route_by_hand():
    w = {"e.gate": torch.tensor([[1.0]], dtype=F), "e.up": torch.tensor([[1.0]], dtype=F),
         "e.down": torch.tensor([[1.0]], dtype=F)}

    def expert(x):
        return float(P.clamped_expert(w, "e.", 2.0, torch.tensor([[x]], dtype=F)))
    swish = lambda a: a / (1 + math.exp(-1.702 * a))
    assert expert(1.0) == pytest.approx(swish(1.0) * 2.0)
    assert expert(9.0) == pytest.approx(swish(2.0) * 3.0)               # both at the limit
    assert expert(-9.0) == pytest.approx(swish(-9.0) * -1.0)            # the gate has no lower limit
    z = torch.log(torch.tensor([[0.5, 0.3, 0.15, 0.05]], dtype=F))
    chosen, weights = P.route(z, torch.tensor([-0.4, 0.0, 0.0, 0.2], dtype=F), 2)
    assert chosen[0].tolist() == [1, 3] and weights[0].tolist() == pytest.approx([0.3 / 0.35, 0.05 / 0.35])
    # the last outputs are identity experts
    x = torch.tensor([[0.7]], dtype=F)
    w = {"e0." + k[2:]: v for k, v in w.items()}
    w.update(router=torch.tensor([[0.0], [0.0]], dtype=F), correction=torch.tensor([0.0, 1.0], dtype=F))
    mlp = {"router": {"experts": 1, "identity": 1, "top": 1}, "expert": {"limit": 2.0}, "shared": None}
    assert float(P.mixture(w, "", mlp, x)) == pytest.approx(0.7)
    mlp["router"]["top"] = 2
    assert float(P.mixture(w, "", mlp, x)) == pytest.approx(0.5 * 0.7 + 0.5 * swish(0.7) * 1.7)


# --------------------------------------------------------------------------- configuration and layout
def test_the_configuration_reader_and_what_it_refuses():
    import gpt_fast_amd as gfa
    from gpt_fast_amd.config.pitenex import ConfigError, DenseMlp, PitenexConfig
    for name, config in CASES.items():
        bare, c = split_ranks(config)
        assert PitenexConfig.from_dict(c.to_dict()) == c, name
        open_ = PitenexConfig.from_dict(bare)
        assert open_ != c and open_.with_ranks(lambda i: config["layers"][i]["mixer"]["right"]["ranks"]) == c
        plan = gfa.config.registry.architecture_of(bare).plan(c)
        assert len(plan.layers) == len(config["layers"]) and all(l.arrangement == "parallel" for l in plan.layers)
        with pytest.raises(ConfigError, match="ranks"):
            gfa.config.registry.architecture_of(bare).plan(open_)
    _, c = split_ranks(CASES["A"])
    a, r, f = c.layers[0].mixer.left, c.layers[0].mixer.right, c.layers[0].mlp
    assert (a.heads, a.kv_heads, a.dim, a.vdim, a.scale, a.chunk, a.rot_dims, a.rot_base) == \
        (6, 2, 24, 32, 0.3, 40, 12, 10000.0)
    assert (r.heads, r.kv_heads, r.dim, r.vdim, r.conv, r.decay_rank, r.gate_rank) == (4, 2, 24, 16, 4, 16, 40)
    assert (f.experts, f.identity, f.top, f.ff, f.limit, f.shared_ff, f.shared_limit) == (7, 3, 3, 40, 1.0, 56, 0.7)
    assert isinstance(c.layers[1].mlp, DenseMlp) and c.layers[2].mlp is None
    assert (c.buckets, c.mul_prev, c.mul_cur, c.residual_mult, c.logit_scale) == (97, 5, 3, 0.6, 0.5)
    assert (c.layers[0].mixer.left_scale, c.layers[0].mixer.right_scale) == (0.8, 1.3)

    def broken(change):
        config = copy.deepcopy(split_ranks(CASES["A"])[0])
        change(config)
        with pytest.raises(ConfigError):
            PitenexConfig.from_dict(config)
    left = lambda c: c["layers"][0]["mixer"]["left"]
    right = lambda c: c["layers"][0]["mixer"]["right"]
    broken(lambda c: c["layers"][0].update(type="other"))
    broken(lambda c: c["layers"][0]["mlp"].update(kind="other"))
    broken(lambda c: c["layers"][0]["mlp"]["router"].update(top=11))
    broken(lambda c: c["layers"][0]["mlp"]["expert"].pop("limit"))
    broken(lambda c: c["layers"][0]["mlp"]["shared"].pop("limit"))
    broken(lambda c: left(c).update(kv_heads=4))
    broken(lambda c: left(c)["rot"].update(dims=7))
    broken(lambda c: left(c)["rot"].update(dims=26))
    broken(lambda c: left(c)["mask"].update(size=0))
    broken(lambda c: left(c).pop("scale"))
    broken(lambda c: right(c).update(kv_heads=3))
    broken(lambda c: right(c).update(conv=0))
    broken(lambda c: c["layers"][0]["mixer"].pop("left_scale"))
    broken(lambda c: c["embedding"]["bigram"].pop("mul_cur"))
    broken(lambda c: c.update(layers=[]))
    for preset in ("pitenex-4096", "pitenex-8192"):
        arch, c = gfa.find_preset(preset)
        assert PitenexConfig.from_dict(arch.config_dict(c)) == c
        arch.plan(c)


@pytest.mark.parametrize("name", sorted(CASES))
def test_the_layout_names_every_parameter_of_the_model_and_the_tensors_give_the_ranks(tmp_path, name):
    import gpt_fast_amd as gfa
    from gpt_fast_amd.parts.base import Runtime
    from gpt_fast_amd.parts.model import DecoderModel
    from gpt_fast_amd.weights.bindings import load_parameters
    folder = make_folder(tmp_path, name, seed=1)
    arch, c = gfa.read_model_folder(folder)
    assert [(l.mixer.right.decay_rank, l.mixer.right.gate_rank) for l in c.layers] == \
        [l["mixer"]["right"]["ranks"] for l in CASES[name]["layers"]]
    model = DecoderModel(arch.plan(c), Runtime(torch.float32, "cpu"))
    declared = model.parameters()
    assert {b.target for b in arch.bindings(c).bindings} == set(declared)
    params = load_parameters(folder, arch.layouts(c), "float32", None)
    for target, p in declared.items():
        assert tuple(params[target].shape) == tuple(p.shape), target
    assert params["head"].data_ptr() == params["embed"].data_ptr()     # the head is the table itself
    _, w = P.load_folder(folder)
    model.bind(params)
    for i, layer in enumerate(CASES[name]["layers"]):
        mixer, p = model.blocks[i].mixer, f"l{i}.mix."
        # the joined first matrix: the left's rows, then the right's, each part where its kernel looks
        # for it; the second matrices of decay and gate with zeros between them
        m, right = layer["mixer"]["right"], mixer.branches[1]
        at = mixer.columns[1]
        assert torch.equal(mixer.w_in[:w[p + "left.q"].shape[0]].double(), w[p + "left.q"])
        assert torch.equal(mixer.w_in[at + right.rows.b:][:m["heads"]].double(), w[p + "right.b"])
        assert torch.equal(mixer.w_in[at + right.rows.g:][:m["ranks"][1]].double(), w[p + "right.g1"])
        n = m["heads"] * m["dim"]
        assert torch.equal(right.w_second[:n, :m["ranks"][0]].double(), w[p + "right.a2"])
        assert not right.w_second[:n, right.rows.a_rank:].any() and not right.w_second[n:, :right.rows.a_rank].any()
        assert mixer.wo.shape == (c.width, w[p + "left.o"].shape[1] + w[p + "right.o"].shape[1])
    assert model.parameter_count(exclude_embedding=False) == sum(
        t.numel() for k, t in params.items() if k != "head")
    needs = model.cache_needs()
    assert len(needs) == len(c.layers) + 1 and len(declared) == len(params)
    assert {"term_join", "scored_attention", "gated_delta", "delta_chunks", "short_conv"} <= set(model.kernel_libraries())


def test_wrong_tensors_are_named_together(tmp_path):
    import gpt_fast_amd as gfa
    from gpt_fast_amd.weights.bindings import WeightsError, load_parameters

    def fewer(t):
        del t["l1.mix.left.sink"]
        t["l0.norm1.b"] = t["l0.norm1.b"][:-1].clone()
        t["l1.norm2"] = torch.ones(96)
    folder = make_folder(tmp_path, "A", seed=2, patch=fewer, tag="fewer")
    arch, c = gfa.read_model_folder(folder)
    with pytest.raises(WeightsError) as e:
        load_parameters(folder, arch.layouts(c), "float32", None)
    for name in ("l1.mix.left.sink", "l0.norm1.b", "l1.norm2"):
        assert name in str(e.value)


def test_parts_refuse_what_they_cannot_do():
    from gpt_fast_amd.config.spec import (GatedDeltaSpec, GatedFeedForwardSpec, LayerSpec, NormedAttentionSpec, NormSpec,
                                          ParallelMixerSpec, RoutedExpertsSpec)
    from gpt_fast_amd.parts.base import BLOCKS, FEED_FORWARDS, MIXERS, Runtime
    from gpt_fast_amd.parts.model import _Arranged
    rt = Runtime(torch.float32, "cpu")
    left = NormedAttentionSpec(16, 2, 1, 8, 8, None, 0.3, chunk=4, sink=True)
    right = GatedDeltaSpec(16, 2, 1, 8, 8, 2, 1e-5, decay_rank=4, gate_rank=4)
    pair = (("a", left), ("b", right))
    with pytest.raises(ValueError):
        MIXERS.build(ParallelMixerSpec(16, pair, scales=(1.0,)), rt)
    with pytest.raises(ValueError):
        MIXERS.build(ParallelMixerSpec(16, pair), rt)
    with pytest.raises(ValueError):
        MIXERS.build(NormedAttentionSpec(16, 2, 1, 8, 8, None, 0.3, chunk=0), rt)
    with pytest.raises(ValueError):
        FEED_FORWARDS.build(RoutedExpertsSpec(16, 4, 7, 8, identity=2), rt)
    with pytest.raises(ValueError):
        FEED_FORWARDS.build(RoutedExpertsSpec(16, 4, 2, 8, activation="clamped_swish", gated=True), rt)
    with pytest.raises(Exception):
        FEED_FORWARDS.build(GatedFeedForwardSpec(16, 8, "clamped_swish"), rt)
    norm = NormSpec(16, 1e-5, kind="layer", bias=True)
    with pytest.raises(ValueError):
        BLOCKS.build(_Arranged(LayerSpec("l", ParallelMixerSpec(16, pair, scales=(1.0, 1.0)), norm, arrangement="parallel",
                                         feed_forward=GatedFeedForwardSpec(16, 8), feed_forward_norm=norm)), rt)
    with pytest.raises(TypeError):
        BLOCKS.build(_Arranged(LayerSpec("l", left, NormSpec(16, 1e-5, kind="none"), arrangement="post_norm",
                                         mixer_out_norm=norm)), rt)


def test_pages_of_chunks_that_ended_come_back():
    """A sequence of hundreds of tokens in chunks of 40 holds a page or two, not all of its pages."""
    from gpt_fast_amd.cache.store import Cache
    from gpt_fast_amd.config.spec import NormedAttentionSpec
    from gpt_fast_amd.parts.base import MIXERS, Runtime
    part = MIXERS.build(NormedAttentionSpec(16, 2, 1, 8, 8, None, 0.3, chunk=40, sink=True), Runtime(torch.float32, "cpu"))
    cache = Cache([part.cache_need()], [None], max_tokens=64 * 4, max_sequences=1, dtype=torch.float32, device="cpu")
    slot = cache.acquire()
    cache.extend(slot, 100)
    for _ in range(400):
        cache.extend(slot, 1)
        first = cache.length(slot) - 1
        held = cache.page_list(0, slot)
        assert all(held[p] >= 0 for p in range(first // 40 * 40 // 64, first // 64 + 1))    # what the token sees
        assert sum(p >= 0 for p in held) <= 3
    cache.check()
    # the prompt work counts a chunk's triangle, not the square
    part.wqkv = part.wo = None
    assert part.step_flops([80], [0]) - part.step_flops([40], [0]) == pytest.approx(part.step_flops([40], [40]))


def test_random_cases_are_read_and_run_by_the_plain_implementation(tmp_path):
    for seed in (1, 2):
        config = random_case(seed)
        folder = write_model(os.path.join(str(tmp_path), f"r{seed}"), config, seed)
        cfg, w = P.load_folder(folder)
        toks = util.random_tokens(cfg["vocab"], 30, seed)
        outs = []
        logits = P.forward(w, cfg, toks, outs)
        assert logits.shape == (30, cfg["vocab"]) and torch.isfinite(logits).all() and len(outs) == len(cfg["layers"])
        # causal: the logits of a prefix are the prefix of the logits
        assert util.rel_err(P.forward(w, cfg, toks[:11]), logits[:11]) < 1e-9
