"""CPU tests of Bikadra: what fixes the plain implementation of tests/plain_bikadra.py beside its
equations (hand-made cases and identities of each mechanism), the configuration reader, the
checkpoint layout against the model's parameters, and the plan's run order and cache needs."""
import copy
import math
import os

import pytest
import torch

import plain_bikadra as P
import util
from bikadra_cases import CASES, make_folder, random_case, write_model

F = torch.float64


# --------------------------------------------------------------------------- the plain implementation
def test_streams_by_hand():
    """Two streams of one element: 2 and 5.  in (1, 10): 52.  mix [from, to] = ((1, 100), (1000,
    10000)), out (0.5, 0.25), y = 8: stream 1 = 2 + 5000 + 4, stream 2 = 200 + 50000 + 2."""
    X = torch.tensor([[[2.0]], [[5.0]]], dtype=F)
    assert float(P.stream_read(X, torch.tensor([1.0, 10.0], dtype=F))) == 52.0
    new = P.stream_write(X, torch.tensor([[1.0, 100.0], [1000.0, 10000.0]], dtype=F),
                         torch.tensor([0.5, 0.25], dtype=F), torch.tensor([[8.0]], dtype=F))
    assert new.flatten().tolist() == [5006.0, 50202.0]
    # identity mix, all ones: every stream is a plain residual sum
    new = P.stream_write(X, torch.eye(2, dtype=F), torch.ones(2, dtype=F), torch.tensor([[8.0]], dtype=F))
    assert new.flatten().tolist() == [10.0, 13.0]


def test_norm_and_activation():
    x = torch.tensor([[3.0, -4.0]], dtype=F)
    assert util.rel_err(P.rms_norm(x, torch.tensor([2.0, 1.0], dtype=F), 0.5),
                        torch.tensor([[6.0, -4.0]], dtype=F) / math.sqrt(13.0)) < 1e-12
    z = torch.linspace(-4, 4, 33, dtype=F)
    assert util.rel_err(P.gelu_tanh(z), torch.nn.functional.gelu(z, approximate="tanh")) < 1e-12
    assert util.rel_err(P.softplus(torch.tensor([-40.0, 0.0, 40.0], dtype=F)),
                        torch.tensor([math.exp(-40.0), math.log(2.0), 40.0], dtype=F)) < 1e-12


def test_rotation_pairs_sign_and_relative_positions():
    rot = {"dims": 6, "base": 100.0}
    x = torch.zeros(1, 1, 8, dtype=F)
    x[0, 0, 0] = 1.0
    y = P.rotate_half(x, torch.tensor([2]), rot)
    # pair 0 is (0, 3) and turns by 2 radians; elements 6 and 7 pass
    assert abs(float(y[0, 0, 0]) - math.cos(2.0)) < 1e-12 and abs(float(y[0, 0, 3]) - math.sin(2.0)) < 1e-12
    g = torch.Generator().manual_seed(1)
    q, k = torch.randn(1, 1, 8, generator=g, dtype=F), torch.randn(1, 1, 8, generator=g, dtype=F)
    assert torch.equal(P.rotate_half(q, torch.tensor([9]), rot)[..., 6:], q[..., 6:])
    assert util.rel_err(P.rotate_half(q, torch.tensor([0]), rot), q) < 1e-15

    def dot(i, j):
        return float((P.rotate_half(q, torch.tensor([i]), rot) * P.rotate_half(k, torch.tensor([j]), rot)).sum())
    assert dot(17, 11) == pytest.approx(dot(106, 100), abs=1e-10)
    assert abs(dot(17, 11) - dot(17, 12)) > 1e-3


def test_the_rescaled_ladder_by_hand_and_against_the_library_s():
    """dims 8, base 100, original 64, factor 4, fast 16, slow 2: place(16) = -0.39 -> lo 0, place(2)
    = 1.41 -> hi 2; ramp = 0, 1/2, 1, 1."""
    from gpt_fast_amd.config.spec import PositionSpec
    from gpt_fast_amd.parts.position import frequencies_and_trig_scale
    rot = {"dims": 8, "base": 100.0, "scaling": {"factor": 4.0, "original": 64, "fast": 16.0, "slow": 2.0}}
    f, grow = P.rotary_frequencies(rot)
    plain = [100.0 ** (-2.0 * i / 8) for i in range(4)]
    want = [plain[0], plain[1] * (0.5 / 4 + 0.5), plain[2] / 4, plain[3] / 4]
    assert util.rel_err(f, torch.tensor(want, dtype=F)) < 1e-12
    assert grow == pytest.approx(0.1 * math.log(4.0) + 1.0)
    for name in ("A", "B", "C", "O"):
        for layer in CASES[name]["layers"]:
            r = layer["mixer"].get("rot")
            if layer["type"] != "latent_attention" or not r:
                continue
            sc = None if "scaling" not in r else (("rope_type", "yarn"),) + tuple(r["scaling"].items())
            freqs, trig = frequencies_and_trig_scale(PositionSpec(rotary_dim=r["dims"], base=r["base"],
                                                                  layout="half", scaling=sc))
            f, grow = P.rotary_frequencies(r)
            assert util.rel_err(freqs, f) < 1e-6 and trig == pytest.approx(grow)


def test_attention_is_the_library_function_s_and_scaled_as_given():
    g = torch.Generator().manual_seed(3)
    q, k, v = (torch.randn(7, 2, 5, generator=g, dtype=F) for _ in range(3))
    want = torch.nn.functional.scaled_dot_product_attention(
        q.transpose(0, 1), k.transpose(0, 1), v.transpose(0, 1), is_causal=True, scale=0.7).transpose(0, 1)
    assert util.rel_err(P.causal_attention(q, k, v, 0.7), want) < 1e-12


def test_latent_attention_in_the_latent_s_space_is_the_same():
    """Keys and values written out per head against the form with one kv head whose key is the
    latent and the rotated part and whose value is the latent."""
    m = CASES["A"]["layers"][0]["mixer"]
    H, d, dr, dv, R, Q, D, T = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"], m["q_rank"], 20, 9
    g = torch.Generator().manual_seed(4)
    w = {n: torch.randn(*s, generator=g, dtype=F) * 0.3 for n, s in
         {"dq": (Q, D), "uq": (H * (d + dr), Q), "dkv": (R + dr, D), "uk": (H * d, R), "uv": (H * dv, R),
          "g": (H, D), "o": (D, H * dv)}.items()}
    w["dq.norm"], w["dkv.norm"] = torch.rand(Q, generator=g, dtype=F), torch.rand(R, generator=g, dtype=F)
    h = torch.randn(T, D, generator=g, dtype=F)
    want = P.latent_attention(w, "", m, 1e-5, h)
    pos = torch.arange(T)
    q = (P.rms_norm(h @ w["dq"].T, w["dq.norm"], 1e-5) @ w["uq"].T).view(T, H, d + dr)
    kv = h @ w["dkv"].T
    c = P.rms_norm(kv[:, :R], w["dkv.norm"], 1e-5)
    key = torch.cat([c[:, None], P.rotate_half(kv[:, None, R:], pos, m["rot"])], -1).expand(T, H, R + dr)
    uk, uv = w["uk"].view(H, d, R), w["uv"].view(H, dv, R)
    query = torch.cat([torch.einsum("thd,hdr->thr", q[..., :d], uk), P.rotate_half(q[..., d:], pos, m["rot"])], -1)
    lat = P.causal_attention(query, key, c[:, None].expand(T, H, R), m["scale"])
    lat = lat * torch.sigmoid(h @ w["g"].T)[..., None]                 # the gate commutes with w_uv
    got = torch.einsum("thr,hvr->thv", lat, uv).reshape(T, H * dv) @ w["o"].T
    assert util.rel_err(got, want) < 1e-10


def test_short_convolution_against_the_library_s_convolution_and_by_hand():
    g = torch.Generator().manual_seed(2)
    x, taps, bias = (torch.randn(*s, generator=g, dtype=F) for s in ((9, 5), (5, 4), (5,)))
    want = torch.nn.functional.conv1d(torch.nn.functional.pad(x.T[None], (3, 0)), taps[:, None], bias, groups=5)[0].T
    assert util.rel_err(P.short_convolution(x, taps, bias), want) < 1e-12
    y = P.short_convolution(torch.tensor([[1.0], [10.0], [100.0]], dtype=F), torch.tensor([[3.0, 2.0]], dtype=F),
                            torch.tensor([0.5], dtype=F))
    assert y.flatten().tolist() == [2.5, 23.5, 230.5]


def test_the_state_space_cell_has_its_closed_form_and_uses_its_groups():
    g = torch.Generator().manual_seed(5)
    T, H, dv, G, N = 7, 4, 3, 2, 5
    x, B, C = (torch.randn(*s, generator=g, dtype=F) for s in ((T, H, dv), (T, G, N), (T, G, N)))
    dt = torch.rand(T, H, generator=g, dtype=F)
    A_log, D = torch.randn(H, generator=g, dtype=F), torch.randn(H, generator=g, dtype=F)
    y = P.state_space(x, B, C, dt, A_log, D)
    for t in (0, 3, 6):
        for h in range(H):
            want = D[h] * x[t, h]
            for s in range(t + 1):
                decay = torch.exp(-torch.exp(A_log[h]) * dt[s + 1:t + 1, h].sum())
                want = want + decay * dt[s, h] * (B[s, h // 2] @ C[t, h // 2]) * x[s, h]
            assert util.rel_err(y[t, h], want) < 1e-10
    # causal
    x2 = x.clone()
    x2[4:] = 9.0
    assert torch.equal(P.state_space(x2, B, C, dt, A_log, D)[:4], y[:4])


def test_the_gate_comes_before_the_norm_and_every_part_has_its_own():
    y, z = torch.tensor([[1.0, 2.0, 3.0, 4.0]], dtype=F), torch.tensor([[0.0, 1.0, 2.0, -1.0]], dtype=F)
    w = torch.tensor([1.0, 1.0, 1.0, 2.0], dtype=F)
    u = [0.0, 2 / (1 + math.exp(-1)), 3 * 2 / (1 + math.exp(-2)), 4 * -1 / (1 + math.exp(1))]
    r1, r2 = math.sqrt((u[0] ** 2 + u[1] ** 2) / 2 + 0.1), math.sqrt((u[2] ** 2 + u[3] ** 2) / 2 + 0.1)
    want = torch.tensor([[u[0] / r1, u[1] / r1, u[2] / r2, 2 * u[3] / r2]], dtype=F)
    assert util.rel_err(P.gated_group_norm(y, z, w, 2, 0.1), want) < 1e-12


def test_the_run_order():
    assert P.run_order({"layers": [0] * 6, "loop": {"start": 1, "stop": 4, "times": 2}}) == [0, 1, 2, 3, 1, 2, 3, 4, 5]
    assert P.run_order({"layers": [0] * 2}) == [0, 1]
    from gpt_fast_amd.architectures.bikadra import bikadra_plan
    from gpt_fast_amd.config.bikadra import BikadraConfig
    for name, config in CASES.items():
        plan = bikadra_plan(BikadraConfig.from_dict(config))
        assert [r.layer for r in plan.order] == P.run_order(config), name
        assert all(r.cache_from is None for r in plan.order)           # each pass has its own cache


# --------------------------------------------------------------------------- configuration and layout
def test_the_configuration_reader_and_what_it_refuses():
    import gpt_fast_amd as gfa
    from gpt_fast_amd.config.bikadra import BikadraConfig, ConfigError
    for name, config in CASES.items():
        c = BikadraConfig.from_dict(config)
        assert BikadraConfig.from_dict(c.to_dict()) == c, name
        plan = gfa.config.registry.architecture_of(config).plan(c)
        assert len(plan.layers) == len(config["layers"]) and plan.streams == config["streams"]
    c = BikadraConfig.from_dict(CASES["A"])
    m = c.layers[0].mixer
    assert (m.heads, m.dim, m.rot_dim, m.vdim, m.q_rank, m.kv_rank, m.scale) == (6, 24, 16, 16, 40, 48, 0.3)
    assert m.rot.scaling == (4.0, 64.0, 16.0, 2.0) and c.layers[2].mlp is None and c.layers[0].mlp.ff == 136
    m = c.layers[1].mixer
    assert (m.heads, m.vdim, m.state, m.groups, m.conv, m.norm_groups) == (6, 16, 24, 3, 3, 4)
    assert c.streams == 3 and c.embedding_scale == 1.5 and c.logit_softcap == 20.0
    assert (c.loop.start, c.loop.stop, c.loop.times) == (1, 3, 3)

    def broken(change):
        config = copy.deepcopy(CASES["A"])
        change(config)
        with pytest.raises(ConfigError):
            BikadraConfig.from_dict(config)
    broken(lambda c: c["layers"][0].update(type="other"))
    broken(lambda c: c["layers"][0]["mlp"].update(kind="moe"))
    broken(lambda c: c["layers"][1]["mixer"].update(groups=4))
    broken(lambda c: c["layers"][1]["mixer"].update(norm_groups=7))
    broken(lambda c: c["layers"][1]["mixer"].pop("conv"))
    broken(lambda c: c["layers"][1]["mixer"].update(state=0))
    broken(lambda c: c["layers"][0]["mixer"]["rot"].update(dims=7))
    broken(lambda c: c["layers"][0]["mixer"]["rot"].update(dims=18))
    broken(lambda c: c["layers"][0]["mixer"].pop("kv_rank"))
    broken(lambda c: c["loop"].update(stop=9))
    broken(lambda c: c.pop("streams"))
    broken(lambda c: c.update(layers=[]))
    for preset in ("bikadra-4096", "bikadra-8192"):
        arch, c = gfa.find_preset(preset)
        assert BikadraConfig.from_dict(arch.config_dict(c)) == c


def test_a_plan_of_several_streams_takes_only_layers_that_work_on_them():
    import dataclasses

    import gpt_fast_amd as gfa
    arch = gfa.config.registry.architecture("Bikadra")
    plan = arch.plan(arch.read_config(CASES["A"]))
    plan.layers[1] = dataclasses.replace(plan.layers[1], streams=None, arrangement="pre_norm")
    with pytest.raises(ValueError, match="streams"):
        plan.validate()


@pytest.mark.parametrize("name", sorted(CASES))
def test_the_layout_names_every_parameter_of_the_model(tmp_path, name):
    import gpt_fast_amd as gfa
    from gpt_fast_amd.parts.base import Runtime
    from gpt_fast_amd.parts.model import DecoderModel
    from gpt_fast_amd.weights.bindings import load_parameters
    arch = gfa.config.registry.architecture_of(CASES[name])
    c = arch.read_config(CASES[name])
    model = DecoderModel(arch.plan(c), Runtime(torch.float32, "cpu"))
    declared = model.parameters()
    layout = arch.bindings(c)
    assert {b.target for b in layout.bindings} == set(declared)
    folder = make_folder(tmp_path, name, seed=1)
    params = load_parameters(folder, arch.layouts(c), "float32", None)
    for target, p in declared.items():
        assert tuple(params[target].shape) == tuple(p.shape), target
    assert params["head"].data_ptr() == params["embed"].data_ptr()     # the head is the table itself
    _, w = P.load_folder(folder)
    for i, layer in enumerate(CASES[name]["layers"]):
        m = layer["mixer"]
        if layer["type"] == "latent_attention":
            down = params[f"l{i}.mix.w_down"].double()
            assert torch.equal(down[-m["heads"]:], w[f"l{i}.mix.g"])   # the gates' rows come last
            assert torch.equal(down[:m["q_rank"]], w[f"l{i}.mix.dq"])
        assert (f"l{i}.hc2.mix" in params) == (layer["mlp"] is not None)
    needs = model.cache_needs()
    assert len(needs) == len(P.run_order(CASES[name])) and len(declared) == len(params)
    assert {"streams", "state_space", "short_conv", "scored_attention"} <= set(model.kernel_libraries())


def test_what_a_layer_without_a_feed_forward_stores_for_it_is_not_used(tmp_path):
    import gpt_fast_amd as gfa
    from gpt_fast_amd.weights.bindings import WeightsError, load_parameters

    def patch(t):
        t["l2.norm2"] = torch.ones(96)
        t["l2.hc2.mix"] = torch.eye(3)
    folder = make_folder(tmp_path, "A", seed=2, patch=patch, tag="more")
    arch, c = gfa.read_model_folder(folder)
    assert "l2.norm2.weight" not in load_parameters(folder, arch.layouts(c), "float32", None)

    def fewer(t):
        del t["l1.mix.conv.b"]
        t["l0.hc1.in"] = t["l0.hc1.in"][:-1].clone()
        t["l1.norm3"] = torch.ones(96)
    folder = make_folder(tmp_path, "A", seed=2, patch=fewer, tag="fewer")
    with pytest.raises(WeightsError) as e:
        load_parameters(folder, arch.layouts(c), "float32", None)
    for name in ("l1.mix.conv.b", "l0.hc1.in", "l1.norm3"):
        assert name in str(e.value)


def test_random_cases_are_read_and_run_by_the_plain_implementation(tmp_path):
    from gpt_fast_amd.config.bikadra import BikadraConfig
    for seed in (1, 2):
        config = random_case(seed)
        BikadraConfig.from_dict(config)
        folder = write_model(os.path.join(str(tmp_path), f"r{seed}"), config, seed)
        cfg, w = P.load_folder(folder)
        toks = util.random_tokens(cfg["vocab"], 30, seed)
        outs = []
        logits = P.forward(w, cfg, toks, outs)
        assert logits.shape == (30, cfg["vocab"]) and torch.isfinite(logits).all() and len(outs) == len(P.run_order(cfg))
        # causal: the logits of a prefix are the prefix of the logits
        assert util.rel_err(P.forward(w, cfg, toks[:11]), logits[:11]) < 1e-9
