"""The Pitenex decoder as data: its plan and its checkpoint layout.

Plan: the embedded rows plus an embedding of the pair (previous token, token); the layers
``config.json`` lists, each with one layer norm (weight and bias) whose rows the mixer and the
feed-forward both read, and ``x <- x + residual_mult (mixer(h) + ff(h))``; the mixer is a weighted sum
of an attention (interleaved rotary pairs, chunks of positions, a learned sink per head) and a gated
delta rule with a decay per key channel; the feed-forward is gated with the tanh form of gelu, or a
mixture of clamped gated experts of which some hand their input on, or absent.  The final norm's
rows go through the embedding table itself, times a constant.

Checkpoint layout: ``embed``, ``bigram``, ``l<i>.norm1`` (+ ``.b``), ``l<i>.mix.left.<name>``,
``l<i>.mix.right.<name>``, ``l<i>.mlp.<name>``, ``final.norm`` (+ ``.b``); linear weights [out, in].
Projections that read the same input are joined into one matrix when they are loaded.
"""
import torch

from ..config.pitenex import ConfigError, DenseMlp, MoeMlp, PitenexConfig
from ..config.registry import Architecture, register_architecture
from ..config.spec import (GatedDeltaSpec, GatedFeedForwardSpec, LayerSpec, ModelPlan, NormedAttentionSpec,
                           NormSpec, PairEmbeddingSpec, ParallelMixerSpec, PositionSpec, RoutedExpertsSpec, Run)
from ..weights.bindings import Binding, CheckpointLayout, Source

PAIR_TABLE = "pair_embedding"


def _mixer_spec(c: PitenexConfig, m) -> ParallelMixerSpec:
    a, r = m.left, m.right
    position = PositionSpec(kind="none")
    if a.rot_dims:
        position = PositionSpec(kind="rope", rotary_dim=a.rot_dims, base=a.rot_base, layout="interleaved")
    left = NormedAttentionSpec(dim=c.width, n_heads=a.heads, n_kv_heads=a.kv_heads, head_dim=a.dim,
                               value_dim=a.vdim, position=position, scale=a.scale, chunk=a.chunk, sink=True)
    if not (r.decay_rank and r.gate_rank):
        raise ConfigError("Pitenex: the ranks of the delta rule's decay and gate are neither in the "
                          "configuration nor known from a checkpoint")
    right = GatedDeltaSpec(dim=c.width, n_heads=r.heads, n_kv_heads=r.kv_heads, key_dim=r.dim, value_dim=r.vdim,
                           conv_taps=r.conv, eps=c.norm_eps, unit_eps=1e-6, gate="sigmoid",
                           decay_rank=r.decay_rank, gate_rank=r.gate_rank)
    return ParallelMixerSpec(dim=c.width, branches=(("left", left), ("right", right)),
                             scales=(m.left_scale, m.right_scale))


def _feed_forward_spec(c: PitenexConfig, mlp):
    if mlp is None:
        return None
    if isinstance(mlp, DenseMlp):
        return GatedFeedForwardSpec(c.width, mlp.ff, "gelu_tanh")
    assert isinstance(mlp, MoeMlp)
    return RoutedExpertsSpec(dim=c.width, n_experts=mlp.experts, top=mlp.top, hidden=mlp.ff,
                             shared_hidden=mlp.shared_ff, activation="clamped_swish", weight_eps=1e-20,
                             scoring="softmax", choice_correction=True, gated=True, identity=mlp.identity,
                             limit=mlp.limit, shared_limit=mlp.shared_limit if mlp.shared_ff else None)


def pitenex_plan(c: PitenexConfig) -> ModelPlan:
    def norm():
        return NormSpec(c.width, c.norm_eps, kind="layer", bias=True)

    layers = [LayerSpec(name=f"l{i}", arrangement="parallel", result_scale=c.residual_mult,
                        mixer=_mixer_spec(c, l.mixer), mixer_norm=norm(),
                        feed_forward=_feed_forward_spec(c, l.mlp), mixer_name="mix", mixer_norm_name="norm1",
                        feed_forward_name="mlp")
              for i, l in enumerate(c.layers)]
    adds = ()
    if c.buckets:
        adds = (PairEmbeddingSpec(dim=c.width, buckets=c.buckets, mul_prev=c.mul_prev, mul_cur=c.mul_cur,
                                  name=PAIR_TABLE),)
    plan = ModelPlan(
        dim=c.width, vocab_size=c.vocab, layers=layers, order=[Run(i) for i in range(len(layers))],
        final_norm=norm(), tie_embeddings=True, max_positions=c.max_positions, embedding_name="embed",
        final_norm_name="final.norm", head_name="head", input_adds=adds,
        logit_scale=None if c.logit_scale == 1.0 else c.logit_scale)
    plan.validate()
    return plan


def pitenex_bindings(c: PitenexConfig) -> CheckpointLayout:
    D, V = c.width, c.vocab
    b = [Binding("embed", (Source("embed", (V, D)),))]
    if c.buckets:
        b.append(Binding(PAIR_TABLE + ".table", (Source("bigram", (c.buckets + 1, D)),)))

    def vector(target, name, shape, init="norm"):
        return Binding(target, (Source(name, shape, init),), role="vector")

    def norm(target, name):
        return [vector(target + ".weight", name, (D,)), vector(target + ".bias", name + ".b", (D,), "around_zero")]

    for i, l in enumerate(c.layers):
        p = f"l{i}."
        a, r = l.mixer.left, l.mixer.right
        H, G, d, dv = a.heads, a.kv_heads, a.dim, a.vdim
        x = p + "mix.left."
        b += norm(p + "norm1", p + "norm1")
        b += [
            Binding(x + "wqkv", (Source(x + "q", (H * d, D)), Source(x + "k", (G * d, D)),
                                 Source(x + "v", (G * dv, D))), combine=torch.cat),
            vector(x + "sink", x + "sink", (H,), "unit"),
            Binding(x + "wo", (Source(x + "o", (D, H * dv)),)),
        ]
        H, G, d, dv = r.heads, r.kv_heads, r.dim, r.vdim
        x = p + "mix.right."
        b += [
            # rows of q, k, v (the convolved channels), beta, the first matrices of decay and gate
            Binding(x + "w_in", (Source(x + "q", (G * d, D)), Source(x + "k", (G * d, D)),
                                 Source(x + "v", (H * dv, D)), Source(x + "b", (H, D)),
                                 Source(x + "a1", (r.decay_rank, D)), Source(x + "g1", (r.gate_rank, D))),
                    combine=torch.cat),
            Binding(x + "taps", (Source(x + "q.conv", (G * d, r.conv), "unit"),
                                 Source(x + "k.conv", (G * d, r.conv), "unit"),
                                 Source(x + "v.conv", (H * dv, r.conv), "unit")),
                    role="vector", combine=torch.cat),
            vector(x + "A_log", x + "A_log", (H,), "around_zero"),
            Binding(x + "w_a2", (Source(x + "a2", (H * d, r.decay_rank)),)),
            vector(x + "dt_bias", x + "dt_bias", (H * d,), "around_zero"),
            Binding(x + "w_g2", (Source(x + "g2", (H * dv, r.gate_rank)),)),
            vector(x + "norm", x + "norm", (dv,)),
            Binding(x + "wo", (Source(x + "o", (D, H * dv)),)),
        ]
        f, x = l.mlp, p + "mlp."
        if isinstance(f, DenseMlp):
            b += [Binding(x + "w13", (Source(x + "gate", (f.ff, D)), Source(x + "up", (f.ff, D))),
                          combine=torch.cat),
                  Binding(x + "w2", (Source(x + "down", (D, f.ff)),))]
        elif f is not None:
            n = f.experts
            b += [
                Binding(x + "w_router", (Source(x + "router", (n + f.identity, D)),)),
                vector(x + "correction", x + "correction", (n + f.identity,), "around_zero"),
                # an expert's gate rows and then its up rows; the experts stacked
                Binding(x + "w_up", tuple(Source(f"{x}e{e}.{part}", (f.ff, D))
                                          for e in range(n) for part in ("gate", "up")),
                        combine=lambda parts, n=n: torch.cat(parts).view(n, -1, parts[0].shape[1])),
                Binding(x + "w_down", tuple(Source(f"{x}e{e}.down", (D, f.ff)) for e in range(n)),
                        combine=torch.stack),
            ]
            if f.shared_ff:
                b += [Binding(x + "shared_up", (Source(x + "shared.gate", (f.shared_ff, D)),
                                                Source(x + "shared.up", (f.shared_ff, D))), combine=torch.cat),
                      Binding(x + "shared_down", (Source(x + "shared.down", (D, f.shared_ff)),))]
    b += norm("final.norm", "final.norm")
    # the output head is the embedding table
    b.append(Binding("head", (Source("head", (V, D)),), alias_of="embed"))
    return CheckpointLayout(tuple(b))


def pitenex_sizes_from_tensors(c: PitenexConfig, shapes: dict) -> PitenexConfig:
    """The ranks of decay and gate, where the configuration leaves them to the checkpoint."""
    def rank(i, name):
        shape = shapes.get(f"l{i}.mix.right.{name}", ())
        return int(shape[0]) if len(shape) == 2 else 0
    return c.with_ranks(lambda i: (rank(i, "a1"), rank(i, "g1")))


def pitenex_sizes(c: PitenexConfig) -> dict:
    """The sizes that the layers share, flat; per-layer sizes as short strings."""
    kinds = "".join("-" if l.mlp is None else ("d" if isinstance(l.mlp, DenseMlp) else "e") for l in c.layers)
    out = {"n_layer": len(c.layers), "dim": c.width, "vocab_size": c.vocab, "norm_eps": c.norm_eps,
           "feed_forward_kinds": kinds, "pair_buckets": c.buckets, "residual_mult": c.residual_mult}
    a, r = c.layers[0].mixer.left, c.layers[0].mixer.right
    out["left"] = f"{a.heads} heads of {a.dim}, {a.kv_heads} kv heads, values {a.vdim}, chunks of {a.chunk}"
    out["right"] = (f"{r.heads} heads of {r.dim} x {r.vdim}, {r.kv_heads} key heads, {r.conv} taps, ranks "
                    f"{r.decay_rank} and {r.gate_rank}")
    for l in c.layers:
        f = l.mlp
        if isinstance(f, DenseMlp) and "intermediate_size" not in out:
            out["intermediate_size"] = f.ff
        if isinstance(f, MoeMlp) and "experts" not in out:
            out["experts"] = f"{f.experts} of {f.ff} and {f.identity} identity, top {f.top}, shared {f.shared_ff}"
    return out


PITENEX = register_architecture(Architecture(
    names=("Pitenex", "pitenex"),
    read_config=PitenexConfig.from_dict,
    plan=pitenex_plan,
    bindings=pitenex_bindings,
    config_dict=PitenexConfig.to_dict,
    presets=PitenexConfig.from_name,
    describe=pitenex_sizes,
    layer_count_key="layers",
    sizes_from_tensors=pitenex_sizes_from_tensors,
))
