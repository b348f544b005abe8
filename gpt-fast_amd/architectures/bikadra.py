"""The Bikadra decoder as data: its plan and its checkpoint layout.

Plan: the embedded rows times a constant, copied into several streams; the layers
``config.json`` lists, each a block whose sublayers read a weighted sum of the streams through
an RMS norm and whose results move all streams at once (hyper-connections); the mixer is latent
attention with half-split rotary pairs on a rescaled ladder and a gate per head, or a
state-space cell (Mamba-2) behind a short convolution; the feed-forward two matrices with the
tanh form of gelu, or none.  The layers ``loop.start .. loop.stop - 1`` run ``loop.times`` times
in a row with the same weights, each run with a cache entry of its own.  The sum of the streams
goes through the final norm and the embedding table itself, and the logits are capped.

Checkpoint layout: ``embed``, ``l<i>.norm1`` / ``.norm2``, ``l<i>.hc1.in`` / ``.out`` / ``.mix`` (and
``hc2``), ``l<i>.mix.<name>``, ``l<i>.mlp.up`` / ``.down``, ``final.norm``; linear weights
[out, in].  Projections that read the same input are joined into one matrix when they are
loaded.
"""
import torch

from ..config.bikadra import BikadraConfig, LatentMixer, StateSpaceMixer
from ..config.registry import Architecture, register_architecture
from ..config.spec import (DenseFeedForwardSpec, LatentAttentionSpec, LayerSpec, ModelPlan, NormSpec,
                           PositionSpec, Run, StateSpaceSpec)
from ..weights.bindings import Binding, CheckpointLayout, Source


def _position(rot):
    if rot is None:
        return PositionSpec(kind="none")
    scaling = None
    if rot.scaling is not None:
        factor, original, fast, slow = rot.scaling
        scaling = (("rope_type", "yarn"), ("factor", factor), ("original", original),
                   ("fast", fast), ("slow", slow))
    return PositionSpec(kind="rope", rotary_dim=rot.dims, base=rot.base, layout="half", scaling=scaling)


def _mixer_spec(c: BikadraConfig, m):
    if isinstance(m, LatentMixer):
        return LatentAttentionSpec(dim=c.width, n_heads=m.heads, head_dim=m.dim, rot_dim=m.rot_dim,
                                   value_dim=m.vdim, q_rank=m.q_rank, kv_rank=m.kv_rank, scale=m.scale,
                                   eps=c.norm_eps, position=_position(m.rot), head_gate=True)
    assert isinstance(m, StateSpaceMixer)
    return StateSpaceSpec(dim=c.width, n_heads=m.heads, value_dim=m.vdim, state=m.state,
                          n_groups=m.groups, conv_taps=m.conv, norm_groups=m.norm_groups,
                          eps=c.norm_eps)


def _order(c: BikadraConfig):
    n = len(c.layers)
    if c.loop is None:
        return [Run(i) for i in range(n)]
    a, b = c.loop.start, c.loop.stop
    return [Run(i) for i in list(range(a)) + list(range(a, b)) * c.loop.times + list(range(b, n))]


def bikadra_plan(c: BikadraConfig) -> ModelPlan:
    def norm():
        return NormSpec(c.width, c.norm_eps)

    layers = []
    for i, l in enumerate(c.layers):
        has_ff = l.mlp is not None
        layers.append(LayerSpec(
            name=f"l{i}", arrangement="hyper_connected", streams=c.streams,
            mixer=_mixer_spec(c, l.mixer), mixer_norm=norm(),
            feed_forward=DenseFeedForwardSpec(c.width, l.mlp.ff, "gelu_tanh") if has_ff else None,
            feed_forward_norm=norm() if has_ff else None,
            mixer_name="mix", mixer_norm_name="norm1", mixer_streams_name="hc1",
            feed_forward_name="mlp", feed_forward_norm_name="norm2", feed_forward_streams_name="hc2"))
    plan = ModelPlan(
        dim=c.width, vocab_size=c.vocab, layers=layers, order=_order(c), final_norm=norm(),
        tie_embeddings=True, max_positions=c.max_positions, embedding_name="embed",
        final_norm_name="final.norm", head_name="head", streams=c.streams,
        embedding_scale=None if c.embedding_scale == 1.0 else c.embedding_scale,
        logit_softcap=c.logit_softcap)
    plan.validate()
    return plan


def bikadra_bindings(c: BikadraConfig) -> CheckpointLayout:
    D, V, S = c.width, c.vocab, c.streams
    b = [Binding("embed", (Source("embed", (V, D)),))]

    def vector(target, name, shape, init="norm"):
        return Binding(target, (Source(name, shape, init),), role="vector")

    for i, l in enumerate(c.layers):
        p = f"l{i}."
        m = l.mixer
        for q in (1, 2) if l.mlp is not None else (1,):
            b += [vector(f"{p}norm{q}.weight", f"{p}norm{q}", (D,)),
                  vector(f"{p}hc{q}.in", f"{p}hc{q}.in", (S,), "share"),
                  vector(f"{p}hc{q}.out", f"{p}hc{q}.out", (S,)),
                  vector(f"{p}hc{q}.mix", f"{p}hc{q}.mix", (S, S), "near_identity")]
        x = p + "mix."
        if isinstance(m, LatentMixer):
            H, d, dr, dv, R = m.heads, m.dim, m.rot_dim, m.vdim, m.kv_rank
            b += [
                # rows of the query latent, of the kv latent with the rotated key part, of the gate
                Binding(x + "w_down", (Source(x + "dq", (m.q_rank, D)), Source(x + "dkv", (R + dr, D)),
                                       Source(x + "g", (H, D))), combine=torch.cat),
                vector(x + "q_norm", x + "dq.norm", (m.q_rank,)),
                vector(x + "kv_norm", x + "dkv.norm", (R,)),
                Binding(x + "w_uq", (Source(x + "uq", (H * (d + dr), m.q_rank)),)),
                Binding(x + "w_uk", (Source(x + "uk", (H * d, R)),)),
                Binding(x + "w_uv", (Source(x + "uv", (H * dv, R)),)),
                Binding(x + "wo", (Source(x + "o", (D, H * dv)),)),
            ]
        else:
            assert isinstance(m, StateSpaceMixer)
            H, inner = m.heads, m.heads * m.vdim
            C = inner + 2 * m.groups * m.state
            b += [
                Binding(x + "w_in", (Source(x + "in", (inner + C + H, D)),)),
                vector(x + "taps", x + "conv", (C, m.conv), "unit"),
                vector(x + "conv_bias", x + "conv.b", (C,), "around_zero"),
                vector(x + "dt_bias", x + "dt_bias", (H,), "around_zero"),
                vector(x + "A_log", x + "A_log", (H,), "around_zero"),
                vector(x + "skip", x + "D", (H,)),
                vector(x + "norm", x + "norm", (inner,)),
                Binding(x + "wo", (Source(x + "o", (D, inner)),)),
            ]
        if l.mlp is not None:
            b += [Binding(p + "mlp.w_up", (Source(p + "mlp.up", (l.mlp.ff, D)),)),
                  Binding(p + "mlp.w_down", (Source(p + "mlp.down", (D, l.mlp.ff)),))]
    b.append(vector("final.norm.weight", "final.norm", (D,)))
    # the output head is the embedding table (without its factor)
    b.append(Binding("head", (Source("head", (V, D)),), alias_of="embed"))
    # a layer without a feed-forward has no second sublayer: what is stored for it is not used
    unused = tuple(rf"^l{i}\.(norm2|hc2\..*)$" for i, l in enumerate(c.layers) if l.mlp is None)
    return CheckpointLayout(tuple(b), ignored=unused)


def bikadra_sizes(c: BikadraConfig) -> dict:
    """The sizes that the layers share, flat; per-layer sizes as short strings."""
    letter = {"latent_attention": "c", "mamba2": "m"}
    out = {"n_layer": len(c.layers), "dim": c.width, "vocab_size": c.vocab, "norm_eps": c.norm_eps,
           "streams": c.streams, "layer_kinds": "".join(letter[l.type] for l in c.layers)}
    if c.loop is not None:
        out["loop"] = f"layers {c.loop.start}..{c.loop.stop - 1} x {c.loop.times}"
    for l in c.layers:
        m = l.mixer
        if isinstance(m, LatentMixer) and "latent_attention" not in out:
            out["latent_attention"] = (f"{m.heads} heads of {m.dim} + {m.rot_dim}, values {m.vdim}, latents "
                                       f"{m.q_rank} and {m.kv_rank}, gated heads")
        if isinstance(m, StateSpaceMixer) and "mamba2" not in out:
            out["mamba2"] = (f"{m.heads} heads of {m.vdim}, {m.state} states, {m.groups} groups, "
                             f"{m.conv} taps, {m.norm_groups} norm groups")
        if l.mlp is not None and "intermediate_size" not in out:
            out["intermediate_size"] = l.mlp.ff
    return out


BIKADRA = register_architecture(Architecture(
    names=("Bikadra", "bikadra"),
    read_config=BikadraConfig.from_dict,
    plan=bikadra_plan,
    bindings=bikadra_bindings,
    config_dict=BikadraConfig.to_dict,
    presets=BikadraConfig.from_name,
    describe=bikadra_sizes,
    layer_count_key="layers",
))
