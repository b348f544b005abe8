"""Small Bikadra configurations for the tests; they differ from each other in every size and
option.  Weights are drawn by the library's random-weights mode and may be patched before
they are written."""
import json
import os

import torch


def _rot(dims, base, scaling=None):
    r = {"dims": dims, "base": base}
    if scaling is not None:
        r["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    return r


def _latent(heads, dim, rot_dim, vdim, q_rank, kv_rank, scale, rot, ff=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank,
         "kv_rank": kv_rank, "scale": scale}
    if rot is not None:
        m["rot"] = rot
    return {"type": "latent_attention", "mixer": m, "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def _mamba(heads, vdim, state, groups, conv, norm_groups, ff=None):
    return {"type": "mamba2",
            "mixer": {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": conv,
                      "norm_groups": norm_groups},
            "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def _model(width, vocab, eps, streams, embed_scale, cap, layers, loop=None):
    d = {"architecture": "Bikadra", "vocab": vocab, "width": width, "norm": {"eps": eps},
         "streams": streams, "embedding": {"scale": embed_scale}, "layers": layers}
    if cap is not None:
        d["logit_softcap"] = cap
    if loop is not None:
        d["loop"] = dict(zip(("start", "stop", "times"), loop))
    return d


CASES = {
    # attention first; three streams; more norm groups than groups; values of another size than
    # the unrotated part; a ladder whose ramp lies inside it; a layer without a feed-forward; two
    # middle layers three times over
    "A": _model(96, 300, 1e-5, 3, 1.5, 20.0, [
        _latent(6, 24, 16, 16, 40, 48, 0.3, _rot(16, 10000.0, (4.0, 64, 16.0, 2.0)), ff=136),
        _mamba(6, 16, 24, 3, 3, 4, ff=72),
        _latent(2, 16, 8, 40, 24, 32, 0.2, _rot(8, 300.0, (2.0, 40, 8.0, 1.0))),
        _mamba(4, 24, 16, 2, 4, 2, ff=104),
    ], loop=(1, 3, 3)),
    # one stream; one head, one group, one norm group, one tap (no convolution); a plain ladder;
    # no factor on the embedding, no cap, no loop
    "B": _model(104, 211, 1e-6, 1, 1.0, None, [
        _mamba(1, 40, 12, 1, 1, 1, ff=60),
        _latent(3, 20, 4, 12, 28, 20, 0.4, _rot(4, 50.0), ff=44),
        _mamba(8, 8, 48, 4, 2, 8, ff=36),
    ]),
    # two streams; as many groups as heads; values wider than 128 and more states than 128; five
    # taps; one attention head; a ladder rescaled throughout (the ramp ends before it); the first
    # layer alone twice over
    "C": _model(64, 97, 1e-5, 2, 0.25, 5.0, [
        _mamba(2, 144, 8, 2, 5, 3, ff=40),
        _latent(1, 32, 32, 64, 72, 64, 0.15, _rot(32, 100.0, (2.0, 16, 1000.0, 500.0)), ff=24),
        _mamba(3, 32, 136, 1, 4, 6),
    ], loop=(0, 1, 2)),
    # a width and sizes that are multiples of two only and five streams: no kernel's fast form
    # applies; a loop around everything that goes round once; a rotated part that is half rotated
    "O": _model(50, 131, 1e-5, 5, 0.7, 12.0, [
        _latent(3, 10, 6, 6, 14, 10, 0.3, _rot(4, 90.0, (3.0, 40, 8.0, 1.0)), ff=18),
        _mamba(3, 10, 6, 1, 3, 5, ff=22),
    ], loop=(0, 2, 1)),
}


def random_case(seed):
    """A configuration drawn from sizes that kernels treat differently, two to five layers in any
    order, now and then one without a feed-forward, one to four streams, a loop somewhere."""
    import random
    rng = random.Random(seed)
    width = rng.choice([128, 192, 256, 384, 448])
    layers = []
    for _ in range(rng.randint(2, 5)):
        ff = None if rng.random() < 0.15 else rng.choice([96, 128, 200, 320])
        if rng.random() < 0.5:
            rot_dim = rng.choice([8, 16, 32, 64])
            scaling = None if rng.random() < 0.3 else (rng.choice([2.0, 4.0, 8.0]), rng.choice([64, 256, 1024]),
                                                       rng.choice([16.0, 32.0]), rng.choice([1.0, 2.0]))
            layers.append(_latent(rng.choice([2, 4, 6, 8, 12]), rng.choice([16, 32, 48, 64]), rot_dim,
                                  rng.choice([16, 32, 48, 64]), rng.choice([48, 64, 128]),
                                  rng.choice([32, 64, 96, 144, 256]), rng.choice([0.0625, 0.125, 0.2]),
                                  _rot(rot_dim, rng.choice([1e4, 5e5]), scaling), ff=ff))
        else:
            heads, vdim = rng.choice([2, 4, 6, 8, 12]), rng.choice([16, 32, 64, 96])
            layers.append(_mamba(heads, vdim, rng.choice([16, 32, 64, 96, 128]),
                                 rng.choice([g for g in (1, 2, 3, 4) if heads % g == 0]), rng.randint(2, 5),
                                 rng.choice([g for g in (1, 2, 3, 4, 8) if heads * vdim % g == 0]), ff=ff))
    n = len(layers)
    start = rng.randint(0, n - 1)
    loop = None if rng.random() < 0.3 else (start, rng.randint(start + 1, n), rng.choice([1, 2, 3]))
    return _model(width, rng.choice([263, 500, 1000]), rng.choice([1e-5, 1e-6]), rng.randint(1, 4),
                  rng.choice([1.0, 4.0]), rng.choice([None, 25.0]), layers, loop)


def write_model(folder, config, seed, dtype="bfloat16", std=0.08, patch=None):
    """A model folder of ``config`` with seeded random weights; ``patch(tensors)`` may change
    them before they are written.  Decays are spread from fast to slow, the step sizes from
    small to large, and the streams' mixes are neither symmetric nor near the identity, so that a
    transposed mix or a stream that is left out shows."""
    import gpt_fast_amd as gfa
    from gpt_fast_amd.weights.random_init import random_checkpoint
    from gpt_fast_amd.weights.safetensors_io import write_safetensors
    arch = gfa.config.registry.architecture_of(config)
    cfg = arch.read_config(config)
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(config, f)
    tensors = random_checkpoint(arch.bindings(cfg), seed, dtype, std=std, norm_std=0.2, tie=True)
    g = torch.Generator().manual_seed(seed + 1)
    for name in sorted(tensors):
        t = tensors[name]
        if name.endswith(".A_log"):
            tensors[name] = (torch.rand(t.shape, generator=g) * 4.0 - 3.0).to(t.dtype)
        elif name.endswith(".dt_bias"):
            tensors[name] = (torch.randn(t.shape, generator=g) * 1.5 - 1.5).to(t.dtype)
        elif name.endswith(".conv"):
            tensors[name] = (torch.randn(t.shape, generator=g) * 0.7).to(t.dtype)
        elif name.endswith(".conv.b"):
            tensors[name] = (torch.randn(t.shape, generator=g) * 0.4).to(t.dtype)
        elif name.endswith((".hc1.in", ".hc2.in")):
            tensors[name] = (torch.randn(t.shape, generator=g) * 0.5 + 0.6).to(t.dtype)
        elif name.endswith((".hc1.out", ".hc2.out")):
            tensors[name] = (torch.randn(t.shape, generator=g) * 0.6 + 0.9).to(t.dtype)
        elif name.endswith((".hc1.mix", ".hc2.mix")):
            S = t.shape[0]
            tensors[name] = (torch.randn(t.shape, generator=g) * (0.5 / S) + 0.8 * torch.eye(S)).to(t.dtype)
        elif name.endswith(".mix.g"):
            tensors[name] = (torch.randn(t.shape, generator=g) * 0.2).to(t.dtype)
    if patch is not None:
        patch(tensors)
    write_safetensors(os.path.join(folder, "model.safetensors"), tensors)
    return folder


def make_folder(tmp, name, seed=0, dtype="bfloat16", patch=None, tag=""):
    folder = os.path.join(str(tmp), f"bikadra_{name}_{dtype}_{seed}{tag}")
    if not os.path.isdir(folder):
        write_model(folder, CASES[name], seed, dtype, patch=patch)
    return folder
