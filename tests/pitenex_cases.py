"""Small Pitenex configurations for the tests; they differ from each other in every size and
option.  Weights are drawn by the library's random-weights mode and may be patched before they
are written."""
import json
import os

import torch


def _left(heads, kv, dim, vdim, chunk, rot, scale):
    d = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale, "mask": {"size": chunk}}
    if rot is not None:
        d["rot"] = {"dims": rot[0], "base": rot[1]}
    return d


def _right(heads, kv, dim, vdim, conv, ranks):
    """The ranks are kept apart: config.json does not hold them, the tensors do."""
    return {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "conv": conv, "ranks": ranks}


def _dense(ff):
    return {"kind": "dense", "ff": ff}


def _moe(experts, identity, top, ff, limit, shared=None):
    return {"kind": "moe", "expert": {"ff": ff, "limit": limit},
            "router": {"experts": experts, "identity": identity, "top": top},
            "shared": None if shared is None else {"ff": shared[0], "limit": shared[1]}}


def _layer(left, right, scales, mlp):
    return {"type": "parallel", "mlp": mlp,
            "mixer": {"left": left, "right": right, "left_scale": scales[0], "right_scale": scales[1]}}


def _model(width, vocab, eps, pair, mult, logit_scale, layers):
    return {"architecture": "Pitenex", "vocab": vocab, "width": width, "norm": {"eps": eps},
            "embedding": {"bigram": dict(zip(("buckets", "mul_prev", "mul_cur"), pair))},
            "residual_mult": mult, "logit_scale": logit_scale, "layers": layers}


CASES = {
    # chunks that begin inside pages, keys and values of different sizes, half of a head rotated,
    # unequal ranks; experts first, then a dense feed-forward, then none
    "A": _model(96, 300, 1e-5, (97, 5, 3), 0.6, 0.5, [
        _layer(_left(6, 2, 24, 32, 40, (12, 10000.0), 0.3), _right(4, 2, 24, 16, 4, (16, 40)), (0.8, 1.3),
               _moe(7, 3, 3, 40, 1.0, (56, 0.7))),
        _layer(_left(2, 1, 16, 48, 100, (16, 300.0), 0.25), _right(6, 3, 40, 24, 2, (24, 8)), (1.1, 0.9),
               _dense(136)),
        _layer(_left(4, 4, 32, 16, 64, (8, 500.0), 0.2), _right(2, 2, 16, 48, 3, (8, 24)), (1.0, 0.7), None),
    ]),
    # one head on either side, one tap (no convolution), no rotation, ranks that are no multiples of
    # eight and a rank of one, every expert chosen, no identity and no shared expert
    "B": _model(104, 211, 1e-6, (64, 29, 13), 1.0, 1.0, [
        _layer(_left(1, 1, 20, 12, 7, None, 0.4), _right(1, 1, 12, 40, 1, (5, 1)), (1.0, 1.0), _dense(60)),
        _layer(_left(8, 8, 8, 24, 33, (4, 50.0), 0.35), _right(8, 1, 20, 10, 5, (1, 13)), (0.5, 1.5),
               _moe(4, 0, 4, 24, 0.5)),
    ]),
    # key channels beyond what the chunks' kernels take, values wider than a pass of theirs, a head of
    # 128 on both sides, one expert and one identity expert of which one is chosen, a chunk of one
    "C": _model(128, 97, 1e-5, (1000, 2, 11), 0.4, 2.0, [
        _layer(_left(4, 2, 128, 128, 130, (128, 1000.0), 0.09), _right(2, 1, 144, 32, 3, (32, 16)), (1.2, 0.8),
               _moe(1, 1, 1, 48, 3.0, (32, 2.0))),
        _layer(_left(3, 1, 64, 80, 1, (2, 77.0), 0.15), _right(3, 3, 128, 144, 4, (16, 48)), (0.9, 1.1),
               _dense(40)),
        _layer(_left(2, 2, 48, 64, 256, (32, 5000.0), 0.2), _right(2, 2, 64, 64, 2, (64, 64)), (1.0, 1.0),
               _moe(12, 4, 2, 64, 1.5, (24, 0.4))),
    ]),
    # a width and sizes that are multiples of two only: no kernel's fast form applies
    "O": _model(50, 131, 1e-5, (13, 3, 1), 0.8, 0.7, [
        _layer(_left(3, 3, 10, 6, 10, (6, 90.0), 0.3), _right(3, 1, 10, 14, 3, (6, 10)), (0.7, 1.2),
               _moe(5, 2, 2, 18, 0.8, (22, 1.1))),
        _layer(_left(5, 1, 6, 18, 50, (2, 40.0), 0.4), _right(2, 1, 6, 10, 4, (2, 3)), (1.0, 1.0), _dense(30)),
    ]),
}


def random_case(seed):
    """A configuration drawn from sizes that kernels treat differently."""
    import random
    rng = random.Random(seed)
    width = rng.choice([128, 192, 256, 384, 448])
    layers = []
    for _ in range(rng.randint(2, 4)):
        lk, rk = rng.choice([1, 2, 3]), rng.choice([1, 2, 3])
        dim = rng.choice([16, 32, 40, 64, 128])
        left = _left(lk * rng.choice([1, 2, 4]), lk, dim, rng.choice([16, 32, 48, 64]),
                     rng.choice([17, 48, 64, 90, 128, 200]), (rng.choice([dim, dim // 2]), rng.choice([1e3, 5e5])),
                     rng.choice([0.0625, 0.125, 0.2]))
        right = _right(rk * rng.choice([1, 2, 3]), rk, rng.choice([16, 32, 64, 80, 128]), rng.choice([16, 32, 64, 96]),
                       rng.randint(1, 5), (rng.choice([8, 24, 32, 64]), rng.choice([8, 16, 40])))
        r = rng.random()
        if r < 0.4:
            mlp = _dense(rng.choice([96, 128, 200]))
        elif r < 0.9:
            experts, identity = rng.choice([4, 9, 20]), rng.choice([0, 1, 2, 5])
            mlp = _moe(experts, identity, rng.randint(1, 4), rng.choice([32, 40, 64]), rng.choice([0.7, 2.0]),
                       None if rng.random() < 0.2 else (rng.choice([32, 72]), rng.choice([0.5, 1.5])))
        else:
            mlp = None
        layers.append(_layer(left, right, (rng.choice([0.7, 1.0, 1.3]), rng.choice([0.8, 1.0, 1.2])), mlp))
    return _model(width, rng.choice([263, 500, 1000]), rng.choice([1e-5, 1e-6]),
                  (rng.choice([61, 521, 1024]), rng.choice([3, 29]), rng.choice([1, 5])),
                  rng.choice([0.5, 0.9]), rng.choice([0.5, 1.0]), layers)


def split_ranks(config):
    """(config.json without the ranks, the library's configuration with them)."""
    from gpt_fast_amd.config.pitenex import PitenexConfig
    import copy
    bare, full = copy.deepcopy(config), copy.deepcopy(config)
    for plain, whole in zip(bare["layers"], full["layers"]):
        plain["mixer"]["right"].pop("ranks")
        decay, gate = whole["mixer"]["right"].pop("ranks")
        whole["mixer"]["right"].update(decay_rank=decay, gate_rank=gate)
    return bare, PitenexConfig.from_dict(full)


def write_model(folder, config, seed, dtype="bfloat16", std=0.08, patch=None):
    """A model folder of ``config`` with seeded random weights; ``patch(tensors)`` may change them
    before they are written.  Decays are spread from fast to slow, the sinks weigh as much as a few
    keys, and the experts' products are large enough to be clamped."""
    import gpt_fast_amd as gfa  # noqa: F401
    from gpt_fast_amd.architectures.pitenex import pitenex_bindings
    from gpt_fast_amd.weights.random_init import random_checkpoint
    from gpt_fast_amd.weights.safetensors_io import write_safetensors
    bare, cfg = split_ranks(config)
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(bare, f)
    tensors = random_checkpoint(pitenex_bindings(cfg), seed, dtype, std=std, norm_std=0.2, tie=True)
    g = torch.Generator().manual_seed(seed + 1)
    for name in sorted(tensors):
        t = tensors[name]
        if name.endswith(".A_log"):
            tensors[name] = (torch.rand(t.shape, generator=g) * 4.0 - 3.5).to(t.dtype)
        elif name.endswith(".dt_bias"):
            tensors[name] = (torch.randn(t.shape, generator=g) * 1.5 - 2.0).to(t.dtype)
        elif name.endswith(".conv"):
            tensors[name] = (torch.randn(t.shape, generator=g) * 0.7).to(t.dtype)
        elif name.endswith(".sink"):
            tensors[name] = (torch.randn(t.shape, generator=g) + 1.0).to(t.dtype)
        elif name.endswith((".a2", ".g2")):
            tensors[name] = (torch.randn(t.shape, generator=g) * 0.3).to(t.dtype)
        elif name.endswith((".router",)):
            tensors[name] = (torch.randn(t.shape, generator=g) * 0.2).to(t.dtype)
        elif name.endswith(".correction"):
            tensors[name] = (torch.randn(t.shape, generator=g) * 0.05).to(t.dtype)
        elif name in ("embed", "bigram"):
            tensors[name] = (torch.randn(t.shape, generator=g) * 0.4).to(t.dtype)
    if patch is not None:
        patch(tensors)
    write_safetensors(os.path.join(folder, "model.safetensors"), tensors)
    return folder


def make_folder(tmp, name, seed=0, dtype="bfloat16", patch=None, tag=""):
    folder = os.path.join(str(tmp), f"pitenex_{name}_{dtype}_{seed}{tag}")
    if not os.path.isdir(folder):
        write_model(folder, CASES[name], seed, dtype, patch=patch)
    return folder
