"""Typed configuration of the Pitenex decoder: a stack whose layers are listed one by one in
``config.json``; in every layer an attention inside chunks and a gated delta rule stand side by
side, and the feed-forward (gated, or a mixture of experts, or none) beside both.

    {"architecture": "Pitenex", "vocab": V, "width": D, "norm": {"eps": e},
     "embedding": {"bigram": {"buckets", "mul_prev", "mul_cur"}},
     "residual_mult": m, "logit_scale": c,
     "layers": [{"type": "parallel",
                 "mixer": {"left": {"heads", "kv_heads", "dim", "vdim", "scale", "mask": {"size"},
                                    "rot": {"dims", "base"}},
                           "right": {"heads", "kv_heads", "dim", "vdim", "conv"},
                           "left_scale", "right_scale"},
                 "mlp": {"kind": "dense", "ff"}
                        | {"kind": "moe", "router": {"experts", "identity", "top"},
                           "expert": {"ff", "limit"}, "shared": {"ff", "limit"} | null}
                        | null}, ...]}

Every size and constant is read from there; nothing is assumed equal between layers.  The ranks of
the delta rule's decay and gate ("decay_rank", "gate_rank" of "right") may be left to the
checkpoint's tensors.
"""
import dataclasses
from dataclasses import dataclass
from typing import Optional, Tuple


class ConfigError(ValueError):
    pass


def _need(d: dict, key: str, where: str):
    if not isinstance(d, dict) or key not in d:
        raise ConfigError(f"Pitenex config.json: {where} lacks '{key}'")
    return d[key]


def _size(d: dict, key: str, where: str, default: Optional[int] = None) -> int:
    v = int(_need(d, key, where) if default is None else d.get(key, default))
    if v < 1:
        raise ConfigError(f"Pitenex config.json: {where}.{key} {v} must be at least 1")
    return v


def _divides(heads: int, kv_heads: int, where: str) -> None:
    if heads % kv_heads:
        raise ConfigError(f"Pitenex config.json: {where}: {heads} heads do not divide into {kv_heads} kv_heads")


@dataclass(frozen=True)
class ChunkAttention:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    chunk: Optional[int]          # positions per chunk; None: all earlier keys are seen
    rot_dims: int
    rot_base: float

    def to_dict(self) -> dict:
        d = {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim,
             "scale": self.scale}
        if self.chunk is not None:
            d["mask"] = {"size": self.chunk}
        if self.rot_dims:
            d["rot"] = {"dims": self.rot_dims, "base": self.rot_base}
        return d

    @staticmethod
    def read(d: dict, where: str) -> "ChunkAttention":
        heads, dim = _size(d, "heads", where), _size(d, "dim", where)
        rot, mask = d.get("rot") or {}, d.get("mask") or {}
        dims = int(rot.get("dims", 0))
        a = ChunkAttention(heads=heads, kv_heads=_size(d, "kv_heads", where, heads), dim=dim,
                           vdim=_size(d, "vdim", where, dim), scale=float(_need(d, "scale", where)),
                           chunk=_size(mask, "size", where + ".mask") if mask.get("size") is not None else None,
                           rot_dims=dims, rot_base=float(_need(rot, "base", where + ".rot")) if dims else 0.0)
        _divides(a.heads, a.kv_heads, where)
        if dims < 0 or dims % 2 or dims > dim:
            raise ConfigError(f"Pitenex config.json: {where}.rot.dims {dims} must be even and at most dim {dim}")
        return a


@dataclass(frozen=True)
class ChannelDelta:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int
    decay_rank: int = 0           # 0: the checkpoint's tensors say
    gate_rank: int = 0

    def to_dict(self) -> dict:
        d = {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim, "conv": self.conv}
        if self.decay_rank:
            d["decay_rank"] = self.decay_rank
        if self.gate_rank:
            d["gate_rank"] = self.gate_rank
        return d

    @staticmethod
    def read(d: dict, where: str) -> "ChannelDelta":
        heads, dim = _size(d, "heads", where), _size(d, "dim", where)
        r = ChannelDelta(heads=heads, kv_heads=_size(d, "kv_heads", where, heads), dim=dim,
                         vdim=_size(d, "vdim", where, dim), conv=_size(d, "conv", where),
                         decay_rank=int(d.get("decay_rank", 0)), gate_rank=int(d.get("gate_rank", 0)))
        _divides(r.heads, r.kv_heads, where)
        if r.decay_rank < 0 or r.gate_rank < 0:
            raise ConfigError(f"Pitenex config.json: {where}: ranks {r.decay_rank}, {r.gate_rank}")
        return r


@dataclass(frozen=True)
class ParallelPair:
    left: ChunkAttention
    right: ChannelDelta
    left_scale: float
    right_scale: float

    def to_dict(self) -> dict:
        return {"left": self.left.to_dict(), "right": self.right.to_dict(), "left_scale": self.left_scale,
                "right_scale": self.right_scale}


@dataclass(frozen=True)
class DenseMlp:
    ff: int

    def to_dict(self) -> dict:
        return {"kind": "dense", "ff": self.ff}


@dataclass(frozen=True)
class MoeMlp:
    experts: int
    identity: int
    top: int
    ff: int
    limit: float
    shared_ff: int = 0            # 0: no shared expert
    shared_limit: float = 0.0

    def to_dict(self) -> dict:
        shared = {"ff": self.shared_ff, "limit": self.shared_limit} if self.shared_ff else None
        return {"kind": "moe", "expert": {"ff": self.ff, "limit": self.limit},
                "router": {"experts": self.experts, "identity": self.identity, "top": self.top}, "shared": shared}


@dataclass(frozen=True)
class PitenexLayer:
    mixer: ParallelPair
    mlp: object                   # DenseMlp | MoeMlp | None

    def to_dict(self) -> dict:
        return {"type": "parallel", "mixer": self.mixer.to_dict(),
                "mlp": None if self.mlp is None else self.mlp.to_dict()}


def _read_mlp(mlp, where: str):
    if mlp is None:
        return None
    kind = mlp.get("kind", "dense")
    if kind == "dense":
        return DenseMlp(_size(mlp, "ff", where))
    if kind != "moe":
        raise ConfigError(f"Pitenex config.json: {where}.kind '{kind}': dense or moe")
    router, expert = _need(mlp, "router", where), _need(mlp, "expert", where)
    shared = mlp.get("shared")
    m = MoeMlp(experts=_size(router, "experts", where + ".router"), identity=int(router.get("identity") or 0),
               top=_size(router, "top", where + ".router"), ff=_size(expert, "ff", where + ".expert"),
               limit=float(_need(expert, "limit", where + ".expert")),
               shared_ff=_size(shared, "ff", where + ".shared") if shared else 0,
               shared_limit=float(_need(shared, "limit", where + ".shared")) if shared else 0.0)
    if m.identity < 0 or m.top > m.experts + m.identity:
        raise ConfigError(f"Pitenex config.json: {where}: top {m.top} of {m.experts} experts and {m.identity} "
                          f"identity experts")
    return m


def _read_layer(i: int, d: dict) -> PitenexLayer:
    where = f"layers[{i}]"
    kind = _need(d, "type", where)
    if kind != "parallel":
        raise ConfigError(f"Pitenex config.json: {where} has type '{kind}': parallel")
    m, at = _need(d, "mixer", where), where + ".mixer"
    pair = ParallelPair(left=ChunkAttention.read(_need(m, "left", at), at + ".left"),
                        right=ChannelDelta.read(_need(m, "right", at), at + ".right"),
                        left_scale=float(_need(m, "left_scale", at)),
                        right_scale=float(_need(m, "right_scale", at)))
    return PitenexLayer(pair, _read_mlp(d.get("mlp"), where + ".mlp"))


@dataclass(frozen=True)
class PitenexConfig:
    vocab: int
    width: int
    norm_eps: float
    buckets: int                  # of the table of token pairs; 0: no such table
    mul_prev: int
    mul_cur: int
    residual_mult: float
    logit_scale: float
    layers: Tuple[PitenexLayer, ...]
    max_positions: int = 1 << 20  # the design has no table of positions: a bound for requests

    @staticmethod
    def from_dict(d: dict) -> "PitenexConfig":
        top = "the top level"
        layers = _need(d, "layers", top)
        if not isinstance(layers, list) or not layers:
            raise ConfigError("Pitenex config.json: 'layers' must be a list of at least one layer")
        pair = (d.get("embedding") or {}).get("bigram")
        at = "embedding.bigram"
        return PitenexConfig(
            vocab=_size(d, "vocab", top), width=_size(d, "width", top),
            norm_eps=float(_need(_need(d, "norm", top), "eps", "norm")),
            buckets=_size(pair, "buckets", at) if pair else 0,
            mul_prev=int(_need(pair, "mul_prev", at)) if pair else 0,
            mul_cur=int(_need(pair, "mul_cur", at)) if pair else 0,
            residual_mult=float(d.get("residual_mult", 1.0)), logit_scale=float(d.get("logit_scale", 1.0)),
            layers=tuple(_read_layer(i, l) for i, l in enumerate(layers)),
            max_positions=int(d.get("max_positions", 1 << 20)))

    def to_dict(self) -> dict:
        embedding = {}
        if self.buckets:
            embedding["bigram"] = {"buckets": self.buckets, "mul_prev": self.mul_prev, "mul_cur": self.mul_cur}
        return {"architecture": "Pitenex", "vocab": self.vocab, "width": self.width,
                "norm": {"eps": self.norm_eps}, "embedding": embedding, "residual_mult": self.residual_mult,
                "logit_scale": self.logit_scale, "layers": [l.to_dict() for l in self.layers]}

    def with_ranks(self, ranks) -> "PitenexConfig":
        """The ranks that the configuration leaves open, from ``ranks(layer index) -> (decay, gate)``."""
        layers = []
        for i, l in enumerate(self.layers):
            r = l.mixer.right
            if not (r.decay_rank and r.gate_rank):
                decay, gate = ranks(i)
                r = dataclasses.replace(r, decay_rank=r.decay_rank or decay, gate_rank=r.gate_rank or gate)
                l = dataclasses.replace(l, mixer=dataclasses.replace(l.mixer, right=r))
            layers.append(l)
        return dataclasses.replace(self, layers=tuple(layers))

    # ------------------------------------------------------------------ named shapes
    @staticmethod
    def from_name(name: str) -> "PitenexConfig":
        """Shapes for measurements (random weights): ``pitenex-<width>``."""
        key = name.lower()
        if key not in PRESETS:
            raise KeyError(f"no Pitenex preset '{name}'; known: {sorted(PRESETS)}")
        return PRESETS[key]()


def _stack(width: int, n_layers: int, ff: int, expert_ff: int, shared_ff: int, kv_heads: int,
           vocab: int) -> PitenexConfig:
    """Heads of 128 on both sides, chunks of 8,192 positions, four taps, ranks of 128; of every four
    layers one with a dense feed-forward and three with a mixture of 32 experts, two identity
    experts behind them (top 4) and a shared one."""
    heads = width // 128
    pair = ParallelPair(
        left=ChunkAttention(heads=heads, kv_heads=kv_heads, dim=128, vdim=128, scale=128 ** -0.5, chunk=8192,
                            rot_dims=128, rot_base=500000.0),
        right=ChannelDelta(heads=heads // 2, kv_heads=heads // 4, dim=128, vdim=128, conv=4, decay_rank=128,
                           gate_rank=128),
        left_scale=1.0, right_scale=1.0)
    moe = MoeMlp(experts=32, identity=2, top=4, ff=expert_ff, limit=7.0, shared_ff=shared_ff, shared_limit=7.0)
    layers = tuple(PitenexLayer(pair, DenseMlp(ff) if i % 4 == 3 else moe) for i in range(n_layers))
    return PitenexConfig(vocab=vocab, width=width, norm_eps=1e-6, buckets=65521, mul_prev=8191, mul_cur=131,
                         residual_mult=0.5, logit_scale=1.0, layers=layers)


PRESETS = {
    # the widths, head sizes, vocabulary, experts and feed-forwards of the library's refolix-4096
    # and refolix-8192: per token four routed experts and the shared one are as large as the dense
    # feed-forward
    "pitenex-4096": lambda: _stack(4096, 32, 14336, 2048, 6144, 8, vocab=128256),
    "pitenex-8192": lambda: _stack(8192, 80, 28672, 4096, 12288, 8, vocab=128256),
}
