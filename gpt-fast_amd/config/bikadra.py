"""Typed configuration of the Bikadra decoder: a stack whose layers are listed one by one in
``config.json``; several residual streams stand in place of one; a layer's mixer is latent
attention or a state-space cell (Mamba-2), its feed-forward two matrices or absent; a range of
layers may run several times in a row.

    {"architecture": "Bikadra", "vocab": V, "width": D, "norm": {"eps": e}, "streams": S,
     "embedding": {"scale": c}, "logit_softcap": cap,
     "loop": {"start": a, "stop": b, "times": n},
     "layers": [{"type": "latent_attention",
                 "mixer": {"heads", "dim", "rot_dim", "vdim", "q_rank", "kv_rank", "scale",
                           "rot": {"dims", "base", "scaling": {"factor", "original", "fast",
                                                               "slow"}}},
                 "mlp": {"kind": "dense", "ff"} | null},
                {"type": "mamba2",
                 "mixer": {"heads", "vdim", "state", "groups", "conv", "norm_groups"},
                 "mlp": ...}, ...]}

Every size and constant is read from there; nothing is assumed equal between layers.
"""
from dataclasses import dataclass
from typing import Optional, Tuple


class ConfigError(ValueError):
    pass


def _need(d: dict, key: str, where: str):
    if not isinstance(d, dict) or key not in d:
        raise ConfigError(f"Bikadra config.json: {where} lacks '{key}'")
    return d[key]


def _size(d: dict, key: str, where: str) -> int:
    v = int(_need(d, key, where))
    if v < 1:
        raise ConfigError(f"Bikadra config.json: {where}.{key} {v} must be at least 1")
    return v


@dataclass(frozen=True)
class Rotation:
    """Rotary positions on the first ``dims`` elements of the rotated part; ``scaling`` None or
    (factor, original, fast, slow)."""
    dims: int
    base: float
    scaling: Optional[Tuple[float, float, float, float]] = None

    @staticmethod
    def read(d, where: str) -> Optional["Rotation"]:
        if not d or not int(d.get("dims", 0)):
            return None
        sc = d.get("scaling")
        scaling = None
        if sc:
            scaling = tuple(float(_need(sc, k, where + ".scaling")) for k in ("factor", "original", "fast", "slow"))
        r = Rotation(int(d["dims"]), float(_need(d, "base", where)), scaling)
        if r.dims % 2 or r.dims < 0:
            raise ConfigError(f"Bikadra config.json: {where}.dims {r.dims} must be even")
        return r

    def to_dict(self) -> dict:
        d = {"dims": self.dims, "base": self.base}
        if self.scaling is not None:
            d["scaling"] = dict(zip(("factor", "original", "fast", "slow"), self.scaling))
        return d


@dataclass(frozen=True)
class LatentMixer:
    heads: int
    dim: int                  # unrotated elements of a query / key head
    rot_dim: int              # rotated elements (the keys' part is shared by the heads)
    vdim: int
    q_rank: int
    kv_rank: int
    scale: float
    rot: Optional[Rotation]

    def to_dict(self) -> dict:
        d = {"heads": self.heads, "dim": self.dim, "rot_dim": self.rot_dim, "vdim": self.vdim,
             "q_rank": self.q_rank, "kv_rank": self.kv_rank, "scale": self.scale}
        if self.rot is not None:
            d["rot"] = self.rot.to_dict()
        return d


@dataclass(frozen=True)
class StateSpaceMixer:
    heads: int
    vdim: int
    state: int
    groups: int
    conv: int
    norm_groups: int

    def to_dict(self) -> dict:
        return {"heads": self.heads, "vdim": self.vdim, "state": self.state, "groups": self.groups,
                "conv": self.conv, "norm_groups": self.norm_groups}


@dataclass(frozen=True)
class DenseMlp:
    ff: int

    def to_dict(self) -> dict:
        return {"kind": "dense", "ff": self.ff}


@dataclass(frozen=True)
class BikadraLayer:
    type: str                 # "latent_attention" | "mamba2"
    mixer: object
    mlp: Optional[DenseMlp]

    def to_dict(self) -> dict:
        return {"type": self.type, "mixer": self.mixer.to_dict(),
                "mlp": None if self.mlp is None else self.mlp.to_dict()}


@dataclass(frozen=True)
class Loop:
    """Layers start .. stop - 1 run ``times`` times in a row."""
    start: int
    stop: int
    times: int

    def to_dict(self) -> dict:
        return {"start": self.start, "stop": self.stop, "times": self.times}


def _read_mlp(mlp, where: str) -> Optional[DenseMlp]:
    if mlp is None:
        return None
    if mlp.get("kind", "dense") != "dense":
        raise ConfigError(f"Bikadra config.json: {where}.kind '{mlp.get('kind')}': dense")
    return DenseMlp(_size(mlp, "ff", where))


def _read_layer(i: int, d: dict) -> BikadraLayer:
    where = f"layers[{i}]"
    kind = _need(d, "type", where)
    m = _need(d, "mixer", where)
    at = where + ".mixer"
    if kind == "latent_attention":
        dim = _size(m, "dim", at)
        mixer = LatentMixer(heads=_size(m, "heads", at), dim=dim, rot_dim=int(_need(m, "rot_dim", at)),
                            vdim=int(m.get("vdim", dim)), q_rank=_size(m, "q_rank", at),
                            kv_rank=_size(m, "kv_rank", at), scale=float(_need(m, "scale", at)),
                            rot=Rotation.read(m.get("rot"), at + ".rot"))
        if mixer.rot_dim < 0 or (mixer.rot is not None and mixer.rot.dims > mixer.rot_dim):
            raise ConfigError(f"Bikadra config.json: {at}: {0 if mixer.rot is None else mixer.rot.dims} rotated "
                              f"elements in a part of {mixer.rot_dim}")
    elif kind == "mamba2":
        mixer = StateSpaceMixer(heads=_size(m, "heads", at), vdim=_size(m, "vdim", at),
                                state=_size(m, "state", at), groups=_size(m, "groups", at),
                                conv=_size(m, "conv", at), norm_groups=int(m.get("norm_groups", 1)))
        if mixer.heads % mixer.groups:
            raise ConfigError(f"Bikadra config.json: {at}: {mixer.heads} heads do not divide into "
                              f"{mixer.groups} groups")
        if mixer.norm_groups < 1 or mixer.heads * mixer.vdim % mixer.norm_groups:
            raise ConfigError(f"Bikadra config.json: {at}: {mixer.heads * mixer.vdim} elements do not "
                              f"divide into {mixer.norm_groups} norm groups")
    else:
        raise ConfigError(f"Bikadra config.json: {where} has type '{kind}': latent_attention or mamba2")
    return BikadraLayer(kind, mixer, _read_mlp(d.get("mlp"), where + ".mlp"))


@dataclass(frozen=True)
class BikadraConfig:
    vocab: int
    width: int
    norm_eps: float
    streams: int
    embedding_scale: float
    logit_softcap: Optional[float]
    layers: Tuple[BikadraLayer, ...]
    loop: Optional[Loop] = None
    max_positions: int = 1 << 20       # the design has no table of positions: a bound for requests

    @staticmethod
    def from_dict(d: dict) -> "BikadraConfig":
        layers = _need(d, "layers", "the top level")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("Bikadra config.json: 'layers' must be a list of at least one layer")
        loop = d.get("loop")
        if loop is not None:
            loop = Loop(int(_need(loop, "start", "loop")), int(_need(loop, "stop", "loop")),
                        int(_need(loop, "times", "loop")))
            if not 0 <= loop.start <= loop.stop <= len(layers) or loop.times < 0:
                raise ConfigError(f"Bikadra config.json: loop {loop.to_dict()} does not fit "
                                  f"{len(layers)} layers")
        cap = d.get("logit_softcap")
        return BikadraConfig(
            vocab=_size(d, "vocab", "the top level"), width=_size(d, "width", "the top level"),
            norm_eps=float(_need(_need(d, "norm", "the top level"), "eps", "norm")),
            streams=_size(d, "streams", "the top level"),
            embedding_scale=float((d.get("embedding") or {}).get("scale", 1.0)),
            logit_softcap=None if cap is None else float(cap),
            layers=tuple(_read_layer(i, l) for i, l in enumerate(layers)),
            loop=loop, max_positions=int(d.get("max_positions", 1 << 20)))

    def to_dict(self) -> dict:
        d = {"architecture": "Bikadra", "vocab": self.vocab, "width": self.width,
             "norm": {"eps": self.norm_eps}, "streams": self.streams,
             "embedding": {"scale": self.embedding_scale},
             "layers": [l.to_dict() for l in self.layers]}
        if self.logit_softcap is not None:
            d["logit_softcap"] = self.logit_softcap
        if self.loop is not None:
            d["loop"] = self.loop.to_dict()
        return d

    # ------------------------------------------------------------------ named shapes
    @staticmethod
    def from_name(name: str) -> "BikadraConfig":
        """Shapes for measurements (random weights): ``bikadra-<width>``."""
        key = name.lower()
        if key not in PRESETS:
            raise KeyError(f"no Bikadra preset '{name}'; known: {sorted(PRESETS)}")
        return PRESETS[key]()


def _stack(width: int, n_layers: int, ff: int, vocab: int) -> BikadraConfig:
    """Of every four layers three state-space cells (an inner size of twice the width, heads of
    64 with 128 states, eight groups) and one latent attention (heads of 128, latent of 512,
    rotated part of 64); a feed-forward in every layer; four streams; no loop."""
    heads = width // 128
    layers = []
    for i in range(n_layers):
        if i % 4 == 3:
            mixer = LatentMixer(heads=heads, dim=128, rot_dim=64, vdim=128, q_rank=width * 3 // 8,
                                kv_rank=512, scale=(128 + 64) ** -0.5,
                                rot=Rotation(64, 500000.0, (8.0, 8192.0, 32.0, 1.0)))
            kind = "latent_attention"
        else:
            mixer = StateSpaceMixer(heads=2 * width // 64, vdim=64, state=128, groups=8, conv=4,
                                    norm_groups=8)
            kind = "mamba2"
        layers.append(BikadraLayer(kind, mixer, DenseMlp(ff)))
    return BikadraConfig(vocab=vocab, width=width, norm_eps=1e-6, streams=4, embedding_scale=1.0,
                         logit_softcap=30.0, layers=tuple(layers))


PRESETS = {
    # the widths, vocabulary and feed-forwards of the library's nizedra-4096 and nizedra-8192
    "bikadra-4096": lambda: _stack(4096, 32, 21504, vocab=128256),
    "bikadra-8192": lambda: _stack(8192, 80, 43008, vocab=128256),
}
