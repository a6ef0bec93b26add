"""Configuration of the Lotelix architecture: a decoder whose layers mix by a gated recurrence of single channels
(minGRU), by a windowed attention with sinks, an output gate and values mixed with an earlier layer's, or by an attention
with sigmoid weights beside a gated linear attention; norms in groups; routed experts weighted at their input.

config.json is nested; every size and every constant that may differ between models of the design is read from it:

    architecture    "Lotelix"
    vocab, width
    embedding.scale
    norm.eps, norm.groups
    layers[i].type  "mingru" | "attention" | "parallel"
    layers[i].mixer mingru:    width
                    attention: heads, kv_heads, dim, vdim, scale, mask{size}, v_mix,
                               rot{base, dims, scaling{factor, low, high, original} or null}
                    parallel:  left{heads, kv_heads, dim, vdim, scale, rot{base, dims}}, right{heads, dim, vdim, tau}
    layers[i].mlp   null | {kind: "moe", expert{ff}, router{experts, top}}

One size is in no key: the inner size of the decay projection of a parallel layer's right half is the row count of the
tensor l<i>.mix.right.a1. `sizes_from_tensors` puts it into the parsed file as right.decay_rank before the configuration is
made (a file that holds the key itself is taken at its word).
"""
from __future__ import annotations

from dataclasses import dataclass, field

from .base import ConfigError, ModelConfig, coerce, key
from .kudurax import _num, _section


@dataclass(frozen=True)
class BandScaling:
    factor: float
    low: float
    high: float
    original: float


@dataclass(frozen=True)
class Rotation:
    base: float
    dims: int                       # 0: nothing turns
    scaling: BandScaling | None = None


@dataclass(frozen=True)
class MinGRUConfig:
    width: int


@dataclass(frozen=True)
class AttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot: Rotation
    window: int | None = None
    v_mix: bool = False


@dataclass(frozen=True)
class LinearAttentionConfig:
    heads: int
    dim: int
    vdim: int
    tau: float
    decay_rank: int


@dataclass(frozen=True)
class ParallelConfig:
    left: AttentionConfig
    right: LinearAttentionConfig


@dataclass(frozen=True)
class RoutedConfig:
    ff: int
    experts: int
    top: int


@dataclass(frozen=True)
class LotelixLayer:
    type: str                       # "mingru" | "attention" | "parallel"
    mixer: object
    mlp: RoutedConfig | None


def _rotation(m: dict, where: str, dim: int) -> Rotation:
    rot = m.get("rot")
    if rot is None:
        return Rotation(1.0, 0)
    rot, rw = _section(m, "rot", where), where + "rot."
    dims = _num(rot, "dims", int, rw, positive=False)
    if dims < 0 or dims % 2 or dims > dim:
        raise ConfigError(f"config key {rw}'dims' must be even and at most {dim}, got {dims}")
    scaling = None
    if rot.get("scaling") is not None:
        s, sw = _section(rot, "scaling", rw), rw + "scaling."
        scaling = BandScaling(*(_num(s, k, float, sw) for k in ("factor", "low", "high", "original")))
        if not scaling.high > scaling.low:
            raise ConfigError(f"config key {sw}'high' {scaling.high} must exceed 'low' {scaling.low}")
    return Rotation(_num(rot, "base", float, rw), dims, scaling)


def _attention(m: dict, where: str, windowed: bool) -> AttentionConfig:
    heads, kv = _num(m, "heads", int, where), _num(m, "kv_heads", int, where)
    if heads % kv:
        raise ConfigError(f"config key {where}'heads' {heads} is no multiple of 'kv_heads' {kv}")
    dim = _num(m, "dim", int, where)
    window, v_mix = None, False
    if windowed:
        window = _num(_section(m, "mask", where), "size", int, where + "mask.")
        v_mix = coerce(where + "v_mix", m.get("v_mix") or False, bool)
    return AttentionConfig(heads, kv, dim, _num(m, "vdim", int, where), _num(m, "scale", float, where),
                           _rotation(m, where, dim), window, v_mix)


def _mixer(typ: str, m: dict, where: str):
    if typ == "mingru":
        return MinGRUConfig(_num(m, "width", int, where))
    if typ == "attention":
        return _attention(m, where, True)
    if typ == "parallel":
        r, rw = _section(m, "right", where), where + "right."
        if "decay_rank" not in r:
            raise ConfigError(f"config key {rw}'decay_rank' is neither in the file nor known from the tensor "
                              "'mix.right.a1' (a configuration made without its weights must name it)")
        right = LinearAttentionConfig(_num(r, "heads", int, rw), _num(r, "dim", int, rw), _num(r, "vdim", int, rw),
                                      _num(r, "tau", float, rw), _num(r, "decay_rank", int, rw))
        return ParallelConfig(_attention(_section(m, "left", where), where + "left.", False), right)
    raise ConfigError(f"config key {where[:-6]}'type': unknown mixer {typ!r} (known: 'mingru', 'attention', 'parallel')")


def _feed_forward(f, where: str) -> RoutedConfig | None:
    if f is None:
        return None
    if not isinstance(f, dict) or f.get("kind") != "moe":
        raise ConfigError(f"config key {where}'mlp' must be null or an object of kind 'moe', got {f!r}")
    r, rw = _section(f, "router", where + "mlp."), where + "mlp.router."
    out = RoutedConfig(_num(_section(f, "expert", where + "mlp."), "ff", int, where + "mlp.expert."),
                       _num(r, "experts", int, rw), _num(r, "top", int, rw))
    if out.top > out.experts:
        raise ConfigError(f"config key {rw}'top' {out.top} exceeds 'experts' {out.experts}")
    return out


@dataclass(frozen=True)
class LotelixConfig(ModelConfig):
    vocab: int = key(int)
    width: int = key(int)
    embedding_scale: float = field(default=1.0)
    norm_eps: float = field(default=1e-6)
    norm_groups: int = field(default=1)
    layers: tuple = field(default=())

    ARCHITECTURE = "Lotelix"
    MAX_POSITIONS = (1 << 31) - 1     # the design sets no limit; positions are 32-bit in the batch

    @staticmethod
    def sizes_from_tensors(d: dict, shapes: dict) -> dict:
        """d: the parsed config.json; shapes: tensor name -> shape of the model's weight files. Returns d with the
        sizes that only a tensor's shape gives filled in."""
        layers = d.get("layers")
        if not isinstance(layers, list):
            return d
        out = []
        for i, l in enumerate(layers):
            right = l.get("mixer", {}).get("right") if isinstance(l, dict) and isinstance(l.get("mixer"), dict) else None
            shape = shapes.get(f"l{i}.mix.right.a1")
            if isinstance(right, dict) and "decay_rank" not in right and shape:
                l = dict(l, mixer=dict(l["mixer"], right=dict(right, decay_rank=int(shape[0]))))
            out.append(l)
        return dict(d, layers=out)

    @classmethod
    def extra_from_dict(cls, d: dict) -> dict:
        layers = d.get("layers")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("config key 'layers' must be a non-empty list")
        out = []
        for i, l in enumerate(layers):
            where = f"layers[{i}]."
            if not isinstance(l, dict):
                raise ConfigError(f"config key 'layers[{i}]' must be an object")
            typ = l.get("type")
            out.append(LotelixLayer(typ, _mixer(typ, _section(l, "mixer", where), where + "mixer."),
                                    _feed_forward(l.get("mlp"), where)))
        norm = _section(d, "norm", "")
        groups = _num(norm, "groups", int, "norm.") if norm.get("groups") is not None else 1
        return {"norm_eps": _num(norm, "eps", float, "norm."), "norm_groups": groups, "layers": tuple(out),
                "embedding_scale": _num(_section(d, "embedding", ""), "scale", float, "embedding.", positive=False)}

    def check(self) -> None:
        if self.vocab <= 0 or self.width <= 0:
            raise ConfigError(f"config keys 'vocab' and 'width' must be positive, got {self.vocab} and {self.width}")
        if self.width % self.norm_groups:
            raise ConfigError(f"config key 'norm.groups' {self.norm_groups} does not divide 'width' {self.width}")
        mixing = [i for i, l in enumerate(self.layers) if l.type == "attention" and l.mixer.v_mix]
        sizes = {self.layers[i].mixer.kv_heads * self.layers[i].mixer.vdim for i in mixing}
        if len(sizes) > 1:
            raise ConfigError(f"config key layers: the layers with 'v_mix' ({mixing}) must have values of one size, got {sorted(sizes)}")

    @property
    def first_mixing_layer(self) -> int | None:
        """The layer whose values the later layers with `v_mix` mix theirs with."""
        return next((i for i, l in enumerate(self.layers) if l.type == "attention" and l.mixer.v_mix), None)

    def extra_to_dict(self) -> dict:
        def rot(r: Rotation):
            if r.dims == 0:
                return None
            out = {"base": r.base, "dims": r.dims}
            if r.scaling is not None:
                s = r.scaling
                out["scaling"] = {"factor": s.factor, "low": s.low, "high": s.high, "original": s.original}
            return out

        def attention(a: AttentionConfig):
            out = {"heads": a.heads, "kv_heads": a.kv_heads, "dim": a.dim, "vdim": a.vdim, "scale": a.scale, "rot": rot(a.rot)}
            if a.window is not None:
                out.update(mask={"size": a.window}, v_mix=a.v_mix)
            return out

        def mixer(l: LotelixLayer):
            m = l.mixer
            if l.type == "mingru":
                return {"width": m.width}
            if l.type == "attention":
                return attention(m)
            r = m.right
            return {"left": attention(m.left),
                    "right": {"heads": r.heads, "dim": r.dim, "vdim": r.vdim, "tau": r.tau, "decay_rank": r.decay_rank}}

        def mlp(f: RoutedConfig | None):
            return None if f is None else {"kind": "moe", "expert": {"ff": f.ff}, "router": {"experts": f.experts, "top": f.top}}

        return {"architecture": self.ARCHITECTURE, "embedding": {"scale": self.embedding_scale},
                "norm": {"eps": self.norm_eps, "groups": self.norm_groups},
                "layers": [{"type": l.type, "mixer": mixer(l), "mlp": mlp(l.mlp)} for l in self.layers]}

    def to_dict(self) -> dict:
        out = {"vocab": self.vocab, "width": self.width}
        out.update(self.extra_to_dict())
        return out

    # what programs that know no architecture ask a configuration
    @property
    def vocab_size(self) -> int:
        return self.vocab

    @property
    def hidden_size(self) -> int:
        return self.width

    @property
    def max_position_embeddings(self) -> int:
        return self.MAX_POSITIONS

    @property
    def eos_token_ids(self) -> tuple:
        return ()
