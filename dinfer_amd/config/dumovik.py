"""Configuration of the Dumovik architecture: a decoder whose layers mix by latent attention with an output gate, by softly
capped attention inside chunks of positions (its keys and values possibly another layer's), or by lightning attention (a
recurrent state with a fixed decay a head); norms on the sublayers' outputs only; dense or routed feed-forwards.

config.json is nested; every size and every constant that may differ between models of the design is read from it:

    architecture    "Dumovik"
    vocab, width
    norm.eps
    layers[i].type  "latent_attention" | "attention" | "lightning"
    layers[i].mixer latent_attention: heads, dim, rot_dim, vdim, kv_rank, scale, rot{base, dims}
                    attention:        heads, kv_heads, dim, vdim, scale, softcap (null: no cap), mask{size} (null: every earlier
                                      key), kv_from (optional: the layer whose keys and values this one reads)
                    lightning:        heads, dim, vdim, decay[heads]
    layers[i].mlp   null | {kind: "dense", ff} | {kind: "moe", expert{ff, limit}, router{experts, top}}
"""
from __future__ import annotations

from dataclasses import dataclass, field

from .base import ConfigError, ModelConfig, coerce, key
from .kudurax import _num, _section


@dataclass(frozen=True)
class LatentConfig:
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    kv_rank: int
    scale: float
    rot_base: float
    rot_dims: int


@dataclass(frozen=True)
class AttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    softcap: float | None
    chunk: int | None
    kv_from: int | None = None


@dataclass(frozen=True)
class LightningConfig:
    heads: int
    dim: int
    vdim: int
    decay: tuple


@dataclass(frozen=True)
class FeedForwardConfig:
    kind: str                    # "dense" | "moe"
    ff: int                      # dense: its inner size; moe: an expert's
    limit: float = 0.0
    experts: int = 0
    top: int = 0


@dataclass(frozen=True)
class DumovikLayer:
    type: str                    # "latent_attention" | "attention" | "lightning"
    mixer: object
    mlp: FeedForwardConfig | None


def _mixer(typ: str, m: dict, where: str):
    if typ == "latent_attention":
        if m.get("kv_from") is not None:
            raise ConfigError(f"config key {where}'kv_from': a latent layer has keys and values of its own")
        rot, rw = _section(m, "rot", where), where + "rot."
        out = LatentConfig(*(_num(m, k, int, where) for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank")),
                           _num(m, "scale", float, where), _num(rot, "base", float, rw), _num(rot, "dims", int, rw))
        if out.rot_dims > out.rot_dim or out.rot_dims % 2:
            raise ConfigError(f"config key {rw}'dims' must be even and at most rot_dim {out.rot_dim}, got {out.rot_dims}")
        return out
    if typ == "attention":
        heads, kv = _num(m, "heads", int, where), _num(m, "kv_heads", int, where)
        if heads % kv:
            raise ConfigError(f"config key {where}'heads' {heads} is no multiple of 'kv_heads' {kv}")
        chunk = None if m.get("mask") is None else _num(_section(m, "mask", where), "size", int, where + "mask.")
        softcap = None if m.get("softcap") is None else _num(m, "softcap", float, where)
        source = None if m.get("kv_from") is None else coerce(where + "kv_from", m["kv_from"], int)
        return AttentionConfig(heads, kv, _num(m, "dim", int, where), _num(m, "vdim", int, where),
                               _num(m, "scale", float, where), softcap, chunk, source)
    if typ == "lightning":
        heads, decay = _num(m, "heads", int, where), m.get("decay")
        if not isinstance(decay, list) or len(decay) != heads:
            raise ConfigError(f"config key {where}'decay' must be a list of one number a head ({heads}), got {decay!r}")
        decay = tuple(coerce(f"{where}decay[{h}]", d, float) for h, d in enumerate(decay))
        if not all(0.0 < d <= 1.0 for d in decay):
            raise ConfigError(f"config key {where}'decay' must hold numbers in (0, 1], got {list(decay)}")
        return LightningConfig(heads, _num(m, "dim", int, where), _num(m, "vdim", int, where), decay)
    raise ConfigError(f"config key {where[:-6]}'type': unknown mixer {typ!r} (known: 'latent_attention', 'attention', 'lightning')")


def _feed_forward(f, where: str) -> FeedForwardConfig | None:
    if f is None:
        return None
    if not isinstance(f, dict):
        raise ConfigError(f"config key {where[:-1]!r} must be an object or null, got {f!r}")
    if f.get("kind") == "dense":
        return FeedForwardConfig("dense", _num(f, "ff", int, where))
    if f.get("kind") == "moe":
        e, ew = _section(f, "expert", where), where + "expert."
        r, rw = _section(f, "router", where), where + "router."
        out = FeedForwardConfig("moe", _num(e, "ff", int, ew), _num(e, "limit", float, ew), _num(r, "experts", int, rw),
                                _num(r, "top", int, rw))
        if out.top > out.experts:
            raise ConfigError(f"config key {rw}'top' {out.top} exceeds 'experts' {out.experts}")
        return out
    raise ConfigError(f"config key {where}'kind' must be 'dense' or 'moe', got {f.get('kind')!r}")


@dataclass(frozen=True)
class DumovikConfig(ModelConfig):
    vocab: int = key(int)
    width: int = key(int)
    norm_eps: float = field(default=1e-5)
    layers: tuple = field(default=())

    ARCHITECTURE = "Dumovik"
    MAX_POSITIONS = (1 << 31) - 1     # the design sets no limit; positions are 32-bit in the batch

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
            out.append(DumovikLayer(typ, _mixer(typ, _section(l, "mixer", where), where + "mixer."),
                                    _feed_forward(l.get("mlp"), where + "mlp.")))
        return {"norm_eps": _num(_section(d, "norm", ""), "eps", float, "norm."), "layers": tuple(out)}

    def check(self) -> None:
        if self.vocab <= 0 or self.width <= 0:
            raise ConfigError(f"config keys 'vocab' and 'width' must be positive, got {self.vocab} and {self.width}")
        for i, l in enumerate(self.layers):
            j = l.mixer.kv_from if l.type == "attention" else None
            if j is None:
                continue
            if not (0 <= j < i) or self.layers[j].type != "attention":
                raise ConfigError(f"layers[{i}].mixer.kv_from = {j} must name an earlier attention layer")
            a, b = self.layers[j].mixer, l.mixer
            if a.kv_from is not None:
                raise ConfigError(f"layers[{i}].mixer.kv_from = {j}: that layer has no keys and values of its own")
            if (a.kv_heads, a.dim, a.vdim) != (b.kv_heads, b.dim, b.vdim):
                raise ConfigError(f"layers[{i}] reads the keys and values of layer {j}: their kv_heads, dim and vdim must be equal")

    def kept_keys(self, i: int) -> int | None:
        """How many of the last keys attention layer i's cache must hold: as many as it or a layer that reads it may see
        (None: all of them)."""
        readers = [self.layers[i]] + [l for l in self.layers if l.type == "attention" and l.mixer.kv_from == i]
        sizes = [l.mixer.chunk for l in readers]
        return None if None in sizes else max(sizes)

    def extra_to_dict(self) -> dict:
        def mixer(l: DumovikLayer):
            m = l.mixer
            if l.type == "latent_attention":
                return {"heads": m.heads, "dim": m.dim, "rot_dim": m.rot_dim, "vdim": m.vdim, "kv_rank": m.kv_rank,
                        "scale": m.scale, "rot": {"base": m.rot_base, "dims": m.rot_dims}}
            if l.type == "lightning":
                return {"heads": m.heads, "dim": m.dim, "vdim": m.vdim, "decay": list(m.decay)}
            out = {"heads": m.heads, "kv_heads": m.kv_heads, "dim": m.dim, "vdim": m.vdim, "scale": m.scale,
                   "softcap": m.softcap, "mask": None if m.chunk is None else {"size": m.chunk}}
            if m.kv_from is not None:
                out["kv_from"] = m.kv_from
            return out

        def mlp(f: FeedForwardConfig | None):
            if f is None:
                return None
            if f.kind == "dense":
                return {"kind": "dense", "ff": f.ff}
            return {"kind": "moe", "expert": {"ff": f.ff, "limit": f.limit}, "router": {"experts": f.experts, "top": f.top}}

        return {"architecture": self.ARCHITECTURE, "norm": {"eps": self.norm_eps},
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
