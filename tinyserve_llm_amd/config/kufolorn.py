"""Typed configuration of the Kufolorn decoder, read from the keys of its config.json: one eps for every norm, a cap on the
logits (`logit_softcap`; absent: none) and a list of layers. A layer names its mixer's kind ("delta": a gated delta rule behind
short convolutions; "parallel": attention with a learned sink and retention side by side) with the mixer's sizes and
constants, and an optional feed-forward (dense, or a mixture of capped experts with identity experts, chosen inside groups).
Every size and constant of a model stands here and nowhere else."""

from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Mapping

from tinyserve_llm_amd.config.bafarax import _need
from tinyserve_llm_amd.config.llama import ConfigError


@dataclass(frozen=True)
class KufolornRotation:
    dims: int                    # leading dimensions of a head that turn, pairs (i, i + dims/2); 0: none
    base: float
    factor: float = 1.0          # every frequency is divided by it

    @classmethod
    def from_dict(cls, raw: Mapping[str, Any] | None, where: str) -> "KufolornRotation":
        if not raw:
            return cls(0, 1.0)
        scaling = raw.get("scaling")
        c = cls(dims=int(_need(raw, "dims", where)), base=float(_need(raw, "base", where)),
                factor=1.0 if scaling is None else float(_need(scaling, "factor", where + ".scaling")))
        if c.dims < 0 or c.dims % 2 or not c.base > 0 or not c.factor > 0:
            raise ConfigError(f"{where}: an even number of dims, a positive base and a positive scaling.factor")
        return c

    def to_dict(self) -> dict[str, Any]:
        out: dict[str, Any] = {"base": self.base, "dims": self.dims}
        if self.factor != 1.0:
            out["scaling"] = {"factor": self.factor}
        return out


@dataclass(frozen=True)
class KufolornDelta:
    heads: int
    kv_heads: int                # heads of keys and queries, each shared by heads / kv_heads heads
    dim: int
    vdim: int
    conv: int                    # taps of the short convolutions

    @classmethod
    def from_dict(cls, raw: Mapping[str, Any], where: str) -> "KufolornDelta":
        c = cls(*(int(_need(raw, k, where)) for k in ("heads", "kv_heads", "dim", "vdim", "conv")))
        if min(c.heads, c.kv_heads, c.dim, c.vdim, c.conv) <= 0:
            raise ConfigError(f"{where}: heads, kv_heads, dim, vdim and conv are positive")
        if c.heads % c.kv_heads:
            raise ConfigError(f"{where}.kv_heads: {c.heads} heads do not divide into {c.kv_heads} key and query heads")
        return c

    def to_dict(self) -> dict[str, Any]:
        return {"conv": self.conv, "dim": self.dim, "heads": self.heads, "kv_heads": self.kv_heads, "vdim": self.vdim}


@dataclass(frozen=True)
class KufolornAttention:
    heads: int
    kv_heads: int
    dim: int                     # size of a query / key head
    vdim: int                    # size of a value head
    scale: float
    rot: KufolornRotation

    @classmethod
    def from_dict(cls, raw: Mapping[str, Any], where: str) -> "KufolornAttention":
        c = cls(*(int(_need(raw, k, where)) for k in ("heads", "kv_heads", "dim", "vdim")), scale=float(_need(raw, "scale", where)),
                rot=KufolornRotation.from_dict(raw.get("rot"), where + ".rot"))
        if min(c.heads, c.kv_heads) <= 0 or c.heads % c.kv_heads:
            raise ConfigError(f"{where}.kv_heads: {c.heads} heads do not divide into {c.kv_heads} key/value heads")
        if min(c.dim, c.vdim) <= 0 or c.rot.dims > c.dim:
            raise ConfigError(f"{where}: dim and vdim are positive, rot.dims at most dim")
        return c

    def to_dict(self) -> dict[str, Any]:
        out: dict[str, Any] = {"dim": self.dim, "heads": self.heads, "kv_heads": self.kv_heads, "scale": self.scale, "vdim": self.vdim}
        if self.rot.dims:
            out["rot"] = self.rot.to_dict()
        return out


@dataclass(frozen=True)
class KufolornRetention:
    heads: int
    dim: int
    vdim: int
    decay: tuple[float, ...]     # per head
    rot: KufolornRotation

    @classmethod
    def from_dict(cls, raw: Mapping[str, Any], where: str) -> "KufolornRetention":
        decay = _need(raw, "decay", where)
        if not isinstance(decay, (list, tuple)):
            raise ConfigError(f"{where}.decay: a list, a number per head")
        c = cls(*(int(_need(raw, k, where)) for k in ("heads", "dim", "vdim")), decay=tuple(float(d) for d in decay),
                rot=KufolornRotation.from_dict(raw.get("rot"), where + ".rot"))
        if min(c.heads, c.dim, c.vdim) <= 0 or c.rot.dims > c.dim:
            raise ConfigError(f"{where}: heads, dim and vdim are positive, rot.dims at most dim")
        if len(c.decay) != c.heads or not all(0.0 <= d <= 1.0 for d in c.decay):
            raise ConfigError(f"{where}.decay: a number from 0 to 1 for each of {c.heads} heads")
        return c

    def to_dict(self) -> dict[str, Any]:
        out: dict[str, Any] = {"decay": list(self.decay), "dim": self.dim, "heads": self.heads, "vdim": self.vdim}
        if self.rot.dims:
            out["rot"] = self.rot.to_dict()
        return out


@dataclass(frozen=True)
class KufolornParallel:
    left: KufolornAttention
    right: KufolornRetention
    left_scale: float
    right_scale: float

    @classmethod
    def from_dict(cls, raw: Mapping[str, Any], where: str) -> "KufolornParallel":
        return cls(KufolornAttention.from_dict(_need(raw, "left", where), where + ".left"),
                   KufolornRetention.from_dict(_need(raw, "right", where), where + ".right"),
                   float(_need(raw, "left_scale", where)), float(_need(raw, "right_scale", where)))

    def to_dict(self) -> dict[str, Any]:
        return {"left": self.left.to_dict(), "left_scale": self.left_scale, "right": self.right.to_dict(), "right_scale": self.right_scale}


MIXERS = {"delta": KufolornDelta, "parallel": KufolornParallel}


@dataclass(frozen=True)
class KufolornDense:
    ff: int

    def to_dict(self) -> dict[str, Any]:
        return {"ff": self.ff, "kind": "dense"}


@dataclass(frozen=True)
class KufolornExperts:
    experts: int                 # experts with matrices
    identity: int                # router outputs beyond them, which stand for experts that hand their input through
    top: int
    ff: int                      # width of one expert
    limit: float                 # cap on an expert's two branches
    groups: int = 1              # equal groups of neighbouring router outputs,
    keep: int = 1                # of which this many can be chosen from

    def to_dict(self) -> dict[str, Any]:
        router: dict[str, Any] = {"experts": self.experts, "top": self.top}
        if self.groups > 1:
            router["groups"] = {"count": self.groups, "keep": self.keep}
        if self.identity:
            router["identity"] = self.identity
        return {"expert": {"ff": self.ff, "limit": self.limit}, "kind": "moe", "router": router}


def _mlp(raw: Mapping[str, Any] | None, where: str) -> "KufolornDense | KufolornExperts | None":
    if raw is None:
        return None
    kind = _need(raw, "kind", where)
    if kind == "dense":
        c = KufolornDense(ff=int(_need(raw, "ff", where)))
        if c.ff <= 0:
            raise ConfigError(f"{where}.ff: positive")
        return c
    if kind == "moe":
        router, expert = _need(raw, "router", where), _need(raw, "expert", where)
        groups = router.get("groups")
        count, keep = (int(_need(groups, k, where + ".router.groups")) for k in ("count", "keep")) if groups is not None else (1, 1)
        e = KufolornExperts(experts=int(_need(router, "experts", where + ".router")), identity=int(router.get("identity") or 0),
                            top=int(_need(router, "top", where + ".router")), ff=int(_need(expert, "ff", where + ".expert")),
                            limit=float(_need(expert, "limit", where + ".expert")), groups=count, keep=keep)
        if e.experts <= 0 or e.identity < 0 or e.ff <= 0 or not e.limit > 0:
            raise ConfigError(f"{where}: positive experts, expert.ff and expert.limit, identity not negative")
        size = (e.experts + e.identity) // max(1, e.groups)
        if e.groups < 1 or (e.experts + e.identity) % e.groups or not 1 <= e.keep <= e.groups:
            raise ConfigError(f"{where}.router.groups: {e.experts + e.identity} router outputs in equal groups, of which some are kept")
        if not 1 <= e.top <= e.keep * size:
            raise ConfigError(f"{where}.router.top: between 1 and the {e.keep * size} router outputs of the groups kept")
        return e
    raise ConfigError(f"{where}.kind {kind!r}: 'dense' or 'moe'")


@dataclass(frozen=True)
class KufolornLayer:
    type: str
    mixer: "KufolornDelta | KufolornParallel"
    mlp: "KufolornDense | KufolornExperts | None"

    @classmethod
    def from_dict(cls, raw: Mapping[str, Any], where: str) -> "KufolornLayer":
        kind = _need(raw, "type", where)
        if kind not in MIXERS:
            raise ConfigError(f"{where}.type {kind!r}: one of {sorted(MIXERS)}")
        return cls(kind, MIXERS[kind].from_dict(_need(raw, "mixer", where), where + ".mixer"), _mlp(raw.get("mlp"), where + ".mlp"))

    def to_dict(self) -> dict[str, Any]:
        return {"mixer": self.mixer.to_dict(), "mlp": None if self.mlp is None else self.mlp.to_dict(), "type": self.type}


@dataclass(frozen=True)
class KufolornConfig:
    vocab: int
    width: int
    layers: tuple[KufolornLayer, ...]
    norm_eps: float
    logit_softcap: float = 0.0   # logits leave as cap tanh(logits / cap); 0: as they are
    architecture: str = "Kufolorn"

    @classmethod
    def from_dict(cls, raw: Mapping[str, Any]) -> "KufolornConfig":
        layers = tuple(KufolornLayer.from_dict(l, f"layers[{i}]") for i, l in enumerate(_need(raw, "layers", "config.json")))
        if not layers:
            raise ConfigError("layers: the model has at least one")
        c = cls(vocab=int(_need(raw, "vocab", "config.json")), width=int(_need(raw, "width", "config.json")), layers=layers,
                norm_eps=float(_need(_need(raw, "norm", "config.json"), "eps", "norm")), logit_softcap=float(raw.get("logit_softcap") or 0.0))
        if c.vocab <= 0 or c.width <= 0 or c.norm_eps < 0 or c.logit_softcap < 0:
            raise ConfigError("vocab and width are positive, norm.eps and logit_softcap are not negative")
        return c

    def to_dict(self) -> dict[str, Any]:
        out: dict[str, Any] = {"architecture": self.architecture, "layers": [l.to_dict() for l in self.layers],
                               "norm": {"eps": self.norm_eps}, "vocab": self.vocab, "width": self.width}
        if self.logit_softcap:
            out["logit_softcap"] = self.logit_softcap
        return out
