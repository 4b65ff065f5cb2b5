"""Typed configuration of the Morulix decoder, read from the keys of its config.json: one eps for every norm, a list of
layers, and a stretch of layers that runs several times in a row with the same weights (`loop`; absent: every layer
once). A layer names its mixer's kind ("mamba2": a state-space mixer; "attention": grouped-query attention in a sliding
window; "latent_attention": attention through a low-rank latent without positions) with the mixer's sizes and
constants, and an optional dense feed-forward. Every size and constant of a model stands here and nowhere else."""

from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Mapping

from tinyserve_llm_amd.config.bafarax import _mask_size, _need
from tinyserve_llm_amd.config.llama import ConfigError


@dataclass(frozen=True)
class FrequencyBands:
    """Slows the rotation's frequencies by wavelength: those longer than original / low by `factor`, those shorter than
    original / high not at all, those between by a mix of both."""
    factor: float
    low: float
    high: float
    original: float

    @classmethod
    def from_dict(cls, raw: Mapping[str, Any], where: str) -> "FrequencyBands":
        c = cls(*(float(_need(raw, k, where)) for k in ("factor", "low", "high", "original")))
        if min(c.factor, c.low, c.original) <= 0 or c.high < c.low:
            raise ConfigError(f"{where}: factor, low and original are positive, high is at least low")
        return c

    def to_dict(self) -> dict[str, Any]:
        original = int(self.original) if self.original == int(self.original) else self.original
        return {"factor": self.factor, "high": self.high, "low": self.low, "original": original}


@dataclass(frozen=True)
class MorulixRotation:
    dims: int                    # leading dimensions of a head that turn, pairs (i, i + dims/2); 0: none
    base: float
    bands: FrequencyBands | None = None

    @classmethod
    def from_dict(cls, raw: Mapping[str, Any] | None, where: str) -> "MorulixRotation":
        if not raw:
            return cls(0, 1.0)
        scaling = raw.get("scaling")
        c = cls(dims=int(_need(raw, "dims", where)), base=float(_need(raw, "base", where)),
                bands=FrequencyBands.from_dict(scaling, where + ".scaling") if scaling else None)
        if c.dims < 0 or c.dims % 2 or c.base <= 0:
            raise ConfigError(f"{where}: an even number of dims, a positive base")
        return c

    def to_dict(self) -> dict[str, Any]:
        out: dict[str, Any] = {"base": self.base, "dims": self.dims}
        if self.bands is not None:
            out["scaling"] = self.bands.to_dict()
        return out


@dataclass(frozen=True)
class MorulixAttention:
    heads: int
    kv_heads: int
    dim: int                     # size of a query / key head
    vdim: int                    # size of a value head
    scale: float
    rot: MorulixRotation
    window: int                  # a position sees itself and the window - 1 before it (0: all before it)

    @classmethod
    def from_dict(cls, raw: Mapping[str, Any], where: str) -> "MorulixAttention":
        c = cls(heads=int(_need(raw, "heads", where)), kv_heads=int(_need(raw, "kv_heads", where)), dim=int(_need(raw, "dim", where)),
                vdim=int(_need(raw, "vdim", where)), scale=float(_need(raw, "scale", where)),
                rot=MorulixRotation.from_dict(raw.get("rot"), where + ".rot"), window=_mask_size(raw, where))
        if c.heads <= 0 or c.kv_heads <= 0 or c.heads % c.kv_heads:
            raise ConfigError(f"{where}.kv_heads: {c.heads} heads do not divide into {c.kv_heads} key/value heads")
        if c.dim <= 0 or c.vdim <= 0 or c.rot.dims > c.dim:
            raise ConfigError(f"{where}: dim and vdim are positive, rot.dims at most dim")
        return c

    def to_dict(self) -> dict[str, Any]:
        out: dict[str, Any] = {"dim": self.dim, "heads": self.heads, "kv_heads": self.kv_heads, "scale": self.scale, "vdim": self.vdim}
        if self.window:
            out["mask"] = {"size": self.window}
        if self.rot.dims:
            out["rot"] = self.rot.to_dict()
        return out


@dataclass(frozen=True)
class MorulixLatentAttention:
    heads: int
    dim: int                     # query / key dimensions of a head
    vdim: int
    kv_rank: int                 # size of the latent that keys and values are made from
    scale: float

    @classmethod
    def from_dict(cls, raw: Mapping[str, Any], where: str) -> "MorulixLatentAttention":
        c = cls(heads=int(_need(raw, "heads", where)), dim=int(_need(raw, "dim", where)), vdim=int(_need(raw, "vdim", where)),
                kv_rank=int(_need(raw, "kv_rank", where)), scale=float(_need(raw, "scale", where)))
        if min(c.heads, c.dim, c.vdim, c.kv_rank) <= 0:
            raise ConfigError(f"{where}: heads, dim, vdim and kv_rank are positive")
        return c

    def to_dict(self) -> dict[str, Any]:
        return {"dim": self.dim, "heads": self.heads, "kv_rank": self.kv_rank, "scale": self.scale, "vdim": self.vdim}


@dataclass(frozen=True)
class MorulixMamba2:
    heads: int
    vdim: int                    # channels of a head
    state: int                   # rows of a head's state
    groups: int                  # groups of heads that share their B and C
    conv: int                    # taps of the short convolution
    norm_groups: int             # equal parts of the heads' output that are normalised each by itself

    @classmethod
    def from_dict(cls, raw: Mapping[str, Any], where: str) -> "MorulixMamba2":
        c = cls(*(int(_need(raw, k, where)) for k in ("heads", "vdim", "state", "groups", "conv", "norm_groups")))
        if min(c.heads, c.vdim, c.state, c.groups, c.conv, c.norm_groups) <= 0:
            raise ConfigError(f"{where}: heads, vdim, state, groups, conv and norm_groups are positive")
        if c.heads % c.groups:
            raise ConfigError(f"{where}.groups: {c.heads} heads do not divide into {c.groups} groups")
        if (c.heads * c.vdim) % c.norm_groups:
            raise ConfigError(f"{where}.norm_groups: {c.heads * c.vdim} channels do not divide into {c.norm_groups} parts")
        return c

    def to_dict(self) -> dict[str, Any]:
        return {"conv": self.conv, "groups": self.groups, "heads": self.heads, "norm_groups": self.norm_groups, "state": self.state,
                "vdim": self.vdim}


MIXERS = {"attention": MorulixAttention, "latent_attention": MorulixLatentAttention, "mamba2": MorulixMamba2}


@dataclass(frozen=True)
class MorulixLayer:
    type: str
    mixer: "MorulixAttention | MorulixLatentAttention | MorulixMamba2"
    ff: int | None               # width of the dense feed-forward; None: the layer has none

    @classmethod
    def from_dict(cls, raw: Mapping[str, Any], where: str) -> "MorulixLayer":
        kind = _need(raw, "type", where)
        if kind not in MIXERS:
            raise ConfigError(f"{where}.type {kind!r}: one of {sorted(MIXERS)}")
        mlp, ff = raw.get("mlp"), None
        if mlp is not None:
            if _need(mlp, "kind", where + ".mlp") != "dense":
                raise ConfigError(f"{where}.mlp.kind {mlp['kind']!r}: this decoder has dense feed-forwards")
            ff = int(_need(mlp, "ff", where + ".mlp"))
            if ff <= 0:
                raise ConfigError(f"{where}.mlp.ff: positive")
        return cls(kind, MIXERS[kind].from_dict(_need(raw, "mixer", where), where + ".mixer"), ff)

    def to_dict(self) -> dict[str, Any]:
        return {"mixer": self.mixer.to_dict(), "mlp": None if self.ff is None else {"ff": self.ff, "kind": "dense"}, "type": self.type}


@dataclass(frozen=True)
class MorulixConfig:
    vocab: int
    width: int
    layers: tuple[MorulixLayer, ...]
    norm_eps: float
    # layers loop_start .. loop_stop - 1 run loop_times times in a row, each pass behind its own input; loop_times 0: no
    # looped stretch, every layer once
    loop_start: int = 0
    loop_stop: int = 0
    loop_times: int = 0
    architecture: str = "Morulix"

    @classmethod
    def from_dict(cls, raw: Mapping[str, Any]) -> "MorulixConfig":
        layers = tuple(MorulixLayer.from_dict(l, f"layers[{i}]") for i, l in enumerate(_need(raw, "layers", "config.json")))
        if not layers:
            raise ConfigError("layers: the model has at least one")
        loop, start, stop, times = raw.get("loop"), 0, 0, 0
        if loop:
            start, stop, times = (int(_need(loop, k, "loop")) for k in ("start", "stop", "times"))
            if not 0 <= start < stop <= len(layers) or times < 1:
                raise ConfigError(f"loop {dict(loop)}: 0 <= start < stop <= {len(layers)} layers, times >= 1")
        c = cls(vocab=int(_need(raw, "vocab", "config.json")), width=int(_need(raw, "width", "config.json")), layers=layers,
                norm_eps=float(_need(_need(raw, "norm", "config.json"), "eps", "norm")), loop_start=start, loop_stop=stop, loop_times=times)
        if c.vocab <= 0 or c.width <= 0 or c.norm_eps < 0:
            raise ConfigError("vocab and width are positive, norm.eps is not negative")
        return c

    def to_dict(self) -> dict[str, Any]:
        out: dict[str, Any] = {"architecture": self.architecture, "layers": [l.to_dict() for l in self.layers],
                               "norm": {"eps": self.norm_eps}, "vocab": self.vocab, "width": self.width}
        if self.loop_times:
            out["loop"] = {"start": self.loop_start, "stop": self.loop_stop, "times": self.loop_times}
        return out

    def run_order(self) -> list[tuple[int, int | None]]:
        """The layers in the order they run: (layer, number of the pass that this run begins, else None)."""
        if not self.loop_times:
            return [(i, None) for i in range(len(self.layers))]
        order: list[tuple[int, int | None]] = [(i, None) for i in range(self.loop_start)]
        for t in range(self.loop_times):
            order += [(i, t if i == self.loop_start else None) for i in range(self.loop_start, self.loop_stop)]
        return order + [(i, None) for i in range(self.loop_stop, len(self.layers))]
