"""Configuration of the Kisutar decoder: pre-norm layers with RMS norms, a token shift before every mixer and a learned
sum over all earlier layers' results after every layer; the mixer is latent attention with latent queries, a rotated
part, a sliding window and sinks (a layer may read an earlier layer's latent rows); the feed-forwards a dense layer
with xIELU or experts behind a softmax router, with an optional shared expert.

config.json is nested:
    architecture: "Kisutar"      vocab, width: ints      norm: {eps}
    layers: [{type, mixer: {...}, mlp: {...} | null}, ...]
        type "latent_attention":  mixer {heads, dim, rot_dim, vdim, q_rank, kv_rank, scale, rot: {base, dims}, mask: {size}
                                  (optional: without it every earlier position is seen), kv_from (optional: the layer whose
                                  latent rows and rotated keys it reads)}
        mlp {kind: "dense", ff}
        mlp {kind: "moe", router: {experts, top}, expert: {ff}, shared: {ff} (optional)}
"""
from __future__ import annotations

import dataclasses
from typing import Any, ClassVar, Optional

from .base import ConfigError, ModelConfig

MIXER_SIZES = ("heads", "dim", "rot_dim", "vdim", "q_rank", "kv_rank")


def _is_int(v, minimum=1) -> bool:
    return isinstance(v, int) and not isinstance(v, bool) and v >= minimum


def _is_num(v) -> bool:
    return isinstance(v, (int, float)) and not isinstance(v, bool)


@dataclasses.dataclass
class KisutarConfig(ModelConfig):
    architecture: ClassVar[str] = "Kisutar"
    ignored: ClassVar[frozenset[str]] = ModelConfig.ignored | frozenset({"architecture"})

    vocab: int
    width: int
    layers: list
    norm: dict = dataclasses.field(default_factory=lambda: {"eps": 1e-5})
    max_positions: Optional[int] = None

    def validate(self) -> None:
        self._int("vocab")
        self._int("width")
        if not isinstance(self.norm, dict) or not _is_num(self.norm.get("eps")) or not self.norm["eps"] > 0:
            raise ConfigError("norm.eps must be a positive number")
        if not isinstance(self.layers, list) or not self.layers:
            raise ConfigError("layers must be a non-empty list")
        for i, layer in enumerate(self.layers):
            where = f"layers[{i}]"
            if not isinstance(layer, dict) or layer.get("type") != "latent_attention":
                raise ConfigError(f"{where}.type must be 'latent_attention'")
            self._check_mixer(i, layer.get("mixer"), where + ".mixer")
            self._check_mlp(layer.get("mlp"), where + ".mlp")

    def _check_mixer(self, i: int, m, where: str) -> None:
        lacks = [k for k in MIXER_SIZES + ("scale", "rot") if not isinstance(m, dict) or k not in m]
        if lacks:
            raise ConfigError(f"{where} lacks key(s): {', '.join(lacks)}")
        for k in MIXER_SIZES:
            if not _is_int(m[k]):
                raise ConfigError(f"{where}.{k} must be a positive integer, got {m[k]!r}")
        if not _is_num(m["scale"]) or not m["scale"] > 0:
            raise ConfigError(f"{where}.scale must be a positive number, got {m['scale']!r}")
        rot = m["rot"]
        if not isinstance(rot, dict) or not _is_num(rot.get("base")) or not rot["base"] > 0:
            raise ConfigError(f"{where}.rot.base must be a positive number")
        dims = rot.setdefault("dims", m["rot_dim"])
        if not _is_int(dims, 0) or dims % 2 or dims > m["rot_dim"]:
            raise ConfigError(f"{where}.rot.dims must be an even number of the {m['rot_dim']} rotated channels, got {dims!r}")
        mask = m.get("mask")
        if mask is not None and (not isinstance(mask, dict) or not _is_int(mask.get("size"))):
            raise ConfigError(f"{where}.mask.size must be a positive integer")
        src = m.get("kv_from")
        if src is None:
            return
        if not _is_int(src, 0) or src >= i:
            raise ConfigError(f"{where}.kv_from must name an earlier layer, got {src!r}")
        other = self.layers[src]["mixer"]
        if other.get("kv_from") is not None:
            raise ConfigError(f"{where}.kv_from: layer {src} has no latent rows of its own")
        for k in ("kv_rank", "rot_dim", "rot"):
            if other[k] != m[k]:
                raise ConfigError(f"{where}.{k} {m[k]} is not layer {src}'s {other[k]}")

    @staticmethod
    def _check_mlp(mlp, where: str) -> None:
        if mlp is None:
            return
        if not isinstance(mlp, dict) or mlp.get("kind") not in ("dense", "moe"):
            raise ConfigError(f"{where}.kind must be 'dense' or 'moe' (or mlp null)")
        if mlp["kind"] == "dense":
            if not _is_int(mlp.get("ff")):
                raise ConfigError(f"{where}.ff must be a positive integer")
            return
        try:
            sizes = [mlp["router"]["experts"], mlp["router"]["top"], mlp["expert"]["ff"]]
            if mlp.get("shared") is not None:
                sizes.append(mlp["shared"]["ff"])
        except (KeyError, TypeError) as e:
            raise ConfigError(f"{where} lacks a key ({e})") from None
        if not all(_is_int(v) for v in sizes):
            raise ConfigError(f"{where}: sizes must be positive integers, got {sizes}")
        if sizes[1] > sizes[0]:
            raise ConfigError(f"{where}.router: top {sizes[1]} of {sizes[0]} experts")

    # --------------------------------------------------------------------- derived
    @property
    def vocab_size(self) -> int:
        return self.vocab

    @property
    def hidden_size(self) -> int:
        return self.width

    @property
    def eps(self) -> float:
        return float(self.norm["eps"])

    def to_dict(self) -> dict[str, Any]:
        out = {"architecture": self.architecture}
        out.update(dataclasses.asdict(self))
        if out.get("max_positions") is None:
            out.pop("max_positions", None)
        return out
