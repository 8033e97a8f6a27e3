"""Configuration of the Tobilorn decoder: layers whose sublayers are normed before and after, differential attention
(two softmax maps a head) behind a sliding window that keeps the first tokens, experts behind a softmax router with
identity experts and a shared expert, a narrow input looked up by the token's id in every layer, and a stretch of the
layers that runs several times, every pass beginning with a projection of the stream joined with the embedding.

config.json is nested:
    architecture: "Tobilorn"     vocab, width: ints     norm: {eps}     embedding: {scale}     logit_scale: s
    loop: {start, stop, times} (optional: layers start .. stop - 1 run `times` times in a row)
    token_side: {dim} (optional: channels of a token's own vector in every layer)
    layers: [{type, mixer: {...}, mlp: {...} | null}, ...]
        type "attention":  mixer {heads, kv_heads, dim, vdim, scale, diff, rot: {base, dims} (optional),
                                  mask: {size, keep_first} (optional: without it every earlier position is seen)}
        mlp {kind: "moe", router: {experts, top, identity (optional)}, expert: {ff}, shared: {ff} (optional)}
"""
from __future__ import annotations

import dataclasses
from typing import Any, ClassVar, Optional

from .base import ConfigError, ModelConfig

MIXER_SIZES = ("heads", "kv_heads", "dim", "vdim")


def _is_int(v, minimum=1) -> bool:
    return isinstance(v, int) and not isinstance(v, bool) and v >= minimum


def _is_num(v) -> bool:
    return isinstance(v, (int, float)) and not isinstance(v, bool)


@dataclasses.dataclass
class TobilornConfig(ModelConfig):
    architecture: ClassVar[str] = "Tobilorn"
    ignored: ClassVar[frozenset[str]] = ModelConfig.ignored | frozenset({"architecture"})

    vocab: int
    width: int
    layers: list
    norm: dict = dataclasses.field(default_factory=lambda: {"eps": 1e-5})
    embedding: dict = dataclasses.field(default_factory=lambda: {"scale": 1.0})
    logit_scale: float = 1.0
    loop: Optional[dict] = None
    token_side: Optional[dict] = None
    max_positions: Optional[int] = None

    def validate(self) -> None:
        self._int("vocab")
        self._int("width")
        self._float("logit_scale", positive=False)
        if not isinstance(self.norm, dict) or not _is_num(self.norm.get("eps")) or not self.norm["eps"] > 0:
            raise ConfigError("norm.eps must be a positive number")
        if not isinstance(self.embedding, dict) or not _is_num(self.embedding.get("scale")):
            raise ConfigError("embedding.scale must be a number")
        if self.token_side is not None and (not isinstance(self.token_side, dict) or not _is_int(self.token_side.get("dim"))):
            raise ConfigError("token_side.dim must be a positive integer")
        if not isinstance(self.layers, list) or not self.layers:
            raise ConfigError("layers must be a non-empty list")
        for i, layer in enumerate(self.layers):
            where = f"layers[{i}]"
            if not isinstance(layer, dict) or layer.get("type") != "attention":
                raise ConfigError(f"{where}.type must be 'attention'")
            self._check_mixer(layer.get("mixer"), where + ".mixer")
            self._check_mlp(layer.get("mlp"), where + ".mlp")
        if self.loop is not None:
            lp = self.loop
            ok = isinstance(lp, dict) and all(_is_int(lp.get(k), 0) for k in ("start", "stop")) and _is_int(lp.get("times"))
            if not ok or not lp["start"] < lp["stop"] <= len(self.layers):
                raise ConfigError(f"loop must give 0 <= start < stop <= {len(self.layers)} and times >= 1, got {lp!r}")

    @staticmethod
    def _check_mixer(m, where: str) -> None:
        lacks = [k for k in MIXER_SIZES + ("scale", "diff") if not isinstance(m, dict) or k not in m]
        if lacks:
            raise ConfigError(f"{where} lacks key(s): {', '.join(lacks)}")
        for k in MIXER_SIZES:
            if not _is_int(m[k]):
                raise ConfigError(f"{where}.{k} must be a positive integer, got {m[k]!r}")
        if m["heads"] % m["kv_heads"]:
            raise ConfigError(f"{where}: heads {m['heads']} is no multiple of kv_heads {m['kv_heads']}")
        if not _is_num(m["scale"]) or not m["scale"] > 0:
            raise ConfigError(f"{where}.scale must be a positive number, got {m['scale']!r}")
        if not _is_num(m["diff"]):
            raise ConfigError(f"{where}.diff must be a number, got {m['diff']!r}")
        rot = m.get("rot")
        if rot is not None:
            if not isinstance(rot, dict) or not _is_num(rot.get("base")) or not rot["base"] > 0:
                raise ConfigError(f"{where}.rot.base must be a positive number")
            dims = rot.setdefault("dims", m["dim"])
            if not _is_int(dims, 0) or dims % 2 or dims > m["dim"]:
                raise ConfigError(f"{where}.rot.dims must be an even number of the {m['dim']} channels, got {dims!r}")
        mask = m.get("mask")
        if mask is not None:
            if not isinstance(mask, dict) or not _is_int(mask.get("size")):
                raise ConfigError(f"{where}.mask.size must be a positive integer")
            if not _is_int(mask.setdefault("keep_first", 0), 0):
                raise ConfigError(f"{where}.mask.keep_first must be a number of tokens, got {mask['keep_first']!r}")

    @staticmethod
    def _check_mlp(mlp, where: str) -> None:
        if mlp is None:
            return
        if not isinstance(mlp, dict) or mlp.get("kind") != "moe":
            raise ConfigError(f"{where}.kind must be 'moe' (or mlp null)")
        try:
            r = mlp["router"]
            sizes = [r["experts"], r["top"], mlp["expert"]["ff"]]
            identity = r.setdefault("identity", 0)
            if mlp.get("shared") is not None:
                sizes.append(mlp["shared"]["ff"])
        except (KeyError, TypeError, AttributeError) as e:
            raise ConfigError(f"{where} lacks a key ({e})") from None
        if not all(_is_int(v) for v in sizes) or not _is_int(identity, 0):
            raise ConfigError(f"{where}: sizes must be positive integers, got {sizes} and {identity} identity experts")
        if r["top"] > r["experts"] + identity:
            raise ConfigError(f"{where}.router: top {r['top']} of {r['experts']} + {identity} experts")

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

    def run_order(self) -> list[tuple]:
        """[(layer, the pass of the loop that begins before it, or None)] in the order the layers run."""
        n = len(self.layers)
        if not self.loop:
            return [(i, None) for i in range(n)]
        a, b, times = self.loop["start"], self.loop["stop"], self.loop["times"]
        out: list[tuple] = [(i, None) for i in range(a)]
        for p in range(times):
            out += [(i, p if i == a else None) for i in range(a, b)]
        return out + [(i, None) for i in range(b, n)]

    def to_dict(self) -> dict[str, Any]:
        out = {"architecture": self.architecture}
        out.update(dataclasses.asdict(self))
        for k in ("loop", "token_side", "max_positions"):
            if out.get(k) is None:
                out.pop(k, None)
        return out
