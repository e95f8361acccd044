"""Typed configuration of the Rifizen decoder, read from ``config.json``, and the model it describes.

A Rifizen model is a list of layers over a 32-bit residual stream, each branch between a norm before and a norm behind
it.  A layer's mixer is two mixers side by side that read the same rows: grouped-query attention inside a sliding
window, with unit-RMS queries and keys, capped scores and a bias by distance in place of a rotation; and retention, a
linear attention whose state fades by a constant per head, over rotated queries and keys.  Each result is normed over
the width by a norm of its own, and the branch is half their sum.  The feed-forward is dense (squared relu) or a
mixture of experts whose weights are the softmax over the chosen router outputs; a layer may have none.  A stretch of
layers may run several times in a row with the same weights (``loop``), every pass with a cache of its own and behind a
vector of its own that is added to the stream.  Every size and constant comes from config.json; nothing here knows a
particular model.
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Dict, List, Optional, Tuple

from .llama import ConfigError
from .spec import LayerRun, LayerSpec, ModelSpec, PartSpec

ARCHITECTURE = "Rifizen"
LAYER_TYPES = ("parallel",)
#: config.json names no longest context: angles and states are computed from positions, so the bound is a matter
#: of memory alone; an engine is given its own ``max_model_len`` or pool size
DEFAULT_MAX_POSITIONS = 1 << 20
#: each of a layer's two mixers counts half
PAIR_SCALE = 0.5
#: the slopes of H heads are ``2^(-SLOPE_SPAN (h + 1) / H)``
SLOPE_SPAN = 8.0

_LEFT_KEYS = ("heads", "kv_heads", "dim", "vdim")
_RIGHT_KEYS = ("heads", "dim", "vdim")


def _positive_int(where: str, name: str, v) -> int:
    if not isinstance(v, int) or isinstance(v, bool) or v <= 0:
        raise ConfigError(f"{where}: {name} must be a positive integer, got {v!r}")
    return v


def _count(where: str, name: str, v) -> int:
    if not isinstance(v, int) or isinstance(v, bool) or v < 0:
        raise ConfigError(f"{where}: {name} must be an integer that is not negative, got {v!r}")
    return v


def _number(where: str, name: str, v) -> float:
    if not isinstance(v, (int, float)) or isinstance(v, bool):
        raise ConfigError(f"{where}: {name} must be a number, got {v!r}")
    return float(v)


def _dict(where: str, v, keys) -> Dict[str, Any]:
    if not isinstance(v, dict):
        raise ConfigError(f"{where}: an object is missing")
    lacking = [k for k in keys if k not in v]
    if lacking:
        raise ConfigError(f"{where}: lacks {lacking}")
    return dict(v)


def _left(where: str, d) -> Dict[str, Any]:
    left = _dict(where, d, _LEFT_KEYS + ("scale", "softcap", "mask"))
    for k in _LEFT_KEYS:
        _positive_int(where, k, left[k])
    if left["heads"] % left["kv_heads"]:
        raise ConfigError(f"{where}: {left['heads']} heads are not a multiple of {left['kv_heads']} kv_heads")
    left["scale"] = _number(where, "scale", left["scale"])
    if not _number(where, "softcap", left["softcap"]) > 0:
        raise ConfigError(f"{where}: softcap must be positive, got {left['softcap']!r}")
    mask = _dict(where + ".mask", left["mask"], ("size",))
    left["mask"] = {"size": _positive_int(where + ".mask", "size", mask["size"])}
    return left


def _right(where: str, d) -> Dict[str, Any]:
    right = _dict(where, d, _RIGHT_KEYS + ("decay", "rot"))
    for k in _RIGHT_KEYS:
        _positive_int(where, k, right[k])
    if not isinstance(right["decay"], (list, tuple)) or len(right["decay"]) != right["heads"]:
        raise ConfigError(f"{where}: decay must list a number for each of {right['heads']} heads, got {right['decay']!r}")
    right["decay"] = [_number(where, "decay", v) for v in right["decay"]]
    if not all(0 <= v <= 1 for v in right["decay"]):
        raise ConfigError(f"{where}: decays lie between 0 and 1, got {right['decay']!r}")
    rot = _dict(where + ".rot", right["rot"], ("dims", "base"))
    dims = _count(where + ".rot", "dims", rot["dims"])
    if dims % 2 or dims > right["dim"]:
        raise ConfigError(f"{where}: rot.dims={dims} must be even and at most {right['dim']}")
    if not _number(where + ".rot", "base", rot["base"]) > 0:
        raise ConfigError(f"{where}: rot.base must be positive")
    return right


def _mlp(where: str, mlp) -> Dict[str, Any]:
    mlp = _dict(where, mlp, ("kind",))
    if mlp["kind"] == "dense":
        _positive_int(where, "ff", mlp.get("ff"))
    elif mlp["kind"] == "moe":
        expert = _dict(where + ".expert", mlp.get("expert"), ("ff",))
        router = _dict(where + ".router", mlp.get("router"), ("experts", "top"))
        _positive_int(where + ".expert", "ff", expert["ff"])
        experts = _positive_int(where + ".router", "experts", router["experts"])
        if _positive_int(where + ".router", "top", router["top"]) > experts:
            raise ConfigError(f"{where}.router: {router['top']} choices among {experts} experts")
    else:
        raise ConfigError(f"{where}: kind {mlp['kind']!r} is neither 'dense' nor 'moe'")
    return mlp


def _loop(loop, n_layers: int) -> Optional[Dict[str, int]]:
    if loop is None:
        return None
    loop = _dict("loop", loop, ("start", "stop", "times"))
    start, stop = _count("loop", "start", loop["start"]), _positive_int("loop", "stop", loop["stop"])
    if not start < stop <= n_layers:
        raise ConfigError(f"loop: layers {start} .. {stop - 1} are not a stretch of {n_layers} layers")
    return {"start": start, "stop": stop, "times": _positive_int("loop", "times", loop["times"])}


@dataclass(frozen=True)
class RifizenLayer:
    """One entry of ``layers``: the mixer's sizes and constants and the feed-forward's description (None: none)."""

    type: str
    mixer: Dict[str, Any]
    mlp: Optional[Dict[str, Any]] = None

    def to_dict(self) -> Dict[str, Any]:
        return {"type": self.type, "mixer": self.mixer, "mlp": self.mlp}


@dataclass(frozen=True)
class RifizenConfig:
    vocab: int
    width: int
    layers: Tuple[RifizenLayer, ...]
    norm_eps: float
    loop: Optional[Dict[str, int]] = None
    eos_token_id: Any = None
    architectures: tuple = (ARCHITECTURE,)

    @classmethod
    def from_dict(cls, d: Dict[str, Any]) -> "RifizenConfig":
        missing = [k for k in ("vocab", "width", "layers", "norm") if k not in d]
        if missing:
            raise ConfigError(f"config.json lacks required keys {missing}")
        if not isinstance(d["layers"], list) or not d["layers"]:
            raise ConfigError("config.json: 'layers' must be a list with at least one layer")
        eps = d["norm"].get("eps") if isinstance(d["norm"], dict) else None
        if not isinstance(eps, (int, float)) or not eps > 0:
            raise ConfigError(f"config.json: norm.eps must be positive, got {eps!r}")
        return cls(
            vocab=_positive_int("config", "vocab", d["vocab"]),
            width=_positive_int("config", "width", d["width"]),
            layers=tuple(cls._layer(f"layers[{i}]", entry) for i, entry in enumerate(d["layers"])),
            norm_eps=float(eps),
            loop=_loop(d.get("loop"), len(d["layers"])),
            eos_token_id=d.get("eos_token_id"),
        )

    @staticmethod
    def _layer(where: str, entry) -> RifizenLayer:
        entry = _dict(where, entry, ("type", "mixer"))
        if entry["type"] not in LAYER_TYPES:
            raise ConfigError(f"{where}: type {entry['type']!r} is not one of {list(LAYER_TYPES)}")
        mixer = _dict(where + ".mixer", entry["mixer"], ("left", "right"))
        mixer["left"] = _left(where + ".mixer.left", mixer["left"])
        mixer["right"] = _right(where + ".mixer.right", mixer["right"])
        mlp = entry.get("mlp")
        return RifizenLayer(type=entry["type"], mixer=mixer, mlp=None if mlp is None else _mlp(where + ".mlp", mlp))

    def to_dict(self) -> Dict[str, Any]:
        d: Dict[str, Any] = {
            "architecture": ARCHITECTURE,
            "vocab": self.vocab,
            "width": self.width,
            "norm": {"eps": self.norm_eps},
            "layers": [layer.to_dict() for layer in self.layers],
        }
        if self.loop is not None:
            d["loop"] = dict(self.loop)
        if self.eos_token_id is not None:
            d["eos_token_id"] = self.eos_token_id
        return d


def distance_slopes(heads: int) -> List[float]:
    """What a position of distance costs each head's scores: ``2^(-8 (h + 1) / heads)``."""
    return [2.0 ** (-SLOPE_SPAN * (h + 1) / heads) for h in range(heads)]


def run_order(cfg: RifizenConfig) -> List[LayerRun]:
    """The layers in the order they run: the loop's stretch ``times`` times, step vector t before pass t."""
    n, loop = len(cfg.layers), cfg.loop
    if loop is None:
        return [LayerRun(i) for i in range(n)]
    order = [LayerRun(i) for i in range(loop["start"])]
    for t in range(loop["times"]):
        order += [LayerRun(i, step_vector=t if i == loop["start"] else None) for i in range(loop["start"], loop["stop"])]
    return order + [LayerRun(i) for i in range(loop["stop"], n)]


def _feed_forward_spec(cfg: RifizenConfig, mlp: Dict[str, Any]) -> PartSpec:
    if mlp["kind"] == "dense":
        return PartSpec("dense_relu2", dict(hidden_size=cfg.width, intermediate_size=mlp["ff"]))
    router = mlp["router"]
    return PartSpec("routed", dict(hidden_size=cfg.width, expert_size=mlp["expert"]["ff"], num_experts=router["experts"], top=router["top"],
                                   correction=False, normalize=True, router_bias=True))


def rifizen_model_spec(cfg: RifizenConfig) -> ModelSpec:
    """The model as data: one ``LayerSpec`` per layer, named ``l<i>`` as its tensors are."""

    def norm():
        return PartSpec("rmsnorm", dict(size=cfg.width, eps=cfg.norm_eps, stream_dtype="float32"))

    specs: List[LayerSpec] = []
    for i, layer in enumerate(cfg.layers):
        left, right = layer.mixer["left"], layer.mixer["right"]
        rot = right["rot"]
        parts = {
            "norm1": norm(),
            "left": PartSpec("attention", dict(
                hidden_size=cfg.width, num_heads=left["heads"], num_kv_heads=left["kv_heads"], head_dim=left["dim"], qkv_bias=False,
                softmax_scale=float(left["scale"]), window=left["mask"]["size"], position=PartSpec("none", {}), v_head_dim=left["vdim"],
                qk_norm_eps=cfg.norm_eps, softcap=float(left["softcap"]), slopes=distance_slopes(left["heads"]))),
            "right": PartSpec("retention", dict(
                hidden_size=cfg.width, num_heads=right["heads"], head_dim=right["dim"], v_head_dim=right["vdim"], decay=right["decay"],
                norm_eps=cfg.norm_eps, position=PartSpec("none", {}) if rot["dims"] == 0 else PartSpec("rope", dict(
                    head_dim=right["dim"], rotary_dim=rot["dims"], theta=float(rot["base"]), scaling=None, pairing="half", precise=True)))),
            "left_out": norm(),
            "right_out": norm(),
            "norm1b": norm(),
        }
        block = "sandwich_normed_pair"
        if layer.mlp is not None:
            parts.update(norm2=norm(), mlp=_feed_forward_spec(cfg, layer.mlp), norm2b=norm())
        else:
            block += "_mixer"
        specs.append(LayerSpec(name=f"l{i}", block=block, parts=parts, block_params=dict(left_scale=PAIR_SCALE, right_scale=PAIR_SCALE)))
    spec = ModelSpec(
        architecture=ARCHITECTURE,
        hidden_size=cfg.width,
        vocab_size=cfg.vocab,
        max_positions=DEFAULT_MAX_POSITIONS,
        embedding=PartSpec("embedding", dict(vocab_size=cfg.vocab, hidden_size=cfg.width, stream_dtype="float32")),
        layers=specs,
        order=run_order(cfg),
        final_norm=norm(),
        head=PartSpec("lm_head", dict(vocab_size=cfg.vocab, hidden_size=cfg.width, tied=False)),
        step_vectors=cfg.loop["times"] if cfg.loop is not None else 0,
    )
    spec.validate()
    return spec
