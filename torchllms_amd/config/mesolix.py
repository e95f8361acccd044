"""Typed configuration of the Mesolix decoder, read from ``config.json``, and the model it describes.

A Mesolix model is a list of layers over a 32-bit residual stream that a token's embedding and a learned vector of its
position open; every branch stands behind a norm whose weight is stored around zero.  A layer's mixer is attention through
a latent (keys and values of all heads expanded from one normed latent per token, queries from a normed latent of their
own, no positions, a sink per head), grouped-query attention inside a sliding window with a learned bias by bucketed
distance, both with a gate per channel of the heads' outputs, or a state-space mixer whose heads have one decay each
(Mamba-2).  The feed-forward is a gated one between limits or a mixture of experts chosen by sigmoid scores that multiply
the experts' inputs, beside an optional shared expert; a layer may have none.  A layer may use another layer's tensors
(``weights_of``) with a cache of its own.  Every size and constant comes from config.json; nothing here knows a
particular model.
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Dict, List, Optional, Tuple

from .llama import ConfigError
from .spec import LayerRun, LayerSpec, ModelSpec, PartSpec

ARCHITECTURE = "Mesolix"
LAYER_TYPES = ("latent_attention", "attention", "mamba2")
#: the gated feed-forward's activation is ``g * sigmoid(GATE_SLOPE * g)``
GATE_SLOPE = 1.702
#: rows of a bias by distance in a configuration that names none (one made for random weights); a checkpoint's tensors
#: say how many there are
DEFAULT_DISTANCE_ROWS = 32

_SIZES = {
    "latent_attention": ("heads", "dim", "vdim", "q_rank", "kv_rank"),
    "attention": ("heads", "kv_heads", "dim", "vdim"),
    "mamba2": ("heads", "vdim", "state", "groups", "conv", "norm_groups"),
}


def _positive_int(where: str, name: str, v) -> int:
    if not isinstance(v, int) or isinstance(v, bool) or v <= 0:
        raise ConfigError(f"{where}: {name} must be a positive integer, got {v!r}")
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


def _multiple(where: str, m, many: str, few: str) -> None:
    if m[many] % m[few]:
        raise ConfigError(f"{where}: {m[many]} {many} are not a multiple of {m[few]} {few}")


def _mixer(where: str, kind: str, d) -> Dict[str, Any]:
    m = _dict(where, d, _SIZES[kind])
    for k in _SIZES[kind]:
        _positive_int(where, k, m[k])
    if kind == "mamba2":
        _multiple(where, m, "heads", "groups")
        if (m["heads"] * m["vdim"]) % m["norm_groups"]:
            raise ConfigError(f"{where}: {m['heads']} heads of {m['vdim']} channels do not fall into {m['norm_groups']} norm_groups")
        return m
    m["scale"] = _number(where, "scale", m.get("scale"))
    if kind == "attention":
        _multiple(where, m, "heads", "kv_heads")
        _positive_int(where, "bias_max", m.get("bias_max"))
        if m.get("rel_rows") is not None:  # (a checkpoint's tensors say it, see mesolix_sizes_from_tensors)
            _positive_int(where, "rel_rows", m["rel_rows"])
        mask = _dict(where + ".mask", m.get("mask"), ("size",))
        m["mask"] = {"size": _positive_int(where + ".mask", "size", mask["size"])}
    return m


def _mlp(where: str, mlp) -> Dict[str, Any]:
    mlp = _dict(where, mlp, ("kind",))
    if mlp["kind"] == "dense":
        _positive_int(where, "ff", mlp.get("ff"))
        if not _number(where, "limit", mlp.get("limit")) > 0:
            raise ConfigError(f"{where}: limit must be positive, got {mlp['limit']!r}")
    elif mlp["kind"] == "moe":
        expert = _dict(where + ".expert", mlp.get("expert"), ("ff",))
        router = _dict(where + ".router", mlp.get("router"), ("experts", "top"))
        _positive_int(where + ".expert", "ff", expert["ff"])
        experts = _positive_int(where + ".router", "experts", router["experts"])
        if _positive_int(where + ".router", "top", router["top"]) > experts:
            raise ConfigError(f"{where}.router: {router['top']} choices among {experts} experts")
        if mlp.get("shared") is not None:
            _positive_int(where + ".shared", "ff", _dict(where + ".shared", mlp["shared"], ("ff",))["ff"])
    else:
        raise ConfigError(f"{where}: kind {mlp['kind']!r} is neither 'dense' nor 'moe'")
    return mlp


@dataclass(frozen=True)
class MesolixLayer:
    """One entry of ``layers``: the mixer's type, sizes and constants, the feed-forward's description (None: none), and
    the layer whose tensors it uses (None: its own)."""

    type: str
    mixer: Dict[str, Any]
    mlp: Optional[Dict[str, Any]] = None
    weights_of: Optional[int] = None

    def to_dict(self) -> Dict[str, Any]:
        d = {"type": self.type, "mixer": self.mixer, "mlp": self.mlp}
        if self.weights_of is not None:
            d["weights_of"] = self.weights_of
        return d


@dataclass(frozen=True)
class MesolixConfig:
    vocab: int
    width: int
    max_positions: int
    layers: Tuple[MesolixLayer, ...]
    norm_eps: float
    eos_token_id: Any = None
    architectures: tuple = (ARCHITECTURE,)

    @classmethod
    def from_dict(cls, d: Dict[str, Any]) -> "MesolixConfig":
        missing = [k for k in ("vocab", "width", "max_positions", "layers", "norm") if k not in d]
        if missing:
            raise ConfigError(f"config.json lacks required keys {missing}")
        if not isinstance(d["layers"], list) or not d["layers"]:
            raise ConfigError("config.json: 'layers' must be a list with at least one layer")
        eps = d["norm"].get("eps") if isinstance(d["norm"], dict) else None
        if not isinstance(eps, (int, float)) or not eps > 0:
            raise ConfigError(f"config.json: norm.eps must be positive, got {eps!r}")
        layers = tuple(cls._layer(f"layers[{i}]", entry) for i, entry in enumerate(d["layers"]))
        for i, layer in enumerate(layers):
            if layer.weights_of is None:
                continue
            theirs = layers[weights_owner(layers, i)]
            if (layer.type, layer.mixer, layer.mlp) != (theirs.type, theirs.mixer, theirs.mlp):
                raise ConfigError(f"layers[{i}]: differs from layer {layer.weights_of}, whose tensors it uses")
        return cls(
            vocab=_positive_int("config", "vocab", d["vocab"]),
            width=_positive_int("config", "width", d["width"]),
            max_positions=_positive_int("config", "max_positions", d["max_positions"]),
            layers=layers,
            norm_eps=float(eps),
            eos_token_id=d.get("eos_token_id"),
        )

    @staticmethod
    def _layer(where: str, entry) -> MesolixLayer:
        entry = _dict(where, entry, ("type", "mixer"))
        if entry["type"] not in LAYER_TYPES:
            raise ConfigError(f"{where}: type {entry['type']!r} is not one of {list(LAYER_TYPES)}")
        mlp, source = entry.get("mlp"), entry.get("weights_of")
        if source is not None and (not isinstance(source, int) or isinstance(source, bool) or source < 0):
            raise ConfigError(f"{where}: weights_of={source!r} names no layer")
        return MesolixLayer(type=entry["type"], mixer=_mixer(where + ".mixer", entry["type"], entry["mixer"]),
                            mlp=None if mlp is None else _mlp(where + ".mlp", mlp), weights_of=source)

    def to_dict(self) -> Dict[str, Any]:
        d: Dict[str, Any] = {
            "architecture": ARCHITECTURE,
            "vocab": self.vocab,
            "width": self.width,
            "max_positions": self.max_positions,
            "norm": {"eps": self.norm_eps},
            "layers": [layer.to_dict() for layer in self.layers],
        }
        if self.eos_token_id is not None:
            d["eos_token_id"] = self.eos_token_id
        return d


def weights_owner(layers, i: int) -> int:
    """The layer whose tensors layer ``i`` uses in the end (itself without ``weights_of``)."""
    seen = []
    while layers[i].weights_of is not None:
        if i in seen or not layers[i].weights_of < len(layers):
            raise ConfigError(f"layers[{i}]: weights_of={layers[i].weights_of} leads to no layer with tensors of its own")
        seen.append(i)
        i = layers[i].weights_of
    return i


def _mixer_spec(cfg: MesolixConfig, layer: MesolixLayer) -> PartSpec:
    m = layer.mixer
    if layer.type == "latent_attention":
        return PartSpec("latent_attention", dict(
            hidden_size=cfg.width, num_heads=m["heads"], head_dim=m["dim"], rot_dim=0, v_head_dim=m["vdim"], q_rank=m["q_rank"],
            kv_rank=m["kv_rank"], softmax_scale=m["scale"], norm_eps=cfg.norm_eps, position=PartSpec("none", {}), out_gate="channel",
            sinks=True))
    if layer.type == "attention":
        return PartSpec("attention", dict(
            hidden_size=cfg.width, num_heads=m["heads"], num_kv_heads=m["kv_heads"], head_dim=m["dim"], qkv_bias=False,
            softmax_scale=m["scale"], window=m["mask"]["size"], position=PartSpec("none", {}), v_head_dim=m["vdim"], out_gate="channel",
            distance_rows=m.get("rel_rows") or DEFAULT_DISTANCE_ROWS, distance_most=m["bias_max"]))
    return PartSpec("state_space_dual", dict(
        hidden_size=cfg.width, num_heads=m["heads"], v_head_dim=m["vdim"], state_size=m["state"], num_groups=m["groups"],
        conv_taps=m["conv"], norm_groups=m["norm_groups"], norm_eps=cfg.norm_eps))


def _feed_forward_spec(cfg: MesolixConfig, mlp: Dict[str, Any]) -> PartSpec:
    if mlp["kind"] == "dense":
        return PartSpec("swiglu", dict(hidden_size=cfg.width, intermediate_size=mlp["ff"], activation="sigmoid_limited",
                                       limit=float(mlp["limit"]), slope=GATE_SLOPE))
    router = mlp["router"]
    return PartSpec("routed", dict(
        hidden_size=cfg.width, expert_size=mlp["expert"]["ff"], num_experts=router["experts"], top=router["top"],
        shared_size=(mlp.get("shared") or {}).get("ff", 0), shared_gate=False, correction=False, scores="sigmoid", weigh="input"))


def mesolix_sizes_from_tensors(cfg: MesolixConfig, shapes: Dict[str, tuple]) -> MesolixConfig:
    """The configuration with the size that config.json leaves to the tensors: of every windowed attention the rows of
    its table of distances, ``l<i>.mix.rel`` [rows, heads]."""
    layers = []
    for i, layer in enumerate(cfg.layers):
        shape = shapes.get(f"l{weights_owner(cfg.layers, i)}.mix.rel")
        if layer.type == "attention" and shape is not None and len(shape) == 2:
            layer = MesolixLayer(type=layer.type, mixer=dict(layer.mixer, rel_rows=int(shape[0])), mlp=layer.mlp, weights_of=layer.weights_of)
        layers.append(layer)
    return MesolixConfig(vocab=cfg.vocab, width=cfg.width, max_positions=cfg.max_positions, layers=tuple(layers), norm_eps=cfg.norm_eps,
                         eos_token_id=cfg.eos_token_id)


def mesolix_model_spec(cfg: MesolixConfig) -> ModelSpec:
    """The model as data: one ``LayerSpec`` per layer with tensors of its own, named ``l<i>`` as they are; a layer that
    uses another's is one more run of that layer."""

    def norm():
        return PartSpec("rmsnorm", dict(size=cfg.width, eps=cfg.norm_eps, stream_dtype="float32", offset=1.0))

    specs: List[LayerSpec] = []
    at: Dict[int, int] = {}  # layer -> its place among the specs
    for i, layer in enumerate(cfg.layers):
        if layer.weights_of is not None:
            continue
        parts = {"mixer_norm": norm(), "mixer": _mixer_spec(cfg, layer)}
        block = "pre_norm"
        if layer.mlp is not None:
            parts.update(ffn_norm=norm(), ffn=_feed_forward_spec(cfg, layer.mlp))
        else:
            block += "_mixer"
        at[i] = len(specs)
        specs.append(LayerSpec(name=f"l{i}", block=block, parts=parts))
    spec = ModelSpec(
        architecture=ARCHITECTURE,
        hidden_size=cfg.width,
        vocab_size=cfg.vocab,
        max_positions=cfg.max_positions,
        embedding=PartSpec("embedding", dict(vocab_size=cfg.vocab, hidden_size=cfg.width, stream_dtype="float32",
                                             positions=cfg.max_positions)),
        layers=specs,
        order=[LayerRun(at[weights_owner(cfg.layers, i)]) for i in range(len(cfg.layers))],
        final_norm=norm(),
        head=PartSpec("lm_head", dict(vocab_size=cfg.vocab, hidden_size=cfg.width, tied=False)),
    )
    spec.validate()
    return spec
