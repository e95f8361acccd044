"""Small Mesolix configurations for the tests, and model folders with random weights made from them.

The configurations differ from each other in every size and constant, and in what a single model may happen to make
equal or one: heads and groups (one of each among them), sizes of keys, values and latents, windows (a single position
among them), tables of distances (odd numbers of rows, ends before and behind the window), taps (one among them), parts
of the norm, limits, one choice of experts, several and all, with and without a shared expert or any feed-forward, layers
that use the tensors of one before or behind them."""

from __future__ import annotations

from pathlib import Path
from typing import Dict, Optional

import torch


def latent(heads, dim, vdim, q_rank, kv_rank, spread=1.0):
    """``spread``: a factor on the scores (1: of the order of ``make_folder``'s weights, a few units)."""
    return "latent_attention", {"heads": heads, "dim": dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank, "scale": spread / dim ** 0.5}


def windowed(heads, kv_heads, dim, vdim, size, rows=8, most=20, spread=3.0):
    return "attention", {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": spread / dim ** 0.5, "bias_max": most,
                         "rel_rows": rows, "mask": {"size": size}}


def mamba(heads, vdim, state, groups=1, conv=4, norm_groups=1):
    return "mamba2", {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": conv, "norm_groups": norm_groups}


def dense(ff, limit=0.6):
    return {"kind": "dense", "ff": ff, "limit": limit}


def moe(ff, experts, top, shared=None):
    d = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if shared:
        d["shared"] = {"ff": shared}
    return d


def layer(mixer, mlp=None, weights_of: Optional[int] = None):
    d = {"type": mixer[0], "mixer": mixer[1], "mlp": mlp}
    if weights_of is not None:
        d["weights_of"] = weights_of
    return d


def again(layers, i):
    """A layer that uses the tensors of layer ``i`` of ``layers``."""
    return dict(layers[i], weights_of=i)


def model(vocab, width, eps, layers, max_positions=1024):
    return {"architecture": "Mesolix", "vocab": vocab, "width": width, "max_positions": max_positions, "norm": {"eps": eps}, "layers": layers}


_A = [
    layer(latent(4, 16, 24, 40, 24), dense(112)),
    layer(mamba(6, 20, 12, groups=3, conv=4, norm_groups=2), moe(24, 5, 2, shared=40)),
    layer(windowed(4, 2, 16, 24, 24, rows=12, most=20), None),
]
CONFIG_A = model(131, 64, 1e-5, _A + [again(_A, 0), again(_A, 2), again(_A, 1)], max_positions=300)
_B = [
    layer(windowed(8, 2, 32, 32, 48, rows=32, most=40), moe(40, 6, 1)),
    layer(latent(8, 32, 32, 96, 64), None),
    layer(mamba(4, 64, 64, conv=2), dense(72, limit=1.1)),
    layer(windowed(6, 1, 64, 64, 33, rows=9, most=200), moe(16, 3, 3, shared=24)),
    layer(latent(3, 20, 12, 28, 256), dense(40, limit=0.3)),
]
CONFIG_B = model(77, 96, 1e-6, _B + [again(_B, 1)])
_C = [
    layer(mamba(3, 128, 128, conv=1, norm_groups=3), moe(56, 10, 3)),
    layer(latent(20, 40, 72, 56, 128), dense(200, limit=0.5)),
    layer(windowed(1, 1, 40, 80, 100, rows=6, most=64), None),
    layer(windowed(3, 3, 128, 128, 1, rows=2, most=5), moe(32, 4, 2, shared=8)),
]
CONFIG_C = model(200, 128, 1e-4, [dict(_C[2], weights_of=3)] + [_C[0], _C[1], _C[2], _C[3], again([None, _C[0]], 1)])
CONFIGS = {"A": CONFIG_A, "B": CONFIG_B, "C": CONFIG_C}
PAGE_SIZE = {"A": 8, "B": 16, "C": 4}

#: a mixer too small to matter beside the feed-forward that a test is about
TINY = windowed(1, 1, 8, 8, 5, rows=4, most=6)


def single_layer(entry: dict, width: int = 64, vocab: int = 61) -> dict:
    """A model of one layer, for a mechanism alone."""
    return model(vocab, width, 1e-5, [entry])


def make_folder(path, cfg_dict: dict, seed: int = 0, dtype=torch.bfloat16, decisive_router: bool = False) -> Path:
    """A model folder written by the package's random-weights mode, then made harder on faults: projections are scaled up
    so that scores are sharp and gates, states and experts depend on their inputs, sinks and distances weigh as much as
    scores, norms get weights with a spread, step sizes and decays reach from heads that forget within a few tokens to heads that
    keep hundreds.  ``decisive_router``: one channel of the stream is the token's sign (nothing else writes to it) and the
    routers listen to it before all else, their experts' answers standing well apart, so that rounding cannot change a
    choice (what a bfloat16 run is compared on) while tokens of both signs choose differently; without it the choice changes
    from token to token.  The table of distances keeps its number of rows to the tensors: config.json does not name it."""
    import json

    from safetensors.torch import save_file

    from torchllms_amd.config.mesolix import MesolixConfig
    from torchllms_amd.weights import write_model_folder

    folder = write_model_folder(path, MesolixConfig.from_dict(cfg_dict), seed=seed, dtype=dtype)
    cfg, tensors = read_folder(folder)
    for entry in cfg["layers"]:
        entry["mixer"].pop("rel_rows", None)
    (folder / "config.json").write_text(json.dumps(cfg))
    gen = torch.Generator().manual_seed(seed + 1)

    def randn(t):
        return torch.randn(t.shape, generator=gen)

    for name in sorted(tensors):
        t = tensors[name].float()
        leaf = name.split(".", 1)[-1] if name[0] == "l" and name[1].isdigit() else name
        if leaf in ("norm1", "norm2", "final.norm"):
            t = 0.3 * randn(t)
        elif leaf in ("mix.norm", "mix.dq.norm", "mix.dkv.norm"):
            t = 1.0 + 0.3 * randn(t)
        elif name == "embed":
            t = t * 40.0
        elif name == "pos":
            t = t * 20.0
        elif leaf == "mix.sink":
            t = 1.0 + randn(t)
        elif leaf == "mix.rel":
            t = 1.5 * randn(t)
        elif leaf == "mix.A_log":
            t = torch.empty(t.shape).uniform_(-3.0, 1.0, generator=gen)
        elif leaf == "mix.dt_bias":
            t = torch.empty(t.shape).uniform_(-4.0, 0.0, generator=gen)
        elif leaf in ("mix.D", "mix.conv"):
            t = t if leaf == "mix.conv" else 0.5 + 0.5 * randn(t)
        elif leaf == "mix.conv.b":
            t = 0.3 * randn(t)
        elif leaf in ("mix.uq", "mix.uk"):
            t = t * 15.0
        elif leaf.startswith("mix."):
            t = t * 5.0
        elif leaf == "mlp.router":
            t = randn(t) / t.shape[1] ** 0.5 * (0.1 if decisive_router else 2.0)
        elif leaf.startswith("mlp."):
            t = t * 4.0
        elif name == "head":
            t = t * 5.0
        tensors[name] = t
    if decisive_router:
        signs = torch.where(torch.arange(cfg["vocab"]) % 2 == 0, 1.0, -1.0)
        tensors["embed"][:, 1] = 2.5 * signs
        tensors["pos"][:, 1] = 0.0
        for name, t in tensors.items():
            if name.endswith((".mix.o", ".down")):
                t[1] = 0.0
            elif name.endswith(".norm2"):
                t[1] = 0.0
            elif name.endswith(".router"):
                order = torch.randperm(t.shape[0], generator=gen).float()
                apart = min(0.7, 6.0 / t.shape[0])
                t *= min(1.0, apart)
                t[:, 1] = apart * (order - order.mean())
    tensors = {k: v.to(dtype).contiguous() for k, v in tensors.items()}
    save_file(tensors, str(folder / "model.safetensors"), metadata={"format": "pt"})
    return folder


def read_folder(folder) -> (dict, Dict[str, torch.Tensor]):
    """config.json as a dict and the tensors by their checkpoint names, read with safetensors
    directly (not through the package's loader)."""
    import json

    from safetensors import safe_open

    folder = Path(folder)
    with open(folder / "config.json") as f:
        cfg = json.load(f)
    tensors = {}
    with safe_open(str(folder / "model.safetensors"), framework="pt", device="cpu") as f:
        for name in f.keys():
            tensors[name] = f.get_tensor(name)
    return cfg, tensors
