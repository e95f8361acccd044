"""Small Rifizen configurations for the tests, and model folders with random weights made from them.

The configurations differ from each other in every size and constant, and in what a single model may happen to make
equal or one: heads and kv heads (one of each among them), sizes of keys and values on both sides, rotated channels
(all, some, none), windows (a single position among them), caps, decays up to 1 (a head that forgets at once is its
token's value times the sign of q . k but for the norm's eps: rounding shows there, so such heads are tested alone),
dense, routed and no feed-forward, one choice, several and all, a loop from the first layer, to the last, and none."""

from __future__ import annotations

from pathlib import Path
from typing import Dict

import torch


def left(heads, kv_heads, dim, vdim, size, spread=3.0, softcap=8.0):
    """``spread``: the standard deviation of the scores of random unit-RMS queries and keys before the cap."""
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": spread / dim ** 0.5, "softcap": softcap,
            "mask": {"size": size}}


def right(heads, dim, vdim, decay, dims=None, base=10000.0):
    return {"heads": heads, "dim": dim, "vdim": vdim, "decay": list(decay), "rot": {"dims": dim if dims is None else dims, "base": base}}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(ff, experts, top):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}


def layer(lf, rt, mlp=None):
    return {"type": "parallel", "mixer": {"left": lf, "right": rt}, "mlp": mlp}


def model(vocab, width, eps, layers, loop=None):
    d = {"architecture": "Rifizen", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}
    if loop is not None:
        d["loop"] = {"start": loop[0], "stop": loop[1], "times": loop[2]}
    return d


CONFIG_A = model(131, 64, 1e-5, [
    layer(left(4, 2, 16, 24, 24), right(2, 24, 16, [0.9, 0.998]), dense(112)),
    layer(left(2, 1, 24, 16, 33, softcap=4.0), right(3, 16, 40, [0.5, 0.97, 0.9995], dims=8, base=500.0), moe(24, 5, 2)),
    layer(left(6, 3, 8, 12, 17, spread=2.0), right(1, 12, 20, [0.99], dims=0), None),
], loop=(0, 2, 3))
CONFIG_B = model(77, 96, 1e-6, [
    layer(left(6, 1, 64, 64, 48, softcap=30.0), right(3, 32, 48, [0.8, 0.99, 0.9999], dims=16, base=1e6), moe(40, 6, 1)),
    layer(left(3, 3, 32, 16, 40), right(2, 64, 32, [0.97, 0.5]), None),
    layer(left(8, 2, 32, 32, 70, spread=4.0, softcap=12.0), right(4, 16, 16, [0.95, 0.98, 0.99, 0.995], base=50.0), dense(72)),
    layer(left(2, 2, 16, 16, 1), right(2, 8, 64, [1.0, 0.3]), moe(16, 3, 3)),
])
CONFIG_C = model(200, 128, 1e-4, [
    layer(left(2, 1, 128, 128, 29), right(2, 40, 72, [0.999, 0.93], dims=24), moe(56, 10, 3)),
    layer(left(8, 4, 64, 64, 45, softcap=5.0), right(1, 128, 128, [0.9985], dims=64, base=1000.0), moe(32, 4, 2)),
    layer(left(1, 1, 40, 80, 100), right(4, 64, 24, [0.6, 0.9, 0.99, 0.999]), dense(200)),
], loop=(1, 3, 2))
CONFIGS = {"A": CONFIG_A, "B": CONFIG_B, "C": CONFIG_C}
PAGE_SIZE = {"A": 8, "B": 16, "C": 4}

#: sides of a layer too small to matter beside the side that a test is about
TINY_LEFT, TINY_RIGHT = left(1, 1, 8, 8, 5), right(1, 8, 8, [0.9])


def single_layer(entry: dict, width: int = 64, vocab: int = 61, loop=None) -> dict:
    """A model of one layer, for a mechanism alone."""
    return model(vocab, width, 1e-5, [entry], loop=loop)


def make_folder(path, cfg_dict: dict, seed: int = 0, dtype=torch.bfloat16, decisive_router: bool = False) -> Path:
    """A model folder written by the package's random-weights mode, then made harder on faults: projections are scaled up
    so that gates, retention and experts depend on their inputs (the softmax side's queries and keys are normed, so
    the configuration's scale decides how sharp its scores are), norms get weights with a spread, the loop's vectors
    are as large as what they are added to.  ``decisive_router``: the routers' biases stand two apart, so that rounding
    cannot change a choice (what a bfloat16 run is compared on); without it the choice changes from token to token."""
    from safetensors.torch import save_file

    from torchllms_amd.config.rifizen import RifizenConfig
    from torchllms_amd.weights import write_model_folder

    folder = write_model_folder(path, RifizenConfig.from_dict(cfg_dict), seed=seed, dtype=dtype)
    _, tensors = read_folder(folder)
    gen = torch.Generator().manual_seed(seed + 1)
    for name in list(tensors):
        t = tensors[name].float()
        leaf = name.split(".", 1)[-1] if name[0] == "l" and name[1].isdigit() else name
        if leaf in ("norm1", "norm1b", "norm2", "norm2b", "mix.left.out", "mix.right.out", "final.norm"):
            t = 1.0 + 0.3 * torch.randn(t.shape, generator=gen)
        elif name in ("embed", "loop.step"):
            t = t * 40.0
        elif leaf.startswith("mix."):
            t = t * 5.0
        elif leaf == "mlp.router":
            t = (0.05 if decisive_router else 1.0) * torch.randn(t.shape, generator=gen) / t.shape[1] ** 0.5 * 2.0
        elif leaf == "mlp.router.b":
            t = 2.0 * torch.randperm(t.shape[0], generator=gen).float() if decisive_router else 0.7 * torch.randn(t.shape, generator=gen)
        elif leaf.startswith("mlp."):
            t = t * 3.0
        elif name == "head":
            t = t * 5.0
        tensors[name] = t
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
