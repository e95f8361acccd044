"""Rifizen without a GPU: the configuration and what it refuses, the order of execution with its loop, tensor names there
and back, what the cache keeps, and the plain implementation pinned by hand-worked cases and by what taking a
mechanism out does to the logits of the test models."""

import json
import math

import pytest
import torch

from torchllms_amd.cache.manager import group_layers
from torchllms_amd.config import ConfigError, load_config
from torchllms_amd.config.rifizen import RifizenConfig, distance_slopes, rifizen_model_spec, run_order
from torchllms_amd.config.spec import LayerRun
from torchllms_amd.parts.model import Model

from . import rifizen_models as models
from .helpers import random_tokens
from .plain import rifizen as plain


@pytest.mark.parametrize("name", sorted(models.CONFIGS))
def test_configuration_there_and_back(name):
    cfg = RifizenConfig.from_dict(models.CONFIGS[name])
    again = RifizenConfig.from_dict(json.loads(json.dumps(cfg.to_dict())))
    assert again == cfg
    spec = rifizen_model_spec(cfg)
    assert len(spec.layers) == len(cfg.layers) and spec.vocab_size == cfg.vocab
    # the order is the plain implementation's
    assert [(r.layer, r.step_vector) for r in spec.order] == plain.run_order(models.CONFIGS[name])


def _with(cfg, path, value):
    d = json.loads(json.dumps(cfg))
    at = d
    for key in path[:-1]:
        at = at[key]
    if value is None:
        at.pop(path[-1], None)
    else:
        at[path[-1]] = value
    return d


@pytest.mark.parametrize("path,value", [
    (("vocab",), None), (("width",), 0), (("layers",), []), (("norm",), {"eps": 0}), (("layers", 0, "type"), "attention"),
    (("layers", 0, "mixer", "left"), None), (("layers", 0, "mixer", "right"), None), (("layers", 0, "mixer", "left", "heads"), 3),
    (("layers", 0, "mixer", "left", "softcap"), 0.0), (("layers", 0, "mixer", "left", "softcap"), None),
    (("layers", 0, "mixer", "left", "mask"), {}), (("layers", 0, "mixer", "left", "mask", "size"), 0),
    (("layers", 0, "mixer", "left", "scale"), "x"), (("layers", 0, "mixer", "right", "decay"), [0.9]),
    (("layers", 0, "mixer", "right", "decay"), [0.9, 1.5]), (("layers", 0, "mixer", "right", "rot", "dims"), 26),
    (("layers", 0, "mixer", "right", "rot", "dims"), 7), (("layers", 0, "mixer", "right", "rot", "base"), -1.0),
    (("layers", 0, "mlp", "kind"), "glu"), (("layers", 0, "mlp", "ff"), None), (("layers", 1, "mlp", "router", "top"), 6),
    (("layers", 1, "mlp", "expert"), None), (("loop", "stop"), 4), (("loop", "start"), 2), (("loop", "times"), 0), (("loop", "times"), None),
])
def test_configuration_refuses(path, value):
    with pytest.raises(ConfigError):
        RifizenConfig.from_dict(_with(models.CONFIG_A, path, value))


def test_loops():
    """The stretch runs its times in a row, every pass behind its own vector, each run with cache entries of its own;
    without a loop there is no such tensor."""
    two = models.CONFIG_B["layers"]

    def order(loop):
        return run_order(RifizenConfig.from_dict(dict(models.CONFIG_B, loop=loop)))

    assert order({"start": 1, "stop": 3, "times": 2}) == [LayerRun(0), LayerRun(1, step_vector=0), LayerRun(2), LayerRun(1, step_vector=1), LayerRun(2), LayerRun(3)]
    assert order({"start": 3, "stop": 4, "times": 3}) == [LayerRun(0), LayerRun(1), LayerRun(2)] + [LayerRun(3, step_vector=t) for t in range(3)]
    assert order({"start": 0, "stop": 4, "times": 1}) == [LayerRun(0, step_vector=0), LayerRun(1), LayerRun(2), LayerRun(3)]
    assert order(None) == [LayerRun(i) for i in range(len(two))]
    assert "loop.step" not in Model(rifizen_model_spec(RifizenConfig.from_dict(models.CONFIG_B))).param_specs()
    model = Model(rifizen_model_spec(RifizenConfig.from_dict(models.CONFIG_A)))
    assert model.param_specs()["loop.step"].shape == (3, 64)
    assert {key for key, _ in model.cache_needs()} == {(run, side) for run in range(7) for side in ("left", "right")}
    spec = rifizen_model_spec(RifizenConfig.from_dict(models.CONFIG_A))
    bad = type(spec)(**{**vars(spec), "step_vectors": 2})
    with pytest.raises(ValueError, match="step vector"):
        bad.validate()


def test_folder_there_and_back(tmp_path):
    """``write_model_folder`` names every tensor as a checkpoint does and the loader finds every one again."""
    from safetensors.torch import load_file

    from torchllms_amd.weights import load_weights, write_model_folder

    cfg = RifizenConfig.from_dict(models.CONFIG_A)
    folder = write_model_folder(tmp_path / "m", cfg, seed=1, dtype=torch.float32)
    names = set(load_file(str(folder / "model.safetensors")))
    assert {"embed", "head", "final.norm", "loop.step", "l0.norm1", "l0.norm1b", "l0.norm2", "l0.norm2b", "l0.mlp.up", "l0.mlp.down",
            "l1.mlp.router", "l1.mlp.router.b", "l1.mlp.e4.gate", "l1.mix.left.q", "l1.mix.left.out", "l2.mix.right.g", "l2.mix.right.out"} <= names
    assert not {"l2.norm2", "l2.mlp.up", "l0.mlp.router", "l0.mlp.gate", "l0.mix.left.g"} & names
    arch, loaded = load_config(folder)
    assert arch.name == "Rifizen" and loaded == cfg
    model = Model(arch.model_spec(loaded))
    tensors = load_weights(folder, arch.weight_rules(loaded), model.param_specs(), torch.float32, device="cpu")
    assert set(tensors) == set(model.param_specs())
    model.bind(tensors)


def test_what_the_cache_keeps():
    """Pages for the attention of every run (groups by sizes and window), a 32-bit state row for its retention."""
    model = Model(rifizen_model_spec(RifizenConfig.from_dict(models.CONFIG_C)))
    needs = dict(model.cache_needs())
    assert (needs[(0, "left")].num_kv_heads, needs[(0, "left")].head_dim, needs[(0, "left")].v_head_dim, needs[(0, "left")].window) == (1, 128, None, 29)
    assert (needs[(2, "left")].head_dim, needs[(2, "left")].v_head_dim, needs[(2, "left")].window) == (40, 80, 100)
    assert needs[(1, "right")].shape == (128 * 128,) and needs[(1, "right")].dtype == "float32"
    groups, states = group_layers(model.cache_needs())
    assert sorted(g.window for g in groups) == [29, 45, 100] and sum(len(s.run_ids) for s in states) == 5
    # parts refuse what no kernel takes
    wide = json.loads(json.dumps(models.CONFIG_C))
    wide["layers"][0]["mixer"]["right"]["dim"] = 300
    with pytest.raises(ValueError, match="keys of 300 channels"):
        Model(rifizen_model_spec(RifizenConfig.from_dict(wide))).check_sizes(torch.float32)


# ----------------------------------------------------------------------------- the plain implementation pinned
def test_plain_scores_by_hand():
    """One pair of tokens: cap first, then the distance at the head's slope; slopes of a number of heads that is no power
    of two; the mask at its edge."""
    q = torch.tensor([[[3.0], [1.0]], [[2.0], [-4.0]]], dtype=torch.float64)  # two tokens, two heads of one channel
    k = torch.tensor([[[1.0], [1.0]], [[5.0], [0.5]]], dtype=torch.float64)
    s = plain.biased_scores(q, k, 0.5, 2.0)
    assert plain.slopes(2).tolist() == [2.0 ** -4, 2.0 ** -8]
    assert float(s[0, 1, 0]) == pytest.approx(2.0 * math.tanh(2.0 * 1.0 * 0.5 / 2.0) - 2.0 ** -4)
    assert float(s[1, 1, 0]) == pytest.approx(2.0 * math.tanh(-4.0 * 1.0 * 0.5 / 2.0) - 2.0 ** -8)
    assert float(s[0, 1, 1]) == pytest.approx(2.0 * math.tanh(2.0 * 5.0 * 0.5 / 2.0))
    assert plain.slopes(3).tolist() == pytest.approx([2 ** (-8 / 3), 2 ** (-16 / 3), 2 ** -8])
    assert distance_slopes(3) == pytest.approx(plain.slopes(3).tolist(), rel=1e-15)
    assert plain.visible(4, 2).int().tolist() == [[1, 0, 0, 0], [1, 1, 0, 0], [0, 1, 1, 0], [0, 0, 1, 1]]


def test_plain_retention_is_its_unrolled_sum():
    """``o_t = sum_(s <= t) decay^(t - s) (q_t . k_s) v_s``; a state that forgets at once keeps the token alone."""
    gen = torch.Generator().manual_seed(2)
    q, k, v = (torch.randn((9, 2, d), generator=gen, dtype=torch.float64) for d in (4, 4, 3))
    decay = [0.0, 0.8]
    got = plain.retention_states(q, k, v, decay)
    for t in range(9):
        for h in range(2):
            want = sum(decay[h] ** (t - s) * float((q[t, h] * k[s, h]).sum()) * v[s, h] for s in range(t + 1))
            assert torch.allclose(got[t, h], want, atol=1e-12)


def test_plain_rotation_is_relative_and_pairs_halves():
    x, y = torch.randn(1, 1, 8, dtype=torch.float64), torch.randn(1, 1, 8, dtype=torch.float64)
    at = lambda z, p: plain.rotate_half(z, torch.tensor([p]), 6, 100.0)  # noqa: E731
    assert torch.equal(at(x, 5)[..., 6:], x[..., 6:])
    assert torch.allclose((at(x, 9) * at(y, 4)).sum(), (at(x, 105) * at(y, 100)).sum(), atol=1e-10)
    c, s = math.cos(2.0 * 100.0 ** (-2 / 6)), math.sin(2.0 * 100.0 ** (-2 / 6))
    assert float(at(x, 2)[0, 0, 1]) == pytest.approx(float(x[0, 0, 1]) * c - float(x[0, 0, 4]) * s)
    assert float(at(x, 2)[0, 0, 4]) == pytest.approx(float(x[0, 0, 4]) * c + float(x[0, 0, 1]) * s)


def test_plain_router_weights_are_the_softmax_of_the_chosen():
    ids, w = plain.routed_choice(torch.tensor([[0.5, 3.0, -1.0, 2.0]], dtype=torch.float64), 2)
    assert ids.tolist() == [[1, 3]]
    assert w[0].tolist() == pytest.approx([1 / (1 + math.exp(-1.0)), 1 / (1 + math.exp(1.0))])


def _distance(a, b):
    d = a - b
    d = d - d.mean(-1, keepdim=True)
    return float((d.pow(2).mean(-1).sqrt() / b.pow(2).mean().sqrt()).max())


def test_every_mechanism_shows_in_the_logits(tmp_path, monkeypatch):
    """The test models make a fault visible: what taking a mechanism out, or moving an edge by one token, does to the
    logits is a hundred times what the 32-bit comparisons allow (3e-5)."""
    cfg, w = models.read_folder(models.make_folder(tmp_path / "m", models.CONFIG_A, seed=3))
    tokens = random_tokens(80, cfg["vocab"], 1)
    truth = plain.forward(cfg, w, tokens)

    def moved(cfg2=cfg, w2=w, toks=tokens):
        return _distance(plain.forward(cfg2, w2, toks), truth)

    def changed(fn):
        d = json.loads(json.dumps(cfg))
        fn(d)
        return d

    for i in range(3):
        assert moved(changed(lambda d: d["layers"][i]["mixer"]["left"]["mask"].update(size=d["layers"][i]["mixer"]["left"]["mask"]["size"] + 1))) > 3e-3
        assert moved(changed(lambda d: d["layers"][i]["mixer"]["left"].update(softcap=1e9))) > 3e-3
        assert moved(changed(lambda d: d["layers"][i]["mixer"]["right"].update(decay=[x * 0.99 for x in d["layers"][i]["mixer"]["right"]["decay"]]))) > 3e-3
    assert moved(changed(lambda d: d["layers"][0]["mixer"]["right"]["rot"].update(dims=22))) > 3e-3
    assert moved(changed(lambda d: d["layers"][1]["mixer"]["right"]["rot"].update(base=510.0))) > 3e-3
    assert moved(changed(lambda d: d["loop"].update(times=2))) > 3e-3
    assert moved(changed(lambda d: d["layers"][1]["mlp"]["router"].update(top=1))) > 3e-3
    assert moved(w2=dict(w, **{"loop.step": w["loop.step"][[0, 2, 1]]})) > 3e-3
    for name in ("l1.mlp.router.b", "l0.mix.left.out", "l2.mix.right.out", "l0.norm1b", "l1.norm2b"):
        assert moved(w2=dict(w, **{name: torch.ones_like(w[name])})) > 3e-3, name
    assert moved(toks=[(tokens[0] + 1) % cfg["vocab"]] + tokens[1:]) > 3e-3
    # the first token still shows in the last position's logits (retention carries it past every window)
    other = plain.forward(cfg, w, [(tokens[0] + 1) % cfg["vocab"]] + tokens[1:])
    assert _distance(other[-1:], truth[-1:]) > 3e-3
    monkeypatch.setattr(plain, "slopes", lambda heads, dtype=torch.float64: torch.zeros(heads, dtype=dtype))
    assert moved() > 3e-3
