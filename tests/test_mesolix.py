"""Mesolix without a GPU: the configuration and what it refuses, the order of execution with layers that use another's
tensors, tensor names there and back, what the cache keeps, the buckets of distances, and the plain implementation
pinned by hand-worked cases and by what taking a mechanism out does to the logits of the test models."""

import json
import math
from fractions import Fraction

import pytest
import torch

from torchllms_amd.cache.manager import group_layers
from torchllms_amd.config import ConfigError, load_config
from torchllms_amd.config.mesolix import MesolixConfig, mesolix_model_spec, weights_owner
from torchllms_amd.parts.model import Model
from torchllms_amd.parts.positions import distance_bucket_starts, distance_table

from . import mesolix_models as models
from .helpers import random_tokens
from .plain import mesolix as plain


@pytest.mark.parametrize("name", sorted(models.CONFIGS))
def test_configuration_there_and_back(name):
    cfg = MesolixConfig.from_dict(models.CONFIGS[name])
    again = MesolixConfig.from_dict(json.loads(json.dumps(cfg.to_dict())))
    assert again == cfg
    spec = mesolix_model_spec(cfg)
    assert len(spec.order) == len(cfg.layers) and spec.vocab_size == cfg.vocab and spec.max_positions == cfg.max_positions
    # every run is a run of the layer whose tensors the plain implementation would take
    assert [spec.layers[r.layer].name for r in spec.order] == [f"l{plain.owner(models.CONFIGS[name], i)}" for i in range(len(cfg.layers))]


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


_PLAIN_LAYERS = dict(models.CONFIG_A, layers=models.CONFIG_A["layers"][:3])  # (none that uses another's tensors)


@pytest.mark.parametrize("path,value", [
    (("vocab",), None), (("width",), 0), (("max_positions",), None), (("layers",), []), (("norm",), {"eps": 0}), (("layers", 0, "type"), "mamba1"),
    (("layers", 0, "mixer"), None), (("layers", 0, "mixer", "q_rank"), None), (("layers", 0, "mixer", "kv_rank"), -1), (("layers", 0, "mixer", "scale"), "x"),
    (("layers", 0, "mlp", "limit"), 0), (("layers", 0, "mlp", "limit"), None), (("layers", 0, "mlp", "kind"), "glu"), (("layers", 0, "mlp", "ff"), None),
    (("layers", 1, "mixer", "groups"), 4), (("layers", 1, "mixer", "norm_groups"), 7), (("layers", 1, "mixer", "conv"), 0), (("layers", 1, "mixer", "state"), None),
    (("layers", 1, "mlp", "router", "top"), 6), (("layers", 1, "mlp", "expert"), None), (("layers", 1, "mlp", "shared"), {}),
    (("layers", 2, "mixer", "kv_heads"), 3), (("layers", 2, "mixer", "bias_max"), None), (("layers", 2, "mixer", "mask"), {}), (("layers", 2, "mixer", "mask", "size"), 0),
    (("layers", 2, "mixer", "rel_rows"), -3), (("layers", 2, "weights_of"), 0), (("layers", 2, "weights_of"), 2), (("layers", 2, "weights_of"), 9),
    (("layers", 2, "weights_of"), True),
])
def test_configuration_refuses(path, value):
    MesolixConfig.from_dict(_PLAIN_LAYERS)
    with pytest.raises(ConfigError):
        MesolixConfig.from_dict(_with(_PLAIN_LAYERS, path, value))


def test_layers_that_use_the_tensors_of_others():
    """Through one another, forward and backward; a circle leads nowhere; every run keeps a cache entry of its own."""
    one = models.CONFIG_A["layers"][0]
    layers = [dict(one, weights_of=2), dict(one, weights_of=0), one, dict(one, weights_of=1)]
    cfg = MesolixConfig.from_dict(dict(models.CONFIG_A, layers=layers))
    assert [weights_owner(cfg.layers, i) for i in range(4)] == [2, 2, 2, 2]
    spec = mesolix_model_spec(cfg)
    assert [layer.name for layer in spec.layers] == ["l2"] and [r.layer for r in spec.order] == [0, 0, 0, 0]
    assert [key for key, _ in Model(spec).cache_needs()] == [(run, "mixer") for run in range(4)]
    with pytest.raises(ConfigError, match="no layer with tensors"):
        MesolixConfig.from_dict(dict(models.CONFIG_A, layers=[dict(one, weights_of=1), dict(one, weights_of=0)]))


def test_folder_there_and_back(tmp_path):
    """``write_model_folder`` names every tensor as a checkpoint does and the loader finds every one again; the rows of
    the table of distances come from the tensors."""
    from safetensors.torch import load_file

    from torchllms_amd.weights import load_weights

    folder = models.make_folder(tmp_path / "m", models.CONFIG_A, seed=1, dtype=torch.float32)
    names = set(load_file(str(folder / "model.safetensors")))
    assert {"embed", "pos", "head", "final.norm", "l0.norm1", "l0.norm2", "l0.mix.dq", "l0.mix.dq.norm", "l0.mix.uq", "l0.mix.dkv", "l0.mix.dkv.norm",
            "l0.mix.uk", "l0.mix.uv", "l0.mix.sink", "l0.mix.g", "l0.mix.o", "l0.mlp.gate", "l0.mlp.up", "l0.mlp.down", "l1.mix.in", "l1.mix.conv",
            "l1.mix.conv.b", "l1.mix.dt_bias", "l1.mix.A_log", "l1.mix.D", "l1.mix.norm", "l1.mix.o", "l1.mlp.router", "l1.mlp.e4.gate",
            "l1.mlp.shared.up", "l2.mix.q", "l2.mix.k", "l2.mix.v", "l2.mix.rel", "l2.mix.g", "l2.mix.o"} <= names
    assert not {n for n in names if n.startswith(("l3.", "l4.", "l5."))} and not {"l2.norm2", "l2.mlp.up", "l0.mlp.router"} & names
    arch, loaded = load_config(folder)
    assert "rel_rows" not in json.loads((folder / "config.json").read_text())["layers"][2]["mixer"]
    assert arch.name == "Mesolix" and loaded == MesolixConfig.from_dict(models.CONFIG_A)
    model = Model(arch.model_spec(loaded))
    tensors = load_weights(folder, arch.weight_rules(loaded), model.param_specs(), torch.float32, device="cpu")
    assert set(tensors) == set(model.param_specs())
    model.bind(tensors)


def test_what_the_cache_keeps():
    """A latent a token, pages behind a window, a 32-bit state row with the convolution's last inputs."""
    model = Model(mesolix_model_spec(MesolixConfig.from_dict(models.CONFIG_A)))
    needs = dict(model.cache_needs())
    assert sorted(key[0] for key in needs) == [0, 1, 2, 3, 4, 5]
    assert (needs[(0, "mixer")].num_kv_heads, needs[(0, "mixer")].head_dim, needs[(0, "mixer")].window, needs[(0, "mixer")].values_in_keys) == (1, 24, 0, True)
    assert (needs[(4, "mixer")].num_kv_heads, needs[(4, "mixer")].head_dim, needs[(4, "mixer")].v_head_dim, needs[(4, "mixer")].window) == (2, 16, 24, 24)
    assert needs[(1, "mixer")].dtype == "float32" and needs[(1, "mixer")].shape == (3 * (120 + 2 * 3 * 12) + 6 * 20 * 12,)
    groups, states = group_layers(model.cache_needs())
    assert sorted(g.window for g in groups) == [0, 24] and sum(len(s.run_ids) for s in states) == 2
    wide = json.loads(json.dumps(_PLAIN_LAYERS))
    wide["layers"][1]["mixer"]["state"] = 300
    with pytest.raises(ValueError, match="states of 300 channels"):
        Model(mesolix_model_spec(MesolixConfig.from_dict(wide))).check_sizes(torch.float32)
    flat = json.loads(json.dumps(_PLAIN_LAYERS))
    flat["layers"][2]["mixer"]["bias_max"] = 6  # (half of twelve rows: no logarithmic buckets)
    with pytest.raises(ValueError, match="logarithmic buckets"):
        Model(mesolix_model_spec(MesolixConfig.from_dict(flat)))


def test_buckets_of_distances():
    """Against the formula where no edge is near, against exact fractions everywhere, against the plain implementation;
    edges that are powers (a logarithm may come out below them)."""
    assert distance_bucket_starts(8, 64) == [4, 8, 16, 32]
    assert distance_bucket_starts(16, 8 ** 9) == [8, 64, 512, 4096, 8 ** 5, 8 ** 6, 8 ** 7, 8 ** 8]
    for rows, most in ((16, 240), (32, 128), (7, 50), (2, 3), (3, 9), (12, 20), (33, 1000), (64, 77)):
        half = rows // 2
        table = distance_table(torch.arange(rows, dtype=torch.float32)[:, None], most, 0)[0].long().tolist()
        for n in range(2 * most):
            got = table[min(n, len(table) - 1)]
            assert got == plain.bucket(n, rows, most), (rows, most, n)
            if n < half:
                assert got == n
                continue
            x = math.log(n / half) / math.log(most / half) * (rows - half)
            if abs(x - round(x)) > 1e-6:
                assert got == min(rows - 1, half + math.floor(x)), (rows, most, n)
            else:
                t = round(x)
                assert Fraction(n, half) ** (rows - half) >= Fraction(most, half) ** t
                assert got == min(rows - 1, half + t)
    # a window cuts the table, the last bucket ends it
    rel = torch.randn(8, 3)
    assert distance_table(rel, 64, 10).shape == (3, 10) and distance_table(rel, 64, 1000).shape == (3, 33)
    assert torch.equal(distance_table(rel, 64, 1000)[:, 32], rel[7]) and torch.equal(distance_table(rel, 64, 10)[:, 9], rel[5])


# ----------------------------------------------------------------------------- the plain implementation pinned
def test_plain_sink_and_masks_by_hand():
    """Two keys of equal score beside a sink: each gets 1 / (2 + exp(sink - score))."""
    s = torch.tensor([[[1.0, float("-inf")], [1.0, 1.0]]], dtype=torch.float64)
    p = plain.softmax_with_sink(s, torch.tensor([2.0], dtype=torch.float64))
    assert float(p[0, 1, 0]) == pytest.approx(1 / (2 + math.exp(1.0))) and float(p[0, 0, 0]) == pytest.approx(1 / (1 + math.exp(1.0)))
    assert float(p[0, 0, 1]) == 0.0
    assert plain.causal(3).int().tolist() == [[1, 0, 0], [1, 1, 0], [1, 1, 1]]
    assert plain.within(4, 2).int().tolist() == [[1, 0, 0, 0], [1, 1, 0, 0], [0, 1, 1, 0], [0, 0, 1, 1]]
    bias = plain.distance_bias(torch.tensor([[1.0], [2.0], [3.0], [4.0]]), 5, 8)  # rows 0, 1, then 2..3 and 4.. up to 8
    assert bias[0].tolist() == [[1, 0, 0, 0, 0], [2, 1, 0, 0, 0], [3, 2, 1, 0, 0], [3, 3, 2, 1, 0], [4, 3, 3, 2, 1]]


def test_plain_states_are_their_unrolled_sum():
    """``y_t = sum_(s <= t) exp(-exp(A) sum_(s < r <= t) dt_r) dt_s (C_t . B_s) x_s``."""
    gen = torch.Generator().manual_seed(2)
    x, B, C = (torch.randn((9, 2, d), generator=gen, dtype=torch.float64) for d in (3, 4, 4))
    dt = torch.rand((9, 2), generator=gen, dtype=torch.float64)
    log_a = torch.tensor([-1.0, 0.7], dtype=torch.float64)
    got = plain.ssd_states(x, B, C, dt, log_a)
    for t in range(9):
        for h in range(2):
            want = sum(math.exp(-math.exp(log_a[h]) * float(dt[s + 1 : t + 1, h].sum())) * dt[s, h] * (C[t, h] @ B[s, h]) * x[s, h] for s in range(t + 1))
            assert torch.allclose(got[t, h], want, atol=1e-12)


def test_plain_convolution_gate_and_router_by_hand():
    out = plain.causal_conv(torch.tensor([[1.0], [2.0], [4.0]]), torch.tensor([[10.0, 1.0]]), torch.tensor([0.5]))
    assert out[:, 0].tolist() == [1.5, 12.5, 24.5]  # the last column of the taps is the current token's
    w = {"gate": torch.tensor([[3.0]]), "up": torch.tensor([[-5.0]]), "down": torch.tensor([[1.0]])}
    assert float(plain.clamped_glu(torch.tensor([[1.0]]), w, "", 2.0)) == pytest.approx(2.0 / (1 + math.exp(-3.404)) * -1.0)
    assert float(plain.clamped_glu(torch.tensor([[-1.0]]), w, "", 2.0)) == pytest.approx(-3.0 / (1 + math.exp(1.702 * 3)) * 3.0)
    ids, weights = plain.routed_choice(torch.tensor([[0.5, 3.0, -1.0, 2.0]], dtype=torch.float64), 2)
    assert ids.tolist() == [[1, 3]] and weights[0].tolist() == pytest.approx([1 / (1 + math.exp(-3.0)), 1 / (1 + math.exp(-2.0))])
    assert float(plain.softplus(torch.tensor(-40.0, dtype=torch.float64))) == pytest.approx(math.exp(-40.0))


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

    def mixers(d, kind):
        return [entry["mixer"] for entry in d["layers"] if entry["type"] == kind]

    assert moved(changed(lambda d: [m["mask"].update(size=25) for m in mixers(d, "attention")])) > 3e-3
    assert moved(changed(lambda d: [m["mask"].update(size=23) for m in mixers(d, "attention")])) > 3e-3
    assert moved(changed(lambda d: [m.update(bias_max=21) for m in mixers(d, "attention")])) > 3e-3
    assert moved(changed(lambda d: [m.update(scale=m["scale"] * 1.05) for m in mixers(d, "latent_attention")])) > 3e-3
    assert moved(changed(lambda d: [m.update(norm_groups=1) for m in mixers(d, "mamba2")])) > 3e-3
    assert moved(changed(lambda d: [entry["mlp"].update(limit=0.65) for entry in d["layers"] if entry["mlp"] and entry["mlp"]["kind"] == "dense"])) > 3e-3
    assert moved(changed(lambda d: [entry["mlp"]["router"].update(top=1) for entry in d["layers"] if entry["mlp"] and entry["mlp"]["kind"] == "moe"])) > 3e-3
    assert moved(changed(lambda d: d["layers"].pop(3))) > 3e-3  # (a layer that uses another's tensors)
    for name, value in (("l0.mix.sink", -30.0), ("l0.mix.dkv.norm", 1.0), ("l0.mix.dq.norm", 1.0), ("l1.mix.D", 0.0), ("l1.mix.conv.b", 0.0),
                        ("l1.mix.norm", 1.0), ("l1.mix.dt_bias", -2.0), ("l1.mix.A_log", -1.0), ("l2.mix.rel", 0.0), ("l0.norm1", 0.0), ("final.norm", 0.0),
                        ("l1.mlp.shared.down", 0.0), ("l0.mix.g", 0.0), ("l2.mix.g", 0.0), ("pos", 0.0)):
        assert moved(w2=dict(w, **{name: torch.full_like(w[name], value)})) > 3e-3, name
    assert moved(w2=dict(w, pos=w["pos"].roll(1, 0))) > 3e-3
    assert moved(w2=dict(w, **{"l1.mix.conv": w["l1.mix.conv"].flip(1)})) > 3e-3
    # the first token still shows in the last position's logits
    other = plain.forward(cfg, w, [(tokens[0] + 1) % cfg["vocab"]] + tokens[1:])
    assert _distance(other[-1:], truth[-1:]) > 3e-4
    monkeypatch.setattr(plain, "mixture", lambda h, w, p, mlp: plain.expert(h, w, p + "shared.") + sum(
        plain.routed_choice(h @ w[p + "router"].T, mlp["router"]["top"])[1][:, j : j + 1]
        * torch.stack([plain.expert(h[t : t + 1], w, f"{p}e{int(plain.routed_choice(h @ w[p + 'router'].T, mlp['router']['top'])[0][t, j])}.")[0] for t in range(h.shape[0])])
        for j in range(mlp["router"]["top"])))
    assert moved() > 3e-3  # (weights behind the experts instead of before them)
