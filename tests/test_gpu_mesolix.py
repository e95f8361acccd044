"""The Mesolix decoder in the engine against the plain implementation of tests/plain/mesolix.py: every mechanism alone,
whole prompts against decoding token by token, portions down to two tokens, mixed batches with pages and state slots
that are used again, keys far back and at the edges of every window and bucket, layers that use another's tensors, long
decoding from recorded graphs, and greedy generation through ``LLM.generate`` and the scheduler; on three small
configurations that differ in every size, in 32-bit and in bfloat16.  The kernels that are new with this design are also
compared alone, on inputs made so that a fault shows."""

import json

import pytest
import torch

from . import mesolix_models as models
from . import schedules
from .helpers import random_tokens
from .plain import mesolix as plain
from .test_gpu_engine import run_trace
from .test_gpu_rifizen import _paged, assert_within_rounding, distance

pytestmark = pytest.mark.gpu

LENGTHS = {"A": [70, 41, 100, 35, 50, 33], "B": [66, 40, 130, 35, 90], "C": [45, 150, 37, 64, 120]}
FP32_TOL = 3e-5
BF16_TOL = 5e-2
DEV = "cuda:0"


def truth_of(cfg, weights, requests):
    out = {rid: plain.forward(cfg, weights, toks) for rid, toks in requests.items()}
    scale = float(torch.cat([(t - t.mean(-1, keepdim=True)).flatten() for t in out.values()]).pow(2).mean().sqrt())
    return out, scale


def folder_for(dtype, path, cfg_dict, **kw):
    """The model a run in ``dtype`` is compared on: bfloat16 runs get routers whose choice no rounding changes, the 32-bit
    runs, which are the sharp ones, get routers whose choice changes from token to token."""
    return models.make_folder(path / dtype, cfg_dict, decisive_router=dtype == "bfloat16", **kw)


class Case:
    def __init__(self, name, tmp):
        from torchllms_amd.engine import Engine

        self.name = name
        self.folders = {dt: folder_for(dt, tmp / name, models.CONFIGS[name], seed=11) for dt in ("float32", "bfloat16")}
        self.cfg = models.CONFIGS[name]
        self.requests = {f"r{i}": random_tokens(n, self.cfg["vocab"], 100 + i) for i, n in enumerate(LENGTHS[name])}
        self.truths = {dt: truth_of(*models.read_folder(f), self.requests) for dt, f in self.folders.items()}
        self.traces = {
            "whole": schedules.whole(self.requests),
            "tail": schedules.tail(self.requests),
            "portions": schedules.portions(self.requests),
            "mixed": schedules.mixed(self.requests),
        }
        page = models.PAGE_SIZE[name]
        pool_tokens = max(schedules.max_live_tokens(t) for t in self.traces.values())
        self.engines = {
            dt: Engine.from_folder(self.folders[dt], dtype=dt, page_size=page, num_pages=-(-pool_tokens // page), max_seqs=4)
            for dt in ("float32", "bfloat16")
        }
        self._results = {}

    def result(self, dtype, schedule):
        key = (dtype, schedule)
        if key not in self._results:
            self._results[key] = run_trace(self.engines[dtype], self.traces[schedule])
        return self._results[key]

    def distances(self, dtype, result):
        truth, scale = self.truths[dtype]
        return {(rid, pos): distance(row, truth[rid][pos], scale) for (rid, pos), row in result.items()}


@pytest.fixture(scope="module")
def cases(tmp_path_factory):
    tmp = tmp_path_factory.mktemp("mesolix")
    return {name: Case(name, tmp) for name in models.CONFIGS}


@pytest.mark.parametrize("schedule", ["whole", "tail", "portions", "mixed"])
@pytest.mark.parametrize("name", ["A", "B", "C"])
def test_float32_matches_the_plain_model(cases, name, schedule):
    case = cases[name]
    got = case.result("float32", schedule)
    assert len(got) == sum(len(t) for t in case.requests.values())
    dists = case.distances("float32", got)
    where = max(dists, key=dists.get)
    assert dists[where] < FP32_TOL, f"{name}/{schedule}: first look at {where}, distance {dists[where]}"


@pytest.mark.parametrize("schedule", ["tail", "portions", "mixed"])
@pytest.mark.parametrize("name", ["A", "B", "C"])
def test_float32_does_not_depend_on_the_schedule(cases, name, schedule):
    """Every 32-bit kernel adds in an order fixed by the element it computes (blocks of keys aligned to positions, the
    recurrence token by token, the experts pair by pair, a row's sums by its width), so cutting, batching, pages and
    slots change no bit."""
    case = cases[name]
    ref = case.result("float32", "whole")
    got = case.result("float32", schedule)
    diff = sorted(k for k in ref if not torch.equal(ref[k], got[k]))
    assert not diff, f"{name}/{schedule}: {len(diff)} positions differ, first {diff[0]}"


@pytest.mark.parametrize("schedule", ["whole", "tail", "portions", "mixed"])
@pytest.mark.parametrize("name", ["A", "B", "C"])
def test_bfloat16_stays_within_rounding(cases, name, schedule):
    case = cases[name]
    assert_within_rounding(case.distances("bfloat16", case.result("bfloat16", schedule)).values(), BF16_TOL, f"{name}/{schedule}")


# ----------------------------------------------------------------------------- every mechanism alone
_L, _W, _M = models.latent, models.windowed, models.mamba
ALONE = {
    "latent": models.layer(_L(4, 24, 40, 30, 56)),
    "latent_one_head": models.layer(_L(1, 16, 16, 8, 16)),
    "latent_odd_sizes": models.layer(_L(3, 10, 7, 13, 18)),
    "latent_wide": models.layer(_L(2, 48, 32, 64, 320)),
    "latent_matrix_cores": models.layer(_L(6, 32, 24, 40, 64)),
    "latent_matrix_cores_groups": models.layer(_L(24, 16, 16, 40, 128)),
    "latent_matrix_cores_uneven_heads": models.layer(_L(17, 16, 8, 24, 32)),
    "latent_matrix_cores_256": models.layer(_L(12, 64, 64, 96, 256)),
    "windowed": models.layer(_W(4, 2, 24, 40, 30, rows=12, most=25)),
    "windowed_one_head": models.layer(_W(1, 1, 16, 16, 100, rows=7, most=60)),
    "windowed_sees_itself_alone": models.layer(_W(4, 2, 16, 16, 1)),
    "windowed_no_edge": models.layer(_W(5, 5, 16, 24, 5000, rows=20, most=150)),
    "windowed_one_row": models.layer(_W(2, 1, 16, 24, 20, rows=1, most=1)),
    "windowed_odd_sizes": models.layer(_W(3, 1, 10, 6, 19, rows=5, most=11)),
    "windowed_matrix_cores": models.layer(_W(8, 2, 64, 64, 150, rows=32, most=100)),
    "windowed_matrix_cores_one_kv_head": models.layer(_W(6, 1, 128, 128, 130, rows=16, most=300)),
    "windowed_matrix_cores_wider_values": models.layer(_W(4, 2, 32, 64, 45, rows=10, most=40)),
    "windowed_matrix_cores_256": models.layer(_W(2, 1, 256, 256, 70, rows=8, most=64)),
    "mamba": models.layer(_M(6, 24, 40, groups=2, conv=4, norm_groups=3)),
    "mamba_one_head": models.layer(_M(1, 40, 16, conv=2)),
    "mamba_no_history": models.layer(_M(4, 16, 24, groups=4, conv=1, norm_groups=4)),
    "mamba_odd_sizes": models.layer(_M(3, 10, 7, conv=3, norm_groups=5)),
    "mamba_parts_across_heads": models.layer(_M(4, 36, 16, groups=2, conv=5, norm_groups=6)),
    "mamba_matrix_cores": models.layer(_M(4, 64, 128, groups=2, conv=4, norm_groups=2)),
    "mamba_matrix_cores_wide": models.layer(_M(2, 128, 64, conv=3)),
    "mamba_wide_heads": models.layer(_M(2, 200, 32, conv=4)),
    "mamba_wide_states": models.layer(_M(2, 32, 256, groups=2, conv=4)),
    "dense": models.layer(models.TINY, models.dense(136)),
    "dense_narrow": models.layer(models.TINY, models.dense(9, limit=0.2)),
    "routed": models.layer(models.TINY, models.moe(40, 8, 3, shared=24)),
    "routed_one_choice": models.layer(models.TINY, models.moe(33, 5, 1)),
    "routed_all_chosen": models.layer(models.TINY, models.moe(16, 3, 3, shared=9)),
    "routed_many": models.layer(models.TINY, models.moe(8, 70, 6)),
}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("what", sorted(ALONE))
def test_a_mechanism_alone(tmp_path, what, dtype):
    """A model of one layer, a prompt in one step and, in a second request, the same tokens in portions and one by one."""
    from torchllms_amd.engine import Engine, StepEntry

    folder = folder_for(dtype, tmp_path / what, models.single_layer(ALONE[what]), seed=5)
    cfg, weights = models.read_folder(folder)
    tokens = random_tokens(275, cfg["vocab"], 9)
    truth, scale = truth_of(cfg, weights, {"r": tokens})
    engine = Engine.from_folder(folder, dtype=dtype, page_size=8, num_pages=80, max_seqs=2)
    engine.admit("whole")
    whole = engine.step([StepEntry("whole", tokens, list(range(len(tokens))))]).cpu()
    engine.admit("cut")
    rows, at = [], 0
    for n in (5, 2, 30, 1, 1, 1, 17, 2, 1, 1, 13, 1, 150, 1, 1, 47, 1):
        rows.append(engine.step([StepEntry("cut", tokens[at : at + n], list(range(n)))]).cpu())
        at += n
        engine.cache.check_invariants()
    assert at == len(tokens)
    cut = torch.cat(rows)
    for name, got in (("whole", whole), ("cut", cut)):
        dists = [distance(got[i], truth["r"][i], scale) for i in range(len(tokens))]
        if dtype == "float32":
            assert max(dists) < FP32_TOL, f"{what}/{name}: {max(dists)} at {dists.index(max(dists))}"
        else:
            assert_within_rounding(dists, BF16_TOL, f"{what}/{name}")
    if dtype == "float32":
        assert torch.equal(whole, cut)


# ----------------------------------------------------------------------------- a bias by table in the attention kernels
def _plain_attention(q, keys, values, pos, window, keep, scale, cap, table, sinks, group):
    """One query [Hq, d] at position ``pos`` over keys [n, Hk, d] / values [n, Hk, dv]: it sees j <= pos with
    pos - j < window (0: all) or j < keep; a score is capped (cap > 0), then gains its head's entry of ``table`` [Hq, L] at the
    distance (past the end: the last); a sink per head or none."""
    out = []
    js = [j for j in range(pos + 1) if not window or pos - j < window or j < keep]
    dist = torch.tensor([pos - j for j in js])
    for h in range(q.shape[0]):
        g = h // group
        s = (keys[js, g].double() @ q[h].double()) * scale
        if cap > 0:
            s = cap * torch.tanh(s / cap)
        if table is not None:
            s = s + table[h, dist.clamp(max=table.shape[1] - 1)].double()
        e = torch.exp(s - s.max())
        total = e.sum() + (torch.exp(sinks[h].double() - s.max()) if sinks is not None else 0.0)
        out.append((e / total) @ values[js, g].double())
    return torch.stack(out)


def _spiky_table(Hq, entries, gen):
    """A table whose neighbours differ by several units, so that a distance that is one off decides."""
    return torch.randn((Hq, entries), generator=gen) * 3.0


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("Hq,Hk,d,dv,page,window,keep,cap,entries", [(4, 2, 16, 16, 8, 37, 0, 0.0, 37), (8, 4, 24, 40, 4, 37, 11, 9.0, 20), (6, 2, 64, 32, 16, 0, 0, 0.0, 90),
                                                                     (2, 2, 7, 5, 3, 37, 5, 0.0, 1)])
def test_plain_attention_with_a_table_of_distances(Hq, Hk, d, dv, page, window, keep, cap, entries, dtype):
    """Windows with and without kept first positions, and none; tables as long as the window and shorter; with sinks.
    Single tokens by one wave, blocks of keys side by side and a prompt's portion through tiles, against the formula and
    bit by bit against each other."""
    from torchllms_amd.kernels import ops

    gen = torch.Generator().manual_seed(Hq * 100 + d)
    n, scale = 300, 0.3
    table, sinks = _spiky_table(Hq, entries, gen), torch.randn(Hq, generator=gen) * 2 + 2
    keys, values = torch.randn((n, Hk, d), generator=gen), torch.randn((n, Hk, dv), generator=gen)
    positions = [0, 5, 10, 11, 12, 36, 37, 38, 46, 47, 48, 63, 64, 100, 128, 200, 255, 256, 299]
    queries = torch.randn((len(positions), Hq, d), generator=gen)
    if dtype == torch.bfloat16:
        keys, values, queries = (t.to(dtype).float() for t in (keys, values, queries))

    def formula(q, p, table=table, sinks=sinks):
        return _plain_attention(q, keys, values, p, window, keep, scale, cap, table, sinks, Hq // Hk)

    want = torch.stack([formula(queries[i], p) for i, p in enumerate(positions)])
    tol = 1e-5 if dtype == torch.float32 else 2e-2
    for other in (dict(sinks=None), dict(table=table.roll(1, 1))):  # (they do decide)
        if entries > 1 or "sinks" in other:
            off = torch.stack([formula(queries[i], p, **other) for i, p in enumerate(positions)])
            assert (want - off).abs().max() > (20 if dtype == torch.float32 else 5) * tol, other
    k_pages, v_pages, pages = _paged(keys, values, page, 120, gen)
    kp, vp = k_pages.to(DEV, dtype), v_pages.to(DEV, dtype)
    bt = pages.to(DEV).view(1, -1)
    q = queries.reshape(len(positions), Hq * d).to(DEV, dtype)
    pos = torch.tensor(positions, dtype=torch.int32, device=DEV)
    seq = torch.zeros(len(positions), dtype=torch.int32, device=DEV)
    kw = dict(v_head_dim=dv, keep_first=keep, softcap=cap, distances=table.to(DEV), sinks=sinks.to(DEV))
    alone = ops.attention_generic(q, Hq, Hk, d, kp, vp, seq, pos, bt, window, scale, **kw).float().cpu().view(len(positions), Hq, dv)
    assert (alone.double() - want).abs().max() < tol * max(1.0, float(want.abs().max())), (alone.double() - want).abs().max()
    split = ops.attention_generic_split(q, Hq, Hk, d, kp, vp, seq, pos, bt, window, scale, longest=window or n, **kw).float().cpu().view_as(alone)
    assert torch.equal(split, alone)
    for first in (0, 3, 30, 120, 260):
        ps = list(range(first, first + 40))
        qs = queries[torch.arange(40) % len(positions)].reshape(40, Hq * d).to(DEV, dtype)
        tiled = ops.attention_generic(qs, Hq, Hk, d, kp, vp, torch.zeros(40, dtype=torch.int32, device=DEV),
                                      torch.tensor(ps, dtype=torch.int32, device=DEV), bt, window, scale, **kw).cpu()
        for i in (0, 7, 8, 9, 20, 39):
            one = ops.attention_generic(qs[i : i + 1], Hq, Hk, d, kp, vp, seq[:1], torch.tensor(ps[i : i + 1], dtype=torch.int32, device=DEV),
                                        bt, window, scale, **kw).cpu()
            assert torch.equal(tiled[i : i + 1], one), (first, i)
            ref = formula(qs[i].float().cpu().view(Hq, d), ps[i])
            assert (one.float().view(Hq, dv).double() - ref).abs().max() < tol * max(1.0, float(ref.abs().max()))


@pytest.mark.parametrize("Hq,Hk,d,dv,page,window,entries", [
    (8, 2, 128, 128, 16, 200, 200), (4, 4, 64, 128, 16, 70, 30), (16, 1, 64, 64, 8, 500, 400), (4, 2, 256, 256, 16, 100, 90), (6, 2, 128, 128, 16, 64, 64),
    (2, 2, 32, 96, 16, 33, 33), (3, 1, 128, 128, 32, 1, 1), (8, 2, 32, 32, 16, 600, 100), (4, 2, 64, 64, 16, 0, 150)])
def test_matrix_core_attention_with_a_table_of_distances(Hq, Hk, d, dv, page, window, entries):
    """The split-KV decode kernel and the tiled prefill kernel against the plain kernel (which the test above holds
    against the formula): tables that lie in a block's LDS and (many heads, many entries) ones that do not, tiles of keys
    whose distances all lie behind the table's end, all inside it, and on either side; single tokens, and portions that
    begin before, at and behind the window's first full reach; the key at a window's lower edge stands out."""
    from torchllms_amd.kernels import ops

    gen = torch.Generator().manual_seed(Hq + d + window)
    n, scale = 700, 0.7 / d ** 0.5
    table = _spiky_table(Hq, entries, gen)
    if window:  # the last distance a window lets in, and the first it does not, would weigh the most
        table[:, -1] = 6.0
    keys = torch.randn((n, Hk, d), generator=gen).to(torch.bfloat16)
    values = torch.randn((n, Hk, dv), generator=gen).to(torch.bfloat16)
    k_pages, v_pages, pages = _paged(keys.float(), values.float(), page, 2 * (n // page) + 9, gen)
    kp, vp = k_pages.to(DEV, torch.bfloat16), v_pages.to(DEV, torch.bfloat16)
    bt = pages.to(DEV).view(1, -1)
    positions = sorted({min(max(p, 0), n - 1) for p in (0, 1, 15, 16, window - 1, window, window + 1, window + 17, 300, 511, 512, 699)})
    q = torch.randn((len(positions), Hq * d), generator=gen).to(DEV, torch.bfloat16)
    pos = torch.tensor(positions, dtype=torch.int32, device=DEV)
    seq = torch.zeros(len(positions), dtype=torch.int32, device=DEV)
    kw = dict(distances=table.to(DEV))
    want = ops.attention_generic(q, Hq, Hk, d, kp, vp, seq, pos, bt, window, scale, v_head_dim=dv, **kw).float()
    flat = ops.attention_generic(q, Hq, Hk, d, kp, vp, seq, pos, bt, window, scale, v_head_dim=dv).float()
    assert window == 1 or (want - flat).abs().max() > 0.3  # (the table does decide)
    for split in (None, 64, 128):
        got = torch.zeros((len(positions), Hq * dv), dtype=torch.bfloat16, device=DEV)
        for at in range(0, dv, d):
            ops.attention_decode(q, Hq, Hk, d, kp, vp, seq, pos, bt, window, scale, min(max(positions) + 1, window + 15) if window else max(positions) + 1,
                                 out=got, split_size=split, v_offset=at, **kw)
        assert (got.float() - want).abs().max() < 3e-2 * max(1.0, float(want.abs().max())), (split, (got.float() - want).abs().max())
    qpt = ops.prefill_queries_per_tile(Hq, Hk, d)
    for first, count in ((0, 700), (0, 40), (3, 90), (max(window - 1, 0), 130), (window + 20, 77), (500, 200), (690, 10)):
        if first + count > n:
            continue
        ps = list(range(first, first + count))
        q = torch.randn((count, Hq * d), generator=gen).to(DEV, torch.bfloat16)
        qo = torch.tensor([0, count], dtype=torch.int32, device=DEV)
        kv = torch.tensor([first + count], dtype=torch.int32, device=DEV)
        rows, q0s = ops.prefill_tiles([0, count], 0, 1, qpt, [first + count], window)
        tiles = torch.tensor([rows, q0s], dtype=torch.int32, device=DEV)
        want = ops.attention_generic(q, Hq, Hk, d, kp, vp, torch.zeros(count, dtype=torch.int32, device=DEV),
                                     torch.tensor(ps, dtype=torch.int32, device=DEV), bt, window, scale, v_head_dim=dv, **kw).float()
        for groups in (1, 2):
            got = torch.zeros((count, Hq * dv), dtype=torch.bfloat16, device=DEV)
            for at in range(0, dv, d):
                ops.attention_prefill(q, Hq, Hk, d, kp, vp, qo, kv, bt, tiles[0], tiles[1], window, scale, got, key_groups=groups, v_offset=at, **kw)
            err = (got.float() - want).abs().max(dim=1).values
            assert float(err.max()) < 3e-2 * max(1.0, float(want.abs().max())), (first, count, groups, int(err.argmax()) + first, float(err.max()))


@pytest.mark.parametrize("H,per,d,page", [(32, 16, 64, 16), (20, 10, 128, 8), (12, 6, 256, 16), (9, 9, 32, 16)])
def test_groups_of_query_heads_over_one_head_of_the_pages(H, per, d, page):
    """Attention through a latent: groups of query heads as kv heads of their own that all read the pages' one head as keys
    and values, with a sink a head, against the formula (where a far key stands out) for single tokens and portions."""
    from torchllms_amd.kernels import ops

    gen = torch.Generator().manual_seed(H + d)
    n, scale = 500, 0.5 / d ** 0.5
    rows = torch.randn((n, 1, d), generator=gen).to(torch.bfloat16)
    sinks = torch.randn(H, generator=gen) + 3.0 * d * scale  # (as much as the key that stands out)
    k_pages, _, pages = _paged(rows.float(), rows.float(), page, n // page + 40, gen)
    kp, bt = k_pages.to(DEV, torch.bfloat16), pages.to(DEV).view(1, -1)
    dev = sinks.to(DEV)
    kw = dict(sinks=dev, key_heads=1, value_heads=1)

    def queries(ps):
        q = torch.randn((len(ps), H, d), generator=gen)
        for i, p in enumerate(ps):
            q[i] += rows[max(p - 400, p % 7), 0].float() * 3.0  # (a key far back)
        return q.to(torch.bfloat16)

    ps = [0, 1, 15, 16, 17, 100, 255, 256, 499]
    q = queries(ps)
    want = torch.stack([_plain_attention(q[i].float(), rows, rows, p, 0, 0, scale, 0.0, None, sinks, H) for i, p in enumerate(ps)])
    no_sink = torch.stack([_plain_attention(q[i].float(), rows, rows, p, 0, 0, scale, 0.0, None, None, H) for i, p in enumerate(ps)])
    assert (want - no_sink).abs().max() > 0.3
    for split in (None, 64):
        got = ops.attention_decode(q.view(len(ps), H * d).to(DEV), H, H // per, d, kp, kp, torch.zeros(len(ps), dtype=torch.int32, device=DEV),
                                   torch.tensor(ps, dtype=torch.int32, device=DEV), bt, 0, scale, 500, split_size=split, **kw)
        assert (got.float().cpu().view(len(ps), H, d).double() - want).abs().max() < 3e-2 * float(want.abs().max())
    qpt = ops.prefill_queries_per_tile(H, H // per, d)
    for first, count in ((0, 130), (350, 150)):
        ps = list(range(first, first + count))
        q = queries(ps)
        rows_t, q0s = ops.prefill_tiles([0, count], 0, 1, qpt, [first + count], 0)
        tiles = torch.tensor([rows_t, q0s], dtype=torch.int32, device=DEV)
        for groups in (1, 2):
            got = torch.zeros((count, H * d), dtype=torch.bfloat16, device=DEV)
            ops.attention_prefill(q.view(count, H * d).to(DEV), H, H // per, d, kp, kp, torch.tensor([0, count], dtype=torch.int32, device=DEV),
                                  torch.tensor([first + count], dtype=torch.int32, device=DEV), bt, tiles[0], tiles[1], 0, scale, got, key_groups=groups, **kw)
            for i in (0, 1, 31, 32, count - 1):
                ref = _plain_attention(q[i].float(), rows, rows, ps[i], 0, 0, scale, 0.0, None, sinks, H)
                assert (got[i].float().cpu().view(H, d).double() - ref).abs().max() < 3e-2 * max(1.0, float(ref.abs().max())), (first, groups, i)


# ----------------------------------------------------------------------------- the state-space recurrence alone
def _ssd_inputs(n, H, dv, N, G, seed):
    """x | B | C rows and a column of step sizes a head, with a B that stands out early and a C that asks for it late."""
    gen = torch.Generator().manual_seed(seed)
    xbc = torch.randn((n, H * dv + 2 * G * N), generator=gen)
    xbc[5, H * dv : H * dv + G * N] *= 4.0
    xbc[n - 9, H * dv + G * N :] = xbc[5, H * dv : H * dv + G * N]
    dt = torch.randn((n, H + 3), generator=gen)
    dt[7] = 25.0  # (softplus of a large number is the number)
    bias = torch.linspace(-5.0, 0.5, H)
    A = -torch.exp(torch.linspace(-4.0, 1.0, H))
    return xbc, dt, bias, A, torch.randn(H, generator=gen)


def _plain_ssd(xbc, dt, bias, A, D, G, dv, N):
    xbc, H, n = xbc.double(), A.numel(), xbc.shape[0]
    x, B, C = xbc.split([H * dv, G * N, G * N], dim=1)
    x = x.reshape(n, H, dv)
    B, C = (u.reshape(n, G, N).repeat_interleave(H // G, dim=1) for u in (B, C))
    step = plain.softplus(dt[:, :H].double() + bias.double())
    y = plain.ssd_states(x, B, C, step, torch.log(-A.double())) + D.double()[None, :, None] * x
    return y.reshape(n, H * dv)


def _run(ops, xbc, dt, vectors, state, rows, slots, G, dv, N, **kw):
    H = vectors[0].numel()
    return ops.ssd(xbc, dt[:, :H], *vectors, state, 4, rows, slots, G, dv, N, **kw)


SSDS = [(6, 24, 16, 3), (1, 33, 200, 1), (3, 5, 7, 1), (4, 128, 128, 2), (2, 300, 64, 2), (4, 20, 36, 4)]


@pytest.mark.parametrize("H,dv,N,G", SSDS)
def test_ssd_kernel(H, dv, N, G):
    """One row, the same tokens as steps of one request through another slot (the same bits and the same state), rows of
    several requests; heads that forget at once beside heads that keep for hundreds of tokens."""
    from torchllms_amd.kernels import ops

    n = 300
    xbc, dt, *vectors = _ssd_inputs(n, H, dv, N, G, dv + 2)
    want = _plain_ssd(xbc, dt, *vectors, G, dv, N)
    x, d, vec = xbc.to(DEV), dt.to(DEV), [v.to(DEV) for v in vectors]
    state = torch.zeros((3, H * dv * N + 4), device=DEV)
    i32 = lambda *v: torch.tensor(v, dtype=torch.int32, device=DEV)  # noqa: E731
    whole = _run(ops, x, d, vec, state, i32(0, n), i32(0), G, dv, N).cpu()
    bound = 2e-5 * float(want.abs().max())
    assert (whole.double() - want).abs().max() < bound, (whole.double() - want).abs().max()
    assert float(state[0, :4].abs().max()) == 0.0 and float(state[1].abs().max()) == 0.0
    state2 = torch.zeros_like(state)
    out, at = [], 0
    for m in [1, 1, 15, 16, 17, 2, 1, 33, 1, 64, 1, 1, 100, 1, 5, 1, 40]:
        out.append(_run(ops, x[at : at + m].contiguous(), d[at : at + m], vec, state2, i32(0, m), i32(1), G, dv, N).cpu())
        at += m
    assert at == n
    assert torch.equal(torch.cat(out), whole) and torch.equal(state2[1], state[0])
    batch = _run(ops, x, d, vec, torch.zeros_like(state), i32(0, 100, 101, n), i32(2, 0, 1), G, dv, N).cpu()
    assert torch.equal(batch[:100], whole[:100])
    want3 = _plain_ssd(xbc[101:], dt[101:], *vectors, G, dv, N)
    assert (batch[101:].double() - want3).abs().max() < 2e-5 * float(want3.abs().max())
    assert (want3[: n - 101] - want[101:]).abs().max() > 1e-3 * want.abs().max()  # (what lies before matters)


@pytest.mark.parametrize("H,dv,N,G", [(6, 24, 16, 3), (2, 64, 128, 1), (4, 128, 128, 2), (3, 40, 64, 1), (4, 36, 104, 4), (8, 100, 8, 2)])
def test_ssd_by_segments(H, dv, N, G):
    """bfloat16 rows: a prompt's segments side by side against the walk and the formula (of the rounded inputs), the state
    they leave, portions of all lengths that go on from each other's states, single tokens in front of several prompts,
    and the other slots untouched."""
    from torchllms_amd.kernels import ops

    n = 333
    xbc, dt, *vectors = _ssd_inputs(n, H, dv, N, G, dv + 3)
    xbc, dt = xbc.to(torch.bfloat16), dt.to(torch.bfloat16)
    want = _plain_ssd(xbc.float(), dt.float(), *vectors, G, dv, N)
    x, d, vec = xbc.to(DEV), dt.to(DEV), [v.to(DEV) for v in vectors]
    i32 = lambda *v: torch.tensor(v, dtype=torch.int32, device=DEV)  # noqa: E731
    assert ops.ssd_segments_supported(torch.bfloat16, H, dv, N, G)

    def segments(*bounds):
        return ops.ScanSegments(list(bounds), DEV, ops.SSD_SEGMENT)

    walked, state = torch.zeros((5, H * dv * N + 4), device=DEV), torch.zeros((5, H * dv * N + 4), device=DEV)
    by_walk = _run(ops, x, d, vec, walked, i32(0, n), i32(3), G, dv, N).cpu()
    got = _run(ops, x, d, vec, state, i32(0, n), i32(3), G, dv, N, segments=segments(0, n)).cpu()
    top = float(want.abs().max())
    assert (by_walk.double() - want).abs().max() < 2e-5 * top
    assert (got.double() - want).abs().max() < 2e-5 * top, (got.double() - want).abs().max() / top  # (results are 32-bit)
    assert (state[3] - walked[3]).abs().max() < 1e-5 * walked[3].abs().max()
    assert float(state[[0, 1, 2, 4]].abs().max()) == 0.0 and float(state[3, :4].abs().max()) == 0.0
    state.zero_()
    out, at = [], 0
    for m in [63, 64, 65, 2, 5, 128, 6]:
        out.append(_run(ops, x[at : at + m].contiguous(), d[at : at + m], vec, state, i32(0, m), i32(2), G, dv, N, segments=segments(0, m)).cpu())
        at += m
    assert at == n
    assert (torch.cat(out).double() - want).abs().max() < 2e-5 * top
    assert (state[2] - walked[3]).abs().max() < 1e-5 * walked[3].abs().max()
    # two single tokens, then two prompts of one step
    state = torch.zeros_like(walked)
    mixed = _run(ops, x, d, vec, state, i32(0, 1, 2, 100, n), i32(4, 0, 2, 1), G, dv, N, segments=segments(2, 100, n), single_rows=2).cpu()
    for lo, hi in ((0, 1), (1, 2), (2, 100), (100, n)):
        ref = _plain_ssd(xbc[lo:hi].float(), dt[lo:hi].float(), *vectors, G, dv, N)
        assert (mixed[lo:hi].double() - ref).abs().max() < 2e-5 * float(ref.abs().max()), (lo, hi)
    assert float(state[3].abs().max()) == 0.0


@pytest.mark.parametrize("width,parts", [(64, 1), (96, 8), (1000, 5), (4096, 1), (10240, 2), (20000, 1), (8192, 1), (77, 7), (2055, 1)])
def test_gated_norm_by_parts(width, parts):
    """Every part over its own root mean square (they differ by far), the gate before the norm; z as columns of a wider
    matrix; many rows and one give the same bits."""
    from torchllms_amd.kernels import ops

    gen = torch.Generator().manual_seed(width)
    n = 9
    y, z, w = torch.randn((n, width), generator=gen), torch.randn((n, width + 8), generator=gen) * 2, torch.randn(width, generator=gen)
    y *= torch.logspace(-2, 2, parts).repeat_interleave(width // parts)
    for dtype, tol in ((torch.float32, 1e-5), (torch.bfloat16, 1e-2)):
        zd = z.to(dtype)
        g = (y * plain.silu(zd[:, :width].float())).double().view(n, parts, -1)
        want = plain.over_rms(g, 1e-5).view(n, width) * w.double()
        got = ops.gated_norm(y.to(DEV), zd.to(DEV)[:, :width], w.to(DEV), parts, 1e-5)
        assert got.dtype == dtype and (got.cpu().double() - want).abs().max() < tol * float(want.abs().max())
        assert torch.equal(ops.gated_norm(y.to(DEV)[4:5].contiguous(), zd.to(DEV)[4:5, :width], w.to(DEV), parts, 1e-5), got[4:5])


# ----------------------------------------------------------------------------- the small kernels
@pytest.mark.parametrize("D", [64, 50, 1000, 1024, 2048, 4096, 8192, 16384, 4100, 20, 20000])
def test_branch_into_the_stream_and_norm(D):
    """The stream's sum in 32-bit in place and the norm of the sum; the branch in the model's dtype, in 32-bit, and as the
    slices of a split product; the rows of a gather, which leave the stream alone; many rows and one give the same bits."""
    from torchllms_amd.kernels import ops

    gen = torch.Generator().manual_seed(D)
    n = 37
    x, b, w = torch.randn((n, D), generator=gen) * 3, torch.randn((n, D), generator=gen), torch.randn(D, generator=gen)
    rows = torch.tensor([3, 36, 0, 3], dtype=torch.int32)
    for dtype, tol in ((torch.float32, 1e-5), (torch.bfloat16, 1e-2)):
        for branch_dtype in {torch.float32, dtype}:
            bd = b.to(branch_dtype)
            new = x.double() + bd.double()
            want = plain.over_rms(new, 1e-5) * w.double()
            xs = x.to(DEV).clone()
            got = ops.add_norm(xs, bd.to(DEV), w.to(DEV), 1e-5, dtype)
            assert torch.equal(xs.cpu(), x + bd.float())
            assert got.dtype == dtype and (got.cpu().double() - want).abs().max() < tol * float(want.abs().max())
            one = x.to(DEV)[5:6].clone()
            assert torch.equal(ops.add_norm(one, bd.to(DEV)[5:6].contiguous(), w.to(DEV), 1e-5, dtype), got[5:6])
            keep = x.to(DEV).clone()
            picked = ops.add_norm(keep, bd.to(DEV), w.to(DEV), 1e-5, dtype, rows=rows.to(DEV))
            assert torch.equal(keep.cpu(), x) and torch.equal(picked, got[rows.long().to(DEV)])
        for splits in (1, 2, 5):
            part = torch.randn((splits, n, D), generator=gen)
            xs = x.to(DEV).clone()
            got = ops.add_norm(xs, ops.SplitSums(part.to(DEV), torch.bfloat16), w.to(DEV), 1e-5, dtype)
            total = part[0]
            for k in range(1, splits):
                total = total + part[k]
            assert torch.equal(xs.cpu(), x + total)
            want = plain.over_rms((x + total).double(), 1e-5) * w.double()
            assert (got.cpu().double() - want).abs().max() < tol * float(want.abs().max())


def test_gate_between_limits():
    """The gate's own kernel and the one inside the weight-streaming product, on values beyond the limits on both sides."""
    from torchllms_amd.kernels import ops

    gen = torch.Generator().manual_seed(4)
    for n, F in ((3, 24), (7, 5), (1, 1), (300, 1096)):
        both = torch.randn((n, 2 * F), generator=gen) * 3
        for dtype, tol in ((torch.float32, 1e-6), (torch.bfloat16, 8e-3)):
            b = both.to(dtype).double()
            g, u = b[:, :F].clamp(max=1.5), b[:, F:].clamp(-1.5, 1.5)
            want = g * torch.sigmoid(1.702 * g) * (u + 1)
            got = ops.limited_gate_mul(both.to(DEV, dtype), 1.5, 1.702)
            assert (got.cpu().double() - want).abs().max() < tol * max(1.0, float(want.abs().max()))
    x, w = torch.randn((5, 256), generator=gen).to(DEV, torch.bfloat16), torch.randn((2 * 80, 256), generator=gen).to(DEV, torch.bfloat16) * 0.2
    want = ops.limited_gate_mul(torch.nn.functional.linear(x.float(), w.float()).to(torch.bfloat16), 1.5, 1.702).float()
    for cols in (8, 16):
        got = ops.gemm_stream_glu(x, w, 4, cols, activation="sigmoid_limited", limit=1.5, slope=1.702)
        assert (got.float() - want).abs().max() < 2e-2 * float(want.abs().max())


def test_embedding_with_position_vectors():
    from torchllms_amd.kernels import ops

    gen = torch.Generator().manual_seed(6)
    for D in (64, 50, 4096):
        table, pos = torch.randn((30, D), generator=gen), torch.randn((40, D), generator=gen)
        tokens, at = torch.tensor([3, 29, 0, 3], dtype=torch.int32), torch.tensor([0, 39, 7, 1], dtype=torch.int32)
        for dtype in (torch.float32, torch.bfloat16):
            t, p = table.to(dtype), pos.to(dtype)
            got = ops.embed_scaled(tokens.to(DEV), t.to(DEV), 1.0, at.to(DEV), p.to(DEV))
            assert torch.equal(got.cpu(), t.float()[tokens.long()] + p.float()[at.long()])
            assert torch.equal(ops.embed_scaled(tokens.to(DEV), t.to(DEV), 0.5).cpu(), t.float()[tokens.long()] * 0.5)


def test_router_by_sigmoid_scores_and_weights_of_inputs():
    """The largest sigmoid scores as they are; a pair's expert works on its token's row times its weight, gathered and (few
    pairs) in their own order; results added without a weight."""
    from torchllms_amd.kernels import ops

    gen = torch.Generator().manual_seed(3)
    for E, top in ((10, 3), (12, 1), (6, 6), (70, 8), (512, 2), (1, 1)):
        z = torch.randn((200, E), generator=gen) * 3
        ids, weights = plain.routed_choice(z.double(), top)
        got_ids, got_w = ops.router_topk(z.to(DEV), E, None, top, scores="sigmoid")
        assert torch.equal(got_ids.cpu().long(), ids), (E, top)
        assert (got_w.cpu().double() - weights).abs().max() < 1e-6
    D, F, E, top = 48, 40, 5, 2
    w = {f"e{e}.{n}": torch.randn((F, D) if n != "down" else (D, F), generator=gen) * 0.2 for e in range(E) for n in ("gate", "up", "down")}
    gu = torch.stack([torch.cat([w[f"e{e}.gate"], w[f"e{e}.up"]]) for e in range(E)])
    down = torch.stack([w[f"e{e}.down"] for e in range(E)])
    for n, dtype, tol in ((33, torch.float32, 1e-5), (33, torch.bfloat16, 2e-2), (2, torch.bfloat16, 3e-2)):
        x = torch.randn((n, D), generator=gen).to(dtype)
        ids, weights = plain.routed_choice(torch.randn((n, E), generator=gen), top)
        wd = {k: v.to(dtype).double() for k, v in w.items()}
        want = torch.stack([sum(plain.expert(weights[t, j].double() * x[t : t + 1].double(), wd, f"e{int(ids[t, j])}.")[0] for j in range(top)) for t in range(n)])
        behind = torch.stack([sum(weights[t, j].double() * plain.expert(x[t : t + 1].double(), wd, f"e{int(ids[t, j])}.")[0] for j in range(top)) for t in range(n)])
        assert (want - behind).abs().max() > 5 * tol * want.abs().max()
        xd, idd, wts = x.to(DEV), ids.int().to(DEV), weights.float().to(DEV)
        rows, pos, offsets = ops.expert_gather(xd, idd, E, input_weights=wts)
        y = ops.expert_down_rows(ops.expert_glu_rows(rows, gu.to(DEV, dtype), offsets), down.to(DEV, dtype), offsets)
        got = ops.expert_combine(y, pos, idd, None, E, xd).cpu().double()
        assert (got - want).abs().max() < tol * float(want.abs().max())
        if n == 2:
            y = ops.expert_pair_products(xd, gu.to(DEV, dtype), down.to(DEV, dtype), idd, input_weights=wts)
            own = torch.arange(n * top, dtype=torch.int32, device=DEV).view(n, top)
            got = ops.expert_combine(y, own, idd, None, E, xd).cpu().double()
            assert (got - want).abs().max() < tol * float(want.abs().max())


# ----------------------------------------------------------------------------- far keys, edges, slots, long decoding
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_prompts_with_sharp_attention_and_long_memory(tmp_path, dtype):
    """Sharp scores through the latents and windows of up to 300 positions make queries look at a few keys anywhere, and slow
    decays keep what the first tokens wrote: a lost page, a key one off or a state that was not carried shows at late
    positions; whole, in portions that end at and beside page borders, window edges and segments, and decoded."""
    from torchllms_amd.engine import Engine, StepEntry

    layers = [
        models.layer(_L(8, 32, 32, 48, 64, spread=1.5), models.moe(32, 4, 2, shared=16)),
        models.layer(_W(8, 2, 32, 32, 300, rows=16, most=200, spread=5.0), None),
        models.layer(_M(4, 32, 64, groups=2, conv=4, norm_groups=2), models.dense(80)),
        models.layer(_W(4, 1, 32, 64, 129, rows=10, most=400, spread=5.0), None),
        models.layer(_L(3, 24, 16, 20, 40, spread=1.5), models.dense(64)),
    ]
    cfg_dict = models.model(97, 64, 1e-5, layers + [models.again(layers, 2), models.again(layers, 0)])
    folder = folder_for(dtype, tmp_path / "m", cfg_dict, seed=3)
    cfg, weights = models.read_folder(folder)
    tokens = random_tokens(700, cfg["vocab"], 5)
    truth, scale = truth_of(cfg, weights, {"r": tokens})
    engine = Engine.from_folder(folder, dtype=dtype, page_size=16, num_pages=2 * 45, max_seqs=2)
    tol = FP32_TOL if dtype == "float32" else BF16_TOL
    engine.admit("w")
    whole = engine.step([StepEntry("w", tokens, list(range(700)))]).cpu()
    engine.free("w")
    engine.admit("c")
    rows, at = [], 0
    for n in [16, 15, 1, 2, 30, 33, 31, 64, 63, 1, 129, 127, 2, 100] + [1] * 86:
        rows.append(engine.step([StepEntry("c", tokens[at : at + n], list(range(n)))]).cpu())
        at += n
        engine.cache.check_invariants()
    assert at == 700
    assert [-1 in engine.cache.block_table("c", i) for i, g in enumerate(engine.cache.groups)] == [g.window > 0 for g in engine.cache.groups]  # the windows gave pages back
    cut = torch.cat(rows)
    for name, got in (("whole", whole), ("cut", cut)):
        dists = [distance(got[i], truth["r"][i], scale) for i in range(700)]
        if dtype == "float32":
            assert max(dists) < tol, f"{name}: distance {max(dists)} at {dists.index(max(dists))}"
        else:
            assert_within_rounding(dists, tol, name)
    if dtype == "float32":
        assert torch.equal(whole, cut)
        # dropping what lies far back would be seen: the truth of the last 100 tokens alone is another
        short = plain.forward(cfg, weights, tokens[600:])
        assert min(distance(short[i], truth["r"][600 + i], scale) for i in range(50, 100)) > 100 * tol


def test_positions_end_with_their_vectors(tmp_path):
    """The last position runs, the next is refused before anything is launched; no engine can be asked for longer contexts."""
    from torchllms_amd.engine import Engine, StepEntry

    cfg_dict = dict(models.CONFIG_A, max_positions=70)
    folder = models.make_folder(tmp_path / "m", cfg_dict, seed=8)
    cfg, weights = models.read_folder(folder)
    tokens = random_tokens(70, cfg["vocab"], 3)
    truth, scale = truth_of(cfg, weights, {"r": tokens})
    engine = Engine.from_folder(folder, dtype="float32", page_size=8, num_pages=20, max_seqs=2)
    engine.admit("r")
    engine.step([StepEntry("r", tokens[:68], [])])
    got = torch.cat([engine.step([StepEntry("r", [t], [0])]).cpu() for t in tokens[68:]])
    assert max(distance(got[i], truth["r"][68 + i], scale) for i in range(2)) < FP32_TOL
    with pytest.raises(ValueError, match="max_model_len=70"):
        engine.step([StepEntry("r", [1], [0])])
    with pytest.raises(ValueError, match="71 exceeds the 70 positions"):
        Engine.from_folder(folder, dtype="float32", page_size=8, num_pages=20, max_seqs=2, max_model_len=71, beyond_max_positions=True)


def test_a_slot_that_is_used_again_starts_from_zero(tmp_path):
    """One state slot and few pages: each request takes over what the one before left (states, pages of keys) and must
    not see any of it."""
    from torchllms_amd.engine import Engine, StepEntry

    folder = models.make_folder(tmp_path / "m", models.CONFIG_A, seed=8)
    cfg, weights = models.read_folder(folder)
    requests = {f"q{i}": random_tokens(n, cfg["vocab"], 30 + i) for i, n in enumerate([50, 3, 64, 20])}
    truth, scale = truth_of(cfg, weights, requests)
    engine = Engine.from_folder(folder, dtype="float32", page_size=8, num_pages=8, max_seqs=1)
    for rid, toks in requests.items():
        engine.admit(rid)
        head = max(len(toks) - 5, 1)
        rows = [engine.step([StepEntry(rid, toks[:head], list(range(head)))]).cpu()]
        rows += [engine.step([StepEntry(rid, [t], [0])]).cpu() for t in toks[head:]]
        engine.free(rid)
        got = torch.cat(rows)
        assert max(distance(got[i], truth[rid][i], scale) for i in range(len(toks))) < FP32_TOL, rid
    engine.cache.check_invariants()


@pytest.mark.parametrize("name", ["A", "B"])
def test_long_decoding_from_recorded_steps(tmp_path, name):
    """Three requests decode 150 tokens together, over window edges, through layers that use another's tensors: the steps
    are replayed from HIP graphs after the first few, states move on with every replay, pages behind the windows go back,
    and the logits stay the plain model's."""
    from torchllms_amd.engine import Engine, StepEntry

    requests = {f"d{i}": random_tokens(170 + 7 * i, models.CONFIGS[name]["vocab"], 60 + i) for i in range(3)}
    for dtype, tol in (("float32", FP32_TOL), ("bfloat16", BF16_TOL)):
        folder = folder_for(dtype, tmp_path / "m", models.CONFIGS[name], seed=12)
        truth, scale = truth_of(*models.read_folder(folder), requests)
        engine = Engine.from_folder(folder, dtype=dtype, page_size=16, num_pages=40, max_seqs=3)
        for rid in requests:
            engine.admit(rid)
        engine.step([StepEntry(rid, toks[: len(toks) - 150], []) for rid, toks in requests.items()])
        dists = []
        for j in range(150):
            entries = [StepEntry(rid, [toks[len(toks) - 150 + j]], [0]) for rid, toks in requests.items()]
            logits = engine.step(entries).cpu()
            for row, (rid, toks) in zip(logits, requests.items()):
                dists.append(distance(row, truth[rid][len(toks) - 150 + j], scale))
        engine.cache.check_invariants()
        if dtype == "float32":
            assert max(dists) < tol, f"{dtype}: {max(dists)}"
        else:
            assert_within_rounding(dists, tol, dtype)
        assert engine.graphs is not None and any(g.replays > 100 for g in engine.graphs.graphs.values())


# ----------------------------------------------------------------------------- through the entry point
def test_greedy_generation_through_the_entry_point(tmp_path):
    """``LLM.generate``: the scheduler admits, cuts prompts into portions under a small token budget, decodes
    everybody together and frees; the tokens are the plain model's."""
    from torchllms_amd.inference import LLM

    folder = models.make_folder(tmp_path / "m", models.CONFIG_A, seed=4)
    cfg, weights = models.read_folder(folder)
    prompts = [random_tokens(n, cfg["vocab"], 40 + n) for n in (5, 37, 1, 64, 22)]
    new = 20

    def plain_greedy(prompt):
        toks = list(prompt)
        for _ in range(new):
            toks.append(int(plain.forward(cfg, weights, toks)[-1].argmax()))
        return toks[len(prompt):]

    llm = LLM(str(folder), precision="float32", max_len=128, max_bsz=3, page_size=8, max_num_batched_tokens=24)
    results = llm.generate(prompt_token_ids=prompts, temperature=0.0, max_new_tokens=new)
    for p, r in zip(prompts, results):
        assert r.token_ids == plain_greedy(p)
    llm.engine.cache.check_invariants()
    assert llm.engine.cache.live == []
    llm16 = LLM(str(folder), precision="bfloat16", max_len=128, max_bsz=3, page_size=8)
    for p, r in zip(prompts, llm16.generate(prompt_token_ids=prompts, temperature=0.0, max_new_tokens=4)):
        logits = plain.forward(cfg, weights, p)[-1]
        assert logits[r.token_ids[0]] >= logits.max() - 0.1 * float(logits.std())


def test_a_preempted_request_starts_again_from_clean_state(tmp_path):
    """Too few pages for four requests: the scheduler takes the youngest off, gives its pages and its slot away and
    later computes it again from its prompt and what it had generated; the sampled tokens are those of the run with
    room for everybody."""
    from torchllms_amd.inference import LLM

    folder = models.make_folder(tmp_path / "m", models.CONFIG_B, seed=9)
    cfg, _ = models.read_folder(folder)
    prompts = [random_tokens(n, cfg["vocab"], 80 + n) for n in (30, 25, 28, 21)]
    ample = LLM(str(folder), precision="float32", max_len=96, max_bsz=4, page_size=8)
    want = ample.generate(prompt_token_ids=prompts, temperature=0.8, max_new_tokens=30, seed=7)
    tight = LLM(str(folder), precision="float32", max_len=96, max_bsz=4, page_size=8, num_pages=20)
    got = tight.generate(prompt_token_ids=prompts, temperature=0.8, max_new_tokens=30, seed=7)
    assert tight.last_stats["preemptions"] > 0
    assert [r.token_ids for r in got] == [r.token_ids for r in want]
    tight.engine.cache.check_invariants()


def test_generate_command_line_with_random_weights(tmp_path):
    """The generate program given nothing but a config.json: ``--random-weights --seed`` draws the weights that
    ``write_model_folder`` would write for that seed, so the plain model can say which tokens to expect."""
    import json
    import subprocess
    import sys
    from pathlib import Path

    from torchllms_amd.config.mesolix import MesolixConfig
    from torchllms_amd.weights import write_model_folder

    root = Path(__file__).resolve().parent.parent
    folder = tmp_path / "only_config"
    folder.mkdir()
    (folder / "config.json").write_text(json.dumps(models.CONFIG_C))
    prompt = random_tokens(13, models.CONFIG_C["vocab"], 21)
    proc = subprocess.run(
        [sys.executable, "-m", "torchllms_amd.inference.generate", "--model", str(folder), "--dtype", "float32", "--random-weights",
         "--seed", "7", "--max-new-tokens", "6", "--prompt-ids", *map(str, prompt)],
        capture_output=True, text=True, cwd=root, timeout=300,
    )
    assert proc.returncode == 0, proc.stderr[-2000:]
    got = [int(t) for t in proc.stdout.split()[-6:]]
    written = write_model_folder(tmp_path / "written", MesolixConfig.from_dict(models.CONFIG_C), seed=7, dtype=torch.float32)
    cfg, weights = models.read_folder(written)
    toks = list(prompt)
    for _ in range(6):
        toks.append(int(plain.forward(cfg, weights, toks)[-1].argmax()))
    assert got == toks[len(prompt):]


def test_trace_replay_program(tmp_path):
    """``bin/trace_run`` as a user starts it: steps on standard input, logits files out, a pool for the live tokens
    only, four slots."""
    import json
    import subprocess
    import sys
    from pathlib import Path

    import numpy as np

    folder = models.make_folder(tmp_path / "m", models.CONFIG_C, seed=6)
    cfg, weights = models.read_folder(folder)
    requests = {f"t{i}": random_tokens(n, cfg["vocab"], 70 + i) for i, n in enumerate([80, 33, 120, 64, 50, 90])}
    truth, scale = truth_of(cfg, weights, requests)
    steps = schedules.mixed(requests)
    out = tmp_path / "out"
    prog = Path(__file__).resolve().parents[1] / "bin" / "trace_run"
    run = subprocess.run([sys.executable, str(prog), "--model", str(folder), "--dtype", "float32", "--out", str(out), "--max-tokens",
                          str(schedules.max_live_tokens(steps))], input="\n".join(json.dumps(s) for s in steps) + "\n",
                         capture_output=True, text=True, timeout=600)
    assert run.returncode == 0, run.stderr[-2000:]
    assert [ln for ln in run.stdout.splitlines() if ln.startswith("done")] == [f"done {s['step']}" for s in steps]
    for s, where in zip(steps, schedules.positions_of(steps)):
        if not where:
            continue
        got = torch.from_numpy(np.fromfile(out / f"{s['step']}.f32", dtype="<f4").reshape(len(where), cfg["vocab"]))
        for (rid, pos), row in zip(where, got):
            assert distance(row, truth[rid][pos], scale) < FP32_TOL, (s["step"], rid, pos)


ODD = {
    "width_50": models.model(33, 50, 1e-5, [
        models.layer(_L(3, 10, 6, 11, 14), models.moe(14, 3, 2, shared=9)),
        models.layer(_M(3, 14, 6, groups=3, conv=3, norm_groups=7), models.dense(30)),
        models.layer(_W(2, 1, 12, 10, 7, rows=5, most=9), None),
    ]),
    "width_52": models.model(70, 52, 1e-5, [
        models.layer(_W(4, 4, 20, 4, 1000, rows=11, most=70), models.dense(21)),
        models.layer(_M(2, 5, 9, conv=2), models.moe(9, 2, 1)),
        models.layer(_L(1, 7, 9, 5, 22), None),
    ]),
}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(ODD))
def test_widths_that_are_no_multiple_of_eight(tmp_path, name, dtype):
    """Rows that no 16-byte load fits, heads of a handful of channels: the kernels' plain forms."""
    from torchllms_amd.engine import Engine, StepEntry

    folder = folder_for(dtype, tmp_path / name, ODD[name], seed=2)
    cfg, weights = models.read_folder(folder)
    tokens = random_tokens(90, cfg["vocab"], 4)
    truth, scale = truth_of(cfg, weights, {"r": tokens})
    engine = Engine.from_folder(folder, dtype=dtype, page_size=4, num_pages=60, max_seqs=2)
    engine.admit("whole")
    whole = engine.step([StepEntry("whole", tokens, list(range(90)))]).cpu()
    engine.admit("cut")
    rows, at = [], 0
    for n in (3, 2, 40, 1, 1, 35, 1, 1, 1, 5):
        rows.append(engine.step([StepEntry("cut", tokens[at : at + n], list(range(n)))]).cpu())
        at += n
    assert at == 90
    cut = torch.cat(rows)
    for what, got in (("whole", whole), ("cut", cut)):
        dists = [distance(got[i], truth["r"][i], scale) for i in range(90)]
        if dtype == "float32":
            assert max(dists) < FP32_TOL, f"{name}/{what}: {max(dists)}"
        else:
            assert_within_rounding(dists, 2 * BF16_TOL, f"{name}/{what}")
    if dtype == "float32":
        assert torch.equal(whole, cut)


# ----------------------------------------------------------------------------- random configurations
def random_config(seed: int) -> dict:
    """A Mesolix configuration drawn from a seed: every size, constant and the order of layers."""
    import random

    rng = random.Random(seed)
    layers = []
    for _ in range(rng.randint(1, 5)):
        kind = rng.choice(["latent", "windowed", "mamba"])
        if kind == "latent":
            mixer = _L(rng.choice([1, 2, 3, 8, 18]), rng.choice([8, 20, 32, 64]), rng.choice([8, 20, 32, 72]), rng.choice([16, 40, 64]),
                       rng.choice([16, 32, 40, 64, 96, 128, 256, 300]), spread=rng.choice([0.5, 1.0]))
        elif kind == "windowed":
            kv = rng.choice([1, 2, 3])
            dim = rng.choice([8, 16, 24, 32, 48, 64, 128])
            rows = rng.choice([1, 2, 5, 8, 16, 31, 32])
            mixer = _W(kv * rng.choice([1, 2, 4]), kv, dim, rng.choice([dim, dim, 2 * dim if dim <= 64 else dim, 8, 40, 72]),
                       rng.choice([1, 7, 16, 33, 64, 129, 1000]), rows=rows, most=rows // 2 + rng.choice([1, 2, 17, 100, 500]),
                       spread=rng.choice([0.5, 2.0, 4.0]))
        else:
            groups = rng.choice([1, 2, 3])
            heads, dv = groups * rng.choice([1, 2, 4]), rng.choice([4, 8, 20, 32, 64, 100, 128, 136])
            parts = [p for p in (1, 2, 3, 4, 8) if (heads * dv) % p == 0]
            mixer = _M(heads, dv, rng.choice([4, 8, 20, 32, 64, 96, 128, 192]), groups=groups, conv=rng.choice([1, 2, 4, 5]), norm_groups=rng.choice(parts))
        experts = rng.choice([1, 2, 4, 6, 9, 12])
        mlp = rng.choice([None, models.dense(rng.choice([24, 60, 128]), limit=rng.choice([0.3, 0.8, 5.0])),
                          models.moe(rng.choice([16, 24, 40, 72]), experts, rng.randint(1, experts), shared=rng.choice([None, 24, 30]))])
        layers.append(models.layer(mixer, mlp))
    for _ in range(rng.choice([0, 0, 1, 2])):
        layers.append(models.again(layers, rng.choice([i for i, entry in enumerate(layers) if "weights_of" not in entry])))
    return models.model(rng.choice([50, 97, 256, 301]), rng.choice([40, 64, 72, 96, 128, 160]), rng.choice([1e-5, 1e-6, 1e-3]), layers)


@pytest.mark.parametrize("seed", range(10))
def test_random_configurations(tmp_path, seed):
    """Sizes nobody chose: a prompt whole, and the same tokens in portions, single tokens and beside a second
    request, in both dtypes, against the plain model."""
    import random

    from torchllms_amd.engine import Engine, StepEntry

    cfg_dict = random_config(5000 + seed)
    rng = random.Random(seed)
    requests = {"a": random_tokens(rng.randint(120, 330), cfg_dict["vocab"], seed), "b": random_tokens(rng.randint(20, 90), cfg_dict["vocab"], seed + 50)}
    page = rng.choice([4, 8, 16, 32])
    # (drawn constants can let a head's norm divide by little, where 32-bit rounding is magnified several times, in the
    # plain model run in 32-bit as well; a wrong key, mask or state is a hundred times the bound)
    for dtype, tol in (("float32", 1e-4), ("bfloat16", 2 * BF16_TOL)):
        folder = folder_for(dtype, tmp_path / "m", cfg_dict, seed=seed)
        truth, scale = truth_of(*models.read_folder(folder), requests)
        seen = []
        engine = Engine.from_folder(folder, dtype=dtype, page_size=page, num_pages=2 * (-(-420 // page)) + 4, max_seqs=3)
        engine.admit("w")
        whole = engine.step([StepEntry("w", requests["a"], list(range(len(requests["a"]))))]).cpu()
        engine.free("w")
        for i, row in enumerate(whole):
            d = distance(row, truth["a"][i], scale)
            seen.append(d)
            assert dtype == "bfloat16" or d < tol, f"{dtype} whole at {i}: {d}  {cfg_dict}"
        at = {"a": 0, "b": 0}
        engine.admit("a")
        engine.admit("b")
        while at["a"] < len(requests["a"]) or at["b"] < len(requests["b"]):
            entries = []
            for rid in ("a", "b"):
                left = len(requests[rid]) - at[rid]
                if left and rng.random() < 0.8:
                    n = min(left, rng.choice([1, 1, 2, 3, 17, 40, 64, 130]))
                    entries.append(StepEntry(rid, requests[rid][at[rid] : at[rid] + n], list(range(n))))
            if not entries:
                continue
            logits = engine.step(entries).cpu()
            engine.cache.check_invariants()
            k = 0
            for e in entries:
                for w in e.want:
                    d = distance(logits[k], truth[e.rid][at[e.rid] + w], scale)
                    seen.append(d)
                    assert dtype == "bfloat16" or d < tol, f"{dtype} {e.rid} at {at[e.rid] + w} in a step of {[len(x.tokens) for x in entries]}: {d}  {cfg_dict}"
                    if dtype == "float32" and e.rid == "a":
                        assert torch.equal(logits[k], whole[at["a"] + w])
                    k += 1
                at[e.rid] += len(e.tokens)
        if dtype == "bfloat16":
            assert_within_rounding(seen, tol, f"{cfg_dict}")
        del engine
