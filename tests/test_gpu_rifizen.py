"""The Rifizen decoder in the engine against the plain implementation of tests/plain/rifizen.py: every mechanism alone,
whole prompts against decoding token by token, portions down to two tokens, mixed batches with pages and state slots
that are used again, keys far back and at the edges of every window, loops, long decoding from recorded graphs, and
greedy generation through ``LLM.generate`` and the scheduler; on three small configurations that differ in every size,
in 32-bit and in bfloat16.  The kernels that are new with this design are also compared alone, on inputs made so that a
fault shows."""

import pytest
import torch

from . import rifizen_models as models
from . import schedules
from .helpers import random_tokens
from .plain import rifizen as plain
from .test_gpu_engine import run_trace

pytestmark = pytest.mark.gpu

LENGTHS = {"A": [70, 41, 100, 35, 50, 33], "B": [66, 40, 130, 35, 90], "C": [45, 150, 37, 64, 120]}
#: distances are measured as a replay of a trace is judged: the difference of two rows of logits with its mean taken
#: off, root mean square over the vocabulary, over the root mean square of the truth
FP32_TOL = 3e-5
BF16_TOL = 5e-2
DEV = "cuda:0"


def distance(got: torch.Tensor, truth: torch.Tensor, scale: float) -> float:
    d = got.double() - truth.double()
    d = d - d.mean()
    return float(d.pow(2).mean().sqrt()) / scale


def truth_of(cfg, weights, requests):
    out = {rid: plain.forward(cfg, weights, toks) for rid, toks in requests.items()}
    scale = float(torch.cat([(t - t.mean(-1, keepdim=True)).flatten() for t in out.values()]).pow(2).mean().sqrt())
    return out, scale


def folder_for(dtype, path, cfg_dict, **kw):
    """The model a run in ``dtype`` is compared on: bfloat16 runs get routers whose choice no rounding changes, the 32-bit
    runs, which are the sharp ones, get routers whose choice changes from token to token."""
    return models.make_folder(path / dtype, cfg_dict, decisive_router=dtype == "bfloat16", **kw)


def assert_within_rounding(dists, tol, what):
    """bfloat16 against the plain model: all but 5% of the positions lie under the bound, and their mean under half of
    it (a position or two, the same in every schedule, where a norm divides by little, magnify rounding; a fault of a
    kernel moves every position)."""
    d = sorted(dists)
    keep = d[: max(len(d) - max(len(d) * 5 // 100, 1), 1)]
    assert keep[-1] < tol, f"{what}: {sum(x >= tol for x in d)} of {len(d)} positions at or over {tol}, the worst kept {keep[-1]}"
    assert sum(keep) / len(keep) < tol / 2, f"{what}: mean distance {sum(keep) / len(keep)}"


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
    tmp = tmp_path_factory.mktemp("rifizen")
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
_L, _R, _TL, _TR = models.left, models.right, models.TINY_LEFT, models.TINY_RIGHT
ALONE = {
    "attention": models.layer(_L(4, 2, 24, 40, 30), _TR),
    "attention_one_head": models.layer(_L(1, 1, 16, 16, 100, softcap=3.0), _TR),
    "attention_odd_sizes": models.layer(_L(3, 1, 10, 6, 19), _TR),
    "attention_sees_itself_alone": models.layer(_L(4, 2, 16, 16, 1), _TR),
    "attention_no_edge": models.layer(_L(5, 5, 16, 24, 5000), _TR),
    "attention_matrix_cores": models.layer(_L(8, 2, 64, 64, 50), _TR),
    "attention_matrix_cores_wide": models.layer(_L(6, 1, 128, 128, 130, softcap=20.0), _TR),
    "attention_matrix_cores_wider_values": models.layer(_L(4, 2, 32, 64, 45), _TR),
    "attention_matrix_cores_256": models.layer(_L(2, 1, 256, 256, 70), _TR),
    "retention": models.layer(_TL, _R(4, 24, 40, [0.9, 0.99, 0.999, 0.5])),
    "retention_matrix_cores": models.layer(_TL, _R(3, 128, 128, [0.9, 0.995, 0.9998])),
    "retention_wide_values": models.layer(_TL, _R(2, 64, 200, [0.97, 0.9995], dims=32)),
    "retention_wide_keys": models.layer(_TL, _R(1, 256, 32, [0.995], dims=100)),
    "retention_odd_sizes": models.layer(_TL, _R(3, 18, 70, [0.9, 0.99, 0.7], dims=6)),
    "retention_no_rotation": models.layer(_TL, _R(2, 32, 64, [0.999, 0.9], dims=0)),
    "retention_keeps_all_and_nothing": models.layer(_TL, _R(2, 16, 16, [1.0, 0.0])),
    "both_sides": models.layer(_L(2, 1, 32, 32, 16), _R(2, 32, 16, [0.99, 0.8])),
    "dense": models.layer(_TL, _TR, models.dense(136)),
    "dense_narrow": models.layer(_TL, _TR, models.dense(9)),
    "routed": models.layer(_TL, _TR, models.moe(40, 8, 3)),
    "routed_one_choice": models.layer(_TL, _TR, models.moe(33, 5, 1)),
    "routed_all_chosen": models.layer(_TL, _TR, models.moe(16, 3, 3)),
    "routed_many": models.layer(_TL, _TR, models.moe(8, 70, 6)),
}
LOOPS = {"both_sides": (0, 1, 4), "dense": (0, 1, 1), "routed": (0, 1, 2)}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("what", sorted(ALONE))
def test_a_mechanism_alone(tmp_path, what, dtype):
    """A model of one layer (for some in a loop), a prompt in one step and, in a second request, the same tokens in
    portions and one by one."""
    from torchllms_amd.engine import Engine, StepEntry

    folder = folder_for(dtype, tmp_path / what, models.single_layer(ALONE[what], loop=LOOPS.get(what)), seed=5)
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
    # (a head's norm may divide by a root mean square that comes near zero at a position or two, where 32-bit rounding
    # shows larger, in the plain model too: a position's bound is the usual one, or three times what the plain model run
    # in 32-bit is away from the 64-bit truth there)
    own = plain.forward(cfg, weights, tokens, dtype=torch.float32) if dtype == "float32" else None
    for name, got in (("whole", whole), ("cut", cut)):
        dists = [distance(got[i], truth["r"][i], scale) for i in range(len(tokens))]
        if dtype == "float32":
            over = [(i, d) for i, d in enumerate(dists) if d >= max(FP32_TOL, 3 * distance(own[i], truth["r"][i], scale))]
            assert not over, f"{what}/{name}: {over[:5]}"
        else:
            assert_within_rounding(dists, BF16_TOL, f"{what}/{name}")
    if dtype == "float32":
        assert torch.equal(whole, cut)


# ----------------------------------------------------------------------------- the bias by distance in the attention kernels
def _paged(keys, values, page, n_pages, gen):
    """Keys [n, Hk, d] and values [n, Hk, dv] of one request in pages handed out in a shuffled order; the pool holds
    other numbers everywhere else.  Returns (k_pages, v_pages, block table row)."""
    n = keys.shape[0]
    order = torch.randperm(n_pages, generator=gen)[: -(-n // page)]
    k_pages = torch.randn((n_pages, keys.shape[1], page, keys.shape[2]), generator=gen) * 3
    v_pages = torch.randn((n_pages, values.shape[1], page, values.shape[2]), generator=gen) * 3
    for j in range(n):
        k_pages[order[j // page], :, j % page] = keys[j]
        v_pages[order[j // page], :, j % page] = values[j]
    return k_pages, v_pages, order.to(torch.int32)


def _plain_attention(q, keys, values, pos, window, keep, scale, cap, slopes, group):
    """One query [Hq, d] at position ``pos`` over keys [n, Hk, d] / values [n, Hk, dv]: it sees j <= pos with
    pos - j < window or j < keep; a score is capped (cap > 0), then loses its head's slope times the distance."""
    out = []
    js = [j for j in range(pos + 1) if pos - j < window or j < keep]
    dist = torch.tensor([pos - j for j in js], dtype=torch.float64)
    for h in range(q.shape[0]):
        g = h // group
        s = (keys[js, g].double() @ q[h].double()) * scale
        if cap > 0:
            s = cap * torch.tanh(s / cap)
        p = torch.softmax(s - slopes[h] * dist, 0)
        out.append(p @ values[js, g].double())
    return torch.stack(out)


def _edge_queries(positions, keys, Hq, window, keep, scale, slopes, cap, gen):
    """Queries that like the keys on both sides of the window's lower edge (and of the kept positions') more than what
    their distance costs, so that a mask or a distance that is one off decides."""
    d = keys.shape[2]
    q = torch.randn((len(positions), Hq, d), generator=gen)
    for i, p in enumerate(positions):
        edge = [j for j in (p - window + 1, p - window, keep - 1, keep) if 0 <= j <= p]
        for h in range(Hq):
            q[i, h] = sum(keys[j, h // (Hq // keys.shape[1])].float() for j in edge) * (6.0 / (scale * d)) + 0.3 * q[i, h]
    return q


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("Hq,Hk,d,dv,page,keep,cap", [(4, 2, 16, 16, 8, 0, 9.0), (8, 4, 24, 40, 4, 11, 0.0), (6, 2, 64, 32, 16, 5, 20.0), (2, 2, 7, 5, 3, 0, 5.0)])
def test_plain_attention_with_a_bias_by_distance(Hq, Hk, d, dv, page, keep, cap, dtype):
    """A window of 37 over 300 keys (for some with kept first positions, whose distances are the true ones); single
    tokens by one wave, blocks of keys side by side and a prompt's portion through tiles, against the formula and bit by
    bit against each other."""
    from torchllms_amd.kernels import ops

    gen = torch.Generator().manual_seed(Hq * 100 + d)
    n, window, scale = 300, 37, 0.3
    slopes = torch.tensor([0.1 * 2.0 ** -h for h in range(Hq)])
    keys, values = torch.randn((n, Hk, d), generator=gen), torch.randn((n, Hk, dv), generator=gen)
    positions = [0, 5, 10, 11, 12, 36, 37, 38, 46, 47, 48, 63, 64, 100, 128, 200, 255, 256, 299]
    queries = _edge_queries(positions, keys, Hq, window, keep, scale, slopes, cap, gen)
    if dtype == torch.bfloat16:
        keys, values, queries = (t.to(dtype).float() for t in (keys, values, queries))
    args = (keys, values)
    want = torch.stack([_plain_attention(queries[i], *args, p, window, keep, scale, cap, slopes, Hq // Hk) for i, p in enumerate(positions)])
    tol = 1e-5 if dtype == torch.float32 else 2e-2
    for other in (dict(window=window + 1), dict(slopes=slopes * 0), dict(slopes=slopes * 1.5)):  # (they do decide)
        kw = dict(window=window, slopes=slopes, **{}) | other
        off = torch.stack([_plain_attention(queries[i], *args, p, kw["window"], keep, scale, cap, kw["slopes"], Hq // Hk) for i, p in enumerate(positions)])
        assert (want - off).abs().max() > (20 if dtype == torch.float32 else 5) * tol, other
    k_pages, v_pages, table = _paged(keys, values, page, 120, gen)
    kp, vp = k_pages.to(DEV, dtype), v_pages.to(DEV, dtype)
    bt = table.to(DEV).view(1, -1)
    q = queries.reshape(len(positions), Hq * d).to(DEV, dtype)
    pos = torch.tensor(positions, dtype=torch.int32, device=DEV)
    seq = torch.zeros(len(positions), dtype=torch.int32, device=DEV)
    kw = dict(v_head_dim=dv, keep_first=keep, softcap=cap, slopes=slopes.to(DEV))
    alone = ops.attention_generic(q, Hq, Hk, d, kp, vp, seq, pos, bt, window, scale, **kw).float().cpu().view(len(positions), Hq, dv)
    assert (alone.double() - want).abs().max() < tol * max(1.0, float(want.abs().max())), (alone.double() - want).abs().max()
    split = ops.attention_generic_split(q, Hq, Hk, d, kp, vp, seq, pos, bt, window, scale, longest=window, **kw).float().cpu().view_as(alone)
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
            ref = _plain_attention(qs[i].float().cpu().view(Hq, d), *args, ps[i], window, keep, scale, cap, slopes, Hq // Hk)
            assert (one.float().view(Hq, dv).double() - ref).abs().max() < tol * max(1.0, float(ref.abs().max()))


@pytest.mark.parametrize("Hq,Hk,d,dv,page,window,cap", [
    (8, 2, 128, 128, 16, 200, 15.0), (4, 4, 64, 128, 16, 70, 0.0), (16, 1, 64, 64, 8, 1000, 30.0), (4, 2, 256, 256, 16, 100, 10.0),
    (6, 2, 128, 128, 16, 64, 0.0), (2, 2, 32, 96, 16, 33, 6.0), (3, 1, 128, 128, 32, 1, 8.0)])
def test_matrix_core_attention_with_a_bias_by_distance(Hq, Hk, d, dv, page, window, cap):
    """The split-KV decode kernel and the tiled prefill kernel against the plain kernel (which the test above holds
    against the formula): capped and uncapped scores less the distance, queries that like the keys at the window's edges;
    single tokens, and portions that begin before, at and behind the window's first full reach."""
    from torchllms_amd.kernels import ops

    gen = torch.Generator().manual_seed(Hq + d + window)
    n, scale = 700, 0.7 / d ** 0.5
    slopes = torch.tensor([2.0 ** (-8.0 * (h + 1) / Hq) for h in range(Hq)])
    keys = torch.randn((n, Hk, d), generator=gen).to(torch.bfloat16)
    values = torch.randn((n, Hk, dv), generator=gen).to(torch.bfloat16)
    k_pages, v_pages, table = _paged(keys.float(), values.float(), page, 2 * (n // page) + 9, gen)
    kp, vp = k_pages.to(DEV, torch.bfloat16), v_pages.to(DEV, torch.bfloat16)
    bt = table.to(DEV).view(1, -1)
    dev_slopes = slopes.to(DEV)

    def queries_for(positions):
        q = _edge_queries(positions, keys, Hq, window, 0, scale, slopes, cap, gen)
        return q.reshape(len(positions), Hq * d).to(DEV, torch.bfloat16)

    positions = sorted({min(max(p, 0), n - 1) for p in (0, 1, 15, 16, window - 1, window, window + 1, window + 17, 300, 511, 512, 699)})
    q = queries_for(positions)
    pos = torch.tensor(positions, dtype=torch.int32, device=DEV)
    seq = torch.zeros(len(positions), dtype=torch.int32, device=DEV)
    kw = dict(softcap=cap, slopes=dev_slopes)
    want = ops.attention_generic(q, Hq, Hk, d, kp, vp, seq, pos, bt, window, scale, v_head_dim=dv, **kw).float()
    flat = ops.attention_generic(q, Hq, Hk, d, kp, vp, seq, pos, bt, window, scale, v_head_dim=dv, softcap=cap).float()
    assert window == 1 or (want - flat).abs().max() > 0.3  # (the bias does decide)
    for split in (None, 64, 128):
        got = torch.zeros((len(positions), Hq * dv), dtype=torch.bfloat16, device=DEV)
        for at in range(0, dv, d):
            ops.attention_decode(q, Hq, Hk, d, kp, vp, seq, pos, bt, window, scale, min(max(positions) + 1, window + 15), out=got,
                                 split_size=split, v_offset=at, **kw)
        assert (got.float() - want).abs().max() < 3e-2 * max(1.0, float(want.abs().max())), (split, (got.float() - want).abs().max())
    qpt = ops.prefill_queries_per_tile(Hq, Hk, d)
    for first, count in ((0, 700), (0, 40), (3, 90), (window - 1, 130), (window + 20, 77), (500, 200), (690, 10)):
        if first + count > n:
            continue
        ps = list(range(first, first + count))
        q = queries_for(ps)
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


# ----------------------------------------------------------------------------- retention alone
def _retention_inputs(n, H, dk, dv, dims, seed):
    """A projection [n, 2 H dk + 2 H dv] = q | k | v | gate with a key that stands out early and a query that asks for
    it late, and the step's table of cosines and sines."""
    gen = torch.Generator().manual_seed(seed)
    proj = torch.randn((n, 2 * H * dk + 2 * H * dv), generator=gen)
    proj[5, H * dk : 2 * H * dk] *= 4.0
    proj[n - 9, : H * dk] = proj[5, H * dk : 2 * H * dk]
    i = torch.arange(max(dims // 2, 1), dtype=torch.float64)
    ang = torch.arange(n, dtype=torch.float64)[:, None] * (1000.0 ** (-2.0 * i / max(dims, 1)))[None, :]
    table = torch.stack([torch.cos(ang), torch.sin(ang)], dim=-1).float().contiguous()
    return proj, (table if dims else None)


def _plain_retention(proj, H, dk, dv, dims, decay, eps, first=0):
    """Rows ``first ..`` of a sequence as one that starts there (their own positions, a zero state)."""
    proj = proj.double()
    n = proj.shape[0]
    q, k = proj[:, : H * dk].view(n, H, dk), proj[:, H * dk : 2 * H * dk].view(n, H, dk)
    v, g = proj[:, 2 * H * dk : 2 * H * dk + H * dv].view(n, H, dv), proj[:, 2 * H * dk + H * dv :]
    pos = torch.arange(n) + first
    q, k = plain.rotate_half(q, pos, dims, 1000.0), plain.rotate_half(k, pos, dims, 1000.0) * dk ** -0.5
    o = plain.over_rms(plain.retention_states(q, k, v, decay), eps)
    return o.reshape(n, H * dv) * plain.silu(g)


RETENTIONS = [(4, 16, 24, 16, [0.5, 0.9, 0.99, 0.9995]), (1, 200, 33, 64, [0.999]), (3, 7, 5, 0, [0.9, 0.0, 1.0]), (2, 128, 128, 128, [0.99, 0.99995]),
              (2, 64, 300, 32, [0.98, 0.999]), (2, 36, 20, 6, [0.99, 0.7])]


def _run(ops, proj, table, dims, decay, eps, state, rows, slots, H, dk, dv, **kw):
    return ops.retention(proj, 0, H * dk, 2 * H * dk, 2 * H * dk + H * dv, table, dims, decay, eps, state, 4, rows, slots, H, dk, dv, **kw)


@pytest.mark.parametrize("H,dk,dv,dims,decay", RETENTIONS)
def test_retention_kernel(H, dk, dv, dims, decay):
    """One row, the same tokens as steps of one request through another slot (the same bits and the same state), rows of
    several requests; a head that forgets at once beside heads that keep for thousands of tokens."""
    from torchllms_amd.kernels import ops

    n, eps = 300, 1e-5
    proj, table = _retention_inputs(n, H, dk, dv, dims, dk + 2)
    want = _plain_retention(proj, H, dk, dv, dims, decay, eps)
    x, cs, dec = proj.to(DEV), table.to(DEV) if table is not None else None, torch.tensor(decay, device=DEV)
    state = torch.zeros((3, H * dv * dk + 4), device=DEV)
    i32 = lambda *v: torch.tensor(v, dtype=torch.int32, device=DEV)  # noqa: E731
    whole = _run(ops, x, cs, dims, dec, eps, state, i32(0, n), i32(0), H, dk, dv).cpu()
    bound = 2e-4 * float(want.abs().max())
    assert (whole.double() - want).abs().max() < bound, (whole.double() - want).abs().max()
    assert float(state[0, :4].abs().max()) == 0.0 and float(state[1].abs().max()) == 0.0
    state2 = torch.zeros_like(state)
    out, at = [], 0
    for m in [1, 1, 15, 16, 17, 2, 1, 33, 1, 64, 1, 1, 100, 1, 5, 1, 40]:
        cut = cs[at : at + m].contiguous() if cs is not None else None
        out.append(_run(ops, x[at : at + m].contiguous(), cut, dims, dec, eps, state2, i32(0, m), i32(1), H, dk, dv).cpu())
        at += m
    assert at == n
    assert torch.equal(torch.cat(out), whole) and torch.equal(state2[1], state[0])
    batch = _run(ops, x, cs, dims, dec, eps, torch.zeros_like(state), i32(0, 100, 101, n), i32(2, 0, 1), H, dk, dv).cpu()
    assert torch.equal(batch[:100], whole[:100])
    want3 = _plain_retention(proj[101:], H, dk, dv, dims, decay, eps, first=101)
    assert (batch[101:].double() - want3).abs().max() < 2e-4 * float(want3.abs().max())
    if max(decay) > 0.99:  # what lies far back matters
        assert (want3[n - 9 - 101] - want[n - 9]).abs().max() > 1e-2 * want.abs().max()


@pytest.mark.parametrize("H,dk,dv,dims,decay", [(4, 16, 24, 16, [0.5, 0.9, 0.99, 0.9995]), (2, 128, 128, 128, [0.99, 0.99995]), (3, 100, 36, 40, [0.9, 0.0, 1.0]),
                                                (1, 64, 128, 0, [0.999]), (2, 32, 64, 8, [0.9, 0.9999])])
def test_retention_by_segments(H, dk, dv, dims, decay):
    """bfloat16 projections: a prompt's segments side by side against the walk and the formula (of the rounded inputs), the
    state they leave, portions of all lengths that go on from each other's states, single tokens in front of several
    prompts, and the other slots untouched."""
    from torchllms_amd.kernels import ops

    n, eps = 333, 1e-5
    proj, table = _retention_inputs(n, H, dk, dv, dims, dk + 3)
    proj = proj.to(torch.bfloat16)
    want = _plain_retention(proj.float(), H, dk, dv, dims, decay, eps)
    x, cs, dec = proj.to(DEV), table.to(DEV) if table is not None else None, torch.tensor(decay, device=DEV)
    i32 = lambda *v: torch.tensor(v, dtype=torch.int32, device=DEV)  # noqa: E731
    assert ops.retention_segments_supported(torch.bfloat16, dk, dv, dims)

    def segments(*bounds):
        return ops.ScanSegments(list(bounds), DEV, ops.RETENTION_SEGMENT)

    walked, state = torch.zeros((5, H * dv * dk + 4), device=DEV), torch.zeros((5, H * dv * dk + 4), device=DEV)
    by_walk = _run(ops, x, cs, dims, dec, eps, walked, i32(0, n), i32(3), H, dk, dv).float().cpu()
    got = _run(ops, x, cs, dims, dec, eps, state, i32(0, n), i32(3), H, dk, dv, segments=segments(0, n)).float().cpu()
    top = float(want.abs().max())
    assert (got.double() - want).abs().max() < 1e-2 * top and (got - by_walk).abs().max() < 1e-2 * top
    assert (state[3] - walked[3]).abs().max() < 1e-5 * walked[3].abs().max()
    assert float(state[[0, 1, 2, 4]].abs().max()) == 0.0 and float(state[3, :4].abs().max()) == 0.0
    state.zero_()
    out, at = [], 0
    for m in [63, 64, 65, 2, 5, 128, 6]:
        cut = cs[at : at + m].contiguous() if cs is not None else None
        out.append(_run(ops, x[at : at + m].contiguous(), cut, dims, dec, eps, state, i32(0, m), i32(2), H, dk, dv, segments=segments(0, m)).float().cpu())
        at += m
    assert at == n
    assert (torch.cat(out).double() - want).abs().max() < 1e-2 * top
    assert (state[2] - walked[3]).abs().max() < 1e-5 * walked[3].abs().max()
    # two single tokens, then two prompts of one step
    state = torch.zeros_like(walked)
    mixed = _run(ops, x, cs, dims, dec, eps, state, i32(0, 1, 2, 100, n), i32(4, 0, 2, 1), H, dk, dv, segments=segments(2, 100, n), single_rows=2).float().cpu()
    for lo, hi in ((0, 1), (1, 2), (2, 100), (100, n)):
        ref = _plain_retention(proj[lo:hi].float(), H, dk, dv, dims, decay, eps, first=lo)
        assert (mixed[lo:hi].double() - ref).abs().max() < 1e-2 * float(ref.abs().max()), (lo, hi)
    assert float(state[3].abs().max()) == 0.0


# ----------------------------------------------------------------------------- the small kernels
@pytest.mark.parametrize("D", [64, 50, 1000, 1024, 2048, 4096, 8192, 4100, 20])
def test_pair_of_norms_into_the_stream(D):
    """Both results normed, their weighted sum normed again into the 32-bit stream, a vector added, the next norm's rows;
    without the vector and without a next norm; many rows and one give the same bits."""
    from torchllms_amd.kernels import ops

    gen = torch.Generator().manual_seed(D)
    n = 37
    a, b, x = (torch.randn((n, D), generator=gen) * s for s in (1.0, 30.0, 2.0))
    wa, wb, wp, wn, add = (torch.randn(D, generator=gen) for _ in range(5))
    rms = lambda z, e: z / torch.sqrt((z * z).mean(-1, keepdim=True) + e)  # noqa: E731
    for dtype, tol in ((torch.float32, 1e-5), (torch.bfloat16, 2e-2)):
        ad, bd = a.to(dtype).double(), b.to(dtype).double()
        y = 0.5 * rms(ad, 1e-5) * wa.double() + 0.25 * rms(bd, 1e-3) * wb.double()
        for vec in (None, add):
            new = x.double() + rms(y, 1e-6) * wp.double() + (vec.double() if vec is not None else 0.0)
            want = rms(new, 1e-4) * wn.double()
            xs = x.to(DEV).clone()
            rest = (wp.to(DEV), 1e-6)
            vd = vec.to(DEV) if vec is not None else None
            pair = lambda s, lo, hi, **kw: ops.pair_norm_add_norm(s, a.to(DEV, dtype)[lo:hi].contiguous(), wa.to(DEV), 1e-5, 0.5,  # noqa: E731
                                                                  b.to(DEV, dtype)[lo:hi].contiguous(), wb.to(DEV), 1e-3, 0.25, *rest, add=vd, **kw)
            rows = pair(xs, 0, n, next_weight=wn.to(DEV), next_eps=1e-4)
            assert (xs.cpu().double() - new).abs().max() < 1e-5 * float(new.abs().max())
            assert rows.dtype == dtype and (rows.cpu().double() - want).abs().max() < tol * float(want.abs().max())
            one = x.to(DEV)[5:6].clone()
            assert torch.equal(pair(one, 5, 6, next_weight=wn.to(DEV), next_eps=1e-4), rows[5:6]) and torch.equal(one, xs[5:6])
            alone = x.to(DEV).clone()
            assert pair(alone, 0, n) is None and torch.equal(alone, xs)
            # the branch as one result
            single = x.double() + rms(bd, 1e-6) * wp.double() + (vec.double() if vec is not None else 0.0)
            xs = x.to(DEV).clone()
            rows = ops.post_norm_add_norm(xs, b.to(DEV, dtype), *rest, wn.to(DEV), 1e-4, add=vd)
            assert (xs.cpu().double() - single).abs().max() < 1e-5 * float(single.abs().max())
            assert (rows.cpu().double() - rms(single, 1e-4) * wn.double()).abs().max() < tol * 4 * float(wn.abs().max())


def test_squared_relu():
    from torchllms_amd.kernels import ops

    for shape in ((3, 24), (7, 5), (1, 1), (300, 4096)):
        x = torch.randn(shape, generator=torch.Generator().manual_seed(shape[1]))
        for dtype in (torch.float32, torch.bfloat16):
            got = ops.relu_square_(x.to(DEV, dtype)).cpu()
            want = torch.relu(x.to(dtype).float()) ** 2
            assert torch.equal(got, want.to(dtype))


def test_router_with_a_bias_against_the_plain_choice():
    """Biases that turn the choice, also where the score without them is vanishing."""
    from torchllms_amd.kernels import ops

    gen = torch.Generator().manual_seed(3)
    for E, top in ((10, 3), (12, 2), (6, 6), (70, 8), (512, 1), (1, 1)):
        z = torch.randn((200, E), generator=gen) * 3
        bias = torch.randn(E, generator=gen) * 4
        z[:20] *= 10.0
        ids, weights = plain.routed_choice(z.double() + bias.double(), top)
        got_ids, got_w = ops.router_topk(z.to(DEV), E, None, top, normalize=True, bias=bias.to(DEV))
        assert torch.equal(got_ids.cpu().long(), ids), (E, top)
        assert (got_w.cpu().double() - weights).abs().max() < 1e-5
        if 1 < top < E:
            assert not torch.equal(plain.routed_choice(z.double(), top)[0], ids)


# ----------------------------------------------------------------------------- far keys, edges, slots, long decoding
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_prompts_with_sharp_attention_and_long_memory(tmp_path, dtype):
    """Sharp scores under small slopes make queries look at a few keys anywhere in windows of up to 300 positions, and
    decays near one keep what the first tokens wrote: a lost page, a key one off or a state that was not carried shows
    at late positions; whole, in portions that end at and beside page borders, window edges and segments, and decoded."""
    from torchllms_amd.engine import Engine, StepEntry

    cfg_dict = models.model(97, 64, 1e-5, [
        models.layer(_L(8, 2, 32, 32, 300, spread=5.0, softcap=15.0), _R(2, 32, 32, [0.995, 0.9998]), models.moe(32, 4, 2)),
        models.layer(_L(4, 1, 32, 64, 129, spread=5.0, softcap=12.0), _R(3, 64, 24, [0.9, 0.999, 0.9999], dims=16, base=1e5), None),
        models.layer(_L(2, 2, 24, 16, 257, spread=4.0, softcap=20.0), _R(1, 20, 140, [0.9995]), models.dense(80)),
    ], loop=(1, 3, 2))
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
    assert all(-1 in engine.cache.block_table("c", g) for g in range(len(engine.cache.groups)))  # the windows gave pages back
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
    """Three requests decode 150 tokens together, over window edges, through a loop (A): the steps are replayed from HIP
    graphs after the first few, states move on with every replay, pages behind the windows go back, and the logits stay
    the plain model's."""
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

    from torchllms_amd.config.rifizen import RifizenConfig
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
    written = write_model_folder(tmp_path / "written", RifizenConfig.from_dict(models.CONFIG_C), seed=7, dtype=torch.float32)
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


def test_a_step_vector_before_layers_of_another_arrangement(tmp_path):
    """The order's step vectors are the model's, not the design's: layers with one norm before each branch, run twice in
    a row, get them too (added by the model where no layer's kernel does it)."""
    from dataclasses import replace

    from torchllms_amd.config.llama import LlamaConfig, llama_model_spec
    from torchllms_amd.config.registry import get_architecture
    from torchllms_amd.config.spec import LayerRun
    from torchllms_amd.engine import Engine, StepEntry
    from torchllms_amd.parts.model import Model
    from torchllms_amd.weights.random_init import random_tensors

    from .helpers import TINY_B

    cfg = LlamaConfig.from_dict(TINY_B)
    base = llama_model_spec(cfg)
    order = [LayerRun(0), LayerRun(1, step_vector=1), LayerRun(1, step_vector=0), LayerRun(2)]
    logits = {}
    for scale in (0.0, 1.0):
        spec = replace(base, order=order, step_vectors=2)
        tensors = random_tensors(Model(spec).param_specs(), 3, torch.float32)
        tensors["loop.step"] = tensors["loop.step"] * 50.0 * scale
        arch = replace(get_architecture("LlamaForCausalLM"), model_spec=lambda _cfg, spec=spec: spec)
        engine = Engine(arch, cfg, {k: v.to(DEV) for k, v in tensors.items()}, torch.float32, page_size=8, num_pages=16, max_seqs=2)
        tokens = random_tokens(40, TINY_B["vocab_size"], 2)
        engine.admit("w")
        whole = engine.step([StepEntry("w", tokens, list(range(40)))]).cpu()
        engine.admit("c")
        cut = torch.cat([engine.step([StepEntry("c", tokens[:30], list(range(30)))]).cpu()]
                        + [engine.step([StepEntry("c", [t], [0])]).cpu() for t in tokens[30:]])
        assert torch.equal(whole, cut)
        logits[scale] = whole
    assert (logits[0.0] - logits[1.0]).abs().max() > 1e-2


ODD = {
    "width_50": models.model(33, 50, 1e-5, [
        models.layer(_L(3, 1, 10, 6, 9), _R(2, 6, 10, [0.9, 0.99]), models.moe(14, 3, 2)),
        models.layer(_L(2, 1, 12, 10, 7), _R(3, 14, 5, [0.8, 0.95, 0.99], dims=4), models.dense(30)),
        models.layer(_L(1, 1, 6, 7, 11), _R(1, 3, 9, [0.97], dims=2), None),
    ], loop=(1, 2, 2)),
    "width_52": models.model(70, 52, 1e-5, [
        models.layer(_L(2, 2, 4, 12, 5), _R(2, 4, 4, [0.5, 0.999]), models.dense(21)),
        models.layer(_L(4, 4, 20, 4, 1000), _R(1, 12, 8, [0.99], dims=8), models.moe(9, 2, 1)),
    ], loop=(0, 2, 2)),
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
    """A Rifizen configuration drawn from a seed: every size, constant, the order of layers and the loop."""
    import random

    rng = random.Random(seed)
    layers = []
    n = rng.randint(1, 5)
    for _ in range(n):
        kv = rng.choice([1, 2, 3])
        dim = rng.choice([8, 16, 24, 32, 48, 64, 128])
        lf = _L(kv * rng.choice([1, 2, 4]), kv, dim, rng.choice([dim, dim, 2 * dim if dim <= 64 else dim, 8, 40, 72]),
                rng.choice([1, 7, 16, 33, 64, 129, 1000]), spread=rng.choice([0.5, 2.0, 4.0]), softcap=rng.choice([2.0, 10.0, 50.0]))
        heads, dk = rng.choice([1, 2, 3, 5]), rng.choice([4, 8, 20, 32, 64, 96, 128, 192])
        rt = _R(heads, dk, rng.choice([8, 24, 32, 64, 100, 128, 136]), [rng.choice([0.3, 0.5, 0.9, 0.97, 0.99, 0.999, 1.0]) for _ in range(heads)],
                dims=rng.choice([0, dk // 4 * 2, dk]), base=rng.choice([100.0, 10000.0, 1000000.0]))
        experts = rng.choice([1, 2, 4, 6, 9, 12])
        mlp = rng.choice([None, models.dense(rng.choice([24, 60, 128])), models.moe(rng.choice([16, 24, 40, 72]), experts, rng.randint(1, experts))])
        layers.append(models.layer(lf, rt, mlp))
    start = rng.randint(0, n - 1)
    loop = rng.choice([None, (start, rng.randint(start + 1, n), rng.choice([1, 2, 3]))])
    return models.model(rng.choice([50, 97, 256, 301]), rng.choice([40, 64, 72, 96, 128, 160]), rng.choice([1e-5, 1e-6, 1e-3]), layers, loop=loop)


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
