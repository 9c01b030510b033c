"""Lukupel on the GPU against the plain implementation (tests/plain_lukupel.py): every mechanism alone and together, under
every way of cutting requests into steps, in 32-bit and in bfloat16."""
from __future__ import annotations

import copy

import numpy as np
import pytest
import torch

import lukupel_models as lm
import plain_lukupel as plain
import replay

pytestmark = pytest.mark.gpu

F32_TOL = 2e-4          # of a row's root mean square; honest 32-bit arithmetic is at 1e-5
# bfloat16 against the unrounded plain model, in units of what rounding alone does: the plain model with the values
# that are kept in bfloat16 rounded (narrow models with weights of order one; a head whose read all but cancels is normed to
# full size, rounding errors and all, so single rows stray far while the others stay close). The average row and the row
# that 97 in 100 stay below are held; a fault of a kernel moves many rows by their whole size.
BF16_MEAN, BF16_MOST, BF16_FLOOR = 1.5, 2.0, 4e-3


def _engine(tmp_path, cfg, seed, dtype, weights=None, **kw):
    from llmengine import Engine
    store = torch.float32 if dtype == "fp32" else torch.bfloat16
    folder, weights = lm.write_model(tmp_path, cfg, seed, store, weights)
    return Engine(folder, dtype, deterministic=True, **kw), weights


def _tokens(n, vocab, seed):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def _reference(cfg, weights, requests):
    w = {k: v.float() for k, v in weights.items()}
    return {rid: plain.forward(cfg, w, ids).numpy() for rid, ids in requests.items()}


def _honest(cfg, weights, requests, ref):
    """(average, 97 in 100) of the errors of rounding alone."""
    with plain.bfloat16_storage():
        e = _errors(_rows(_reference(cfg, weights, requests)), ref)
    return float(np.mean(e)), float(np.quantile(e, 0.97))


def _as_rounding(got, ref, honest) -> bool:
    e = _errors(got, ref)
    return np.mean(e) < BF16_MEAN * honest[0] + BF16_FLOOR and np.quantile(e, 0.97) < BF16_MOST * honest[1] + 2 * BF16_FLOOR


def _errors(got: dict, ref: dict) -> list[float]:
    return [float(np.sqrt(np.mean((row - ref[rid][pos]) ** 2)) / np.sqrt(np.mean(ref[rid][pos] ** 2)))
            for rid, rows in got.items() for pos, row in rows.items()]


def _worst(got, ref) -> float:
    return max(_errors(got, ref))


def _mean(got, ref) -> float:
    return float(np.mean(_errors(got, ref)))


def _covered(got: dict, requests: dict) -> bool:
    return all(sorted(got[rid]) == list(range(len(ids))) for rid, ids in requests.items())


def _stacked(got: dict) -> dict:
    return {rid: np.stack([rows[p] for p in sorted(rows)]) for rid, rows in got.items()}


def _rows(stacked: dict) -> dict:
    return {rid: {p: rows[p] for p in range(len(rows))} for rid, rows in stacked.items()}


def _pool(engine, steps, page, slots):
    """As many pages as the live requests need and `slots` state slots: pages and slots are used again."""
    return engine.new_cache(replay.trace_peak_tokens(steps, page) // page, page, slots)


ONE_LAYER = {
    "chunked": lm.config([lm.chunked(ff=None)]),
    "chunked_sharp": lm.config([lm.chunked(chunk=9, sharp=4.0, ff=None)]),
    "chunked_without_chunks": lm.config([lm.chunked(chunk=0, sharp=3.0, ff=None)]),
    "chunked_chunks_of_one": lm.config([lm.chunked(chunk=1, ff=None)]),
    "chunked_chunks_of_a_page": lm.config([lm.chunked(chunk=8, sharp=3.0, ff=None)]),
    "chunked_one_long_chunk": lm.config([lm.chunked(chunk=500, ff=None)]),
    "chunked_no_rotation_one_head": lm.config([lm.chunked(heads=1, kv_heads=1, dim=20, vdim=20, dims=0, chunk=17, sharp=3.0, ff=None)]),
    "chunked_whole_head_rotated_no_factor": lm.config([lm.chunked(heads=6, kv_heads=3, dim=8, vdim=6, dims=8, factor=0, chunk=12, ff=None)]),
    "chunked_wide_heads": lm.config([lm.chunked(heads=2, kv_heads=1, dim=136, vdim=70, dims=70, chunk=19, scale=0.2, ff=None)], width=36),
    "memory": lm.config([lm.mlstm()]),
    "memory_one_head_of_one": lm.config([lm.mlstm(heads=1, dim=1, vdim=1)]),
    "memory_wide": lm.config([lm.mlstm(heads=1, dim=70, vdim=40, gate_cap=20.0)]),
    "memory_widest_keys": lm.config([lm.mlstm(heads=2, dim=256, vdim=3)]),
    "memory_many_small_heads": lm.config([lm.mlstm(heads=9, dim=4, vdim=2, gate_cap=1.0)]),
    "memory_wide_values": lm.config([lm.mlstm(heads=2, dim=6, vdim=300)]),
    "memory_gates_far_apart": lm.config([lm.mlstm(heads=4, gate_cap=40.0)], embedding_scale=12.0),
    "squared_rectifier": lm.config([lm.chunked(ff=24)]),
    "squared_rectifier_behind_a_memory": lm.config([lm.mlstm(ff=33)]),
    "one_layer_three_times": lm.config([lm.mlstm(ff=12), lm.mlstm(ff=12, weights_of=0), lm.mlstm(ff=12, weights_of=0)]),
    "a_chunked_layer_twice": lm.config([lm.chunked(chunk=7, ff=None), lm.mlstm(), lm.chunked(chunk=7, ff=None, weights_of=0)]),
    "tensors_of_a_later_layer": lm.config([lm.mlstm(weights_of=1), lm.mlstm()]),
    "width_of_30_nothing_scaled": lm.config([lm.chunked(heads=5, kv_heads=5, dim=6, vdim=6, dims=2, ff=9), lm.mlstm()], width=30, vocab=33,
                                            residual_mult=1.0, embedding_scale=1.0),
    "logits_far_above_the_cap": lm.config([lm.mlstm()], logit_softcap=0.5),
}


@pytest.mark.parametrize("name", sorted(ONE_LAYER))
def test_each_mechanism_alone_whole_token_by_token_and_in_portions(tmp_path, name):
    cfg = ONE_LAYER[name]
    engine, weights = _engine(tmp_path, cfg, 3, "fp32")
    requests = {"a": _tokens(41, cfg["vocab"], 1), "b": _tokens(1, cfg["vocab"], 2)}
    ref = _reference(cfg, weights, requests)
    for steps in (replay.whole(requests), replay.tail_one_by_one(requests, tail=40), replay.portions(requests),
                  replay.portions(requests, sizes=(2,))):
        got = replay.run_trace(engine, _pool(engine, steps, 8, 2), steps)
        assert _covered(got, requests)
        assert _worst(got, ref) < F32_TOL


@pytest.mark.parametrize("dtype", ["fp32", "bf16"])
@pytest.mark.parametrize("cfg_name", ["MIXED", "ALIGNED"])
def test_every_schedule_gives_the_plain_logits(tmp_path, cfg_name, dtype):
    cfg = getattr(lm, cfg_name)
    engine, weights = _engine(tmp_path, cfg, 11, dtype)
    V = cfg["vocab"]
    requests = {"long": _tokens(150, V, 5), "one": _tokens(1, V, 6), "two": _tokens(2, V, 7), "mid": _tokens(49, V, 8),
                "page": _tokens(32, V, 9), "more": _tokens(65, V, 10)}
    ref = _reference(cfg, weights, requests)
    honest = _honest(cfg, weights, requests, ref) if dtype == "bf16" else None
    schedules = {
        "whole": replay.whole(requests),
        "tail": replay.tail_one_by_one(requests, tail=40),
        "portions": replay.portions(requests),
        "portions of two": replay.portions(requests, sizes=(2,)),
        "mixed": replay.mixed(requests, max_live=3, seed=1),
        "mixed, other cuts": replay.mixed(requests, max_live=2, sizes=(2, 17, 3, 61), seed=2),
    }
    first = None
    for what, steps in schedules.items():
        for page in (16, 8):
            cache = _pool(engine, steps, page, 3)
            got = replay.run_trace(engine, cache, steps)
            assert _covered(got, requests), what
            if dtype == "fp32":
                assert _worst(got, ref) < F32_TOL, (what, page)
            else:
                first = first or _stacked(got)
                assert _as_rounding(got, ref, honest) and _as_rounding(got, first, honest), (what, page)
            assert not cache.manager.live_requests()


@pytest.mark.parametrize("seed", range(10))
def test_configurations_drawn_at_random(tmp_path, seed):
    """Layers of both kinds in any order with sizes, head counts, chunks and constants drawn at random, in both precisions
    against the plain model, with prompts long enough for the memory's chunks."""
    cfg = lm.random_config(seed)
    V = cfg["vocab"]
    requests = {"a": _tokens(300 + 17 * seed, V, seed), "b": _tokens(1 + 11 * seed, V, seed + 50), "c": _tokens(130, V, seed + 90)}
    schedules = [replay.whole(requests), replay.tail_one_by_one(requests, tail=40 + 20 * seed),
                 replay.portions(requests, sizes=(64, 2, 33, 200, 7, 1, 129)), replay.mixed(requests, max_live=3, sizes=(50, 3, 24, 2, 210), seed=seed)]
    weights = lm.make_weights(cfg, seed, torch.bfloat16)
    ref = _reference(cfg, weights, requests)
    honest = _honest(cfg, weights, requests, ref)
    for dtype in ("fp32", "bf16"):
        w = {k: v.float() for k, v in weights.items()} if dtype == "fp32" else weights
        engine, _ = _engine(tmp_path / dtype, cfg, seed, dtype, weights=w)
        for steps in schedules:
            got = replay.run_trace(engine, _pool(engine, steps, 16, 3), steps)
            assert _covered(got, requests)
            if dtype == "fp32":
                assert _worst(got, ref) < 1.5 * F32_TOL
            else:
                assert _as_rounding(got, ref, honest)


MATRIX_CORES = {
    # three heads on one key/value head (a wavefront's 16 rows are 5 tokens and a third), key entries of 48 (a slab and a
    # half), values of 80, chunks that end inside blocks of keys; memories whose sizes fill no tile or slab exactly
    "three_heads": lm.config([lm.chunked(heads=3, kv_heads=1, dim=48, vdim=80, dims=24, chunk=37, scale=0.4, sharp=2.0, ff=None),
                              lm.mlstm(heads=2, dim=24, vdim=16), lm.mlstm(heads=3, dim=8, vdim=112)], width=32),
    # every head with keys of its own (a tile holds one head of 16 tokens), heads of 16 and of 128; wide memories
    "heads_of_their_own": lm.config([lm.chunked(heads=4, kv_heads=4, dim=16, vdim=32, dims=16, chunk=50, scale=0.7, sharp=2.0, ff=None),
                                     lm.chunked(heads=2, kv_heads=2, dim=128, vdim=128, chunk=100, scale=0.3, ff=None),
                                     lm.mlstm(heads=2, dim=128, vdim=256), lm.mlstm(heads=1, dim=256, vdim=240)], width=32),
    # 24 heads on two key/value heads (a token's heads fill a tile and a half), no chunks, chunks of 130
    "many_heads": lm.config([lm.chunked(heads=24, kv_heads=2, dim=32, vdim=16, dims=8, chunk=0, scale=0.5, sharp=2.0, ff=None),
                             lm.chunked(heads=8, kv_heads=1, dim=64, vdim=64, dims=32, chunk=130, scale=0.3, sharp=2.0, ff=None),
                             lm.mlstm(heads=5, dim=64, vdim=64), lm.mlstm(heads=2, dim=104, vdim=176)], width=32),
}


@pytest.mark.parametrize("name", sorted(MATRIX_CORES))
def test_the_matrix_core_kernels_at_other_sizes(tmp_path, name, monkeypatch):
    """bfloat16 on the matrix cores against the same model on the plain-precision attention and the row-by-row memory (what
    differs is the order of sums and the rounding of what enters the memory), under every schedule, and both against the
    plain model."""
    from llmengine.ops import KernelChoices, mlstm
    cfg = MATRIX_CORES[name]
    engine, weights = _engine(tmp_path, cfg, 21, "bf16")
    slow_engine, _ = _engine(tmp_path / "plain", cfg, 21, "bf16", weights=weights, kernel_choices=KernelChoices(fast_attention=False))
    V = cfg["vocab"]
    requests = {"a": _tokens(300, V, 1), "b": _tokens(21, V, 2), "c": _tokens(1, V, 3)}
    ref = _reference(cfg, weights, requests)
    honest = _honest(cfg, weights, requests, ref)
    with monkeypatch.context() as mp:
        mp.setattr(mlstm, "CHUNK_FROM", mlstm.NEVER)
        slow = _stacked(replay.run_trace(slow_engine, slow_engine.new_cache(32, 16, 3), replay.whole(requests)))
    for steps in (replay.whole(requests), replay.tail_one_by_one(requests, tail=150), replay.portions(requests, sizes=(33, 2, 64, 7, 1, 128, 41)),
                  replay.mixed(requests, max_live=3, sizes=(50, 3, 24, 2), seed=4)):
        got = replay.run_trace(engine, _pool(engine, steps, 16, 3), steps)
        assert _covered(got, requests)
        assert _as_rounding(got, slow, honest) and _as_rounding(got, ref, honest)


class _Step:
    """What the memory's operation reads of a step."""

    def __init__(self, lens, slots):
        dev = "cuda"
        self.num_tokens, self.num_seqs, self.new_lens = sum(lens), len(lens), list(lens)
        starts = np.concatenate([[0], np.cumsum(lens)])
        self.q_start = torch.tensor(starts, dtype=torch.int32, device=dev)
        self.seq_idx = torch.tensor(np.repeat(np.arange(len(lens)), lens), dtype=torch.int32, device=dev)
        self.slots = torch.tensor(slots, dtype=torch.int32, device=dev)

    def buffer(self, name, shape, dtype):
        t = torch.empty(shape, dtype=dtype, device="cuda")
        return t.fill_(float("nan"))                        # (scratch memory may hold anything)


@pytest.mark.parametrize("heads, dim, vdim, cap, lens", [
    (2, 32, 48, 6.0, [300, 1, 64, 130]), (3, 128, 256, 15.0, [257]), (1, 256, 64, 4.0, [128, 5, 129]), (2, 40, 112, 10.0, [48, 47, 200]),
    (4, 64, 64, 30.0, [1, 1, 500, 1]), (2, 8, 16, 2.0, [640]), (1, 200, 240, 8.0, [127, 1, 128]), (3, 56, 32, 5.0, [1, 2, 3, 4, 1]),
    (2, 128, 256, 9.0, [1, 1, 1]), (5, 17, 33, 9.0, [1, 1]), (1, 256, 300, 9.0, [1, 1, 1, 1])])
def test_the_memory_kernels_against_the_recurrence(heads, dim, vdim, cap, lens, monkeypatch):
    """The memory's operation on rows, states and levels drawn at random: every form (the walk, chunks, the kernel for steps
    of single rows) against the recurrence in float64 (rows
    and states afterwards), requests of every length side by side, slots in any order, the others untouched."""
    from llmengine import ops
    g = torch.Generator().manual_seed(heads * 1000 + dim + vdim)
    rnd = lambda *s: torch.randn(*s, generator=g, dtype=torch.float64)
    T, S, n_slots = sum(lens), len(lens), len(lens) + 2
    qk, hv = heads * dim, heads * vdim
    cols = ops.mlstm.MlstmColumns(q=0, k=qk, v=2 * qk, g=2 * qk + hv, i=2 * qk + 2 * hv, f=2 * qk + 2 * hv + heads)
    width = (2 * qk + 2 * hv + 2 * heads + 15) // 16 * 16
    p = rnd(T, width)
    p[:, cols.f:cols.f + heads] = p[:, cols.f:cols.f + heads] * 2 + 3
    p[:, cols.i:cols.i + heads] *= 3
    # (values that bfloat16 holds, so that both forms are given the same q, k and v)
    p[:, :cols.g] = p[:, :cols.g].to(torch.bfloat16).double()
    p = p.float().double()
    bias, norm_w = rnd(2 * heads).float(), (rnd(hv) * 0.2 + 1).float()
    slots = torch.randperm(n_slots, generator=g)[:S].tolist()
    memory, level = rnd(n_slots, heads, vdim + 1, dim).float(), rnd(n_slots, heads, 1).expand(-1, -1, vdim + 1).float().contiguous()
    step = _Step(lens, slots)
    w = {"i": torch.eye(heads, dtype=torch.float64), "i.b": bias[:heads].double(), "f": torch.eye(heads, dtype=torch.float64), "f.b": bias[heads:].double()}
    want = torch.empty(T, hv, dtype=torch.float64)
    want_mem, want_lev = memory.double().clone(), level.double().clone()
    eps, scale, at = 1e-5, 0.7, 0
    for s, n in enumerate(lens):
        rows = p[at:at + n]
        li = plain.soft_bounded(rows[:, cols.i:cols.i + heads] + w["i.b"], cap)
        lf = -torch.log1p(torch.exp(-plain.soft_bounded(rows[:, cols.f:cols.f + heads] + w["f.b"], cap)))
        M = memory[slots[s]].double()
        state = (M[:, :vdim].transpose(1, 2).clone(), M[:, vdim].clone(), level[slots[s], :, 0].double().clone())
        o, state = plain.matrix_memory(rows[:, :qk].view(n, heads, dim) * dim ** -0.5, rows[:, qk:2 * qk].view(n, heads, dim),
                                       rows[:, 2 * qk:2 * qk + hv].view(n, heads, vdim), li, lf, state=state)
        want[at:at + n] = scale * plain.rms_unit(o, eps).reshape(n, hv) * norm_w.double() * torch.sigmoid(rows[:, cols.g:cols.g + hv])
        want_mem[slots[s], :, :vdim], want_mem[slots[s], :, vdim] = state[0].transpose(1, 2), state[1]
        want_lev[slots[s]] = state[2][:, None]
        at += n
    rel = lambda a, b: float((a.double().cpu() - b).abs().max() / b.abs().max())
    for dtype, chunk_from, single in ((torch.float32, None, True), (torch.float32, None, False), (torch.bfloat16, ops.mlstm.NEVER, False),
                                      (torch.bfloat16, 48, True), (torch.bfloat16, 2, False)):
        monkeypatch.setattr(ops.mlstm, "SINGLE_ROWS", single)
        mem, lev = memory.cuda(), level.cuda()
        # (the result is a column range of a wider buffer, as beside another mixer)
        wide = torch.full((T, hv + 32), 7.0, dtype=dtype, device="cuda")
        ops.mlstm.mlstm(p.float().cuda(), cols, bias.cuda(), cap, mem, lev, norm_w.cuda(), step, wide[:, 16:16 + hv], heads, dim, vdim, eps,
                        scale, chunk_from=chunk_from)
        tol = 3e-5 if dtype == torch.float32 else 1e-2
        assert rel(wide[:, 16:16 + hv].float(), want) < tol, (dtype, chunk_from)
        assert bool((wide[:, :16] == 7).all()) and bool((wide[:, 16 + hv:] == 7).all())
        assert rel(mem, want_mem) < 2e-5 and rel(lev, want_lev) < 2e-5, (dtype, chunk_from)
        rest = [x for x in range(n_slots) if x not in slots]
        assert torch.equal(mem.cpu()[rest], memory[rest]) and torch.equal(lev.cpu()[rest], level[rest])


def test_the_memory_refuses_what_it_cannot_hold():
    from llmengine import ops
    from llmengine.config import parse_config
    from llmengine.config.registry import resolve
    step = _Step([2], [0])
    p = torch.zeros(2, 64, device="cuda")
    cols = ops.mlstm.MlstmColumns(q=0, k=8, v=16, g=24, i=32, f=33)
    args = lambda **kw: dict(dict(p=p, cols=cols, gate_bias=torch.zeros(2, device="cuda"), cap=1.0, memory=torch.zeros(1, 1, 9, 8, device="cuda"),
                                  level=torch.zeros(1, 1, 9, device="cuda"), norm_w=torch.ones(8, device="cuda"), step=step,
                                  out=torch.zeros(2, 8, device="cuda"), heads=1, dim=8, vdim=8, eps=1e-5), **kw)
    ops.mlstm.mlstm(**args())
    for kw in (dict(cap=0.0), dict(p=p[:, :33]), dict(memory=torch.zeros(1, 1, 8, 8, device="cuda")), dict(dim=300), dict(out=torch.zeros(3, 8, device="cuda"))):
        with pytest.raises(ops.KernelError):
            ops.mlstm.mlstm(**args(**kw))
    model = resolve("Lukupel").build_model(parse_config(lm.config([lm.mlstm(dim=257), lm.chunked(dim=300, ff=None)])))
    assert [r.split(":")[0] for r in model.tree_refusals()] == ["l0.mix", "l1.mix"]


@pytest.mark.parametrize("M, N, K", [(1, 48, 64), (16, 320, 96), (40, 100, 64), (70, 512, 256), (130, 1000, 72), (300, 4096, 128), (1030, 640, 64)])
def test_the_squared_rectifier_in_the_products_epilogue(M, N, K):
    from llmengine import ops
    g = torch.Generator().manual_seed(M)
    x, w = torch.randn(M, K, generator=g), torch.randn(N, K, generator=g) * K ** -0.5
    scratch = lambda shape, dtype: torch.full(shape, float("nan"), dtype=dtype, device="cuda")
    for dtype, tol in ((torch.float32, 1e-5), (torch.bfloat16, 1e-2)):
        xd, wd = x.to(dtype).cuda(), w.to(dtype).cuda()
        want = torch.relu(xd.double().cpu() @ wd.double().cpu().T) ** 2
        for wt in [wd] + ([ops.block_weight(wd)] if ops.can_block(wd) else []):
            out = torch.full((M, N), 5.0, dtype=dtype, device="cuda")
            ops.gemm_squared_relu(xd, wt, out, scratch)
            assert float((out.double().cpu() - want).abs().max() / want.abs().max()) < tol


def test_scaled_residual_and_capped_logits():
    from llmengine import ops
    g = torch.Generator().manual_seed(3)
    for T, H in ((5, 28), (3, 256), (2, 30), (4, 2056)):
        y, h, w = (torch.randn(*s, generator=g) for s in ((T, H), (T, H), (H,)))
        want = h.double() + 0.3 * w.double() * plain.rms_unit(y.double(), 1e-5)
        for dtype in (torch.float32, torch.bfloat16):
            hd, x = h.cuda(), torch.empty(T, H, dtype=dtype, device="cuda")
            ops.norm_add(y.cuda(), w.cuda(), hd, 1e-5, None, x, scale=0.3)
            assert torch.allclose(hd.double().cpu(), want, atol=1e-5) and torch.equal(x, hd.to(dtype))
    z = torch.randn(7, 33, generator=g) * 40
    zd = z.cuda()
    ops.soft_cap_(zd, 11.0)
    assert torch.allclose(zd.double().cpu(), 11.0 * torch.tanh(z.double() / 11.0), atol=1e-5)
    with pytest.raises(ops.KernelError):
        ops.soft_cap_(zd, 0.0)


@pytest.mark.parametrize("dtype", ["fp32", "bf16"])
def test_a_batch_of_unequal_requests_against_each_alone(tmp_path, dtype):
    cfg = lm.ALIGNED
    engine, _ = _engine(tmp_path, cfg, 12, dtype)
    V = cfg["vocab"]
    requests = {"a": _tokens(170, V, 1), "b": _tokens(3, V, 2), "c": _tokens(1, V, 3), "d": _tokens(50, V, 4)}
    alone = _stacked(replay.run_trace(engine, engine.new_cache(11, 16, 1), replay.whole(requests)))
    together = [{"step": 0, "entries": [{"id": r, "tokens": ids, "want": list(range(len(ids)))} for r, ids in requests.items()],
                 "end": list(requests)}]
    got = replay.run_trace(engine, engine.new_cache(17, 16, 4), together)
    assert _worst(got, alone) < (1e-5 if dtype == "fp32" else 2e-2)


@pytest.mark.parametrize("dtype", ["fp32", "bf16"])
def test_a_slot_that_is_used_again_starts_from_an_empty_memory(tmp_path, dtype):
    """One state slot: the second request takes the slot the first one left, and must not find its memory there."""
    cfg = lm.config([lm.mlstm(heads=2, dim=16, vdim=32, gate_cap=9.0)], width=32)
    store = torch.float32 if dtype == "fp32" else torch.bfloat16
    engine, weights = _engine(tmp_path, cfg, 5, dtype, weights=lm.make_weights(cfg, 5, store, remember=6.0))
    requests = {"first": _tokens(90, cfg["vocab"], 1), "second": _tokens(65, cfg["vocab"], 2)}
    ref = _reference(cfg, weights, requests)
    cache = engine.new_cache(8, 16, 1)
    for steps in (replay.whole(requests), replay.portions(requests, sizes=(9, 2, 50)), replay.tail_one_by_one(requests, tail=10)):
        got = replay.run_trace(engine, cache, steps)
        assert _worst(got, ref) < F32_TOL if dtype == "fp32" else _as_rounding(got, ref, _honest(cfg, weights, requests, ref))


@pytest.mark.parametrize("dtype", ["fp32", "bf16"])
def test_memories_that_last_hundreds_of_tokens(tmp_path, dtype):
    """Forget gates near one: a token written hundreds of places back is still read. Portions of hundreds of tokens run in
    chunks, beside other requests' single tokens and short portions, and need not end where a chunk ends. In the plain model
    the early token shows; the engine follows it with and without that token, in every schedule."""
    cfg = lm.config([lm.mlstm(heads=2, dim=24, vdim=16, gate_cap=9.0), lm.mlstm(heads=3, dim=32, vdim=48, gate_cap=12.0)], width=32)
    store = torch.float32 if dtype == "fp32" else torch.bfloat16
    engine, weights = _engine(tmp_path, cfg, 6, dtype, weights=lm.make_weights(cfg, 6, store, remember=7.0))
    V = cfg["vocab"]
    long = _tokens(530, V, 1)
    changed = list(long)
    changed[20] = (long[20] + 1) % V
    requests = {"long": long, "other": _tokens(260, V, 2), "short": _tokens(12, V, 3)}
    ref = _reference(cfg, weights, requests)
    far = _reference(cfg, weights, {"long": changed})["long"]
    moved = np.sqrt(np.mean((far[400:] - ref["long"][400:]) ** 2)) / np.sqrt(np.mean(ref["long"][400:] ** 2))
    assert moved > 10 * F32_TOL
    cut = lambda rid, a, b: {"id": rid, "tokens": requests[rid][a:b], "want": list(range(b - a))}
    mixed = [{"step": 0, "entries": [cut("long", 0, 201), cut("short", 0, 1)], "end": []},
             {"step": 1, "entries": [cut("short", 1, 3), cut("long", 201, 457), cut("other", 0, 193)], "end": []},
             {"step": 2, "entries": [cut("other", 193, 260), cut("long", 457, 458), cut("short", 3, 4)], "end": ["other"]},
             {"step": 3, "entries": [cut("long", 458, 530), cut("short", 4, 12)], "end": ["long", "short"]}]
    for steps in (mixed, replay.whole(requests), replay.tail_one_by_one(requests, tail=140), replay.portions(requests, sizes=(47, 48, 2, 127, 129))):
        got = replay.run_trace(engine, _pool(engine, steps, 16, 3), steps)
        assert _covered(got, requests)
        assert _worst(got, ref) < F32_TOL if dtype == "fp32" else _as_rounding(got, ref, _honest(cfg, weights, requests, ref))


@pytest.mark.parametrize("dtype", ["fp32", "bf16"])
def test_far_keys_page_borders_and_chunk_edges(tmp_path, dtype):
    """Sharp softmaxes over a long prompt: the layer without chunks finds its keys anywhere among hundreds, the others stand
    on keys of their chunks (40 and 24 tokens: edges inside pages, at page borders and across them), the memory carries over
    hundreds of tokens; in prompts cut anywhere and in decoding behind many chunks."""
    layers = [lm.chunked(heads=4, kv_heads=2, dim=32, vdim=32, dims=8, chunk=0, scale=2.0, ff=None)] + copy.deepcopy(lm.ALIGNED["layers"][:4])
    layers[2]["mixer"]["scale"] *= 3.0
    layers[4]["mixer"]["scale"] *= 3.0
    cfg = lm.config(layers + [lm.borrow(layers, 2)], width=64, vocab=128)
    engine, weights = _engine(tmp_path, cfg, 13, dtype)
    V = cfg["vocab"]
    requests = {"far": _tokens(700, V, 1), "edge": _tokens(90, V, 2)}
    ref = _reference(cfg, weights, requests)
    honest = _honest(cfg, weights, requests, ref) if dtype == "bf16" else None
    first = None
    for steps in (replay.whole(requests), replay.tail_one_by_one(requests, tail=70), replay.portions(requests, sizes=(33, 2, 64, 7, 16, 1, 41)),
                  replay.mixed(requests, max_live=2, prompt_frac=0.8, sizes=(50, 3, 24, 2), seed=4)):
        got = replay.run_trace(engine, _pool(engine, steps, 16, 2), steps)
        assert _covered(got, requests)
        if dtype == "fp32":
            assert _worst(got, ref) < 2 * F32_TOL       # (scores several times larger carry their rounding into the weights)
        else:
            first = first or _stacked(got)
            assert _as_rounding(got, ref, honest) and _as_rounding(got, first, honest)


def _hand_made(chunk: int):
    """A single layer whose scores are made by hand: a query of token id 1 scores a key of id 2 far above all others and
    the key's value moves the row. Queries and keys are normed per head, so what singles the key out is its direction: the
    key matrix spreads ordinary tokens over many entries and id 2 over one."""
    D = 16
    cfg = lm.config([lm.chunked(heads=1, kv_heads=1, dim=D, vdim=D, dims=0, chunk=chunk, scale=2.0, ff=None)], width=D, vocab=9,
                    embedding_scale=1.0)
    weights = lm.make_weights(cfg, 31, torch.float32)
    wk = torch.eye(D)
    wk[0, 0], wk[0, 1], wk[1, 1], wk[3, 3] = 0.0, 1.0, 0.0, 0.0      # a key's entry 0 is the stream's entry 1
    wv = torch.zeros(D, D)
    wv[3, 3] = 1.0                                                   # a value carries the stream's entry 3
    weights["l0.mix.q"], weights["l0.mix.k"], weights["l0.mix.v"] = torch.eye(D), wk, wv
    weights["embed"] = torch.randn(9, D, generator=torch.Generator().manual_seed(5)) * 0.3
    weights["embed"][:, 3] = 0
    weights["embed"][1] = 0
    weights["embed"][1, 0] = 6.0
    weights["embed"][2] = 0
    weights["embed"][2, 1] = 5.0
    weights["embed"][2, 3] = 4.0                    # what the row carries when the key is seen
    return cfg, weights


@pytest.mark.parametrize("dtype", ["fp32", "bf16"])
def test_one_key_stands_out_at_the_chunk_s_edges_and_far_back(tmp_path, dtype):
    """Where the one key lies (the first of the query's chunk, the last of the chunk in front, at a page border; far back
    where there are no chunks) decides the row, for queries at the chunk's start, inside it and at its end; the engine
    follows the plain model in each place, in a prompt, in portions that end at the edge and decoded."""
    base = [[3, 4, 5, 6, 7, 8][i % 6] for i in range(200)]
    cases = [(24, q, at, at is not None and at // 24 == q // 24) for q in (168, 191, 180)
             for at in (None, q // 24 * 24 - 1, q // 24 * 24 - 24, *([q // 24 * 24] if q % 24 else []), *([176] if q > 176 else []))]
    cases += [(0, 199, at, at is not None) for at in (None, 7, 16, 190)]
    engines = {c: _engine(tmp_path / str(c), _hand_made(c)[0], 31, dtype, weights={k: v.to(torch.float32 if dtype == "fp32" else torch.bfloat16)
                                                                                  for k, v in _hand_made(c)[1].items()}) for c in (24, 0)}
    alone = {}
    for chunk, q, at, seen in cases:
        cfg = _hand_made(chunk)[0]
        engine, weights = engines[chunk]
        ids = list(base[:q + 1])
        if at is not None:
            ids[at] = 2
        ids[q] = 1
        requests = {"r": ids}
        ref = _reference(cfg, weights, requests)
        for steps in (replay.whole(requests), replay.tail_one_by_one(requests, tail=3), replay.portions(requests, sizes=(24, 48, 2, 70)),
                      replay.portions(requests, sizes=(q, 1))):
            got = replay.run_trace(engine, _pool(engine, steps, 16, 1), steps)
            assert _worst(got, ref) < (F32_TOL if dtype == "fp32" else 2e-2), (chunk, q, at)
        row = ref["r"][q]
        if at is None:
            alone[chunk, q] = row
        else:
            moved = float(np.sqrt(np.mean((row - alone[chunk, q]) ** 2)) / np.sqrt(np.mean(alone[chunk, q] ** 2)))
            assert (moved > 0.1) if seen else (moved < 1e-6), (chunk, q, at)


def test_pages_of_earlier_chunks_are_given_back_and_used_again(tmp_path):
    """A pool with pages for one chunk and the next portion only: a long request lives in it, since pages of chunks that no
    later token reads are given back."""
    cfg = lm.config([lm.chunked(chunk=32, ff=12), lm.mlstm(), lm.chunked(chunk=20, ff=None)])
    engine, weights = _engine(tmp_path, cfg, 8, "fp32")
    ids = _tokens(300, cfg["vocab"], 1)
    ref = _reference(cfg, weights, {"r": ids})
    for sizes in ((8, 5, 1, 2), (1,)):
        cache = engine.new_cache(6, 8, 1)
        got = replay.run_trace(engine, cache, replay.portions({"r": ids}, sizes=sizes))
        assert _covered(got, {"r": ids}) and _worst(got, ref) < F32_TOL
        assert cache.manager.free_pages("chunk32") == 6 and cache.manager.free_pages("chunk20") == 6


def test_long_decoding_through_recorded_steps(tmp_path):
    """300 tokens one by one after a short prompt: chunks end many times, their pages are given back and used again, the
    memory is carried, and the recorded step is replayed."""
    cfg = lm.MIXED
    engine, weights = _engine(tmp_path, cfg, 14, "fp32")
    ids = _tokens(310, cfg["vocab"], 4)
    ref = _reference(cfg, weights, {"r": ids})
    got = replay.run_trace(engine, engine.new_cache(20, 16, 2), replay.tail_one_by_one({"r": ids}, tail=300))
    assert _covered(got, {"r": ids}) and _worst(got, ref) < F32_TOL
    assert engine.runner.graph_replays >= 299


def test_long_decoding_in_bfloat16_on_the_matrix_cores(tmp_path):
    cfg = lm.ALIGNED
    engine, weights = _engine(tmp_path, cfg, 18, "bf16")
    ids = _tokens(200, cfg["vocab"], 4)
    ref = _reference(cfg, weights, {"r": ids})
    honest = _honest(cfg, weights, {"r": ids}, ref)
    whole = _stacked(replay.run_trace(engine, engine.new_cache(16, 16, 1), replay.whole({"r": ids})))
    got = replay.run_trace(engine, engine.new_cache(16, 16, 2), replay.tail_one_by_one({"r": ids}, tail=190))
    assert _as_rounding(got, whole, honest) and _as_rounding(got, ref, honest)
    assert engine.runner.graph_replays >= 189


@pytest.mark.parametrize("cfg_name", ["MIXED", "ALIGNED"])
def test_sums_that_are_split_as_serving_does(tmp_path, cfg_name):
    """Without the promise of one order of sums, steps of few rows cut a sublayer's last product over k and add the parts
    into a buffer that the norm behind it leaves as zeros; whole prompts, portions and recorded steps follow one another."""
    from llmengine import Engine
    cfg = getattr(lm, cfg_name)
    folder, weights = lm.write_model(tmp_path, cfg, 19)
    engine = Engine(folder, "bf16")
    V = cfg["vocab"]
    requests = {"a": _tokens(130, V, 1), "b": _tokens(70, V, 2), "c": _tokens(5, V, 3)}
    ref = _reference(cfg, weights, requests)
    honest = _honest(cfg, weights, requests, ref)
    for steps in (replay.tail_one_by_one(requests, tail=30), replay.whole(requests), replay.mixed(requests, max_live=3, sizes=(70, 3, 24, 2), seed=4),
                  replay.portions(requests, sizes=(64, 65, 2))):
        got = replay.run_trace(engine, _pool(engine, steps, 16, 3), steps)
        assert _covered(got, requests) and _as_rounding(got, ref, honest)


@pytest.mark.parametrize("page", [4, 12, 24, 64])
def test_pages_of_other_sizes(tmp_path, page):
    """Values are written eight tokens a piece where pages hold whole pieces, and token by token otherwise."""
    cfg = lm.config([lm.chunked(chunk=30, sharp=2.0, ff=None), lm.chunked(heads=2, kv_heads=1, dim=16, vdim=20, chunk=0, ff=12)])
    engine, weights = _engine(tmp_path, cfg, 25, "fp32")
    V = cfg["vocab"]
    requests = {"a": _tokens(150, V, 1), "b": _tokens(39, V, 2)}
    ref = _reference(cfg, weights, requests)
    for steps in (replay.whole(requests), replay.portions(requests, sizes=(17, 31, 2, 50)), replay.mixed(requests, max_live=2, sizes=(40, 3, 21), seed=1)):
        got = replay.run_trace(engine, _pool(engine, steps, page, 2), steps)
        assert _covered(got, requests) and _worst(got, ref) < F32_TOL


def test_several_requests_decode_together_over_the_chunks_edges(tmp_path):
    """Four requests of unequal lengths decode side by side through recorded steps; each crosses its chunks' edges at
    another step, and one ends and another takes its slot and pages on the way."""
    cfg = lm.MIXED
    engine, weights = _engine(tmp_path, cfg, 24, "fp32")
    V = cfg["vocab"]
    requests = {f"r{i}": _tokens(30 + 9 * i, V, 60 + i) for i in range(6)}
    ref = _reference(cfg, weights, requests)
    steps = replay.mixed(requests, max_live=4, prompt_frac=0.2, seed=7)
    got = replay.run_trace(engine, _pool(engine, steps, 16, 4), steps)
    assert _covered(got, requests) and _worst(got, ref) < F32_TOL
    assert engine.runner.graph_replays > 20


def test_first_tokens_of_a_sequence(tmp_path):
    cfg = lm.MIXED
    engine, weights = _engine(tmp_path, cfg, 15, "fp32")
    requests = {f"n{n}": _tokens(n, cfg["vocab"], 30 + n) for n in range(1, 7)}
    ref = _reference(cfg, weights, requests)
    for steps in (replay.whole(requests), replay.tail_one_by_one(requests, tail=8), replay.mixed(requests, max_live=4, seed=3)):
        got = replay.run_trace(engine, engine.new_cache(8, 16, 4), steps)
        assert _worst(got, ref) < F32_TOL


def test_greedy_generation_through_the_entry_point_and_the_scheduler(tmp_path):
    cfg = lm.MIXED
    engine, weights = _engine(tmp_path, cfg, 16, "fp32")
    prompts = [_tokens(9, cfg["vocab"], 1), _tokens(30, cfg["vocab"], 2), _tokens(1, cfg["vocab"], 3)]
    new = 12
    w = {k: v.float() for k, v in weights.items()}

    def plain_greedy(ids):
        ids = list(ids)
        for _ in range(new):
            ids.append(int(plain.forward(cfg, w, ids)[-1].argmax()))
        return ids

    want = [plain_greedy(p) for p in prompts]
    for p, out_want in zip(prompts, want):
        out, finish = engine.generate(p, new)
        assert out == out_want and finish == "length"
    from llmengine import BlockManager, ContinuousBatchScheduler
    sched = ContinuousBatchScheduler(engine, BlockManager(num_blocks=12, block_size=16), max_concurrent=2,
                                     max_prefill_tokens_per_step=16)
    for p in prompts:
        sched.enqueue(p, new)
    sched.run_until_idle()
    assert [r.token_ids for r in sched.results] == want


def test_the_trace_runner_replays_a_model_of_this_design(tmp_path):
    import json
    import os
    import subprocess
    import sys
    cfg = lm.MIXED
    folder, weights = lm.write_model(tmp_path / "model", cfg, 17, torch.float32)
    requests = {"a": _tokens(40, cfg["vocab"], 1), "b": _tokens(21, cfg["vocab"], 2)}
    steps = replay.mixed(requests, max_live=2, seed=5)
    ref = _reference(cfg, weights, requests)
    out = tmp_path / "out"
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    p = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", folder, "--dtype", "float32",
                        "--out", str(out), "--max-tokens", str(replay.trace_peak_tokens(steps))],
                       input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True, timeout=600)
    assert p.returncode == 0, p.stderr[-2000:]
    assert [l for l in p.stdout.splitlines() if l.startswith("done")] == [f"done {s['step']}" for s in steps]
    done = {rid: 0 for rid in requests}
    for s in steps:
        rows = np.fromfile(out / f"{s['step']}.f32", dtype="<f4").reshape(-1, cfg["vocab"])
        r = 0
        for e in s["entries"]:
            for w in e["want"]:
                want = ref[e["id"]][done[e["id"]] + w]
                assert np.sqrt(np.mean((rows[r] - want) ** 2)) / np.sqrt(np.mean(want ** 2)) < F32_TOL
                r += 1
            done[e["id"]] += len(e["tokens"])


def test_the_command_line_generates_with_random_weights_of_this_design(tmp_path):
    import json
    import os
    import subprocess
    import sys
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    cfgf = tmp_path / "cfg.json"
    cfgf.write_text(json.dumps(lm.ALIGNED))
    pf = tmp_path / "prompts.txt"
    pf.write_text("1 2 3\n7,8,9,10,11\n")
    out = subprocess.run([sys.executable, os.path.join(root, "bin", "llmengine-cli"), "--random", str(cfgf), "--seed", "3",
                          "--prompt-file", str(pf), "--max-new-tokens", "4", "--temperature", "0.7"],
                         capture_output=True, text=True, timeout=300)
    assert out.returncode == 0, out.stderr[-2000:]
    recs = [json.loads(line) for line in out.stdout.strip().splitlines()]
    assert [len(r["token_ids"]) for r in recs] == [7, 9] and all(r["finish_reason"] == "length" for r in recs)
