"""Diporax on the GPU against the plain implementation (tests/plain_diporax.py): every mechanism alone and together, under
every way of cutting requests into steps, in 32-bit and in bfloat16."""
from __future__ import annotations

import numpy as np
import pytest
import torch

import diporax_models as dm
import plain_diporax as plain
import replay

pytestmark = pytest.mark.gpu

F32_TOL = 2e-4          # of a row's root mean square; honest 32-bit arithmetic is at 1e-5
# bfloat16 against the unrounded plain model, in units of what rounding alone does: the plain model with the values that are
# kept in bfloat16 rounded. Without experts the average row and the row that 97 in 100 stay below are held; with experts, where
# rounding swaps close calls between two of them now and then, the row that half and the one that 80 in 100 stay below.
BF16_MEAN, BF16_MOST, BF16_FLOOR = 1.5, 2.0, 4e-3


def _engine(tmp_path, cfg, seed, dtype, weights=None, **kw):
    from llmengine import Engine
    store = torch.float32 if dtype == "fp32" else torch.bfloat16
    folder, weights = dm.write_model(tmp_path, cfg, seed, store, weights)
    return Engine(folder, dtype, deterministic=kw.pop("deterministic", True), **kw), weights


def _tokens(n, vocab, seed):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def _reference(cfg, weights, requests):
    w = {k: v.float() for k, v in weights.items()}
    return {rid: plain.forward(cfg, w, ids).numpy() for rid, ids in requests.items()}


def _has_experts(cfg):
    return any(l.get("mlp") for l in cfg["layers"])


def _summary(e, cfg):
    return (float(np.median(e)), float(np.quantile(e, 0.8))) if _has_experts(cfg) else (float(np.mean(e)), float(np.quantile(e, 0.97)))


def _honest(cfg, weights, requests, ref):
    """What rounding alone does, in the two numbers that are held."""
    with plain.bfloat16_storage():
        return _summary(_errors(_rows(_reference(cfg, weights, requests)), ref), cfg)


def _as_rounding(got, ref, honest, cfg) -> bool:
    a, b = _summary(_errors(got, ref), cfg)
    return a < BF16_MEAN * honest[0] + BF16_FLOOR and b < BF16_MOST * honest[1] + 2 * BF16_FLOOR


def _errors(got: dict, ref: dict) -> list[float]:
    return [float(np.sqrt(np.mean((row - ref[rid][pos]) ** 2)) / np.sqrt(np.mean(ref[rid][pos] ** 2)))
            for rid, rows in got.items() for pos, row in rows.items()]


def _worst(got, ref) -> float:
    return max(_errors(got, ref))


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
    "latent": dm.config([dm.latent()], side=0),
    "latent_sharp": dm.config([dm.latent(sharp=6.0)], side=0),
    "latent_one_head": dm.config([dm.latent(heads=1, dim=4, rot_dim=2, vdim=3, kv_rank=5, q_rank=6)], side=0),
    "latent_without_scaling": dm.config([dm.latent(factor=0)], side=0),
    "latent_wider_than_a_wavefront": dm.config([dm.latent(heads=2, dim=20, rot_dim=10, vdim=24, kv_rank=72, q_rank=80)], side=0),
    "lightning": dm.config([dm.lightning()], side=0),
    "lightning_one_head_of_one": dm.config([dm.lightning(heads=1, dim=1, vdim=1, decay=(0.9,))], side=0),
    "lightning_decays_of_nothing_and_one": dm.config([dm.lightning(decay=(0.0, 1.0, 0.5))], side=0),
    "lightning_wide_keys": dm.config([dm.lightning(heads=2, dim=256, vdim=3, decay=(0.9, 0.99))], side=0),
    "lightning_wide_values": dm.config([dm.lightning(heads=2, dim=6, vdim=300, decay=(0.9, 0.99))], side=0),
    "lightning_many_small_heads": dm.config([dm.lightning(heads=9, dim=4, vdim=2, decay=[0.1 * (i + 1) for i in range(9)])], side=0),
    "full": dm.config([dm.full()], side=0),
    "full_sharp": dm.config([dm.full(sharp=5.0)], side=0),
    "full_without_cap_scaling_or_mixing": dm.config([dm.full(softcap=0, factor=0, v_mix=False)], side=0),
    "full_one_tap": dm.config([dm.full(conv=1)], side=0),
    "full_seven_taps": dm.config([dm.full(conv=7)], side=0),
    "full_no_convolution": dm.config([dm.full(conv=0)], side=0),
    "full_no_rotation_one_head": dm.config([dm.full(heads=1, kv_heads=1, dim=20, vdim=20, dims=0)], side=0),
    "full_whole_head_rotated": dm.config([dm.full(heads=6, kv_heads=3, dim=8, vdim=6, dims=8)], side=0),
    "full_wide_heads": dm.config([dm.full(heads=2, kv_heads=1, dim=136, vdim=70, dims=70, scale=0.08)], side=0, width=36),
    "values_that_mix_over_three_layers": dm.config([dm.full(), dm.full(heads=4, kv_heads=4, dim=6, vdim=5, dims=4), dm.full(v_mix=False, vdim=3), dm.full()], side=0),
    "experts_one_of_three": dm.config([dm.lightning(mlp=dm.moe(experts=3, top=1))], side=0),
    "experts_all_of_four": dm.config([dm.lightning(mlp=dm.moe(experts=4, top=4, ff=7))], side=0),
    "experts_five_of_seventy_none_shared": dm.config([dm.lightning(mlp=dm.moe(experts=70, top=5, ff=6, shared=0))], side=0),
    "one_expert": dm.config([dm.lightning(mlp=dm.moe(experts=1, top=1, ff=33, shared=5))], side=0),
    "token_input": dm.config([dm.lightning(), dm.lightning()], side=5),
    "token_input_wide_behind_experts": dm.config([dm.lightning(mlp=dm.moe())], side=70),
    "token_input_of_one": dm.config([dm.full()], side=1, width=30),
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
@pytest.mark.parametrize("cfg_name", ["MIXED", "ALIGNED", "NO_EXPERTS"])
def test_every_schedule_gives_the_plain_logits(tmp_path, cfg_name, dtype):
    cfg = getattr(dm, cfg_name)
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
                assert _as_rounding(got, ref, honest, cfg) and _as_rounding(got, first, honest, cfg), (what, page)
            assert not cache.manager.live_requests()


@pytest.mark.parametrize("seed", range(10))
def test_configurations_drawn_at_random(tmp_path, seed):
    """Layers of all kinds in any order with sizes, head counts and constants drawn at random, in both precisions against the
    plain model, with prompts long enough for the memory's chunks."""
    cfg = dm.random_config(seed)
    V = cfg["vocab"]
    requests = {"a": _tokens(300 + 17 * seed, V, seed), "b": _tokens(1 + 11 * seed, V, seed + 50), "c": _tokens(130, V, seed + 90)}
    schedules = [replay.whole(requests), replay.tail_one_by_one(requests, tail=40 + 10 * seed),
                 replay.portions(requests, sizes=(64, 2, 33, 200, 7, 1, 129)), replay.mixed(requests, max_live=3, sizes=(50, 3, 24, 2, 210), seed=seed)]
    weights = dm.make_weights(cfg, seed, torch.bfloat16)
    ref = _reference(cfg, weights, requests)
    honest = _honest(cfg, weights, requests, ref)
    for dtype in ("fp32", "bf16"):
        w = {k: v.float() for k, v in weights.items()} if dtype == "fp32" else weights
        engine, _ = _engine(tmp_path / dtype, cfg, seed, dtype, weights=w)
        for steps in schedules:
            got = replay.run_trace(engine, _pool(engine, steps, 16, 3), steps)
            assert _covered(got, requests)
            if dtype == "fp32":
                # (a close call between two experts' 32-bit scores may fall the other way in single rows)
                assert np.quantile(_errors(got, ref), 0.99 if _has_experts(cfg) else 1.0) < 1.5 * F32_TOL
            else:
                assert _as_rounding(got, ref, honest, cfg)


MATRIX_CORES = {
    # latent rows that fill no whole chunk of 32 entries (64 + 24, 80 + 16, 48 + 8), heads that fill no tile
    "latent_rows": dm.config([dm.latent(heads=3, dim=16, rot_dim=24, vdim=16, kv_rank=64, q_rank=32, scale=0.3, sharp=2.0),
                              dm.latent(heads=20, dim=8, rot_dim=16, vdim=8, kv_rank=80, q_rank=24, scale=0.3),
                              dm.latent(heads=1, dim=12, rot_dim=8, vdim=20, kv_rank=48, q_rank=16, scale=0.4)], width=32, side=8),
    # the largest latent, rows of whole chunks
    "latent_wide": dm.config([dm.latent(heads=4, dim=32, rot_dim=64, vdim=32, kv_rank=512, q_rank=64, scale=0.15),
                              dm.latent(heads=6, dim=64, rot_dim=32, vdim=64, kv_rank=256, q_rank=64, scale=0.15)], width=64, side=8),
    # memories whose sizes fill no tile or slab exactly, the largest ones
    "memories": dm.config([dm.lightning(heads=2, dim=24, vdim=16, decay=(0.9, 0.99)), dm.lightning(heads=3, dim=8, vdim=112, decay=(0.5, 0.97, 0.999)),
                           dm.lightning(heads=2, dim=128, vdim=256, decay=(0.99, 0.7)), dm.lightning(heads=1, dim=256, vdim=240, decay=(0.98,))], width=32, side=8),
    # three heads on one key head, heads of their own, heads of 128 with values of 48, 24 heads on two key heads
    "softmax": dm.config([dm.full(heads=3, kv_heads=1, dim=48, vdim=80, dims=24, scale=0.1, conv=4, v_mix=False),
                          dm.full(heads=4, kv_heads=4, dim=16, vdim=48, dims=16, scale=0.3, softcap=5.0),
                          dm.full(heads=2, kv_heads=2, dim=128, vdim=96, dims=32, scale=0.08, conv=2),
                          dm.full(heads=24, kv_heads=2, dim=32, vdim=16, dims=8, scale=0.2, softcap=0, v_mix=False)], width=32, side=8),
}


@pytest.mark.parametrize("name", sorted(MATRIX_CORES))
def test_the_matrix_core_kernels_at_other_sizes(tmp_path, name, monkeypatch):
    """bfloat16 on the matrix cores against the same model on the plain-precision attention and the row-by-row memory (what
    differs is the order of sums and the rounding of what enters the memory), under every schedule, and both against the
    plain model."""
    from llmengine.ops import KernelChoices, lightning
    cfg = MATRIX_CORES[name]
    engine, weights = _engine(tmp_path, cfg, 21, "bf16")
    slow_engine, _ = _engine(tmp_path / "plain", cfg, 21, "bf16", weights=weights, kernel_choices=KernelChoices(fast_attention=False))
    V = cfg["vocab"]
    requests = {"a": _tokens(300, V, 1), "b": _tokens(21, V, 2), "c": _tokens(1, V, 3)}
    ref = _reference(cfg, weights, requests)
    honest = _honest(cfg, weights, requests, ref)
    with monkeypatch.context() as mp:
        mp.setattr(lightning, "CHUNK_FROM", lightning.NEVER)
        slow = _stacked(replay.run_trace(slow_engine, slow_engine.new_cache(32, 16, 3), replay.whole(requests)))
    for steps in (replay.whole(requests), replay.tail_one_by_one(requests, tail=150), replay.portions(requests, sizes=(33, 2, 64, 7, 1, 128, 41)),
                  replay.mixed(requests, max_live=3, sizes=(50, 3, 24, 2), seed=4)):
        got = replay.run_trace(engine, _pool(engine, steps, 16, 3), steps)
        assert _covered(got, requests)
        assert _as_rounding(got, slow, honest, cfg) and _as_rounding(got, ref, honest, cfg)


class _Step:
    """What the memory's operation reads of a step."""

    def __init__(self, lens, slots, dtype=torch.float32):
        dev = "cuda"
        self.num_tokens, self.num_seqs, self.new_lens, self.act_dtype = sum(lens), len(lens), list(lens), dtype
        starts = np.concatenate([[0], np.cumsum(lens)])
        self.q_start = torch.tensor(starts, dtype=torch.int32, device=dev)
        self.seq_idx = torch.tensor(np.repeat(np.arange(len(lens)), lens), dtype=torch.int32, device=dev)
        self.slots = torch.tensor(slots, dtype=torch.int32, device=dev)

    def buffer(self, name, shape, dtype):
        t = torch.empty(shape, dtype=dtype, device="cuda")
        return t.fill_(float("nan"))                        # (scratch memory may hold anything)


@pytest.mark.parametrize("heads, dim, vdim, lens", [
    (2, 32, 48, [300, 1, 64, 130]), (3, 128, 256, [257]), (1, 256, 64, [128, 5, 129]), (2, 40, 112, [48, 47, 200]), (4, 64, 64, [1, 1, 500, 1]),
    (2, 8, 16, [640]), (1, 200, 240, [127, 1, 128]), (3, 56, 32, [1, 2, 3, 4, 1]), (2, 128, 256, [1, 1, 1]), (5, 17, 33, [1, 1]), (1, 256, 300, [1, 1, 1, 1])])
def test_the_memory_kernels_against_the_recurrence(heads, dim, vdim, lens, monkeypatch):
    """The memory's operation on rows and states drawn at random: every form (the walk, chunks, the kernel for steps of single
    rows) against the recurrence in float64 (rows and states afterwards), requests of every length side by side, slots in any
    order, the others untouched."""
    from llmengine import ops
    g = torch.Generator().manual_seed(heads * 1000 + dim + vdim)
    rnd = lambda *s: torch.randn(*s, generator=g, dtype=torch.float64)
    T, S, n_slots = sum(lens), len(lens), len(lens) + 2
    qk, hv = heads * dim, heads * vdim
    width = (2 * qk + 2 * hv + 15) // 16 * 16 + 8
    p = rnd(T, width).float()
    a = torch.tensor([[0.999, 0.3, 0.9, 1.0, 0.0][h % 5] for h in range(heads)], dtype=torch.float64)
    decay = torch.cat([a, torch.log(a)]).float().cuda()
    slots = torch.randperm(n_slots, generator=g)[:S].tolist()
    memory = rnd(n_slots, heads, vdim, dim).float()
    step = _Step(lens, slots)
    act = plain.silu(p.double())
    wants = {}
    for name, q in (("exact", lambda x: x), ("rounded", lambda x: x.to(torch.bfloat16).double())):
        want, want_mem, at = torch.empty(T, hv, dtype=torch.float64), memory.double().clone(), 0
        for s, n in enumerate(lens):
            rows = q(act[at:at + n])
            o, state = plain.decayed_memory(rows[:, :qk].view(n, heads, dim), rows[:, qk:2 * qk].view(n, heads, dim), rows[:, 2 * qk:2 * qk + hv].view(n, heads, vdim),
                                            a.float().double(), state=memory[slots[s]].double().transpose(1, 2).clone())
            want[at:at + n], want_mem[slots[s]] = o.reshape(n, hv), state.transpose(1, 2)
            at += n
        wants[name] = (want, want_mem)
    rel = lambda x, y: float((x.double().cpu() - y).abs().max() / y.abs().max())
    for chunk_from, single in ((ops.lightning.NEVER, True), (ops.lightning.NEVER, False), (48, True), (2, False)):
        monkeypatch.setattr(ops.lightning, "SINGLE_ROWS", single)
        mem, o = memory.cuda(), torch.full((T, hv), float("nan"), device="cuda")
        ops.lightning.lightning(p.cuda(), 0, qk, 2 * qk, decay, mem, step, o, heads, dim, vdim, chunk_from=chunk_from)
        exact, rounded = wants["exact"], wants["rounded"]
        if chunk_from == ops.lightning.NEVER:
            assert rel(o, exact[0]) < 2e-5 and rel(mem, exact[1]) < 2e-5, (chunk_from, single)
        else:
            # (rows that went through chunks are close to the rounded operands' rows, the others to the exact ones; an activation
            # that lies between two bfloat16 values may fall to either of them)
            at = 0
            for s, n in enumerate(lens):
                chunks = n >= chunk_from and dim % 8 == 0 and vdim % 16 == 0 and not (single and T == S) and max(dim, vdim) <= 256
                want = rounded if chunks else exact
                scale = float(exact[0].abs().max())
                assert float((o[at:at + n].double().cpu() - want[0][at:at + n]).abs().max()) < 4e-4 * scale, (chunk_from, s)
                assert rel(mem[slots[s]], want[1][slots[s]]) < 4e-4, (chunk_from, s)
                at += n
        rest = [x for x in range(n_slots) if x not in slots]
        assert torch.equal(mem.cpu()[rest], memory[rest])


def test_the_memory_refuses_what_it_cannot_hold():
    from llmengine import ops
    step = _Step([2], [0])
    args = lambda **kw: dict(dict(p=torch.zeros(2, 64, device="cuda"), q_col=0, k_col=8, v_col=16, decay=torch.ones(2, device="cuda"),
                                  memory=torch.zeros(1, 1, 8, 8, device="cuda"), step=step, o=torch.zeros(2, 8, device="cuda"), heads=1, dim=8, vdim=8), **kw)
    ops.lightning.lightning(**args())
    for kw in (dict(v_col=60), dict(memory=torch.zeros(1, 1, 9, 8, device="cuda")), dict(dim=300), dict(o=torch.zeros(3, 8, device="cuda")),
               dict(decay=torch.ones(1, device="cuda"))):
        with pytest.raises(ops.KernelError):
            ops.lightning.lightning(**args(**kw))


@pytest.mark.parametrize("T, width", [(1, 18), (3, 256), (2, 2052), (5, 4096), (2, 8200), (4, 6144)])
def test_the_joined_norm_and_its_gate(T, width):
    from llmengine import ops
    g = torch.Generator().manual_seed(width)
    o, w, z = torch.randn(T, width, generator=g) * 3, torch.randn(width, generator=g), torch.randn(T, width + 8, generator=g)
    want = 0.7 * o.double() / torch.sqrt((o.double() ** 2).mean(-1, keepdim=True) + 1e-5) * w.double() * torch.sigmoid(z[:, 4:4 + width].double())
    for dtype, tol in ((torch.float32, 1e-5), (torch.bfloat16, 1e-2)):
        wide = torch.full((T, width + 16), 7.0, dtype=dtype, device="cuda")
        ops.lightning.joined_norm_gate(o.cuda(), w.cuda(), z.cuda()[:, 4:4 + width], wide[:, 8:8 + width], 1e-5, 0.7)
        assert float((wide[:, 8:8 + width].double().cpu() - want).abs().max()) < tol * float(want.abs().max())
        assert bool((wide[:, :8] == 7).all()) and bool((wide[:, 8 + width:] == 7).all())


@pytest.mark.parametrize("H", [28, 64, 2048, 3000, 4096, 8192, 8200])
def test_a_normed_embedding_and_the_tokens_gate(H):
    from llmengine import ops
    g = torch.Generator().manual_seed(H)
    table, w, tokens = torch.randn(48, H, generator=g), torch.randn(H, generator=g), torch.tensor([0, 47, 16, 3, 31], dtype=torch.int32)
    for dtype in (torch.float32, torch.bfloat16):
        t, wt = table.to(dtype), w.to(dtype)
        rows = t.double()[tokens.long()]
        want = rows / torch.sqrt((rows ** 2).mean(-1, keepdim=True) + 1e-5) * wt.double()
        layouts = [t.cuda()] + ([ops.block_weight(t.cuda())] if ops.can_block(t.cuda()) else [])
        for layout in layouts:
            out = torch.empty(5, H, device="cuda")
            ops.token_input.embed_norm(layout, tokens.cuda(), wt.cuda(), 1e-5, out)
            assert torch.allclose(out.double().cpu(), want, atol=2e-5)
        z = torch.randn(5, 24, generator=g)
        for out_dtype, tol in ((torch.float32, 1e-5), (torch.bfloat16, 1e-2)):
            out = torch.empty(5, 12, dtype=out_dtype, device="cuda")
            ops.token_input.token_gate(z.cuda()[:, 8:20], t.cuda(), 7, tokens.cuda(), out)
            want_g = plain.gelu(z[:, 8:20].double()) * t.double()[tokens.long(), 7:19]
            assert torch.allclose(out.double().cpu(), want_g, atol=tol, rtol=tol)
    with pytest.raises(ops.KernelError):
        ops.token_input.token_gate(z.cuda()[:, 8:20], t.cuda(), H - 11, tokens.cuda(), out)


@pytest.mark.parametrize("dtype", ["fp32", "bf16"])
def test_a_batch_of_unequal_requests_against_each_alone(tmp_path, dtype):
    cfg = dm.NO_EXPERTS if dtype == "bf16" else dm.ALIGNED
    engine, _ = _engine(tmp_path, cfg, 12, dtype)
    V = cfg["vocab"]
    requests = {"a": _tokens(170, V, 1), "b": _tokens(3, V, 2), "c": _tokens(1, V, 3), "d": _tokens(50, V, 4)}
    alone = _stacked(replay.run_trace(engine, engine.new_cache(11, 16, 1), replay.whole(requests)))
    together = [{"step": 0, "entries": [{"id": r, "tokens": ids, "want": list(range(len(ids)))} for r, ids in requests.items()],
                 "end": list(requests)}]
    got = replay.run_trace(engine, engine.new_cache(17, 16, 4), together)
    assert _worst(got, alone) < (2e-5 if dtype == "fp32" else 3e-2)


@pytest.mark.parametrize("dtype", ["fp32", "bf16"])
def test_a_slot_that_is_used_again_starts_from_nothing(tmp_path, dtype):
    """One state slot: the second request takes the slot the first one left, and must find neither its memory nor the last rows
    of its convolutions there."""
    cfg = dm.config([dm.lightning(heads=2, dim=16, vdim=32, decay=(0.999, 0.9999)), dm.full(heads=4, kv_heads=2, dim=16, vdim=16, conv=5)], width=32)
    engine, weights = _engine(tmp_path, cfg, 5, dtype)
    requests = {"first": _tokens(90, cfg["vocab"], 1), "second": _tokens(65, cfg["vocab"], 2)}
    ref = _reference(cfg, weights, requests)
    cache = engine.new_cache(8, 16, 1)
    for steps in (replay.whole(requests), replay.portions(requests, sizes=(9, 2, 50)), replay.tail_one_by_one(requests, tail=10)):
        got = replay.run_trace(engine, cache, steps)
        assert _worst(got, ref) < F32_TOL if dtype == "fp32" else _as_rounding(got, ref, _honest(cfg, weights, requests, ref), cfg)


@pytest.mark.parametrize("dtype", ["fp32", "bf16"])
def test_memories_that_last_hundreds_of_tokens(tmp_path, dtype):
    """Decays near one: a token written hundreds of places back is still read. Portions of hundreds of tokens run in chunks,
    beside other requests' single tokens and short portions, and need not end where a chunk ends. In the plain model the early
    token shows; the engine follows it in every schedule."""
    cfg = dm.config([dm.lightning(heads=2, dim=24, vdim=16, decay=(0.9995, 0.999)), dm.lightning(heads=3, dim=32, vdim=48, decay=(0.999, 0.9, 1.0))], width=32)
    engine, weights = _engine(tmp_path, cfg, 6, dtype)
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
        assert _worst(got, ref) < F32_TOL if dtype == "fp32" else _as_rounding(got, ref, _honest(cfg, weights, requests, ref), cfg)


@pytest.mark.parametrize("dtype", ["fp32", "bf16"])
def test_far_keys_and_page_borders(tmp_path, dtype):
    """Sharp softmaxes of both attentions over a long prompt find their keys anywhere among hundreds, in prompts cut anywhere
    and in decoding; positions run past the length the rotations were made for."""
    cfg = dm.config([dm.full(heads=4, kv_heads=2, dim=32, vdim=32, dims=16, conv=3, scale=0.8, softcap=40.0, original=200),
                     dm.latent(heads=4, dim=32, rot_dim=16, vdim=16, kv_rank=64, q_rank=48, scale=0.7, original=200)], width=64, vocab=128)
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
            assert _worst(got, ref) < 4 * F32_TOL       # (scores several times larger carry their rounding into the weights)
        else:
            first = first or _stacked(got)
            assert _as_rounding(got, ref, honest, cfg) and _as_rounding(got, first, honest, cfg)


def _hand_made(kind: str, sink: float = -3.0):
    """A single layer whose scores are made by hand: a query of token id 1 scores a key of id 2 far above all others and the
    key's value moves the row. Queries and keys (or their latents) are normed, so what singles the key out is its direction."""
    D = 16
    if kind == "full":
        layer = dm.full(heads=1, kv_heads=1, dim=D, vdim=D, dims=0, conv=3, softcap=60.0, scale=2.0)
    else:
        layer = dm.latent(heads=1, dim=D, rot_dim=2, vdim=D, kv_rank=D, q_rank=D, scale=2.0, factor=0)
    cfg = dm.config([layer], width=D, vocab=9, side=0)
    w = dm.make_weights(cfg, 31, torch.float32)
    wk, wv = torch.eye(D), torch.zeros(D, D)
    wk[0, 0], wk[0, 1], wk[1, 1], wk[3, 3] = 0.0, 1.0, 0.0, 0.0      # a key's entry 0 is the stream's entry 1
    wv[3, 3] = 1.0                                                   # a value carries the stream's entry 3
    ones = torch.ones(D)
    w["embed.norm"] = ones
    if kind == "full":
        w["l0.mix.q"], w["l0.mix.k"], w["l0.mix.v"], w["l0.mix.q.norm"], w["l0.mix.k.norm"] = torch.eye(D), wk, wv, ones, ones
        for c in "qkv":
            w[f"l0.mix.{c}.b"] = torch.zeros(D)
            w[f"l0.mix.{c}.conv"] = torch.tensor([0.02, -0.03, 1.0]).expand(D, 3).clone()
    else:
        # the latent is the stream itself, normed; its up maps are the key and value maps
        w["l0.mix.dq"], w["l0.mix.dq.norm"], w["l0.mix.dkv.norm"] = torch.eye(D), ones, ones
        w["l0.mix.uq"] = torch.cat([torch.eye(D), torch.zeros(2, D)])
        w["l0.mix.dkv"] = torch.cat([torch.eye(D), torch.zeros(2, D)])
        w["l0.mix.uk"], w["l0.mix.uv"] = wk, wv
        w["l0.mix.sink"] = torch.tensor([sink])
    w["embed"] = torch.randn(9, D, generator=torch.Generator().manual_seed(5)) * 0.3
    w["embed"][:, 3] = 0
    w["embed"][1] = 0
    w["embed"][1, 0] = 6.0
    w["embed"][2] = 0
    w["embed"][2, 1] = 5.0
    w["embed"][2, 3] = 4.0                      # what the row carries when the key is seen
    return cfg, w


@pytest.mark.parametrize("dtype", ["fp32", "bf16"])
@pytest.mark.parametrize("kind", ["full", "latent"])
def test_one_key_stands_out_far_back_and_at_page_borders(tmp_path, kind, dtype):
    """Where the one key lies (the sequence's first token, around a page border, far back, just in front of the query) does not
    matter: the row follows it, in a prompt, in portions and decoded; without it the row is another."""
    cfg, weights = _hand_made(kind)
    store = torch.float32 if dtype == "fp32" else torch.bfloat16
    engine, weights = _engine(tmp_path, cfg, 31, dtype, weights={k: v.to(store) for k, v in weights.items()})
    base = [[3, 4, 5, 6, 7, 8][i % 6] for i in range(200)]
    base[199] = 1
    alone = None
    for at in (None, 0, 7, 15, 16, 47, 190, 197):
        ids = list(base)
        if at is not None:
            ids[at] = 2
        ref = _reference(cfg, weights, {"r": ids})
        for steps in (replay.whole({"r": ids}), replay.tail_one_by_one({"r": ids}, tail=3), replay.portions({"r": ids}, sizes=(24, 48, 2, 70)),
                      replay.portions({"r": ids}, sizes=(199, 1))):
            got = replay.run_trace(engine, _pool(engine, steps, 16, 1), steps)
            assert _worst(got, ref) < (F32_TOL if dtype == "fp32" else 2.5e-2), at
        row = ref["r"][199]
        if at is None:
            alone = row
        else:
            assert float(np.sqrt(np.mean((row - alone) ** 2)) / np.sqrt(np.mean(alone ** 2))) > 0.1, at


@pytest.mark.parametrize("dtype", ["fp32", "bf16"])
@pytest.mark.parametrize("sink", [-40.0, 0.0, 12.0, 60.0])
def test_sinks_that_take_nothing_much_and_nearly_everything(tmp_path, sink, dtype):
    cfg = dm.config([dm.latent(heads=4, dim=16, rot_dim=8, vdim=16, kv_rank=48, q_rank=32, scale=0.3)], width=32, side=4)
    store = torch.float32 if dtype == "fp32" else torch.bfloat16
    weights = dm.make_weights(cfg, 4, store)
    weights["l0.mix.sink"] = torch.tensor([sink, 0.5, sink / 2, -sink], dtype=store)
    engine, weights = _engine(tmp_path, cfg, 4, dtype, weights=weights)
    requests = {"a": _tokens(200, cfg["vocab"], 1), "b": _tokens(2, cfg["vocab"], 2)}
    ref = _reference(cfg, weights, requests)
    honest = _honest(cfg, weights, requests, ref)
    for steps in (replay.whole(requests), replay.tail_one_by_one(requests, tail=150), replay.portions(requests, sizes=(70, 2, 33))):
        got = replay.run_trace(engine, _pool(engine, steps, 16, 2), steps)
        assert _worst(got, ref) < F32_TOL if dtype == "fp32" else _as_rounding(got, ref, honest, cfg)


def test_long_decoding_through_recorded_steps(tmp_path):
    """300 tokens one by one after a short prompt: memories and convolutions are carried, pages fill, the recorded step is
    replayed."""
    cfg = dm.MIXED
    engine, weights = _engine(tmp_path, cfg, 14, "fp32")
    ids = _tokens(310, cfg["vocab"], 4)
    ref = _reference(cfg, weights, {"r": ids})
    got = replay.run_trace(engine, engine.new_cache(20, 16, 2), replay.tail_one_by_one({"r": ids}, tail=300))
    assert _covered(got, {"r": ids}) and _worst(got, ref) < F32_TOL
    assert engine.runner.graph_replays >= 299


def test_long_decoding_in_bfloat16_on_the_matrix_cores(tmp_path):
    cfg = dm.NO_EXPERTS
    engine, weights = _engine(tmp_path, cfg, 18, "bf16")
    ids = _tokens(200, cfg["vocab"], 4)
    ref = _reference(cfg, weights, {"r": ids})
    honest = _honest(cfg, weights, {"r": ids}, ref)
    whole = _stacked(replay.run_trace(engine, engine.new_cache(16, 16, 1), replay.whole({"r": ids})))
    got = replay.run_trace(engine, engine.new_cache(16, 16, 2), replay.tail_one_by_one({"r": ids}, tail=190))
    assert _as_rounding(got, whole, honest, cfg) and _as_rounding(got, ref, honest, cfg)
    assert engine.runner.graph_replays >= 189


@pytest.mark.parametrize("cfg_name", ["MIXED", "ALIGNED", "NO_EXPERTS"])
def test_sums_that_are_split_as_serving_does(tmp_path, cfg_name):
    """Without the promise of one order of sums, steps of few rows cut a sublayer's last product over k and add the parts
    into a buffer that the norm behind it leaves as zeros; whole prompts, portions and recorded steps follow one another."""
    cfg = getattr(dm, cfg_name)
    engine, weights = _engine(tmp_path, cfg, 19, "bf16", deterministic=False)
    V = cfg["vocab"]
    requests = {"a": _tokens(130, V, 1), "b": _tokens(70, V, 2), "c": _tokens(5, V, 3)}
    ref = _reference(cfg, weights, requests)
    honest = _honest(cfg, weights, requests, ref)
    for steps in (replay.tail_one_by_one(requests, tail=30), replay.whole(requests), replay.mixed(requests, max_live=3, sizes=(70, 3, 24, 2), seed=4),
                  replay.portions(requests, sizes=(64, 65, 2))):
        got = replay.run_trace(engine, _pool(engine, steps, 16, 3), steps)
        assert _covered(got, requests) and _as_rounding(got, ref, honest, cfg)


@pytest.mark.parametrize("page", [4, 12, 24, 64])
def test_pages_of_other_sizes(tmp_path, page):
    """Values (also those that mix) are written eight tokens a piece where pages hold whole pieces, and token by token
    otherwise; latent rows lie in pages of any size."""
    cfg = dm.config([dm.full(sharp=3.0), dm.latent(sharp=2.0), dm.full(heads=4, kv_heads=4, dim=16, vdim=5, mlp=dm.moe())])
    engine, weights = _engine(tmp_path, cfg, 25, "fp32")
    V = cfg["vocab"]
    requests = {"a": _tokens(150, V, 1), "b": _tokens(39, V, 2)}
    ref = _reference(cfg, weights, requests)
    for steps in (replay.whole(requests), replay.portions(requests, sizes=(17, 31, 2, 50)), replay.mixed(requests, max_live=2, sizes=(40, 3, 21), seed=1)):
        got = replay.run_trace(engine, _pool(engine, steps, page, 2), steps)
        assert _covered(got, requests) and _worst(got, ref) < F32_TOL


def test_several_requests_decode_together(tmp_path):
    """Four requests of unequal lengths decode side by side through recorded steps; one ends and another takes its slot and
    pages on the way."""
    cfg = dm.MIXED
    engine, weights = _engine(tmp_path, cfg, 24, "fp32")
    V = cfg["vocab"]
    requests = {f"r{i}": _tokens(30 + 9 * i, V, 60 + i) for i in range(6)}
    ref = _reference(cfg, weights, requests)
    steps = replay.mixed(requests, max_live=4, prompt_frac=0.2, seed=7)
    got = replay.run_trace(engine, _pool(engine, steps, 16, 4), steps)
    assert _covered(got, requests) and _worst(got, ref) < F32_TOL
    assert engine.runner.graph_replays > 20


def test_first_tokens_of_a_sequence(tmp_path):
    cfg = dm.MIXED
    engine, weights = _engine(tmp_path, cfg, 15, "fp32")
    requests = {f"n{n}": _tokens(n, cfg["vocab"], 30 + n) for n in range(1, 7)}
    ref = _reference(cfg, weights, requests)
    for steps in (replay.whole(requests), replay.tail_one_by_one(requests, tail=8), replay.mixed(requests, max_live=4, seed=3)):
        got = replay.run_trace(engine, engine.new_cache(8, 16, 4), steps)
        assert _worst(got, ref) < F32_TOL


def test_greedy_generation_through_the_entry_point_and_the_scheduler(tmp_path):
    cfg = dm.MIXED
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
    cfg = dm.MIXED
    folder, weights = dm.write_model(tmp_path / "model", cfg, 17, torch.float32)
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
    cfgf.write_text(json.dumps(dm.ALIGNED))
    pf = tmp_path / "prompts.txt"
    pf.write_text("1 2 3\n7,8,9,10,11\n")
    out = subprocess.run([sys.executable, os.path.join(root, "bin", "llmengine-cli"), "--random", str(cfgf), "--seed", "3",
                          "--prompt-file", str(pf), "--max-new-tokens", "4", "--temperature", "0.7"],
                         capture_output=True, text=True, timeout=300)
    assert out.returncode == 0, out.stderr[-2000:]
    recs = [json.loads(line) for line in out.stdout.strip().splitlines()]
    assert [len(r["token_ids"]) for r in recs] == [7, 9] and all(r["finish_reason"] == "length" for r in recs)
