"""The kernels for steps of few rows (gated products, experts in tiles of 16, the router in one launch, a product with the
per-token table's gate), the experts' sum with the norm behind it, and the short convolution over many rows, each against the
64-bit formula."""
from __future__ import annotations

import numpy as np
import pytest
import torch

pytestmark = pytest.mark.gpu

BF16 = torch.bfloat16


def _gen(seed):
    return torch.Generator().manual_seed(seed)


def _act(name, z):
    return {"silu": z * torch.sigmoid(z), "relu": torch.relu(z), "gelu_tanh": torch.nn.functional.gelu(z, approximate="tanh")}[name]


def _interleave(gate, up, group=16):
    FF, K = gate.shape
    return torch.stack([gate.view(FF // group, group, K), up.view(FF // group, group, K)], 1).reshape(2 * FF, K).contiguous()


def _close(got, want, tol):
    err = float((got.double().cpu() - want).abs().max() / want.abs().max())
    return err < tol


@pytest.mark.parametrize("activation", ["silu", "relu", "gelu_tanh"])
@pytest.mark.parametrize("T, FF, K", [(1, 16, 8), (16, 48, 96), (5, 320, 200), (8, 4096, 2048), (3, 2048, 4096), (17, 64, 64)])
def test_gated_products_of_few_rows(T, FF, K, activation):
    from llmengine import ops
    g = _gen(T + FF)
    x, gate, up = torch.randn(T, K, generator=g).to(BF16), (torch.randn(FF, K, generator=g) * K ** -0.5).to(BF16), (torch.randn(FF, K, generator=g) * K ** -0.5).to(BF16)
    want = _act(activation, x.double() @ gate.double().T) * (x.double() @ up.double().T)
    w = _interleave(gate, up).cuda()
    scratch = lambda shape, dtype: torch.full(shape, float("nan"), dtype=dtype, device="cuda")
    for layout in [w] + ([ops.block_weight(w)] if ops.can_block(w) else []):
        out = torch.full((T, FF), 9.0, dtype=BF16, device="cuda")
        ops.gemm_gated(x.cuda(), layout, out, 16, scratch, activation=activation)
        assert _close(out, want, 1e-2)


@pytest.mark.parametrize("T, E, top, FF, H", [(1, 4, 2, 16, 32), (8, 16, 2, 64, 128), (7, 5, 3, 48, 72), (16, 70, 4, 32, 64), (3, 6, 6, 16, 8), (8, 3, 1, 512, 2048)])
@pytest.mark.parametrize("weigh_input", [False, True])
def test_experts_in_tiles_of_sixteen_rows(T, E, top, FF, H, weigh_input):
    """The router, the plan, both products and the sum of a step of few tokens, as the mixture runs them."""
    from llmengine import ops
    g = _gen(E * 10 + T)
    x = torch.randn(T, H, generator=g).to(BF16)
    gate, up = ((torch.randn(E, FF, H, generator=g) * H ** -0.5).to(BF16) for _ in range(2))
    down = (torch.randn(E, H, FF, generator=g) * FF ** -0.5).to(BF16)
    router = (torch.randn(E + 1, H, generator=g) * H ** -0.5).to(BF16)
    w_gu = torch.stack([_interleave(gate[e], up[e]) for e in range(E)]).cuda()
    dev = dict(device="cuda")
    tile = ops.latent.moe_tile(x.cuda(), w_gu, T * top, E, 16)
    assert tile == 16 or T * top > 4 * E
    tile = 16
    cap = ops.moe_capacity(T * top, E, tile)
    ld = (E + 16) // 16 * 16 + 16
    logits, wts = torch.full((T, ld), 3.0, **dev), torch.empty(T, top, **dev)
    i32 = dict(dtype=torch.int32, device="cuda")
    place_pair, pair_place = torch.full((cap,), 77, **i32), torch.full((T * top,), 77, **i32)
    tile_expert, n_tiles = torch.full((cap // tile,), 77, **i32), torch.full((1,), 77, **i32)
    xd = x.cuda()
    assert ops.latent.moe_decide_fits(xd, router.cuda(), top)
    for _ in range(3):                                      # (again and again on what the last call left)
        ops.latent.moe_decide(xd, router.cuda(), E, top, 1.5, True, logits, wts, tile, place_pair, pair_place, tile_expert, n_tiles)
    z = x.double() @ router.double().T
    assert _close(logits[:, :E + 1], z, 1e-4) and bool((logits[:, E + 1:] == 3).all())
    order = torch.argsort(z[:, :E], dim=1, descending=True)[:, :top]
    soft = 1.5 * torch.softmax(torch.gather(z[:, :E], 1, order), 1)
    assert _close(wts, soft, 1e-4)
    pp, pl, te, nt = place_pair.cpu().numpy(), pair_place.cpu().numpy(), tile_expert.cpu().numpy(), int(n_tiles)
    assert sorted(pp[pp >= 0].tolist()) == list(range(T * top)) and (pp[pl] == np.arange(T * top)).all()
    assert all(te[pl[t * top + k] // tile] == int(order[t, k]) for t in range(T) for k in range(top))
    counts = np.bincount(order.numpy().ravel(), minlength=E)
    assert nt == int(((counts + tile - 1) // tile).sum())
    act, y = torch.full((cap, FF), float("nan"), dtype=BF16, **dev), torch.full((cap, H), float("nan"), **dev)
    ops.moe_gemm(xd, w_gu, True, 16, act, place_pair, tile_expert, n_tiles, tile, top, "silu", pairs=T * top,
                 pair_scale=wts.view(-1) if weigh_input else None)
    ops.moe_gemm(act, down.cuda(), False, 0, y, place_pair, tile_expert, n_tiles, tile, 0, "silu", pairs=T * top)
    want = torch.zeros(T, H, dtype=torch.float64)
    for t in range(T):
        for k in range(top):
            e, c = int(order[t, k]), soft[t, k]
            xin = x[t].double() * (c if weigh_input else 1.0)
            want[t] += (1.0 if weigh_input else c) * ((_act("silu", xin @ gate[e].double().T) * (xin @ up[e].double().T)) @ down[e].double().T)
    out = torch.zeros(T, H, **dev)
    ops.moe_combine(y, pair_place, None if weigh_input else wts, out, False, top=top)
    assert _close(out, want, 2e-2)
    # the sum with a gated shared layer, the norm behind it and the copy of the updated rows
    shared, h, norm_w = torch.randn(T, H, generator=g), torch.randn(T, H, generator=g), torch.randn(H, generator=g)
    total = want + torch.sigmoid(z[:, E:E + 1]) * shared.double()
    new_h = h.double() + 0.5 * norm_w.double() * total / torch.sqrt((total ** 2).mean(-1, keepdim=True) + 1e-5)
    for x_dtype in (BF16, torch.float32, None):
        sd, hd = shared.cuda(), h.cuda()
        x_out = torch.empty(T, H, dtype=x_dtype, **dev) if x_dtype is not None else None
        ops.latent.moe_combine_norm(y, pair_place, None if weigh_input else wts, top, sd, logits[:, E:E + 1], norm_w.cuda(), hd, 1e-5, x_out, 0.5,
                                    clear_shared=x_dtype is None)
        assert _close(hd, new_h, 2e-2) and (x_out is None or torch.equal(x_out, hd.to(x_dtype)))
        assert bool((sd == 0).all()) == (x_dtype is None)
    with pytest.raises(ops.KernelError):
        ops.latent.moe_decide(xd, router.cuda()[:E - 1], E, top, 1.0, True, logits, wts, tile, place_pair, pair_place, tile_expert, n_tiles)


@pytest.mark.parametrize("T, H", [(1, 4), (3, 28), (2, 2048), (5, 2052), (2, 4096), (3, 8192)])
def test_the_experts_sum_with_the_norm_behind_it(T, H):
    from llmengine import ops
    g = _gen(H)
    y, pl = torch.randn(9, H, generator=g), torch.randint(0, 9, (T * 3,), generator=g).to(torch.int32)
    wts, shared, h, w = torch.rand(T, 3, generator=g), torch.randn(T, H, generator=g), torch.randn(T, H, generator=g), torch.randn(H, generator=g)
    for use_wts in (True, False):
        for use_shared in (True, False):
            total = torch.stack([sum((wts[t, k].double() if use_wts else 1.0) * y[int(pl[t * 3 + k])].double() for k in range(3)) for t in range(T)])
            total = total + (shared.double() if use_shared else 0.0)
            want = h.double() + w.double() * total / torch.sqrt((total ** 2).mean(-1, keepdim=True) + 1e-5)
            hd = h.cuda()
            ops.latent.moe_combine_norm(y.cuda(), pl.cuda(), wts.cuda() if use_wts else None, 3, shared.cuda() if use_shared else None, None, w.cuda(), hd, 1e-5, None)
            assert _close(hd, want, 1e-5)


@pytest.mark.parametrize("T, n, K", [(1, 5, 64), (16, 24, 96), (8, 256, 2048), (3, 100, 200)])
def test_a_product_with_the_tables_gate(T, n, K):
    from llmengine import ops
    g = _gen(n)
    x, w = torch.randn(T, K, generator=g).to(BF16), (torch.randn(n, K, generator=g) * K ** -0.5).to(BF16)
    table, tokens = torch.randn(20, 3 * n + 1, generator=g).to(BF16), torch.randint(0, 20, (T,), generator=g).to(torch.int32)
    want = _act("gelu_tanh", x.double() @ w.double().T) * table.double()[tokens.long(), n + 1:2 * n + 1]
    for layout in [w.cuda()] + ([ops.block_weight(w.cuda())] if ops.can_block(w.cuda()) else []):
        out = torch.full((T, n), 9.0, dtype=BF16, device="cuda")
        assert ops.token_input.gemm_token_gate(x.cuda(), layout, table.cuda(), n + 1, tokens.cuda(), out)
        assert _close(out, want, 1e-2)
    many = torch.empty(17, n, dtype=BF16, device="cuda")
    assert not ops.token_input.gemm_token_gate(torch.zeros(17, K, dtype=BF16, device="cuda"), w.cuda(), table.cuda(), 0, torch.zeros(17, dtype=torch.int32, device="cuda"), many)


class _Step:
    def __init__(self, lens, slots):
        self.num_tokens, self.num_seqs, self.new_lens = sum(lens), len(lens), list(lens)
        self.q_start = torch.tensor(np.concatenate([[0], np.cumsum(lens)]), dtype=torch.int32, device="cuda")
        self.seq_idx = torch.tensor(np.repeat(np.arange(len(lens)), lens), dtype=torch.int32, device="cuda")
        self.slots = torch.tensor(slots, dtype=torch.int32, device="cuda")


@pytest.mark.parametrize("K", [1, 2, 3, 4, 5])
@pytest.mark.parametrize("C", [8, 1100])
@pytest.mark.parametrize("lens", [[40], [1, 2, 3, 1, 50, 1, 1, 9], [1] * 33, [5, 4]])
def test_the_short_convolution_over_many_rows_and_requests(lens, C, K):
    from llmengine import ops
    g = _gen(C + K)
    T, S = sum(lens), len(lens)
    slots = torch.randperm(S + 2, generator=g)[:S].tolist()
    x, w = torch.randn(T, C + 12, generator=g), torch.randn(C, K, generator=g)
    bias, in_bias, tail = torch.randn(C, generator=g), torch.randn(C, generator=g), torch.randn(S + 2, K - 1, C, generator=g)
    want, new_tail, at = torch.empty(T, C, dtype=torch.float64), tail.double().clone(), 0
    for s, n in enumerate(lens):
        rows = torch.cat([tail[slots[s]].double(), x[at:at + n, :C].double() + in_bias.double()])
        for i in range(n):
            want[at + i] = bias.double() + (rows[i:i + K] * w.double().T).sum(0)
        new_tail[slots[s]] = rows[n:]
        at += n
    td, out = tail.cuda(), torch.full((T, C + 4), 7.0, device="cuda")
    ops.short_conv(x.cuda()[:, :C], w.cuda(), bias.cuda(), td, _Step(lens, slots), out[:, :C], silu=False, in_bias=in_bias.cuda())
    assert float((out[:, :C].double().cpu() - want).abs().max()) < 1e-5 * float(want.abs().max()) and bool((out[:, C:] == 7).all())
    if K > 1:
        assert float((td.double().cpu() - new_tail).abs().max()) < 1e-6 * max(1.0, float(new_tail.abs().max()))
