"""Diporax on the CPU: the plain implementation (tests/plain_diporax.py) pinned to independent facts, the configuration
reader, the tensor names, the cache specs and the random weights."""
from __future__ import annotations

import copy
import math

import pytest
import torch

import diporax_models as dm
import plain_diporax as plain

F64 = torch.float64


def _rand(*shape, seed=0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=F64)


# ---- the plain implementation's mechanisms -------------------------------------------------------------
def test_a_ramp_of_frequencies_and_its_ends():
    rot = {"base": 100.0, "dims": 8, "scaling": {"factor": 4.0, "original": 500, "fast": 20.0, "slow": 1.0}}
    f, mag = plain.turns(rot)
    base = [100.0 ** (-2.0 * c / 8) for c in range(4)]
    # the pair that makes 20 turns over 500 positions is number 8 ln(500 / (40 pi)) / (2 ln 100) = 1.2, the one for 1 turn 3.8
    assert abs(8 * math.log(500 / (40 * math.pi)) / (2 * math.log(100)) - 1.2) < 0.01
    share = [0.0, 0.0, 1.0 / 3.0, 2.0 / 3.0]                # floor 1, ceil 4: pairs 1 .. 4
    for c in range(4):
        assert abs(float(f[c]) - (base[c] / 4 * share[c] + base[c] * (1 - share[c]))) < 1e-12
    assert abs(mag - (0.1 * math.log(4.0) + 1.0)) < 1e-15
    plain_f, one = plain.turns({"base": 100.0, "dims": 8})
    assert one == 1.0 and torch.allclose(plain_f, torch.tensor(base, dtype=F64))
    from llmengine.parts.frequencies import ramped_frequencies
    g, gmag = ramped_frequencies(8, 100.0, rot["scaling"])
    assert torch.allclose(g, f, rtol=1e-14) and abs(gmag - mag) < 1e-15


@pytest.mark.parametrize("turn, pairs", [(plain.rotate_halves, lambda c: (c, c + 3)), (plain.rotate_neighbours, lambda c: (2 * c, 2 * c + 1))])
def test_rotations_by_hand_and_as_a_function_of_distance(turn, pairs):
    rot = {"base": 30.0, "dims": 6, "scaling": {"factor": 2.0, "original": 40, "fast": 4.0, "slow": 0.5}}
    f, mag = plain.turns(rot)
    x = _rand(1, 2, 8, seed=1)
    y = turn(x, torch.tensor([7]), rot)
    for c in range(3):
        i, j = pairs(c)
        a, b, ang = float(x[0, 1, i]), float(x[0, 1, j]), 7 * float(f[c])
        assert abs(float(y[0, 1, i]) - mag * (a * math.cos(ang) - b * math.sin(ang))) < 1e-12
        assert abs(float(y[0, 1, j]) - mag * (b * math.cos(ang) + a * math.sin(ang))) < 1e-12
    assert torch.equal(y[..., 6:], x[..., 6:])              # the entries behind the rotated ones pass, unscaled
    q, k = _rand(1, 1, 8, seed=2), _rand(1, 1, 8, seed=3)
    dot = lambda i, j: float((turn(q, torch.tensor([i]), rot) * turn(k, torch.tensor([j]), rot)).sum())
    assert abs(dot(40, 31) - dot(9, 0)) < 1e-10 and abs(dot(40, 31) - dot(40, 30)) > 1e-4


def test_one_head_with_a_sink_and_a_cap_by_hand():
    q, k, v = _rand(3, 1, 4, seed=1), _rand(3, 1, 4, seed=2), _rand(3, 1, 2, seed=3)
    sink = torch.tensor([0.7], dtype=F64)
    out = plain.attend(q, k, v, 0.5, softcap=1.5, sink=sink)
    for i in range(3):
        s = [1.5 * math.tanh(0.5 * float(q[i, 0] @ k[j, 0]) / 1.5) for j in range(i + 1)]
        w = [math.exp(x) for x in s]
        total = sum(w) + math.exp(0.7)
        want = sum(a * v[j, 0] for j, a in enumerate(w)) / total
        assert torch.allclose(out[i, 0], want, atol=1e-12)
    assert torch.allclose(plain.attend(q, k, v, 0.5, sink=torch.tensor([-1e3], dtype=F64)), plain.attend(q, k, v, 0.5))
    assert plain.attend(q, k, v, 0.5, sink=torch.tensor([1e3], dtype=F64)).abs().max() < 1e-100
    # grouped heads: heads 0 and 1 read key head 0, heads 2 and 3 key head 1
    q4, k2, v2 = _rand(3, 4, 4, seed=4), _rand(3, 2, 4, seed=5), _rand(3, 2, 2, seed=6)
    o = plain.attend(q4, k2, v2, 0.5)
    for h in range(4):
        assert torch.allclose(o[:, h:h + 1], plain.attend(q4[:, h:h + 1], k2[:, h // 2:h // 2 + 1], v2[:, h // 2:h // 2 + 1], 0.5))


def test_the_convolution_against_the_librarys():
    u, w = _rand(9, 5, seed=1), _rand(5, 4, seed=2)
    want = torch.nn.functional.conv1d(torch.nn.functional.pad(u.T[None], (3, 0)), w[:, None, :], groups=5)[0].T
    assert torch.allclose(plain.causal_conv(u, w), want)
    assert torch.allclose(plain.causal_conv(u[:2], w), want[:2])             # fewer tokens than taps
    assert torch.equal(plain.causal_conv(u, w[:, 3:]), u * w[:, 3])          # one tap


def test_mixed_values_and_which_layers_mix():
    v, first = _rand(3, 2, 4, seed=1), _rand(3, 2, 4, seed=2)
    assert torch.equal(plain.mix_values(v, first, torch.tensor(0.0)), v)
    assert torch.allclose(plain.mix_values(v, first, torch.tensor(1.0)), first)
    assert torch.allclose(plain.mix_values(v, first, torch.tensor([0.25], dtype=F64)), 0.75 * v + 0.25 * first)
    # the first mixing layer's own number changes nothing; the later layers' do; a layer that does not mix neither gives nor takes
    cfg = dm.config([dm.full(v_mix=False), dm.full(), dm.full()], side=0)
    w = {k: t.double() for k, t in dm.make_weights(cfg, 3, torch.float32).items()}
    assert "l0.mix.vmix" not in w and w["l1.mix.vmix"].shape == ()
    ref = plain.forward(cfg, w, [1, 2, 3, 4])
    assert torch.equal(plain.forward(cfg, dict(w, **{"l1.mix.vmix": torch.tensor(9.0)}), [1, 2, 3, 4]), ref)
    assert not torch.allclose(plain.forward(cfg, dict(w, **{"l2.mix.vmix": torch.tensor(0.9)}), [1, 2, 3, 4]), ref)


def test_the_memory_in_closed_form_and_carried_on():
    q, k, v = _rand(7, 2, 3, seed=1), _rand(7, 2, 3, seed=2), _rand(7, 2, 4, seed=3)
    a = [0.6, 1.0]
    o, S = plain.decayed_memory(q, k, v, a)
    for t in range(7):
        for h in range(2):
            want = sum(a[h] ** (t - s) * float(q[t, h] @ k[s, h]) * v[s, h] for s in range(t + 1))
            assert torch.allclose(o[t, h], want, atol=1e-12)
    first, mid = plain.decayed_memory(q[:3], k[:3], v[:3], a)
    rest, end = plain.decayed_memory(q[3:], k[3:], v[3:], a, state=mid)
    assert torch.allclose(torch.cat([first, rest]), o) and torch.allclose(end, S)
    o0, _ = plain.decayed_memory(q, k, v, [0.0, 0.0])       # nothing remembered: every token reads its own write
    assert torch.allclose(o0, (q * k).sum(-1, keepdim=True) * v)


def test_lightning_norms_all_heads_together():
    cfg = dm.config([dm.lightning(heads=2, dim=3, vdim=4, decay=(0.5, 0.9))], side=0, width=8)
    w = plain.sub({k: t.double() for k, t in dm.make_weights(cfg, 2, torch.float32).items()}, "l0.mix.")
    x = _rand(5, 8, seed=4)
    m = cfg["layers"][0]["mixer"]
    o, _ = plain.decayed_memory(plain.silu(x @ w["q"].T).view(5, 2, 3), plain.silu(x @ w["k"].T).view(5, 2, 3), plain.silu(x @ w["v"].T).view(5, 2, 4), m["decay"])
    y = o.reshape(5, 8)
    y = y / torch.sqrt((y * y).mean(-1, keepdim=True) + 1e-5) * w["norm"] * torch.sigmoid(x @ w["g"].T)
    assert torch.allclose(plain.lightning(x, w, m, 1e-5), y @ w["o"].T)


def test_experts_weigh_by_the_softmax_over_the_chosen_and_the_shared_one_is_gated():
    cfg = dm.config([dm.lightning(mlp=dm.moe(experts=4, top=2, shared=6))], side=0)
    w = plain.sub({k: t.double() for k, t in dm.make_weights(cfg, 2, torch.float32).items()}, "l0.mlp.")
    mlp, x = cfg["layers"][0]["mlp"], _rand(6, 28, seed=5)
    got = plain.experts(x, w, mlp)
    z = x @ w["router"].T
    for t in range(6):
        order = sorted(range(4), key=lambda e: -float(z[t, e]))[:2]
        total = sum(math.exp(float(z[t, e])) for e in order)
        want = sum(math.exp(float(z[t, e])) / total * plain.expert(x[t:t + 1], w, f"e{e}")[0] for e in order)
        want = want + plain.expert(x[t:t + 1], w, "shared")[0] / (1 + math.exp(-float(x[t] @ w["shared.sg"][0])))
        assert torch.allclose(got[t], want)
    one = plain.experts(x, w, dict(mlp, router={"experts": 4, "top": 1}, shared=None))       # the one chosen weighs 1
    for t in range(6):
        assert torch.allclose(one[t], plain.expert(x[t:t + 1], w, f"e{int(z[t].argmax())}")[0])


def test_the_tokens_own_input_and_a_layer_by_hand():
    assert abs(float(plain.gelu(torch.tensor(1.3, dtype=F64))) - float(torch.nn.functional.gelu(torch.tensor(1.3, dtype=F64), approximate="tanh"))) < 1e-12
    cfg = dm.config([dm.lightning(), dm.lightning()], side=3)
    w = {k: t.double() for k, t in dm.make_weights(cfg, 7, torch.float32).items()}
    ids = [5, 9, 5]
    _, layers = plain.forward(cfg, w, ids, return_layers=True)
    n = lambda y, g: y / torch.sqrt((y * y).mean(-1, keepdim=True) + 1e-5) * g
    x = n(w["embed"][ids], w["embed.norm"])
    for i in range(2):
        p = f"l{i}."
        x = x + n(plain.lightning(x, plain.sub(w, p + "mix."), cfg["layers"][i]["mixer"], 1e-5), w[p + "norm1"]) * w[p + "ls1"]
        e = w["side.embed"][ids][:, 3 * i:3 * i + 3]
        x = x + n((plain.gelu(x @ w[p + "side.gate"].T) * e) @ w[p + "side.proj"].T, w[p + "side.norm"])
        assert torch.allclose(layers[i], x)


def test_latent_attention_by_hand_and_with_the_key_map_on_the_query():
    cfg = dm.config([dm.latent()], side=0)
    w = plain.sub({k: t.double() for k, t in dm.make_weights(cfg, 4, torch.float32).items()}, "l0.mix.")
    m, x = cfg["layers"][0]["mixer"], _rand(6, 28, seed=6)
    got = plain.latent_attention(x, w, m, 1e-5)
    n, d, r, dv, R = 3, 10, 6, 7, 12
    nrm = lambda y, g: y / torch.sqrt((y * y).mean(-1, keepdim=True) + 1e-5) * g
    q = (nrm(x @ w["dq"].T, w["dq.norm"]) @ w["uq"].T).view(6, n, d + r)
    down = x @ w["dkv"].T
    c, pos = nrm(down[:, :R], w["dkv.norm"]), torch.arange(6)
    kr = plain.rotate_neighbours(down[:, None, R:], pos, m["rot"])[:, 0]
    heads = []
    for h in range(n):
        qa = q[:, h, :d] @ w["uk"][h * d:(h + 1) * d]       # the key map taken onto the query
        s = (qa @ c.T + plain.rotate_neighbours(q[:, h:h + 1, d:], pos, m["rot"])[:, 0] @ kr.T) * m["scale"]
        e = torch.exp(s).tril()
        a = e / (e.sum(-1, keepdim=True) + torch.exp(w["sink"][h]))
        heads.append((a @ c) @ w["uv"][h * dv:(h + 1) * dv].T * torch.sigmoid(x @ w["g"][h])[:, None])
    assert torch.allclose(got, torch.cat(heads, -1) @ w["o"].T, atol=1e-10)


def test_sharp_weights_show_a_far_key_and_a_far_write():
    """What the GPU tests rest on: with the sharp attentions a changed token far back moves later rows, and so does one in the
    memory of a slow decay."""
    for layer in (dm.full(sharp=4.0, softcap=0, v_mix=False), dm.latent(sharp=6.0), dm.lightning(decay=(0.999, 0.9995, 0.99))):
        cfg = dm.config([layer], side=0)
        w = {k: t.double() for k, t in dm.make_weights(cfg, 9, torch.float32).items()}
        ids = torch.randint(0, 61, (120,), generator=torch.Generator().manual_seed(1)).tolist()
        other = list(ids)
        other[15] = (ids[15] + 1) % 61
        a, b = plain.forward(cfg, w, ids), plain.forward(cfg, w, other)
        assert torch.equal(a[:15], b[:15])
        moved = ((a - b)[60:] ** 2).mean(-1).sqrt() / (a[60:] ** 2).mean(-1).sqrt()
        assert float(moved.max()) > 1e-2


# ---- the configuration, the model tree -----------------------------------------------------------------
def _parse(cfg):
    from llmengine.config import parse_config
    return parse_config(cfg)


def _build(cfg):
    from llmengine.config.registry import resolve
    return resolve("Diporax").build_model(_parse(cfg))


def test_the_reader_takes_every_value_from_the_file():
    c = _parse(dm.MIXED)
    assert (c.vocab_size, c.width, c.norm_eps, c.token_dim, len(c.layers), c.eos_token_ids) == (61, 28, 1e-5, 6, 8, ())
    a = c.layers[0]
    assert a.type == "attention" and a.mixer["conv"] == 3 and a.mixer["softcap"] == 8.0 and a.mixer["v_mix"] is True
    assert a.mixer["rot"] == {"dims": 8, "base": 70.0, "scaling": {"factor": 2.5, "original": 90.0, "fast": 8.0, "slow": 0.5}}
    assert a.mlp == {"experts": 5, "top": 2, "ff": 20, "shared_ff": 14} and c.layers[2].mlp is None and c.layers[1].mlp["shared_ff"] is None
    assert c.layers[1].mixer["decay"] == (0.5, 0.93, 0.997) and c.layers[6].mixer["rot"]["scaling"] is None
    assert c.layers[3].mixer["softcap"] == 0.0 and c.layers[3].mixer["v_mix"] is False
    assert _parse(dm.config([dm.lightning()], side=0)).token_dim == 0


@pytest.mark.parametrize("where, change", [
    ("mixer", lambda l: l.update(type="mamba")), ("decay", lambda l: l["mixer"].update(decay=[0.5])), ("decay", lambda l: l["mixer"].update(decay=[0.5, 2.0, 0.1])),
    ("heads", lambda l: l["mixer"].pop("heads")), ("kind", lambda l: l.update(mlp={"kind": "dense", "ff": 8})),
    ("top", lambda l: l.update(mlp=dm.moe(experts=2, top=3))), ("router", lambda l: l.update(mlp={"kind": "moe", "expert": {"ff": 4}}))])
def test_the_reader_names_what_is_wrong(where, change):
    from llmengine.config import ConfigError
    cfg = copy.deepcopy(dm.config([dm.lightning()]))
    change(cfg["layers"][0])
    with pytest.raises(ConfigError, match=where):
        _parse(cfg)


@pytest.mark.parametrize("where, layers", [
    ("kv_heads", [dm.full(heads=5, kv_heads=2)]), ("dims", [dm.full(dims=7)]), ("dims", [dm.full(dims=14)]), ("rot_dim", [dm.latent(rot_dim=5)]),
    ("v_mix", [dm.full(), dm.full(vdim=9)]), ("softcap", [dm.full(softcap=-1.0)])])
def test_the_reader_refuses_sizes_that_do_not_go_together(where, layers):
    from llmengine.config import ConfigError
    with pytest.raises(ConfigError, match=where):
        _parse(dm.config(layers))


def test_tensor_names_and_shapes():
    specs = {n: tuple(s.shape) for n, s in _build(dm.MIXED).named_specs().items()}
    assert specs["embed"] == (61, 28) and specs["embed.norm"] == (28,) and specs["side.embed"] == (61, 48) and specs["head"] == (61, 28)
    l0 = {n[3:]: s for n, s in specs.items() if n.startswith("l0.")}
    assert {n: s for n, s in l0.items() if n.startswith("mix.")} == {
        "mix.q": (72, 28), "mix.k": (24, 28), "mix.v": (20, 28), "mix.g": (6, 28), "mix.o": (28, 60), "mix.q.b": (72,), "mix.k.b": (24,),
        "mix.v.b": (20,), "mix.q.conv": (72, 3), "mix.k.conv": (24, 3), "mix.v.conv": (20, 3), "mix.q.norm": (12,), "mix.k.norm": (12,), "mix.vmix": ()}
    assert l0["norm1"] == l0["norm2"] == l0["ls1"] == l0["ls2"] == l0["side.norm"] == (28,)
    assert l0["side.gate"] == (6, 28) and l0["side.proj"] == (28, 6)
    assert l0["mlp.router"] == (5, 28) and l0["mlp.shared.sg"] == (1, 28) and l0["mlp.shared.down"] == (28, 14) and l0["mlp.e4.up"] == (20, 28)
    assert "l1.mlp.shared.sg" not in specs and "l2.ls2" not in specs and "l2.norm2" not in specs and "l3.mix.vmix" not in specs
    assert {n[7:]: s for n, s in specs.items() if n.startswith("l2.mix.")} == {
        "dq": (18, 28), "dq.norm": (18,), "uq": (48, 18), "dkv": (18, 28), "dkv.norm": (12,), "uk": (30, 12), "uv": (21, 12), "sink": (3,), "g": (3, 28),
        "o": (28, 21)}
    assert {n[7:]: s for n, s in specs.items() if n.startswith("l1.mix.")} == {
        "q": (30, 28), "k": (30, 28), "v": (18, 28), "g": (18, 28), "norm": (18,), "o": (28, 18)}


def test_what_each_mixer_keeps():
    specs = _build(dm.MIXED).cache_specs()
    assert specs[0].kind == "full" and specs[0].state["conv"][0] == (2, 116) and set(specs[0].paged) == {"k", "v"}
    assert specs[1].paged == {} and specs[1].state["memory"][0] == (3, 6, 10)
    assert specs[2].paged == {"rows": (-1, 18)} and specs[7].state["conv"][0] == (0, 116)


def test_sizes_that_no_kernel_takes_are_named():
    model = _build(dm.config([dm.lightning(dim=300), dm.full(dim=300, dims=8), dm.latent(kv_rank=600), dm.full(conv=17)]))
    assert [r.split(":")[0] for r in model.tree_refusals()] == ["l0.mix", "l1.mix", "l2.mix", "l3.mix"]


def test_random_weights_fit_the_model(tmp_path):
    from llmengine.parts.base import Placement
    from llmengine.weights import load_model_weights, write_random_model
    folder = write_random_model(dm.ALIGNED, str(tmp_path), 3, torch.float32)
    model = _build(dm.ALIGNED)
    read = load_model_weights(model, folder, Placement(torch.device("cpu"), torch.float32))
    assert set(read) == set(model.named_specs())
    block = model.layers[0]
    assert len(block.scales) == 2 and torch.equal(block.scales[0], torch.ones(64))           # (scale and norm weight in one)
