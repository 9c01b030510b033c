"""Lukupel on the CPU: the plain implementation (tests/plain_lukupel.py) pinned to independent facts, the configuration
reader, the tensor names, the cache specs and the random weights."""
from __future__ import annotations

import copy
import math

import pytest
import torch

import lukupel_models as lm
import plain_lukupel as plain

F64 = torch.float64


def _rand(*shape, seed=0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=F64)


# ---- the plain implementation's mechanisms -------------------------------------------------------------
def test_rotation_turns_halves_and_depends_on_distance_only():
    rot = {"base": 30.0, "dims": 6, "scaling": {"factor": 2.0}}
    x = _rand(1, 1, 8, seed=1)
    y = plain.rotate_halves(x, torch.tensor([7]), rot)
    for c in range(3):
        a, b, ang = float(x[0, 0, c]), float(x[0, 0, c + 3]), 7 * 30.0 ** (-2.0 * c / 6) / 2.0
        assert abs(float(y[0, 0, c]) - (a * math.cos(ang) - b * math.sin(ang))) < 1e-12
        assert abs(float(y[0, 0, c + 3]) - (b * math.cos(ang) + a * math.sin(ang))) < 1e-12
    assert torch.equal(y[..., 6:], x[..., 6:])                       # the entries behind the rotated ones pass
    q, k = _rand(1, 1, 8, seed=2), _rand(1, 1, 8, seed=3)
    dot = lambda i, j: float((plain.rotate_halves(q, torch.tensor([i]), rot) * plain.rotate_halves(k, torch.tensor([j]), rot)).sum())
    assert abs(dot(40, 31) - dot(9, 0)) < 1e-10 and abs(dot(40, 31) - dot(40, 30)) > 1e-4
    # the factor stretches the positions: twice the factor at twice the position is the same turn
    slow = dict(rot, scaling={"factor": 4.0})
    assert torch.allclose(plain.rotate_halves(x, torch.tensor([14]), slow), y, atol=1e-12)
    assert torch.allclose(plain.pair_frequencies({"base": 30.0, "dims": 6}), plain.pair_frequencies(rot) * 2.0)


def test_queries_and_keys_have_length_root_dim_behind_the_rotation():
    m = {"heads": 4, "kv_heads": 2, "dim": 10, "rot": {"base": 20.0, "dims": 6}}
    x = _rand(5, 12, seed=4)
    w = {"q": _rand(40, 12, seed=5), "k": _rand(20, 12, seed=6)}
    q, k = plain.queries_keys(x, w, m, 1e-12, torch.arange(5))
    assert torch.allclose(q.norm(dim=-1), torch.full((5, 4), 10 ** 0.5, dtype=F64)) and torch.allclose(k.norm(dim=-1), torch.full((5, 2), 10 ** 0.5, dtype=F64))
    # a rotation keeps lengths, so the same norm in front of it gives the same (what the engine's kernel does)
    other = plain.rotate_halves(plain.rms_unit((x @ w["q"].T).view(5, 4, 10), 1e-3), torch.arange(5), m["rot"])
    assert torch.allclose(plain.queries_keys(x, w, m, 1e-3, torch.arange(5))[0], other, atol=1e-12)


def test_who_sees_whom_in_chunks():
    v = plain.visible(7, 3)
    assert v[5].tolist() == [False, False, False, True, True, True, False] and v[6].tolist() == [False] * 6 + [True]
    assert v[2].tolist() == [True, True, True] + [False] * 4 and v[3].tolist() == [False, False, False, True] + [False] * 3
    assert plain.visible(4).tolist() == torch.tril(torch.ones(4, 4, dtype=torch.bool)).tolist()
    assert plain.visible(4, 1).tolist() == torch.eye(4, dtype=torch.bool).tolist()
    assert plain.visible(6, 6).tolist() == plain.visible(6).tolist()


def test_one_head_in_chunks_by_hand_and_chunks_as_sequences_of_their_own():
    T = 5
    q, k, v = _rand(T, 1, 4, seed=7), _rand(T, 1, 4, seed=8), _rand(T, 1, 2, seed=9)
    out = plain.attend(q, k, v, 0.5, plain.visible(T, 3))
    for i in range(T):
        lo = i // 3 * 3
        e = [math.exp(0.5 * float(q[i, 0] @ k[j, 0])) for j in range(lo, i + 1)]
        assert torch.allclose(out[i, 0], sum(a / sum(e) * v[j, 0] for a, j in zip(e, range(lo, i + 1))), atol=1e-12)
    assert torch.allclose(out[3:], plain.attend(q[3:], k[3:], v[3:], 0.5, plain.visible(2)), atol=1e-12)
    six = plain.attend(_rand(4, 6, 3, seed=10), _rand(4, 2, 3, seed=11), _rand(4, 2, 5, seed=12), 1.0, plain.visible(4))
    for h in range(6):                                               # grouped heads read the key head of their group
        alone = plain.attend(_rand(4, 6, 3, seed=10)[:, h:h + 1], _rand(4, 2, 3, seed=11)[:, h // 3:h // 3 + 1],
                             _rand(4, 2, 5, seed=12)[:, h // 3:h // 3 + 1], 1.0, plain.visible(4))
        assert torch.allclose(six[:, h], alone[:, 0], atol=1e-12)


def test_the_matrix_memory_without_its_level_and_carried_on():
    """The level only keeps numbers small: with sums that are not scaled, S_t = sum_s e^(F_t - F_s + i_s) k_s v_s^T (F the
    running sum of f), the read is S^T q / (max(|z . q|, 1) + 1e-6 e^m), with m the level."""
    T, n, d, dv = 9, 2, 3, 4
    q, k, v = _rand(T, n, d, seed=13), _rand(T, n, d, seed=14), _rand(T, n, dv, seed=15)
    i, f = _rand(T, n, seed=16) * 2, -torch.nn.functional.softplus(_rand(T, n, seed=17) * 2)
    out, state = plain.matrix_memory(q, k, v, i, f)
    F = torch.cumsum(f, 0)
    for h in range(n):
        level = 0.0
        for t in range(T):
            level = max(float(f[t, h]) + level, float(i[t, h]))
            wts = torch.exp(F[t, h] - F[:t + 1, h] + i[:t + 1, h])
            num = ((wts * (k[:t + 1, h] @ q[t, h]))[:, None] * v[:t + 1, h]).sum(0)
            zq = float((wts * (k[:t + 1, h] @ q[t, h])).sum())
            assert torch.allclose(out[t, h], num / (max(abs(zq), 1.0) + 1e-6 * math.exp(level)), rtol=1e-9, atol=1e-12)
        assert abs(float(state[2][h]) - level) < 1e-12
    first, mid = plain.matrix_memory(q[:4], k[:4], v[:4], i[:4], f[:4])
    rest, end = plain.matrix_memory(q[4:], k[4:], v[4:], i[4:], f[4:], state=mid)
    assert torch.allclose(torch.cat([first, rest]), out, atol=1e-12) and all(torch.allclose(a, b, atol=1e-12) for a, b in zip(end, state))


def test_the_level_starts_at_zero_and_follows_the_gates():
    one = torch.ones(1, 1, 1, dtype=F64)
    for i in (-3.0, 2.0):
        f = -0.5
        out, (S, z, m) = plain.matrix_memory(one, one, 5 * one, torch.tensor([[i]], dtype=F64), torch.tensor([[f]], dtype=F64))
        top = max(f, i)                                              # the start counts as a level of zero, not as minus infinity
        assert abs(float(m) - top) < 1e-12 and abs(float(S) - 5 * math.exp(i - top)) < 1e-12
        w = math.exp(i - top)
        assert abs(float(out) - 5 * w / (max(w, math.exp(-top)) + 1e-6)) < 1e-9


def test_gates_are_capped_and_the_forget_gate_is_a_sigmoid():
    w = {"i": _rand(2, 5, seed=18), "i.b": _rand(2, seed=19), "f": _rand(2, 5, seed=20), "f.b": _rand(2, seed=21)}
    x = _rand(4, 5, seed=22)
    i, f = plain.log_gates(x, w, 1e6)                                # a cap far away changes nothing
    assert torch.allclose(i, x @ w["i"].T + w["i.b"], atol=1e-6)
    assert torch.allclose(torch.exp(f), torch.sigmoid(x @ w["f"].T + w["f.b"]), atol=1e-6)
    i, f = plain.log_gates(100 * x, w, 2.0)
    assert float(i.abs().max()) <= 2.0 and float(torch.exp(f).max()) <= 1 / (1 + math.exp(-2.0)) + 1e-9
    assert float(torch.exp(f).min()) >= 1 / (1 + math.exp(2.0)) - 1e-9


def test_a_layer_norms_behind_its_sublayers_and_a_borrower_remembers_its_own():
    layers = [lm.chunked(chunk=4, ff=10), lm.mlstm(ff=8)]
    cfg = lm.config(layers + [lm.borrow(layers, 1), lm.borrow(layers, 0)])
    w = {k: v.double() for k, v in lm.make_weights(cfg, 1, torch.float32).items()}
    assert not any(n.startswith(("l2.", "l3.")) for n in w)
    ids = [3, 9, 27, 1, 44, 8, 8, 15]
    logits, seen = plain.forward(cfg, w, ids, return_layers=True)
    eps, c = cfg["norm"]["eps"], cfg["residual_mult"]
    x = w["embed"][torch.tensor(ids)] * cfg["embedding"]["scale"]
    for n, (j, mix) in enumerate(((0, plain.chunked_attention), (1, plain.mlstm), (1, plain.mlstm), (0, plain.chunked_attention))):
        x = x + c * plain.norm(mix(x, plain.sub(w, f"l{j}.mix."), layers[j]["mixer"], eps), w[f"l{j}.norm1"], eps)
        up = torch.relu(x @ w[f"l{j}.mlp.up"].T)
        x = x + c * plain.norm((up * up) @ w[f"l{j}.mlp.down"].T, w[f"l{j}.norm2"], eps)
        assert torch.allclose(seen[n], x, atol=1e-12)
    cap = cfg["logit_softcap"]
    raw = plain.norm(x, w["final.norm"], eps) @ w["embed"].T
    assert torch.allclose(logits, cap * torch.tanh(raw / cap), atol=1e-12) and float(logits.abs().max()) < cap
    # norm weights of zero switch a sublayer off, and a residual factor of zero all of them
    assert torch.allclose(plain.forward(dict(cfg, residual_mult=0.0), w, ids, return_layers=True)[1][3],
                          w["embed"][torch.tensor(ids)] * cfg["embedding"]["scale"], atol=1e-12)


def test_sharp_weights_show_a_chunk_that_is_one_off():
    cfg = lm.config([lm.chunked(chunk=9, sharp=4.0, ff=None)])
    w = lm.make_weights(cfg, 2, torch.float32)
    ids = torch.randint(0, cfg["vocab"], (60,), generator=torch.Generator().manual_seed(3)).tolist()
    ref = plain.forward(cfg, w, ids)
    off = copy.deepcopy(cfg)
    off["layers"][0]["mixer"]["mask"]["size"] = 10
    moved = (plain.forward(off, w, ids) - ref).norm(dim=-1) / ref.norm(dim=-1)
    assert float(moved[:9].max()) < 1e-12 and float(moved[9:].max()) > 0.05 and float(moved[9:].median()) > 1e-3


def test_what_was_written_long_ago_shows_in_the_memory():
    """With the tests' remembering weights a token 150 places back moves the row."""
    cfg = lm.config([lm.mlstm(gate_cap=9.0)])
    w = lm.make_weights(cfg, 4, torch.float32, remember=7.0)
    ids = torch.randint(0, cfg["vocab"], (170,), generator=torch.Generator().manual_seed(5)).tolist()
    other = list(ids)
    other[20] = (ids[20] + 7) % cfg["vocab"]
    a, b = plain.forward(cfg, w, ids), plain.forward(cfg, w, other)
    moved = (a - b).norm(dim=-1) / a.norm(dim=-1)
    assert float(moved[:20].max()) < 1e-12 and float(moved[169]) > 1e-3


# ---- configuration, names, caches ---------------------------------------------------------------------
def _parse(cfg):
    from llmengine.config import parse_config
    return parse_config(cfg)


def _model(cfg):
    from llmengine.config.registry import resolve
    return resolve("Lukupel").build_model(_parse(cfg))


def test_the_reader_takes_every_size_and_constant():
    c = _parse(lm.MIXED)
    assert type(c).__name__ == "LukupelConfig" and c.vocab_size == 61 and c.width == 28 and c.embedding_scale == 2.0
    assert c.norm_eps == 1e-5 and c.residual_mult == 0.7 and c.logit_softcap == 9.0 and len(c.layers) == 10
    a = c.layers[0].mixer
    assert (a["heads"], a["kv_heads"], a["dim"], a["vdim"], a["scale"], a["rot_dims"], a["rot_base"], a["rot_factor"], a["chunk"]) == \
           (6, 2, 12, 10, 0.9, 8, 50.0, 2.0, 11)
    assert c.layers[0].ff == 24 and c.layers[2].ff is None and c.layers[2].mixer["rot_factor"] == 1.0 and c.layers[4].mixer["chunk"] == 0
    assert c.layers[1].mixer == {"heads": 3, "dim": 10, "vdim": 6, "gate_cap": 5.0} and c.layers[3].ff == 20
    assert [l.weights_of for l in c.layers] == [None, None, None, None, None, 1, 0, 3, None, 4]
    # a borrower of a borrower runs on the tensors that the first one borrows; what the file leaves out is neutral
    chain = [lm.mlstm(), lm.mlstm(weights_of=0), lm.mlstm(weights_of=1)]
    assert [l.weights_of for l in _parse(lm.config(chain)).layers] == [None, 0, 0]
    bare = {k: v for k, v in lm.config(chain).items() if k not in ("residual_mult", "logit_softcap", "embedding")}
    assert (_parse(bare).residual_mult, _parse(bare).logit_softcap, _parse(bare).embedding_scale) == (1.0, 0.0, 1.0)


@pytest.mark.parametrize("change, word", [
    (lambda c: c["layers"][0]["mixer"].update(heads=5), "heads"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=14), "dims"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=3), "dims"),
    (lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].update(factor=0), "factor"),
    (lambda c: c["layers"][0]["mixer"]["mask"].update(size=0), "size"),
    (lambda c: c["layers"][1]["mixer"].update(gate_cap=0), "gate_cap"),
    (lambda c: c["layers"][1]["mixer"].pop("vdim"), "vdim"),
    (lambda c: c["layers"][5].update(weights_of=5), "weights_of"),
    (lambda c: c["layers"][5].update(weights_of=40), "weights_of"),
    (lambda c: c["layers"][1].update(weights_of=5), "weights_of"),
    (lambda c: c["layers"][5].update(weights_of=0), "differs from layer 0"),
    (lambda c: c["layers"][6]["mixer"].update(scale=0.5), "differs from layer 0"),
    (lambda c: c["layers"][5].update(mlp={"kind": "dense", "ff": 8}), "differs from layer 1"),
    (lambda c: c["layers"][1].update(type="recurrent"), "recurrent"),
    (lambda c: c["layers"][0]["mlp"].update(kind="moe"), "moe"),
    (lambda c: c.update(logit_softcap=-1.0), "logit_softcap"),
    (lambda c: c.pop("norm"), "norm"),
    (lambda c: c.pop("vocab"), "vocab"),
])
def test_the_reader_refuses_by_key_name(change, word):
    from llmengine.config import ConfigError
    cfg = copy.deepcopy(lm.MIXED)
    change(cfg)
    with pytest.raises(ConfigError, match=word):
        _parse(cfg)


def test_tensor_names_and_shapes():
    specs = _model(lm.MIXED).named_specs()
    shape = lambda n: tuple(specs[n].shape)
    assert shape("embed") == (61, 28) and shape("final.norm") == (28,) and "head" not in specs
    assert shape("l0.mix.q") == (72, 28) and shape("l0.mix.k") == (24, 28) and shape("l0.mix.v") == (20, 28) and shape("l0.mix.o") == (28, 60)
    assert shape("l0.mlp.up") == (24, 28) and shape("l0.mlp.down") == (28, 24) and shape("l0.norm2") == (28,) and "l0.mlp.gate" not in specs
    assert not any("norm" in n for n in specs if n.startswith("l0.mix."))      # queries and keys are normed without weights
    assert sorted(n for n in specs if n.startswith("l1.")) == sorted(
        ["l1.norm1"] + ["l1.mix." + n for n in ("q", "k", "v", "g", "o", "norm", "i", "i.b", "f", "f.b")])
    assert shape("l1.mix.q") == (30, 28) and shape("l1.mix.v") == (18, 28) and shape("l1.mix.g") == (18, 28) and shape("l1.mix.norm") == (18,)
    assert shape("l1.mix.i") == (3, 28) and shape("l1.mix.f.b") == (3,)
    assert {n.split(".")[0] for n in specs} == {"embed", "final", "l0", "l1", "l2", "l3", "l4", "l8"}     # borrowers have none


def test_cache_specs_and_the_schedule():
    model = _model(lm.MIXED)
    specs = model.cache_specs()
    assert sorted(specs) == list(range(10))                                 # every layer remembers by itself, borrowers too
    assert (specs[0].kind, specs[0].window) == ("chunk", 11) and (specs[2].kind, specs[2].window) == ("chunk", 6) and specs[4].kind == "full"
    assert dict(specs[6].paged) == dict(specs[0].paged) == {"k": (2, -1, 12), "v": (2, 10, -1)} and not specs[0].state
    assert dict(specs[1].state) == {"memory": ((3, 7, 10), torch.float32), "level": ((3, 7), torch.float32)} and not specs[1].paged
    assert [(c.layer, c.cache_id, c.write_cache) for c in model.schedule] == [(i, i, True) for i in range(5)] + [
        (1, 5, True), (0, 6, True), (3, 7, True), (5, 8, True), (4, 9, True)]
    from llmengine.cache import plan_groups
    assert [(g.name, g.kind, g.window) for g in plan_groups(specs, 7)] == [("chunk11", "chunk", 11), ("chunk6", "chunk", 6), ("full", "full", 0)]


def test_random_weights_are_written_and_named_as_the_model_reads_them(tmp_path):
    from llmengine.weights import write_random_model
    from llmengine.weights.loader import WeightError, check_names
    from llmengine.weights.safetensors_io import TensorIndex
    folder = write_random_model(lm.ALIGNED, str(tmp_path), 3)
    index = TensorIndex(folder)
    try:
        have = {n: index.entry(n).shape for n in index.names()}
        check_names(_model(lm.ALIGNED), have, folder)
        assert "head" not in have and "embed" in have and not any(n.startswith(("l4.", "l5.")) for n in have)
        with pytest.raises(WeightError, match="l4.norm1"):
            check_names(_model(lm.ALIGNED), dict(have, **{"l4.norm1": (64,)}), folder)
    finally:
        index.close()


def test_layers_need_numbers_of_their_own():
    from llmengine.models import DecoderModel
    m = _model(lm.MIXED)
    with pytest.raises(ValueError, match="different numbers"):
        DecoderModel(m.config, m.embedding, m.layers, m.final_norm, m.head, layer_numbers=[0] * len(m.layers))
