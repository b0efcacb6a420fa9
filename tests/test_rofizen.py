"""Rofizen without a GPU: the configuration, the plain implementation's own mechanisms against hand-made cases, and
the real engine, cache and generation loop driven through the plain stand-ins for the kernels against the plain
implementation."""
import copy
import json
import math
import os

import numpy as np
import pytest
import torch

import plain_ops
import plain_rofizen as pr
from replays import batch_steps, chunk_steps, requests_for, run_steps, tail_steps, whole_steps
from rofizen_tiny import RZ, RZ_A, RZ_B, random_config, write_rofizen, written_config


# ------------------------------------------------------------------ configuration
def test_configuration_reads_writes_and_describes():
    from minfer_amd import config_from_dict
    from minfer_amd.engine.model import expected_tensors
    cfg = config_from_dict(RZ_A)
    assert config_from_dict(cfg.to_dict()).to_dict() == cfg.to_dict()
    spec = cfg.model_spec()
    assert [b.kind for b in spec.blocks] == ["postnorm"] * 4 and spec.blocks[0].params["stream_scale"] == 1.7
    assert spec.embedding.params["scale"] == 3.0 and spec.stop_tokens == ()
    names = expected_tensors(spec)
    assert names["l0.mix.left.q"].shape == (192, 96) and names["l0.mix.left.k.b"].shape == (96,)
    assert names["l0.mix.left.q.norm"].shape == (192,) and names["l0.mix.left.k.norm"].shape == (96,)
    assert names["l0.mix.left.o"].shape == (96, 96) and names["l0.mix.left.o.b"].shape == (96,) and names["l0.mix.left.out"].shape == (96,)
    assert names["l0.mix.right.i"].shape == (3, 96) and names["l0.mix.right.f.b"].shape == (3,)
    assert names["l0.mix.right.norm"].shape == (120,) and names["l0.mix.right.o"].shape == (96, 120)
    assert names["l0.mlp.table"].shape == (300, 2) and names["l0.mlp.table"].below == 6
    assert names["l0.mlp.shared.up"].shape == (72, 96) and names["l0.mlp.shared.sg"].shape == (1, 96)
    assert names["l1.mix.a1"].shape == (5, 96) and names["l1.mix.a2"].shape == (48, 5) and names["l1.mix.norm"].shape == (48,)
    assert names["l1.mlp.down"].shape == (96, 112) and "l1.mlp.up.b" not in names
    assert names["l2.mix.g"].shape == (48, 96) and "l2.mix.norm" not in names
    assert "l3.norm2" not in names and cfg.ignored_tensors() == ("l3.norm2",)
    assert "l0.mlp.shared.up" not in expected_tensors(config_from_dict(RZ_B).model_spec())
    left = spec.blocks[0].mixer.params["left"].params
    assert np.allclose(left["slopes"], [2 ** (-8 / 6), 2 ** (-16 / 6), 2 ** (-4.0), 2 ** (-32 / 6), 2 ** (-40 / 6), 2 ** (-8.0)])


def test_the_rank_of_a_decay_comes_from_the_file():
    from minfer_amd import ConfigError, config_from_dict
    cfg = config_from_dict(written_config(RZ_A))
    with pytest.raises(ConfigError, match="rank"):
        cfg.model_spec()
    with pytest.raises(ConfigError, match="l1.mix.a1"):
        cfg.adopt_tensor_shapes({"l3.mix.a1": (20, 96)})
    cfg.adopt_tensor_shapes({"l1.mix.a1": (5, 96), "l3.mix.a1": (20, 96)})
    assert cfg.to_dict() == config_from_dict(RZ_A).to_dict()


@pytest.mark.parametrize("change, word", [
    (lambda c: c["layers"][0].update(type="conv"), "type"),
    (lambda c: c["layers"][0]["mlp"].update(kind="wide"), "kind"),
    (lambda c: c["layers"][0]["mixer"]["left"].update(kv_heads=4), "kv_heads"),
    (lambda c: c["layers"][0]["mixer"].pop("right"), "heads"),
    (lambda c: c["layers"][0]["mixer"]["right"].update(gate_cap=0.0), "gate_cap"),
    (lambda c: c["layers"][0]["mixer"]["left"]["q_temp"].pop("every"), "every"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(top=7), "router"),
    (lambda c: c["layers"][0]["mlp"]["shared"].pop("ff"), "ff"),
    (lambda c: c["layers"][1]["mixer"].pop("tau"), "tau"),
    (lambda c: c["layers"][2]["mixer"].update(decay=[0.9]), "decay"),
    (lambda c: c["layers"][2]["mixer"].update(decay=[0.9, 1.5]), "decay"),
    (lambda c: c["layers"][2]["mixer"]["rot"].update(dims=42), "dims"),
    (lambda c: c["layers"][2]["mixer"]["rot"].update(dims=7), "dims"),
    (lambda c: c.pop("postln_alpha"), "postln_alpha"),
    (lambda c: c.pop("width"), "width"),
])
def test_configuration_rejections_name_the_key(change, word):
    from minfer_amd import ConfigError, config_from_dict
    raw = copy.deepcopy(RZ_A)
    change(raw)
    with pytest.raises(ConfigError, match=word):
        config_from_dict(raw).model_spec()


def test_tables_are_integers_in_range_and_differ_within_a_row(tmp_path, monkeypatch):
    plain_ops.install(monkeypatch)
    from minfer_amd import WeightError, config_from_dict, load_model, write_random_model
    from minfer_amd.weights.safetensors_io import SafetensorsFile, write_safetensors
    folder = write_rofizen(str(tmp_path / "m"), RZ_A, seed=1)
    path = os.path.join(folder, "model.safetensors")
    f = SafetensorsFile(path)
    whole = {n: f.tensor(n).clone() for n in f.names()}

    def write(table):
        made = dict(whole, **{"l0.mlp.table": table})
        write_safetensors(path, [(n, tuple(t.shape), t.dtype) for n, t in made.items()], lambda n: made[n])
    good = whole["l0.mlp.table"]
    for value, word in ((6, "expert numbers"), (-1, "expert numbers"), (int(good[5, 0]), "twice")):
        bad = good.clone()
        bad[5, 1] = value
        write(bad)
        with pytest.raises(WeightError, match=word):
            load_model(folder, dtype="float32", device="cpu")
    write(good.to(torch.bfloat16))
    with pytest.raises(WeightError, match="not integers"):
        load_model(folder, dtype="float32", device="cpu")
    write(good)
    load_model(folder, dtype="float32", device="cpu")
    # a folder of random weights has such tables too
    random = write_random_model(str(tmp_path / "r"), config_from_dict(RZ_A), seed=3)
    t = SafetensorsFile(os.path.join(random, "model.safetensors")).tensor("l0.mlp.table")
    assert t.dtype == torch.int32 and t.min() >= 0 and t.max() < 6 and bool((t[:, 0] != t[:, 1]).all()) and len(t[:, 0].unique()) == 6
    load_model(random, dtype="bfloat16", device="cpu")


def test_a_stored_norm_without_feed_forward_is_not_used(tmp_path, monkeypatch):
    plain_ops.install(monkeypatch)
    from minfer_amd import load_model
    from minfer_amd.weights.safetensors_io import SafetensorsFile, write_safetensors
    folder = write_rofizen(str(tmp_path / "m"), RZ_A, seed=1)
    path = os.path.join(folder, "model.safetensors")
    f = SafetensorsFile(path)
    made = {n: f.tensor(n).clone() for n in f.names()}
    made["l3.norm2"] = torch.ones(96, dtype=torch.bfloat16)
    write_safetensors(path, [(n, tuple(t.shape), t.dtype) for n, t in made.items()], lambda n: made[n])
    with pytest.warns(UserWarning, match="l3.norm2"):
        load_model(folder, dtype="float32", device="cpu")


# ------------------------------------------------------------------ the plain mechanisms by hand
def test_plain_norms_temperature_and_slopes_by_hand():
    x = np.array([[1.0, 3.0, 5.0, 7.0]])
    assert np.allclose(pr.layer_norm(x, np.array([1.0, 2.0, 1.0, -1.0]), 0.0), np.array([[-3, -2, 1, -3]]) / math.sqrt(5.0))
    assert np.allclose(pr.layer_norm(x, np.ones(4), 4.0), np.array([[-3, -1, 1, 3]]) / 3.0)      # eps inside the root
    assert np.allclose(pr.unit_rms(np.array([3.0, 4.0, 0.0, 0.0]), 0.0), [1.2, 1.6, 0, 0])
    # steps of 4 positions: positions 0 to 2 have none behind them, position 3 the first
    t = pr.query_temperature([0, 2, 3, 6, 7, 30], dict(coef=0.5, every=4))
    assert np.allclose(t, 1 + 0.5 * np.log([1, 1, 2, 2, 3, 8]))
    assert np.allclose(pr.slopes(4), [0.25, 0.0625, 1 / 64, 1 / 256]) and np.allclose(pr.slopes(1), [1 / 256])
    v = np.array([[[1.0, 0.0, 0.0, 2.0, 7.0]]])
    assert np.allclose(pr.rotate_halves(v, [2], 100.0, 4)[0, 0],
                       [math.cos(2.0), -2 * math.sin(0.2), math.sin(2.0), 2 * math.cos(0.2), 7.0])


def test_plain_attention_by_hand():
    """Two tokens, one head: the norm over the whole projection, the cap ahead of the slope, biases, the temperature."""
    eye = np.eye(2)
    w = {"q": eye, "q.b": np.zeros(2), "k": eye, "k.b": np.zeros(2), "v": eye, "v.b": np.array([0.0, 1.0]), "o": eye, "o.b": np.array([5.0, 0.0]),
         "q.norm": np.array([2.0, 1.0]), "k.norm": np.ones(2)}
    m = dict(heads=1, kv_heads=1, dim=2, vdim=2, scale=0.7, softcap=1.5, q_temp=dict(coef=0.4, every=2))
    h = np.array([[3.0, 0.0], [1.0, 1.0]])
    out = pr.sloped_attention(h, w, "", m, 0.0)
    assert np.allclose(out[0], h[0] + [5.0, 1.0])
    q, k0, k1 = np.array([2.0, 1.0]) * (1 + 0.4 * math.log(2.0)), np.array([math.sqrt(2.0), 0.0]), np.array([1.0, 1.0])
    s = [1.5 * math.tanh(q @ k0 * 0.7 / 1.5) - 1 / 256, 1.5 * math.tanh(q @ k1 * 0.7 / 1.5)]
    p = np.exp(s) / np.exp(s).sum()
    assert np.allclose(out[1], p[0] * h[0] + p[1] * h[1] + [5.0, 1.0])
    # two query heads on one kv head share their keys; the norm runs over both heads' values at once
    w2 = dict(w, q=np.vstack([eye, 3 * eye]), **{"q.b": np.zeros(4), "q.norm": np.ones(4), "o": np.eye(2, 4), "k.norm": np.ones(2)})
    m2 = dict(m, heads=2, softcap=None, q_temp=None)
    rows = pr.unit_rms(h @ w2["q"].T, 0.0)
    assert np.allclose((rows[1, 2:] / rows[1, :2]), 3.0)
    s = [rows[1, :2] @ k0 * 0.7 - 2.0 ** -4, rows[1, :2] @ k1 * 0.7]
    p = np.exp(s) / np.exp(s).sum()
    assert np.allclose(pr.sloped_attention(h, w2, "", m2, 0.0)[1], p[0] * h[0] + p[1] * h[1] + [5.0, 1.0])


def test_plain_recurrences_by_hand():
    eye = np.eye(2)
    h = np.array([[1.0, 2.0], [3.0, -1.0]])
    # the decay acts on the rows that belong to key channels
    w = {"q": eye, "k": eye, "v": eye, "g": eye, "o": eye, "norm": np.array([1.0, 2.0]), "a1": np.array([[1.0, 0.0]]),
         "a2": np.array([[0.0], [1.0]]), "a2.b": np.array([0.0, -3.0])}
    m = dict(heads=1, dim=2, vdim=2, tau=2.0)
    d = pr.gla_decay(h, w, "", m)[:, 0]
    assert np.allclose(d, [[math.sqrt(0.5), math.sqrt(1 / (1 + math.exp(2.0)))], [math.sqrt(0.5), math.sqrt(0.5)]])
    S = np.outer(h[0], h[0])
    S = np.diag(d[1]) @ S + np.outer(h[1], h[1])
    o = S.T @ h[1] / math.sqrt(2.0)
    want = o / math.sqrt((o * o).mean()) * [1.0, 2.0] * pr.silu(h[1])
    assert np.allclose(pr.gated_linear_attention(h, w, "", m, 0.0)[1], want)
    # retention: the second token's score with the first depends on their distance alone
    w = {"q": eye, "k": eye, "v": eye, "g": eye, "o": eye}
    m = dict(heads=1, dim=2, vdim=2, decay=[0.25], rot=dict(base=10.0, dims=2))
    turned = np.array([[math.cos(1), -math.sin(1)], [math.sin(1), math.cos(1)]])       # a query at distance one
    o = (0.25 * (turned @ h[1]) @ h[0] * h[0] + h[1] @ h[1] * h[1]) / math.sqrt(2.0)
    assert np.allclose(pr.retention(h, w, "", m, 0.0)[1], o / math.sqrt((o * o).mean()) * pr.silu(h[1]))


def test_plain_matrix_memory_by_hand():
    """Unscaled, S is a sum of exp(i + later f) k v^T; the running maximum starts at 0 and only sets the floor of the
    denominator and what 1e-6 is worth beside it."""
    eye = np.eye(2)
    h = np.array([[1.0, 2.0], [0.5, -1.0]])
    zi, zf = np.array([-2.0, 3.0]), np.array([0.0, 1.0])
    w = {"q": eye, "k": eye, "v": eye, "g": np.zeros((2, 2)), "o": eye, "norm": np.array([1.0, 3.0]),
         "i": np.linalg.solve(h, zi)[None], "i.b": np.zeros(1), "f": np.linalg.solve(h, zf)[None], "f.b": np.zeros(1)}
    m = dict(heads=1, dim=2, vdim=2, gate_cap=4.0)
    cap = lambda z: 4.0 * math.tanh(z / 4.0)
    i, f = [cap(z) for z in zi], [math.log(1 / (1 + math.exp(-cap(z)))) for z in zf]
    got_i, got_f = pr.memory_gates(h, w, "", m)
    assert np.allclose(got_i[:, 0], i) and np.allclose(got_f[:, 0], f)
    weights = [math.exp(i[0] + f[1]), math.exp(i[1])]
    q = h[1] / math.sqrt(2.0)
    num = sum(a * (k @ q) * k for a, k in zip(weights, h))
    den = sum(a * (k @ q) for a, k in zip(weights, h))
    m1 = max(f[0], i[0])
    assert m1 < 0.0                                                     # started at 0, not at minus infinity: f wins over i
    m2 = max(f[1] + m1, i[1])
    o = num * math.exp(-m2) / (max(abs(den) * math.exp(-m2), math.exp(-m2)) + 1e-6)
    eps = 1e-2
    want = o / math.sqrt((o * o).mean() + eps) * [1.0, 3.0] * 0.5
    assert np.allclose(pr.matrix_memory(h, w, "", m, eps)[1], want, rtol=1e-12)


def test_plain_feed_forwards_by_hand():
    w = {"up": np.array([[1.0, 1.0], [1.0, -2.0]]), "down": np.array([[1.0, 0.0], [2.0, 1.0]])}
    assert np.allclose(pr.dense(np.array([[2.0, 1.0]]), w, ""), [[9.0, 18.0]])
    assert np.allclose(pr.dense(np.array([[2.0, -1.0]]), w, ""), [[1.0, 18.0]])
    eye = np.eye(2)
    w = {"table": np.array([[1, 0], [2, 1], [0, 2]]), "shared.sg": np.array([[1.0, 0.0]])}
    for e in range(3):
        w.update({f"e{e}.gate": eye * (e + 1), f"e{e}.up": eye, f"e{e}.down": eye * 10 ** e})
    w.update({"shared.gate": eye, "shared.up": eye, "shared.down": eye * 7})
    h = np.array([[1.0, 2.0], [0.5, -1.0]])
    one = lambda e, x: 10 ** e * pr.silu((e + 1) * x) * x
    mlp = dict(router=dict(experts=3, top=2), shared=dict(ff=2))
    got = pr.table_moe(h, [2, 0], w, "", mlp)
    for t, (a, b) in enumerate(((0, 2), (1, 0))):
        want = 0.5 * one(a, h[t]) + 0.5 * one(b, h[t]) + pr.sigmoid(h[t, 0]) * 7 * pr.silu(h[t]) * h[t]
        assert np.allclose(got[t], want)
    assert np.allclose(pr.table_moe(h, [2, 0], w, "", dict(router=mlp["router"]))[0], 0.5 * one(0, h[0]) + 0.5 * one(2, h[0]))


# ------------------------------------------------------------------ the engine on the stand-ins
def _rel(rows, ref):
    worst = 0.0
    for (rid, p), got in rows.items():
        want = ref[rid][p]
        worst = max(worst, float(np.abs(got - want).max() / max(1e-9, want.std())))
    return worst


@pytest.mark.parametrize("name", list(RZ))
def test_engine_on_stand_ins_agrees_with_plain(tmp_path, monkeypatch, name):
    plain_ops.install(monkeypatch)
    from minfer_amd import Engine, load_model
    folder = write_rofizen(str(tmp_path / name), RZ[name], seed=5)
    assert "rank" not in open(os.path.join(folder, "config.json")).read()
    plain = pr.PlainRofizen.from_folder(folder)
    reqs = requests_for(RZ[name]["vocab"], (1, 7, 70, 33), seed=2)
    ref = {rid: plain.forward(toks) for rid, toks in reqs.items()}
    eng = Engine(load_model(folder, dtype="float32", device="cpu"), max_tokens=64 * 12)
    ids = list(reqs)
    for what, steps in (("whole", whole_steps(reqs)), ("one by one", tail_steps(reqs, tail=9)),
                        ("batches", batch_steps(reqs, [ids[:3], ids[3:]])),
                        ("portions", chunk_steps(reqs, [ids[:2], ids[2:]], sizes=(2, 50, 64, 1, 17)))):
        assert _rel(run_steps(eng, steps), ref) < 1e-4, what
    assert not eng.cache.live_slots()


def test_engine_on_stand_ins_random_configuration(tmp_path, monkeypatch):
    plain_ops.install(monkeypatch)
    from minfer_amd import Engine, load_model
    raw = random_config(np.random.default_rng(14))
    folder = write_rofizen(str(tmp_path / "r"), raw, seed=6)
    plain = pr.PlainRofizen.from_folder(folder)
    reqs = requests_for(raw["vocab"], (3, 40, 60), seed=4)
    ref = {rid: plain.forward(toks) for rid, toks in reqs.items()}
    eng = Engine(load_model(folder, dtype="float32", device="cpu"), max_tokens=64 * 8)
    assert _rel(run_steps(eng, chunk_steps(reqs, [list(reqs)], sizes=(2, 31, 1))), ref) < 1e-4, json.dumps(raw)


def test_only_the_wanted_rows_reach_the_last_experts(tmp_path, monkeypatch):
    """The last layer's experts see the wanted rows alone: their tokens' ids must be those rows' ids, in the form for
    few rows and in the form for many, whose counts the host takes from the ids."""
    plain_ops.install(monkeypatch)
    from minfer_amd import Engine, load_model
    raw = dict(copy.deepcopy(RZ_A), layers=[copy.deepcopy(RZ_A["layers"][0])])
    folder = write_rofizen(str(tmp_path / "w"), raw, seed=9)
    plain = pr.PlainRofizen.from_folder(folder)
    reqs = requests_for(300, (40, 30), seed=8)
    eng = Engine(load_model(folder, dtype="float32", device="cpu"), max_tokens=64 * 4)
    slots = [eng.new_sequence() for _ in reqs]
    for want in ([[0, 3, 39], [17]], [list(range(0, 40, 2)), list(range(29, 4, -1))], [[], [29]], [[], []]):
        got = eng.step(slots, list(reqs.values()), want).numpy()
        ref = np.concatenate([plain.forward(t)[w] for t, w in zip(reqs.values(), want)] or [np.zeros((0, 300))])
        assert got.shape == ref.shape and (not got.size or np.abs(got - ref).max() < 1e-4 * ref.std())
        for s in slots:
            eng.end_sequence(s)
        slots = [eng.new_sequence() for _ in reqs]


@pytest.mark.parametrize("name", ["B", "A"])
def test_greedy_generation_on_stand_ins(tmp_path, monkeypatch, name):
    """`generate` with its scheduler, slots and decode sessions, tokens against the plain model."""
    plain_ops.install(monkeypatch)
    from minfer_amd import Engine, generate, load_model
    from minfer_amd.sampling import SamplingParams
    folder = write_rofizen(str(tmp_path / "gen"), RZ[name], seed=8)
    plain = pr.PlainRofizen.from_folder(folder)
    eng = Engine(load_model(folder, dtype="float32", device="cpu"), max_tokens=64 * 6, max_seqs=2)
    prompts = [[5, 9, 20, 7], [11], [25, 3, 3, 3, 8, 1, 44]]
    res = generate(eng, prompts, SamplingParams(temp=0.0, repeat_penalty=1.0), max_new=5, stop_tokens=[])
    for p, toks in zip(prompts, res.tokens):
        seq = list(p)
        for t in toks:
            assert t == pr.greedy(plain.forward(seq)[-1])
            seq.append(t)
    assert not eng.cache.live_slots()
