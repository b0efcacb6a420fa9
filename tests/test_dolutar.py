"""Dolutar without a GPU: the configuration, the plain implementation's own mechanisms against hand-made cases, what
shared cache entries keep, and the real engine, cache and generation loop driven through the plain stand-ins for the
kernels against the plain implementation."""
import copy
import json
import math

import numpy as np
import pytest
import torch

import plain_dolutar as pd
import plain_ops
from dolutar_tiny import DL, DL_A, DL_B, random_config, write_dolutar
from replays import batch_steps, chunk_steps, requests_for, run_steps, tail_steps, whole_steps


# ------------------------------------------------------------------ configuration
def test_configuration_reads_writes_and_describes():
    from minfer_amd import config_from_dict
    from minfer_amd.engine.model import expected_tensors
    cfg = config_from_dict(DL_A)
    assert config_from_dict(cfg.to_dict()).to_dict() == cfg.to_dict()
    spec = cfg.model_spec()
    assert [b.kind for b in spec.blocks] == ["branch_norm"] * 5
    # readers run on their owner's cache entry and write nothing
    assert [(e.block, e.cache, e.writes_cache) for e in spec.schedule] == \
        [(0, 0, True), (1, 0, False), (2, 2, True), (3, 0, False), (4, 2, False)]
    names = expected_tensors(spec)
    assert names["embed"].shape == (300, 96) and names["bigram"].shape == (98, 96) and names["head"].shape == (300, 96)
    assert names["l0.mix.q"].shape == (128, 96) and names["l0.mix.q.b"].shape == (128,) and names["l0.mix.v"].shape == (32, 96)
    assert names["l0.mix.v.b"].shape == (32,) and names["l0.mix.o"].shape == (96, 64) and "l0.mix.o.b" not in names
    assert names["l0.mix.q.norm"].shape == (32,) and names["l0.mix.sink"].shape == (4,)
    for gone in ("k", "v", "k.b", "v.b", "k.norm"):
        assert "l1.mix." + gone not in names
    assert {"l1.mix.q.b", "l1.mix.q.norm", "l1.mix.sink"} <= set(names)
    assert names["l1.mlp.router"].shape == (8, 96) and names["l1.mlp.correction"].shape == (8,) and "l1.mlp.e6.up" not in names
    assert names["l0.mlp.gate"].shape == (112, 96) and "l2.norm2" not in names and names["l4.norm2"].shape == (96,)
    assert spec.embedding.kind == "token_pair_embedding" and spec.final_norm.get("gain_scale") == 3.0
    plain = config_from_dict(DL_B).model_spec()
    assert plain.embedding.kind == "token_embedding" and plain.final_norm.get("gain_scale") == 1.0


@pytest.mark.parametrize("change, word", [
    (lambda c: c["layers"][0].update(type="conv"), "type"),
    (lambda c: c["layers"][0]["mlp"].update(kind="wide"), "kind"),
    (lambda c: c["layers"][0]["mlp"].pop("limit"), "limit"),
    (lambda c: c["layers"][0]["mixer"].update(kv_heads=3), "kv_heads"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=34), "dims"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=7), "dims"),
    (lambda c: c["layers"][0]["mixer"]["mask"].update(size=0), "size"),
    (lambda c: c["layers"][0]["mixer"].pop("scale"), "scale"),
    (lambda c: c["layers"][3]["mixer"].update(kv_from=1), "kv_from"),
    (lambda c: c["layers"][1]["mixer"].update(kv_from=2), "kv_from"),
    (lambda c: c["layers"][1]["mixer"].update(heads=2), "heads"),
    (lambda c: c["layers"][1]["mixer"]["rot"].update(base=77.0), "rot"),
    (lambda c: c["layers"][1]["mlp"]["router"].update(top=9), "router"),
    (lambda c: c["layers"][1]["mlp"]["expert"].pop("ff"), "ff"),
    (lambda c: c["embedding"]["bigram"].pop("mul_cur"), "mul_cur"),
    (lambda c: c.pop("width"), "width"),
    (lambda c: c.pop("norm"), "eps"),
])
def test_configuration_rejections_name_the_key(change, word):
    from minfer_amd import ConfigError, config_from_dict
    raw = copy.deepcopy(DL_A)
    change(raw)
    with pytest.raises(ConfigError, match=word):
        config_from_dict(raw).model_spec()


# ------------------------------------------------------------------ the plain mechanisms by hand
def test_plain_pair_rows_and_embedding_by_hand():
    assert pd.pair_rows([4, 1, 4, 4], 10, 7, 3) == [10, (28 + 3) % 10, (7 + 12) % 10, (28 + 12) % 10]
    w = {"embed": np.arange(10.0).reshape(5, 2), "bigram": 100.0 * np.arange(22.0).reshape(11, 2)}
    got = pd.embed([4, 1], w, dict(scale=0.5, bigram=dict(buckets=10, mul_prev=7, mul_cur=3)))
    assert np.allclose(got, [[4.0 + 2000.0, 4.5 + 2100.0], [1.0 + 200.0, 1.5 + 300.0]])
    assert np.allclose(pd.embed([4], w, dict(scale=0.5)), [[4.0, 4.5]])


def test_plain_masks_and_sinks_by_hand():
    mask = dict(size=2, keep_first=1)
    assert [j for j in range(6) if pd.visible(4, j, mask)] == [0, 3, 4] and [j for j in range(6) if pd.visible(1, j, mask)] == [0, 1]
    assert [j for j in range(6) if pd.visible(3, j, None)] == [0, 1, 2, 3]
    p = pd.sink_softmax(np.log(np.array([[[1.0, 2.0, 5.0]]])), np.array([[True, True, False]]), np.log(np.array([5.0])))
    assert np.allclose(p, [[[1 / 8, 2 / 8, 0.0]]])
    # the vectorised mask of the attention is `visible`, and the sink takes its share: equal keys, values by position
    T = 5
    w = {"q": np.zeros((1, 1)), "q.b": np.ones(1), "q.norm": np.ones(1), "k": np.zeros((1, 1)), "k.b": np.ones(1), "k.norm": np.ones(1),
         "v": np.ones((1, 1)), "v.b": np.full(1, 0.5), "o": np.ones((1, 1)), "sink": np.array([1.0 + math.log(3.0)])}
    m = dict(heads=1, kv_heads=1, dim=1, vdim=1, scale=1.0, mask=mask)
    h = np.arange(T, dtype=np.float64)[:, None]
    out = pd.attention(h, pd.keys_and_values(h, w, "", m, 0.0), w, "", m, 0.0)
    for i in range(T):
        seen = [j for j in range(T) if pd.visible(i, j, mask)]
        assert np.isclose(out[i, 0], sum(j + 0.5 for j in seen) / (len(seen) + 3.0)), i


def test_plain_query_and_key_norms_come_before_the_rotation_with_their_gains():
    """Gains do not commute with a rotation: worked by hand for one head of four values at position 2."""
    w = {"k": np.eye(4), "k.b": np.array([0.0, 0.0, 0.0, 1.0]), "v": np.eye(4), "v.b": np.zeros(4), "k.norm": np.array([1.0, 2.0, 3.0, 4.0])}
    m = dict(kv_heads=1, dim=4, vdim=4, rot=dict(base=100.0, dims=2))
    h = np.zeros((3, 4))
    h[2] = [3.0, 1.0, 2.0, 1.0]
    k, v = pd.keys_and_values(h, w, "", m, 0.0)
    n = np.array([3.0, 1.0, 2.0, 2.0]) / math.sqrt(18.0 / 4.0) * [1.0, 2.0, 3.0, 4.0]
    want = [n[0] * math.cos(2) - n[1] * math.sin(2), n[1] * math.cos(2) + n[0] * math.sin(2), n[2], n[3]]
    assert np.allclose(k[2, 0], want) and np.allclose(v[2, 0], h[2])
    # four rotated values: the first turns with the third by p, the second with the fourth by p base^(-1/2)
    k4, _ = pd.keys_and_values(h, w, "", dict(m, rot=dict(base=100.0, dims=4)), 0.0)
    assert np.allclose(k4[2, 0], [n[0] * math.cos(2) - n[2] * math.sin(2), n[1] * math.cos(.2) - n[3] * math.sin(.2),
                                  n[2] * math.cos(2) + n[0] * math.sin(2), n[3] * math.cos(.2) + n[1] * math.sin(.2)])


def test_plain_feed_forwards_by_hand():
    h = np.array([[1.0, 2.0]])
    w = {"gate": np.array([[2.0, 0.0], [0.0, -1.0]]), "up": np.array([[1.0, 1.0], [-2.0, 0.0]]), "down": np.eye(2)}
    # gate sums 2 and -2 (clamped from above only), up sums 3 and -2 (clamped on both sides)
    assert np.allclose(pd.clamped_ff(h, w, "", 1.5), [[1.5 / (1 + math.exp(-1.702 * 1.5)) * 2.5, -2 / (1 + math.exp(1.702 * 2)) * -0.5]])
    # two experts and one that hands its input on: scores 1/8, 2/8, 5/8; the correction puts the first ahead of the second
    w = {"router": np.log(np.array([[1.0, 1.0], [2.0, 1.0], [5.0, 1.0]])), "correction": np.array([0.2, 0.0, 0.0]),
         "e0.gate": np.array([[1.0, 0.0]]), "e0.up": np.array([[0.0, 2.0]]), "e0.down": np.array([[1.0], [3.0]]),
         "e1.gate": np.zeros((1, 2)), "e1.up": np.zeros((1, 2)), "e1.down": np.zeros((2, 1))}
    chosen, weights, margins = pd.route(h, w, "", 2)
    assert list(chosen[0]) == [2, 0] and np.allclose(weights[0], [5 / 8, 1 / 8]) and np.isclose(margins[0], 1 / 8 + 0.2 - 2 / 8)
    y = 4.0 / (1 + math.exp(-1.0))
    assert np.allclose(pd.mixture(h, w, "", 2, 2), [[5 / 8 * 1 + y / 8, 5 / 8 * 2 + 3 * y / 8]])


# ------------------------------------------------------------------ the cache
def test_a_shared_entry_keeps_what_any_reader_sees():
    from minfer_amd import config_from_dict
    from minfer_amd.cache.paged import Cache, CacheError, KVRequest, StateRequest, widest_request
    from minfer_amd.engine.model import DecoderModel
    from minfer_amd.parts.base import EMBEDDING_ENTRY
    r = lambda **k: KVRequest(2, 32, v_head_dim=16, **k)
    assert widest_request(r(window=70, keep_first=3), r(window=130, keep_first=5)) == r(window=130, keep_first=5)
    assert widest_request(r(window=130), r(window=70, keep_first=9)) == r(window=130, keep_first=9)
    assert widest_request(r(window=70, keep_first=3), r()) == r() and widest_request(r(), r(window=5)) == r()
    assert widest_request(r(chunk=64), r(chunk=64)) == r(chunk=64)
    assert widest_request(r(chunk=64), r(window=5)) == r() and widest_request(r(chunk=64), r(chunk=128)) == r()
    with pytest.raises(CacheError, match="read as"):
        widest_request(r(), KVRequest(2, 32))
    got = DecoderModel(config_from_dict(DL_A).model_spec(), torch.float32, "cpu").cache_requests()
    assert got == {0: r(window=130, keep_first=5), 2: KVRequest(3, 16, v_head_dim=48), EMBEDDING_ENTRY: StateRequest((1,), torch.int32)}
    # a window of 70 would have given page 1 back at length 198; the reader's 130 holds it until position 257
    cache = Cache(got, max_tokens=64 * 12, max_seqs=2, dtype=torch.float32, device="cpu")
    s = cache.alloc_slot()
    for length, gone in ((198, []), (256, []), (257, [1]), (321, [1, 2])):
        cache.reserve({s: length})
        cache.commit({s: length})
        assert [i for i, p in enumerate(cache.group_of[0].pages[s]) if p < 0] == gone, length
        cache.check_invariants()
    cache.free_slot(s)


def test_an_embedding_with_state_does_not_go_with_a_run_order_that_takes_it_in_again():
    from minfer_amd import config_from_dict
    from minfer_amd.engine.model import DecoderModel
    from minfer_amd.parts.spec import ModelSpec
    import dataclasses
    spec = config_from_dict(DL_A).model_spec()
    again = tuple(dataclasses.replace(e, adds_embedding=(n == 2)) for n, e in enumerate(spec.schedule))
    assert isinstance(spec, ModelSpec)
    with pytest.raises(ValueError, match="state"):
        DecoderModel(dataclasses.replace(spec, schedule=again), torch.float32, "cpu")


# ------------------------------------------------------------------ the engine on the stand-ins
def _rel(rows, ref):
    return max(float(np.abs(got - ref[rid][p]).max() / max(1e-9, ref[rid][p].std())) for (rid, p), got in rows.items())


@pytest.mark.parametrize("name", list(DL))
def test_engine_on_stand_ins_agrees_with_plain(tmp_path, monkeypatch, name):
    plain_ops.install(monkeypatch)
    from minfer_amd import Engine, load_model
    folder = write_dolutar(str(tmp_path / name), DL[name], seed=5)
    plain = pd.PlainDolutar(folder)
    reqs = requests_for(DL[name]["vocab"], (1, 7, 70, 33, 140), seed=2)
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
    raw = random_config(np.random.default_rng(12))
    folder = write_dolutar(str(tmp_path / "r"), raw, seed=6)
    plain = pd.PlainDolutar(folder)
    reqs = requests_for(raw["vocab"], (3, 40, 90), seed=4)
    ref = {rid: plain.forward(toks) for rid, toks in reqs.items()}
    eng = Engine(load_model(folder, dtype="float32", device="cpu"), max_tokens=64 * 8)
    assert _rel(run_steps(eng, chunk_steps(reqs, [list(reqs)], sizes=(2, 31, 1))), ref) < 1e-4, json.dumps(raw)


@pytest.mark.parametrize("name", ["B", "A"])
def test_greedy_generation_on_stand_ins(tmp_path, monkeypatch, name):
    """`generate` with its scheduler, slots and decode sessions, tokens against the plain model."""
    plain_ops.install(monkeypatch)
    from minfer_amd import Engine, generate, load_model
    from minfer_amd.sampling import SamplingParams
    folder = write_dolutar(str(tmp_path / "gen"), DL[name], seed=8)
    plain = pd.PlainDolutar(folder)
    eng = Engine(load_model(folder, dtype="float32", device="cpu"), max_tokens=64 * 6, max_seqs=2)
    prompts = [[5, 9, 20, 7], [11], [25, 3, 3, 3, 8, 1, 44]]
    res = generate(eng, prompts, SamplingParams(temp=0.0, repeat_penalty=1.0), max_new=5, stop_tokens=[])
    for p, toks in zip(prompts, res.tokens):
        seq = list(p)
        for t in toks:
            assert t == pd.greedy(plain.forward(seq)[-1])
            seq.append(t)
    assert not eng.cache.live_slots()


def test_a_sequence_with_pair_rows_is_not_rolled_back(tmp_path, monkeypatch):
    plain_ops.install(monkeypatch)
    from minfer_amd import Engine, load_model
    from minfer_amd.engine.engine import StepError
    eng = Engine(load_model(write_dolutar(str(tmp_path / "t"), DL_A, seed=1), dtype="float32", device="cpu"), max_tokens=256)
    s = eng.new_sequence()
    eng.step([s], [[1, 2, 3, 4]], "last")
    with pytest.raises(StepError, match="state"):
        eng.truncate(s, 2)
