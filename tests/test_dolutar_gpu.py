"""Dolutar on the GPU: each new or extended kernel alone against the plain stand-ins (sinks, clamped gates in every
form of the fused product, experts that hand their input on, pair rows), keys just inside and outside a window and among
and behind the kept first positions, the engine against the plain implementation under every way of cutting requests
into steps, long decoding through the captured step, and the programs."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import plain_dolutar as pd
import plain_ops
from dolutar_tiny import DL, DL_B, attention, dense, moe, random_config, write_dolutar
from paged_cases import DEV, attention_case, pages, rnd, run_logged, step_context
from replays import batch_steps, chunk_steps, requests_for, tail_steps, whole_steps
from tiny import random_tokens

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))

# bfloat16 logits against the 64-bit plain implementation, as fractions of the logits' standard deviation, at three
# layers and growing with the root of their number beyond; 32-bit in absolute terms (times the logits' standard
# deviation where that is above one)
BF16_RMS, BF16_MAX, F32_ABS = 0.04, 0.2, 2e-4
SHARP = 3.0
# a bfloat16 run is compared with the plain implementation taking the run's own choices of experts, which must be the
# plain router's wherever its margin is at least this
CLOSE_CALL = 0.02


def check(engine, steps, plain, reqs, dtype, what, loosen=1.0, f32_abs=F32_ABS):
    routed = plain.routed_layers()
    loosen = loosen * max(1.0, len(plain.c["layers"]) / 3.0) ** 0.5
    rows, routes = run_logged(engine, steps, routed)
    assert rows, "nothing was produced"
    for rid, toks in reqs.items():
        if not any(k[0] == rid for k in rows):
            continue
        forced = None
        if dtype != "float32" and routed:
            forced = {l: np.stack([routes[rid][l][p] for p in range(len(toks))]) for l in routed}
        seen = []
        want_all = plain.forward(toks, forced, seen)
        for l, (choice, margin) in zip(routed, seen):
            for p in range(len(toks)):
                if (rid, p) in rows and margin[p] >= (1e-5 if dtype == "float32" else CLOSE_CALL):
                    assert sorted(routes[rid][l][p].tolist()) == sorted(choice[p].tolist()), \
                        f"{what} [{dtype}]: request {rid} position {p} layer {l}: experts {routes[rid][l][p]} for {choice[p]} (margin {margin[p]:.4f})"
        for p in range(len(toks)):
            if (rid, p) not in rows:
                continue
            got, want = rows[(rid, p)], want_all[p]
            assert np.isfinite(got).all(), f"{what}: non-finite logits at request {rid} position {p}"
            diff, std = got.astype(np.float64) - want, float(want.std())
            if dtype == "float32":
                assert np.abs(diff).max() <= f32_abs * max(1.0, std), \
                    f"{what} [float32]: request {rid} position {p} of {len(toks)}: {np.abs(diff).max():.3e}"
            else:
                rms = float(np.sqrt(np.mean(diff * diff)))
                assert rms <= loosen * BF16_RMS * std and np.abs(diff).max() <= loosen * BF16_MAX * std, \
                    f"{what} [bfloat16]: request {rid} position {p} of {len(toks)}: rms {rms / std:.3f}, max {np.abs(diff).max() / std:.3f}"


# ------------------------------------------------------------------ sinks in the attention kernels
def _attend(form, q, kc, vc, table, pos, seq, lens, new, H, G, D, V, scale, window, keep_first, sink):
    """One launch of the attention in one of its forms; the result on the host."""
    from minfer_amd.kernels import ops
    if form == "stand-in":
        out = torch.empty(sum(new), H * V, dtype=q.dtype)
        plain_ops.capped_attn(q, kc, vc, table, pos, seq, torch.ones(H), out, H, G, D, V, scale, 0.0, window, max(lens),
                              keep_first=keep_first, sink=sink)
        return out.float()
    out = torch.empty(sum(new), H * V, dtype=q.dtype, device=DEV)
    ones = torch.ones(H, device=DEV)
    s = None if sink is None else sink.to(DEV)
    if form == "matrix cores":
        ops.capped_attn_prefill(q.to(DEV), kc.to(DEV), vc.to(DEV), table.to(DEV), step_context(lens, new, table, pos, seq), ones,
                                out, H, G, D, V, scale, 0.0, window, keep_first=keep_first, sink=s)
    else:
        ops.capped_attn(q.to(DEV), kc.to(DEV), vc.to(DEV), table.to(DEV), pos.to(DEV), seq.to(DEV), ones, out, H, G, D, V, scale,
                        0.0, window, max(lens), keep_first=keep_first, sink=s)
    return out.float().cpu()


_WANT = {}


@pytest.mark.parametrize("form, dtype", [("plain", torch.float32), ("plain", torch.bfloat16), ("matrix cores", torch.bfloat16)])
@pytest.mark.parametrize("H, G, D, V, window, keep", [
    (6, 3, 32, 48, 17, 3), (8, 2, 96, 48, 0, 0), (4, 4, 16, 16, 64, 64), (8, 2, 128, 64, 70, 5), (9, 1, 10, 6, 5, 2),
    (2, 1, 64, 128, 33, 32), (3, 3, 20, 12, 40, 130), (16, 4, 64, 64, 128, 0)])
@pytest.mark.parametrize("new", [(1, 130, 3, 1, 40), (1, 64, 64, 300, 65), (1, 1, 1, 1, 1)])
def test_sinks_in_both_attention_kernels(form, dtype, H, G, D, V, window, keep, new):
    """Prompts, portions on held tokens and single tokens (keys split over workgroups), over shuffled pages of a
    poisoned pool; sinks from far below every score to far above."""
    if form == "matrix cores" and (D % 16 or V % 16):
        pytest.skip("sizes the plain kernel takes")
    lens = (1, 130, 64, 300, 65)
    q, kc, vc, table, pos, seq, _ = attention_case(dtype, H, G, D, V, lens, new, 0, 0.0, 3)
    sink = rnd(H, seed=9, scale=2.0)
    sink[0], sink[-1] = 30.0, -40.0
    case = (dtype, H, G, D, V, window, keep, new)
    if case not in _WANT:            # the stand-in walks every (token, head, key) on the host: once per case
        _WANT[case] = _attend("stand-in", q, kc, vc, table, pos, seq, lens, new, H, G, D, V, 0.2, window, keep, sink)
    want = _WANT[case]
    got = _attend(form, q, kc, vc, table, pos, seq, lens, new, H, G, D, V, 0.2, window, keep, sink)
    err = (got - want).abs().max()
    assert torch.isfinite(got).all() and err < (2e-5 if dtype == torch.float32 else 4e-2), float(err)
    # a head whose sink outweighs everything gives next to nothing, relative to which it is right all the same
    big = got.view(-1, H, V)[:, 0], want.view(-1, H, V)[:, 0]
    assert big[1].abs().max() < 1e-5 and (big[0] - big[1]).abs().max() < 0.03 * big[1].abs().max()


@pytest.mark.parametrize("form", ["plain float32", "plain bfloat16", "matrix cores"])
def test_a_sink_by_hand(form):
    """Equal keys (scores of 4) and values of one: n keys in sight weigh n e^4 against a sink of e^s, so the result is
    n e^4 / (n e^4 + e^s), for a prompt's tokens, for single tokens with their keys split, with and without a window, and
    the sink counts once whatever the number of splits."""
    H, G, D, V = 4, 2, 16, 16
    dtype = torch.float32 if form == "plain float32" else torch.bfloat16
    n = 1500
    lens = (n, 70)
    table = pages(lens, 4)
    from minfer_amd.cache.paged import v_page_shape
    kc, vc = torch.full((40, G, 64, D), 1.0, dtype=dtype), torch.full((40,) + v_page_shape(G, V, dtype), 1.0, dtype=dtype)
    sink = torch.tensor([4.0, 4.0 + float(np.log(n)), 9.0, -50.0])
    for new in ((1, 1), (40, 70)):
        pos = torch.cat([torch.arange(l - m, l) for l, m in zip(lens, new)]).to(torch.int32)
        seq = torch.repeat_interleave(torch.arange(2, dtype=torch.int32), torch.tensor(new)).to(torch.int32)
        q = torch.full((sum(new), H * D), 0.25, dtype=dtype)
        for window, keep in ((0, 0), (100, 0), (100, 30)):
            got = _attend("plain" if form.startswith("plain") else form, q, kc, vc, table, pos, seq, lens, new, H, G, D, V, 1.0,
                          window, keep, sink).view(-1, H, V)
            for t in range(sum(new)):
                p = int(pos[t])
                seen = sum(pd.visible(p, j, dict(size=window, keep_first=keep) if window else None) for j in range(p + 1))
                for h in range(H):
                    want = seen / (seen + float(np.exp(float(sink[h]) - 4.0)))
                    assert abs(float(got[t, h, 3]) - want) < (1e-5 if dtype == torch.float32 else 6e-3), (t, h, window, keep)


# the last query stands at position 299: (window, kept first positions, the key's position, seen or not)
EDGES = [(17, 0, 283, True), (17, 0, 282, False), (64, 4, 236, True), (64, 4, 235, False), (64, 4, 3, True), (64, 4, 4, False),
         (100, 64, 63, True), (100, 64, 64, False), (100, 70, 69, True), (100, 70, 70, False), (1, 2, 299, True), (1, 2, 298, False),
         (300, 0, 0, True), (299, 0, 0, False), (0, 0, 0, True)]


@pytest.mark.parametrize("form", ["plain float32", "plain bfloat16", "matrix cores"])
@pytest.mark.parametrize("window, keep, key, inside", EDGES)
def test_a_key_at_an_edge_decides_beside_a_sink_or_is_not_seen(form, window, keep, key, inside):
    """A key made to win the softmax (also over the sink) with a value row of 50s, at the end of a prompt, of a portion
    and for a single token; one position further it leaves no trace."""
    H, G, D, V = 4, 2, 16, 16
    dtype = torch.float32 if form == "plain float32" else torch.bfloat16
    sink = torch.tensor([3.0, -1.0, 2.0, 5.0])
    for lens, new in (((300, 90), (300, 20)), ((300, 90), (45, 1)), ((300, 90), (1, 1))):
        q, kc, vc, table, pos, seq, _ = attention_case(dtype, H, G, D, V, lens, new, 0, 0.0, 5, needle=(0, key, 1))
        got = _attend("plain" if form.startswith("plain") else form, q, kc, vc, table, pos, seq, lens, new, H, G, D, V, 1.0,
                      window, keep, sink)
        row = got[new[0] - 1].view(H, V)
        if inside:
            assert (row[2:] - 50.0).abs().max() < 0.5, (lens, new)
        else:
            assert row[2:].abs().max() < 10.0, (lens, new)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H, G, D, V, rot, q_only", [(6, 3, 24, 40, 16, False), (9, 1, 10, 6, 4, False), (4, 4, 16, 16, 16, True), (6, 2, 128, 64, 32, False)])
def test_query_and_key_gains_before_a_rotation_in_halves(dtype, H, G, D, V, rot, q_only):
    from minfer_amd.cache.paged import v_page_shape
    from minfer_amd.kernels import ops
    held, new = (0, 3, 60, 127), (1, 2, 70, 5)
    n, C = sum(new), H * D + (0 if q_only else G * (D + V))
    qkv = rnd(n, C, seed=1, scale=2.0)
    gains = rnd(D, seed=2) + 1.0, None if q_only else rnd(D, seed=3) + 1.0
    seq = torch.repeat_interleave(torch.arange(4, dtype=torch.int32), torch.tensor(new)).to(torch.int32)
    pos = torch.cat([torch.arange(h, h + m) for h, m in zip(held, new)]).to(torch.int32)
    table = pages([h + m for h, m in zip(held, new)], 7)
    ang = torch.arange(256, dtype=torch.float64)[:, None] * (100.0 ** (-2.0 * torch.arange(rot // 2) / rot))
    rt = (torch.cos(ang).float(), torch.sin(ang).float())
    outs = []
    for side in ("plain", "gpu"):
        dev = "cpu" if side == "plain" else DEV
        mv = lambda t: None if t is None else (tuple(x.to(dev) for x in t) if isinstance(t, tuple) else t.to(dev))
        kc = torch.full((40, G, 64, D), 7.0, dtype=dtype, device=dev)
        vc = torch.full((40,) + v_page_shape(G, V, dtype), 7.0, dtype=dtype, device=dev)
        q = torch.empty(n, H * D, dtype=dtype, device=dev)
        (plain_ops if side == "plain" else ops).qk_norm_prep(
            mv(qkv), mv(gains[0]), mv(gains[1]), 1e-5, True, mv(seq), mv(pos), mv(rt), None, False, mv(table), q, kc, vc, H, G, D, V,
            not q_only, halves=True, q_only=q_only)
        outs.append([t.cpu().float() for t in (q, kc, vc)])
    tol = 3e-5 if dtype == torch.float32 else 1e-2
    for name, a, b in zip(("q", "k pages", "v pages"), *outs):
        assert ((a - b).abs() / b.abs().clamp(min=1.0)).max() < tol, name
    if not q_only:                   # position 2 of the third sequence's first page, worked from the equations
        t = 1 + 2 + (61 - 60)        # its token at position 61
        k = qkv[t, H * D:H * D + D].double().numpy()[None, None]
        want = pd.rotate_halves(pd.rms_norm(k, gains[1].double().numpy(), 1e-5), [61], 100.0, rot)[0, 0]
        got = outs[1][1][int(table[2, 0]), 0, 61].numpy()
        assert np.abs(got - want).max() < (1e-4 if dtype == torch.float32 else 2e-2)


# ------------------------------------------------------------------ clamped gates
GATED_SHAPES = {
    (1, 96, 60): "skinny16_kernel", (3, 37, 896): "skinny16_kernel", (16, 300, 2048): "skinny16_kernel",
    (5, 2048, 896): "stationary16_kernel", (8, 3000, 1024): "stationary16_kernel", (16, 64, 8192): "skinny_ring_kernel",
    (17, 112, 96): "skinny_kernel", (40, 100, 1024): "skinny_ring_kernel", (33, 16416, 512): "panel_kernel",
    (64, 33, 77): "skinny_kernel", (65, 112, 96): "tile_kernel<128,128>", (300, 37, 60): "tile_kernel<128,128>",
    (256, 192, 4096): "tile_kernel<128,128>(split K)", (513, 1024, 512): "tile_dma_kernel<128>",
    (1501, 8170, 128): "tile_dma_kernel<256>", (1000, 8192, 100): "tile_kernel<256,256>"}


@pytest.mark.parametrize("m, nf, k", list(GATED_SHAPES))
def test_clamped_gates_in_every_form_of_the_fused_product(m, nf, k):
    """Sums on both sides of the limit; the last row and column of sizes that fill no tile; with the tiled copy of the
    matrix where there is one; the same rows twice give the same bits."""
    from minfer_amd.kernels import ops
    if ops.cu_count() == 256:
        assert ops.plan_linear(m, (nf + 31) // 32 * 64, k, swiglu=True, aligned=k % 8 == 0)["kernel"] == GATED_SHAPES[(m, nf, k)]
    x = rnd(m, k, seed=1).to(torch.bfloat16)
    wg, wu = ((rnd(nf, k, seed=s) * 2.0 / k ** 0.5).to(torch.bfloat16) for s in (2, 3))
    for limit in (0.7, 3.0):
        want = torch.empty(m, nf, dtype=torch.bfloat16)
        plain_ops.swiglu(torch.cat([x.float() @ wg.float().t(), x.float() @ wu.float().t()], dim=1), want, limit)
        lim = torch.tensor([limit], device=DEV)
        w = ops.interleave_gate_up(wg.to(DEV), wu.to(DEV))
        got, again = (torch.full((m, nf), float("nan"), dtype=torch.bfloat16, device=DEV) for _ in range(2))
        ops.linear_swiglu(x.to(DEV), w, got, limit=lim)
        ops.linear_swiglu(x.to(DEV), w, again, limit=lim)
        assert torch.equal(got, again)
        err = (got.cpu().float() - want.float()).abs() / want.float().abs().clamp(min=0.5)
        assert float(err.max()) < 0.02, (limit, float(err.max()))
        if k % 32 == 0 and m <= 64:
            tiled = torch.full((m, nf), float("nan"), dtype=torch.bfloat16, device=DEV)
            ops.linear_swiglu(x.to(DEV), w, tiled, tiled=ops.tile_weight(w), limit=lim)
            assert (tiled.float() - got.float()).abs().max() < 0.05
    rows = rnd(min(m, 40), 2 * nf, seed=5, scale=2.0)
    for dt in (torch.float32, torch.bfloat16):
        want, got = (torch.empty(rows.shape[0], nf, dtype=dt, device=d) for d in ("cpu", DEV))
        plain_ops.swiglu(rows, want, 1.1)
        ops.swiglu(rows.to(DEV), got, 1.1)
        assert (got.cpu().float() - want.float()).abs().max() < (1e-5 if dt == torch.float32 else 2e-2)


def test_clamped_gates_without_the_limit_are_silu_as_before():
    from minfer_amd.kernels import ops
    for m in (8, 40, 300):
        x, wg, wu = rnd(m, 1024, seed=1).to(torch.bfloat16), rnd(64, 1024, seed=2).to(torch.bfloat16) / 16, rnd(64, 1024, seed=3).to(torch.bfloat16) / 16
        want, got = torch.empty(m, 64, dtype=torch.bfloat16), torch.empty(m, 64, dtype=torch.bfloat16, device=DEV)
        plain_ops.swiglu(torch.cat([x.double() @ wg.double().t(), x.double() @ wu.double().t()], dim=1), want)
        ops.linear_swiglu(x.to(DEV), ops.interleave_gate_up(wg.to(DEV), wu.to(DEV)), got)
        assert ((got.cpu().float() - want.float()).abs() / want.float().abs().clamp(min=0.5)).max() < 0.02


# ------------------------------------------------------------------ routers and experts that hand their input on
def test_softmax_router_with_corrections_and_weights_as_they_are():
    from minfer_amd.kernels import ops
    for E, top, n, K in ((3, 1, 5, 70), (8, 2, 40, 96), (14, 3, 300, 64), (5, 5, 9, 33), (70, 8, 21, 128), (2, 1, 257, 60)):
        corr = rnd(E, seed=E + 2, scale=0.2)
        for xt in (torch.float32, torch.bfloat16):
            x, w = rnd(n, K, seed=E).to(xt), rnd(E, K, seed=E + 1, scale=0.3)
            for norm in (False, True):
                want = [torch.empty(n, E), torch.empty(n, top, dtype=torch.int32), torch.empty(n, top)]
                got = [t.clone().to(DEV) for t in want]
                plain_ops.moe_route(x, w, *want, 1, 1, correction=corr, normalize=norm)
                ops.moe_route(x.to(DEV), w.to(DEV), *got, 1, 1, correction=corr.to(DEV), normalize=norm)
                assert torch.equal(got[1].cpu(), want[1])
                assert (got[2].cpu() - want[2]).abs().max() < 1e-5 and (got[0].cpu() - want[0]).abs().max() < 1e-5
            order, weight, _ = pd.route(x.double().numpy(), {"router": w.double().numpy(), "correction": corr.double().numpy()}, "", top)
            ops.moe_route(x.to(DEV), w.to(DEV), *got, 1, 1, correction=corr.to(DEV), normalize=False)
            assert np.array_equal(got[1].cpu().numpy(), order) and np.abs(got[2].cpu().numpy() - weight).max() < 1e-5


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("experts, identity, top, hidden, ff", [(4, 2, 2, 128, 64), (1, 3, 2, 60, 33), (6, 1, 3, 64, 40), (2, 6, 4, 128, 64), (5, 0, 2, 96, 64)])
def test_the_mixture_alone_in_both_forms(dtype, experts, identity, top, hidden, ff):
    """Few tokens, slices of few tokens, and tokens grouped by expert, with the corrections as they come, set so that
    every token takes only experts that hand their input on, and so that none does; added to rows and stored over them."""
    from minfer_amd.parts import FEED_FORWARDS, PartSpec, Runtime, make_part
    dt = getattr(torch, dtype)
    part = make_part(FEED_FORWARDS, PartSpec("grouped_moe", dict(
        hidden_size=hidden, intermediate_size=ff, n_experts=experts, identity=identity, top=top, act="silu", normalize=False,
        correction="correction", router="router", expert="e{}")), Runtime(dt, DEV), "ffn")
    w = {n: (rnd(*s.shape, seed=i + 1) / (s.shape[-1] ** 0.5 if len(s.shape) == 2 else 10.0)).to(torch.bfloat16)
         for i, (n, s) in enumerate(part.tensor_specs().items())}
    assert w["router"].shape == (experts + identity, hidden)
    for how in ("as they come", "handed on", "never handed on"):
        if how != "as they come":
            if (identity if how == "handed on" else experts) < top:
                continue
            favoured = torch.arange(experts + identity) >= experts
            w["correction"] = torch.where(favoured == (how == "handed on"), 5.0, 0.0).to(torch.bfloat16)
        part.load(lambda n: w[n].to(device=DEV, dtype=dt if "router" not in n else torch.bfloat16))
        wd = {n: t.double().numpy() for n, t in w.items()}
        for n in (1, 16, 17, 130):
            x = rnd(n, hidden, seed=n).to(dt)
            log = []
            ctx = type("Ctx", (), {"_memo": {"route_log": log}, "all_decode": False})()
            for accumulate in (True, False):
                h = rnd(n, hidden, seed=99)
                got = h.to(DEV)
                part.forward(x.to(DEV), got, ctx, accumulate=accumulate)
                chosen = log[-1].cpu().numpy()
                if how == "handed on":
                    assert (chosen >= experts).all()
                want = pd.mixture(x.double().numpy(), wd, "", experts, top, forced=chosen) + (h.double().numpy() if accumulate else 0.0)
                assert np.abs(got.cpu().double().numpy() - want).max() < (1e-5 if dtype == "float32" else 1e-2), (how, n, accumulate)


# ------------------------------------------------------------------ pair rows
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_pair_rows_and_their_state(dtype):
    """Sequences in shuffled slots bring a prompt, portions and single tokens; whatever an earlier sequence left in a
    slot plays no part in a first token; factors whose products pass 32 bits; one bucket; an id outside the table shows."""
    from minfer_amd.kernels import ops
    vocab, d = 50000, 70
    for buckets, mp, mc in ((997, 31, 7), (1, 3, 5), (1009, 2147483, 1999993), (64, 0, 1), (40, -7, 3)):
        table, pairs = rnd(vocab, d, seed=1).to(dtype), rnd(buckets + 1, d, seed=2).to(dtype)
        toks = [random_tokens(vocab, n, 3 + n) for n in (1, 9, 200, 3)]
        slots = [5, 0, 3, 6]
        last = torch.full((8, 1), 12345, dtype=torch.int32, device=DEV)
        at = [0] * 4
        got = [[] for _ in toks]
        for cuts in ((1, 5, 150, 2), (None, 1, 2, 1), (None, 3, 1, None), (None, None, 47, None)):
            live = [b for b, c in enumerate(cuts) if c]
            new = [cuts[b] for b in live]
            i32 = lambda v: torch.tensor(v, dtype=torch.int32, device=DEV)
            ids = i32([t for b in live for t in toks[b][at[b]:at[b] + cuts[b]]])
            pos = i32([p for b in live for p in range(at[b], at[b] + cuts[b])])
            out = torch.empty(sum(new), d, device=DEV)
            ops.embed_pairs(table.to(DEV), pairs.to(DEV), ids, pos, i32([i for i, n in enumerate(new) for _ in range(n)]),
                            i32([0] + np.cumsum(new).tolist()), i32([slots[b] for b in live]), last, mp, mc, out, 1.5)
            r = 0
            for b in live:
                got[b] += out[r:r + cuts[b]].cpu().double().numpy().tolist()
                r += cuts[b]
                at[b] += cuts[b]
        w = {"embed": table.double().numpy(), "bigram": pairs.double().numpy()}
        for b, t in enumerate(toks):
            want = pd.embed(t, w, dict(scale=1.5, bigram=dict(buckets=buckets, mul_prev=mp, mul_cur=mc)))
            assert np.abs(np.array(got[b]) - want).max() < 1e-5, (buckets, mp, mc, b)
            assert int(last[slots[b], 0]) == t[-1]
        assert int(last[1, 0]) == 12345
    out = torch.empty(1, d, device=DEV)
    ops.embed_pairs(table.to(DEV), pairs.to(DEV), i32([vocab]), i32([0]), i32([0]), i32([0, 1]), i32([0]), last, 1, 1, out)
    assert bool(torch.isnan(out).all())


# ------------------------------------------------------------------ the engine
@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    tmp = tmp_path_factory.mktemp("dolutar")
    return {name: write_dolutar(str(tmp / name), raw, seed=i) for i, (name, raw) in enumerate(DL.items())}


@pytest.fixture(scope="module")
def plains(folders):
    return {name: pd.PlainDolutar(f) for name, f in folders.items()}


def engine_for(folder, dtype, max_tokens=64 * 16, **kw):
    from minfer_amd import Engine, load_model
    return Engine(load_model(folder, dtype=dtype, device="cuda:0"), max_tokens=max_tokens, poison_cache=True, **kw)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(DL))
def test_replays_agree_with_plain(folders, plains, name, dtype):
    """Whole; the last tokens one by one (the windows' edges pass over decoded tokens); unequal batches one after
    another (slots and pages used again over a poisoned pool); prompts in portions down to two tokens and one, alone
    and in mixed batches."""
    reqs = requests_for(DL[name]["vocab"], (1, 7, 64, 150, 65, 33, 290), seed=3)
    ids = list(reqs)
    eng = engine_for(folders[name], dtype)
    plain = plains[name]
    check(eng, whole_steps(reqs), plain, reqs, dtype, f"{name} whole")
    check(eng, tail_steps(reqs, tail=80), plain, reqs, dtype, f"{name} last 80 one by one")
    check(eng, batch_steps(reqs, [ids[:4], ids[4:]]), plain, reqs, dtype, f"{name} unequal batches")
    check(eng, chunk_steps(reqs, [ids[:3], ids[3:]]), plain, reqs, dtype, f"{name} portions in batches")
    check(eng, chunk_steps(reqs, [[r] for r in ids], sizes=(2,)), plain, reqs, dtype, f"{name} portions of 2")
    check(eng, chunk_steps(reqs, [[r] for r in ids], sizes=(129, 3, 64)), plain, reqs, dtype, f"{name} portions of 129")
    assert not eng.cache.live_slots()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_batch_of_more_sequences_than_one_launch_of_the_experts_takes(folders, plains, dtype):
    """Twenty sequences that start and decode together: the routed layers' few-token form runs in slices."""
    reqs = requests_for(DL["A"]["vocab"], tuple(3 + (7 * i) % 11 for i in range(20)), seed=12)
    eng = engine_for(folders["A"], dtype, max_tokens=64 * 24)
    check(eng, batch_steps(reqs, [list(reqs)], prompt_frac=0.4), plains["A"], reqs, dtype, "twenty together")
    assert not eng.cache.live_slots()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_steps_in_which_nothing_or_little_is_wanted(folders, plains, dtype):
    """A prompt step that asks for no logits at all, then single tokens of which one sequence's are wanted."""
    eng = engine_for(folders["A"], dtype)
    toks = random_tokens(300, 100, 5)
    a, b = eng.new_sequence(), eng.new_sequence()
    assert tuple(eng.step([a, b], [toks[:90], toks[:50]], [[], []]).shape) == (0, 300)
    got_a = eng.step([a, b], [toks[90:91], toks[50:51]], [[0], []]).cpu().numpy()
    got_b = eng.step([a, b], [toks[91:92], toks[51:52]], [[], [0]]).cpu().numpy()
    for got, n in ((got_a, 91), (got_b, 52)):
        want = plains["A"].forward(toks[:n])[-1]
        tol = F32_ABS * max(1.0, want.std()) if dtype == "float32" else SHARP * BF16_MAX * want.std()
        assert got.shape == (1, 300) and np.abs(got[0] - want).max() <= tol
    eng.end_sequence(a)
    eng.end_sequence(b)


@pytest.mark.parametrize("seed", range(8))
def test_configurations_drawn_at_random(tmp_path, seed):
    """Whatever config.json may say: sizes, orders and options drawn at random, both run types, whole, one by one,
    in batches and in portions."""
    raw = random_config(np.random.default_rng(7000 + seed))
    folder = write_dolutar(str(tmp_path / "m"), raw, seed=seed)
    plain = pd.PlainDolutar(folder)
    reqs = requests_for(raw["vocab"], (1, 9, 70, 200, 131), seed=seed)
    ids = list(reqs)
    for dtype in ("float32", "bfloat16"):
        eng = engine_for(folder, dtype)
        what = f"random configuration {seed} ({json.dumps(raw)[:600]})"
        check(eng, whole_steps(reqs), plain, reqs, dtype, what + " whole", SHARP)
        check(eng, tail_steps(reqs, tail=33), plain, reqs, dtype, what + " one by one", SHARP)
        check(eng, batch_steps(reqs, [ids[:3], ids[3:]]), plain, reqs, dtype, what + " batches", SHARP)
        check(eng, chunk_steps(reqs, [ids[:2], ids[2:]]), plain, reqs, dtype, what + " portions", SHARP)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_sharp_attention_over_windows_and_long_decoding(tmp_path, dtype):
    """Queries' gains raised so that the softmax picks single keys (a key that a window wrongly holds or drops, a kept
    position lost, a sink left out or a page given back too early then moves a row by its whole size): a prompt of 400
    tokens whole, then as 250 + 150 one by one, with windows of 17, 64 and 70 whose edges pass over decoded tokens and
    page edges, a reader of 200 positions on an owner of 40, and kept positions of 3 and 65."""
    raw = dict(architecture="Dolutar", vocab=300, width=96, norm=dict(eps=1e-5), logit_scale=1.5,
               embedding=dict(scale=1.0, bigram=dict(buckets=200, mul_prev=17, mul_cur=3)), layers=[
        dict(attention(4, 2, 32, 16, 0.2, 16, 40, 3), mlp=dense(80, 2.0)),
        dict(attention(4, 2, 32, 16, 0.2, 16, 200, 1, kv_from=0), mlp=moe(6, 2, 40, 1)),
        dict(attention(2, 1, 16, 48, 0.3, 8, 64, 65), mlp=None),
        dict(attention(4, 2, 32, 32, 0.25, 32), mlp=moe(4, 1, 56, 1)),
        dict(attention(4, 2, 32, 32, 0.2, 32, 17, 0, kv_from=3), mlp=None),
        dict(attention(2, 1, 16, 48, 0.3, 8, 70, 0, kv_from=2), mlp=None),
    ])
    folder = write_dolutar(str(tmp_path / "sharp"), raw, seed=21, sharpen=4.0 if dtype == "float32" else 2.0)
    plain = pd.PlainDolutar(folder)
    reqs = {"long": random_tokens(300, 400, 77)}
    eng = engine_for(folder, dtype, max_tokens=64 * 16)
    check(eng, whole_steps(reqs), plain, reqs, dtype, "sharp whole", 1.5, 1e-3)
    check(eng, tail_steps(reqs, tail=150), plain, reqs, dtype, "sharp 250 + 150 one by one", 1.5, 1e-3)


def test_greedy_generation_through_the_entry_point(folders, plains):
    """`LLM.generate`: the scheduler, slots used again (more prompts than slots), the captured decode step; 70 new
    tokens so that every sequence crosses a page edge and the windows' edges while decoding."""
    from minfer_amd import LLM
    llm = LLM(folders["A"], dtype="float32", n_ctx=256, n_slots=2)
    prompts = [random_tokens(300, n, 30 + i) for i, n in enumerate((5, 60, 1, 17))]
    res = llm.generate(prompts, max_new=70, temp=0.0, repeat_penalty=1.0, stop_tokens=[])
    eager = llm.generate(prompts, max_new=70, temp=0.0, repeat_penalty=1.0, stop_tokens=[], use_graph=False)
    assert res.tokens == eager.tokens
    for p, toks in zip(prompts, res.tokens):
        assert len(toks) == 70
        logits = plains["A"].forward(list(p) + toks)
        for i, t in enumerate(toks):
            row = logits[len(p) + i - 1]
            top = np.sort(row)[-2:]
            assert t == pd.greedy(row) or top[1] - top[0] < 1e-3, f"token {i}"
    bf = LLM(folders["A"], dtype="bfloat16", n_ctx=256, n_slots=4)
    a = bf.generate(prompts, max_new=20, temp=0.0, repeat_penalty=1.0, stop_tokens=[]).tokens
    b = bf.generate(prompts, max_new=20, temp=0.0, repeat_penalty=1.0, stop_tokens=[], use_graph=False).tokens
    assert a == b


def test_programs(folders, plains, tmp_path):
    """bin/minfer generates greedily from a Dolutar folder; bin/trace_run replays a batch."""
    env = dict(os.environ, PYTHONPATH=ROOT)
    r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "minfer"), folders["B"], "--prompt-tokens", "5,6,7;9",
                        "--greedy", "--repeat-penalty", "1.0", "-n", "4", "--dtype", "float32", "--n-ctx", "64",
                        "--stop-token", "100000"], capture_output=True, text=True, env=env, timeout=300)
    assert r.returncode == 0, r.stderr
    lines = [l for l in r.stdout.strip().splitlines() if l]
    assert len(lines) == 2
    for line, prompt in zip(lines, ([5, 6, 7], [9])):
        seq = list(prompt)
        for t in (int(x) for x in line.split(",")):
            assert t == pd.greedy(plains["B"].forward(seq)[-1])
            seq.append(t)
    vocab = DL_B["vocab"]
    reqs = requests_for(vocab, (3, 70, 20), seed=9)
    ref = {rid: plains["B"].forward(toks) for rid, toks in reqs.items()}
    steps = batch_steps(reqs, [list(reqs)])
    out = str(tmp_path / "out")
    p = subprocess.Popen([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", folders["B"], "--dtype",
                          "float32", "--out", out, "--max-tokens", "93"], stdin=subprocess.PIPE, stdout=subprocess.PIPE,
                         text=True, bufsize=1)
    rows, pos = {}, {}
    try:
        for st in steps:
            p.stdin.write(json.dumps(st) + "\n")
            p.stdin.flush()
            assert p.stdout.readline().strip() == f"done {st['step']}"
            arr = np.fromfile(os.path.join(out, f"{st['step']}.f32"), dtype="<f4").reshape(-1, vocab)
            i = 0
            for e in st["entries"]:
                for w in e["want"]:
                    rows[(e["id"], pos.get(e["id"], 0) + w)] = arr[i]
                    i += 1
                pos[e["id"]] = pos.get(e["id"], 0) + len(e["tokens"])
        p.stdin.close()
        assert p.wait(timeout=60) == 0
    finally:
        if p.poll() is None:
            p.kill()
    for (rid, place), got in rows.items():
        assert np.abs(got - ref[rid][place]).max() <= F32_ABS * max(1.0, ref[rid][place].std()), f"trace_run: request {rid} position {place}"
