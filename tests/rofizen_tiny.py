"""Small Rofizen configurations that differ in every size and option, a writer of model folders with random weights
whose gains, biases, gates and tables are not the trivial ones, and configurations drawn at random."""
from __future__ import annotations

import copy
import json
import os

import numpy as np
import torch


def gla(heads, dim, vdim, tau, rank):
    """`rank` goes into the tensors' shapes, not into the written config.json."""
    return dict(type="gla", mixer=dict(heads=heads, dim=dim, vdim=vdim, tau=tau, rank=rank))


def retention(heads, dim, vdim, decay, rot_dims, base=10000.0):
    return dict(type="retention", mixer=dict(heads=heads, dim=dim, vdim=vdim, decay=list(decay), rot=dict(base=base, dims=rot_dims)))


def parallel(left, right):
    return dict(type="parallel", mixer=dict(left=left, right=right))


def left(heads, kv_heads, dim, vdim, scale, softcap=None, coef=None, every=None):
    m = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale)
    if softcap is not None:
        m["softcap"] = softcap
    if coef is not None:
        m["q_temp"] = dict(coef=coef, every=every)
    return m


def right(heads, dim, vdim, gate_cap):
    return dict(heads=heads, dim=dim, vdim=vdim, gate_cap=gate_cap)


def dense(ff):
    return dict(kind="dense", ff=ff)


def moe(experts, top, ff, shared=None):
    m = dict(kind="moe", expert=dict(ff=ff), router=dict(experts=experts, top=top))
    if shared is not None:
        m["shared"] = dict(ff=shared)
    return m


# sizes the matrix-core kernels take; the memory wider and narrower than the attention beside it; two experts a
# token; a temperature whose steps of 50 fall inside the prompts
RZ_A = dict(architecture="Rofizen", vocab=300, width=96, norm=dict(eps=1e-5), embedding=dict(scale=3.0), postln_alpha=1.7, layers=[
    dict(parallel(left(6, 3, 32, 16, 0.2, softcap=6.0, coef=0.7, every=50), right(3, 24, 40, 5.0)), mlp=moe(6, 2, 40, shared=72)),
    dict(gla(3, 16, 48, 8.0, 5), mlp=dense(112)),
    dict(retention(2, 40, 24, (0.9, 0.995), 16, base=1000.0), mlp=moe(4, 1, 56, shared=24)),
    dict(gla(2, 64, 32, 2.0, 20), mlp=None),
])

# sizes that are multiples of nothing; one kv head; no cap, no temperature; a decay of one; every expert chosen and
# no shared one; a rotation over two values; layers without feed-forward; an alpha of one
RZ_B = dict(architecture="Rofizen", vocab=97, width=62, norm=dict(eps=1e-4), embedding=dict(scale=0.5), postln_alpha=1.0, layers=[
    dict(retention(3, 12, 7, (1.0, 0.5, 0.97), 2, base=20.0), mlp=moe(3, 3, 21)),
    dict(parallel(left(9, 1, 10, 6, 0.7), right(1, 5, 11, 30.0)), mlp=None),
    dict(gla(1, 9, 70, 1.0, 3), mlp=moe(5, 2, 16, shared=33)),
    dict(parallel(left(2, 2, 12, 20, 0.4, softcap=2.0), right(4, 6, 3, 1.5)), mlp=dense(30)),
])

# one query head a kv head; keys past 64 and values past 128; a temperature at every position; the recurrences' keys
# past what their chunked forms' tiles take in the linear attention (130) and past half of it in the gated one
RZ_C = dict(architecture="Rofizen", vocab=400, width=128, norm=dict(eps=1e-6), embedding=dict(scale=11.0), postln_alpha=2.5, layers=[
    dict(parallel(left(8, 8, 80, 144, 0.1, softcap=30.0, coef=0.3, every=1), right(2, 130, 66, 12.0)), mlp=moe(9, 4, 24, shared=40)),
    dict(retention(1, 130, 64, (0.98,), 130), mlp=dense(64)),
    dict(gla(2, 132, 64, 16.0, 16), mlp=moe(2, 1, 100)),
])

RZ = {"A": RZ_A, "B": RZ_B, "C": RZ_C}


def _bf16(a) -> torch.Tensor:
    return torch.tensor(np.asarray(a, dtype=np.float32)).to(torch.bfloat16)


def written_config(raw: dict) -> dict:
    """config.json as a folder holds it: the ranks of the decays are the tensors' business."""
    out = copy.deepcopy(raw)
    for layer in out["layers"]:
        layer["mixer"].pop("rank", None)
    return out


def write_rofizen(folder: str, raw: dict, seed: int = 0, sharpen: float = 1.0) -> str:
    """config.json and model.safetensors (bfloat16, the tables int32).  Matrices N(0, 1/inputs); gains around one,
    signs included now and then; biases N(0, 0.5); the decays' biases around 2, so that states live long; the
    memory's forget biases around 2 as well, its input biases spread; tables whose rows name different experts.
    `sharpen` multiplies the q gains of the attention (its scores grow with them)."""
    from minfer_amd import config_from_dict
    from minfer_amd.engine.model import expected_tensors
    from minfer_amd.weights.safetensors_io import write_safetensors
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(written_config(raw), f)
    expected = expected_tensors(config_from_dict(raw).model_spec())
    rng = np.random.default_rng(seed)
    made = {}
    for name, ts in expected.items():
        shape = tuple(ts.shape)
        if ts.below is not None:
            made[name] = torch.tensor(np.argsort(rng.random((shape[0], ts.below)), axis=1)[:, :shape[1]].astype(np.int32))
            continue
        if name.endswith((".a2.b", ".f.b")):
            a = 2.0 + rng.standard_normal(shape)
        elif name.endswith(".b"):
            a = 0.5 * rng.standard_normal(shape)
        elif len(shape) == 1:
            a = rng.uniform(0.6, 1.4, shape) * np.where(rng.random(shape) < 0.1, -1.0, 1.0)
            if name.endswith(".q.norm"):
                a = a * sharpen
        elif name == "embed":
            a = rng.standard_normal(shape)
        else:
            a = rng.standard_normal(shape) / np.sqrt(shape[1])
            if name.endswith((".right.i", ".right.f")):
                a = 2.0 * a
        made[name] = _bf16(a)
    write_safetensors(os.path.join(folder, "model.safetensors"), [(n, tuple(t.shape), t.dtype) for n, t in made.items()],
                      lambda n: made[n])
    return folder


def random_config(rng) -> dict:
    """A configuration drawn at random: one to five layers of the three kinds in any order, odd head sizes and counts,
    with and without cap, temperature, shared expert and feed-forward, any number of experts a token."""
    width = int(rng.choice([48, 62, 64, 100, 128, 136]))
    layers = []
    for _ in range(int(rng.integers(1, 6))):
        mlp, draw = None, rng.random()
        if draw > 0.5:
            experts = int(rng.choice([1, 2, 5, 8, 20]))
            mlp = moe(experts, int(rng.integers(1, min(experts, 6) + 1)), int(rng.choice([16, 40, 72])),
                      shared=int(rng.choice([8, 33, 64])) if rng.random() < 0.7 else None)
        elif draw > 0.2:
            mlp = dense(int(rng.choice([16, 33, 128])))
        dim, vdim = int(rng.choice([5, 8, 16, 24, 32, 64, 96, 140])), int(rng.choice([3, 8, 16, 24, 64, 80]))
        heads = int(rng.choice([1, 2, 3, 5]))
        kind = int(rng.integers(0, 3))
        if kind == 0:
            layer = gla(heads, dim, vdim, float(rng.choice([0.5, 1.0, 4.0, 16.0])), int(rng.choice([1, 3, 16, 70])))
        elif kind == 1:
            rot = int(rng.choice([d for d in (2, 4, 6, 8, 16, 32, 64, 96, 140) if d <= dim]))
            layer = retention(heads, dim, vdim, [float(d) for d in rng.choice([0.3, 0.9, 0.99, 0.9995, 1.0], heads)], rot,
                              base=float(rng.choice([100.0, 10000.0, 1000000.0])))
        else:
            kv = int(rng.choice([1, 2, 3]))
            temp = rng.random() < 0.7
            layer = parallel(left(kv * int(rng.choice([1, 2, 3, 10])), kv, dim, vdim, float(rng.choice([0.1, 0.3, 1.0])),
                                  softcap=float(rng.choice([1.0, 5.0, 50.0])) if rng.random() < 0.7 else None,
                                  coef=float(rng.choice([0.1, 0.5, 2.0])) if temp else None,
                                  every=int(rng.choice([1, 7, 64, 100])) if temp else None),
                             right(heads, int(rng.choice([5, 16, 32, 64, 140])), int(rng.choice([3, 16, 24, 80])),
                                   float(rng.choice([1.0, 6.0, 15.0, 40.0]))))
        layers.append(dict(layer, mlp=mlp))
    return dict(architecture="Rofizen", vocab=int(rng.choice([64, 300, 1000])), width=width,
                norm=dict(eps=float(rng.choice([1e-6, 1e-5]))), embedding=dict(scale=float(rng.choice([1.0, 8.0]))),
                postln_alpha=float(rng.choice([1.0, 1.5, 3.0])), layers=layers)
