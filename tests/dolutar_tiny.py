"""Small Dolutar configurations that differ in every size and option, a writer of model folders with random weights
whose gains, biases, sinks and corrections are not the trivial ones, and configurations drawn at random."""
from __future__ import annotations

import copy
import json
import os

import numpy as np
import torch


def attention(heads, kv_heads, dim, vdim, scale, rot_dims, window=None, keep_first=0, base=10000.0, kv_from=None):
    m = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale, rot=dict(base=base, dims=rot_dims))
    if window is not None:
        m["mask"] = dict(size=window, keep_first=keep_first)
    if kv_from is not None:
        m["kv_from"] = kv_from
    return dict(type="attention", mixer=m)


def dense(ff, limit):
    return dict(kind="dense", ff=ff, limit=limit)


def moe(experts, top, ff, identity=0):
    return dict(kind="moe", expert=dict(ff=ff), router=dict(experts=experts, top=top, identity=identity))


# sizes the matrix-core kernels take; an owner with a window of 70 and three kept positions whose readers see 130
# positions back with five kept, and 20 back; a causal owner with a windowed reader; a layer without feed-forward;
# experts that hand their input on, one and two of them
DL_A = dict(architecture="Dolutar", vocab=300, width=96, norm=dict(eps=1e-5), logit_scale=3.0,
            embedding=dict(scale=1.5, bigram=dict(buckets=97, mul_prev=31, mul_cur=5)), layers=[
    dict(attention(4, 2, 32, 16, 0.2, 16, 70, 3), mlp=dense(112, 1.0)),
    dict(attention(4, 2, 32, 16, 0.3, 16, 130, 5, kv_from=0), mlp=moe(6, 2, 40, 2)),
    dict(attention(6, 3, 16, 48, 0.4, 16, base=500.0), mlp=None),
    dict(attention(4, 2, 32, 16, 0.25, 16, 20, 0, kv_from=0), mlp=moe(4, 1, 56, 1)),
    dict(attention(6, 3, 16, 48, 0.5, 16, 33, 0, base=500.0, kv_from=2), mlp=dense(40, 0.3)),
])

# sizes that are multiples of nothing; nine query heads on one kv head; a window of one with five kept positions and
# a reader that sees everything; a rotation over two values; every expert chosen; more experts that hand their input
# on than others; no pair table, no scales
DL_B = dict(architecture="Dolutar", vocab=97, width=60, norm=dict(eps=1e-4), layers=[
    dict(attention(9, 1, 10, 6, 0.7, 4, 1, 5, base=20.0), mlp=moe(3, 3, 20)),
    dict(attention(3, 3, 12, 7, 0.9, 2, 40, 0, base=100.0), mlp=moe(1, 2, 33, 3)),
    dict(attention(9, 1, 10, 6, 0.5, 4, base=20.0, kv_from=0), mlp=dense(37, 2.5)),
])

# a window one longer than a page with a page of kept positions, and a reader with kept positions beyond a page; a
# table of a single bucket; all but two experts hand their input on; a scale of the logits below one
DL_C = dict(architecture="Dolutar", vocab=400, width=128, norm=dict(eps=1e-6), logit_scale=0.4,
            embedding=dict(scale=0.25, bigram=dict(buckets=1, mul_prev=3, mul_cur=1)), layers=[
    dict(attention(8, 2, 64, 64, 0.125, 64, 65, 64), mlp=moe(4, 2, 64, 4)),
    dict(attention(2, 2, 16, 32, 0.25, 8, 64, 1), mlp=moe(2, 4, 64, 6)),
    dict(attention(8, 2, 64, 64, 0.25, 64, 40, 70, kv_from=0), mlp=dense(128, 7.0)),
    dict(attention(8, 8, 16, 16, 1.0, 8, 128, 0), mlp=moe(9, 4, 24)),
])

DL = {"A": DL_A, "B": DL_B, "C": DL_C}


def _bf16(a) -> torch.Tensor:
    return torch.tensor(np.asarray(a, dtype=np.float32)).to(torch.bfloat16)


def write_dolutar(folder: str, raw: dict, seed: int = 0, sharpen: float = 1.0) -> str:
    """config.json and model.safetensors (bfloat16).  Matrices N(0, 1/inputs), gains around one, biases N(0, 0.3), sinks
    N(1, 1) (a good part of a few keys' weight), corrections N(0, 0.1) (they change choices).  `sharpen` multiplies the
    queries' gains: scores grow with it, and with it the sinks, so that single keys decide and the sinks still weigh."""
    from minfer_amd import config_from_dict
    from minfer_amd.engine.model import expected_tensors
    from minfer_amd.weights.safetensors_io import write_safetensors
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(raw, f)
    rng = np.random.default_rng(seed)
    made = {}
    for name, ts in expected_tensors(config_from_dict(raw).model_spec()).items():
        shape = tuple(ts.shape)
        if name.endswith(("norm1", "norm2", ".norm")):
            a = rng.uniform(0.6, 1.4, shape)
            if name.endswith("q.norm"):
                a = a * sharpen
        elif name.endswith(".sink"):
            a = (1.0 + rng.standard_normal(shape)) * sharpen
        elif name.endswith(".correction"):
            a = 0.1 * rng.standard_normal(shape)
        elif name.endswith(".b"):
            a = 0.3 * rng.standard_normal(shape)
        elif name in ("embed", "bigram"):
            a = rng.standard_normal(shape)
        else:
            a = rng.standard_normal(shape) / np.sqrt(shape[1])
            if name.endswith("router"):
                a = a * 0.5          # (it reads the stream itself, which grows with the layers)
        made[name] = _bf16(a)
    write_safetensors(os.path.join(folder, "model.safetensors"),
                      [(n, tuple(t.shape), torch.bfloat16) for n, t in made.items()], lambda n: made[n])
    return folder


def random_config(rng) -> dict:
    """A configuration drawn at random: one to six layers, readers behind owners with masks of their own, with and
    without feed-forward, odd head sizes and counts, windows from one to beyond the prompts, kept positions from none to
    beyond a page, any share of experts that hand their input on."""
    width = int(rng.choice([48, 60, 64, 100, 128, 136]))
    layers, owners = [], []
    for i in range(int(rng.integers(1, 7))):
        draw = rng.random()
        if draw < 0.15:
            mlp = None
        elif draw < 0.45:
            mlp = dense(int(rng.choice([16, 37, 64, 100])), float(rng.choice([0.3, 1.0, 7.0])))
        else:
            experts, identity = int(rng.integers(1, 9)), int(rng.choice([0, 1, 2, 5]))
            mlp = moe(experts, int(rng.integers(1, min(6, experts + identity) + 1)), int(rng.choice([16, 40, 64, 72])), identity)
        mask = None
        if rng.random() < 0.8:
            mask = dict(size=int(rng.choice([1, 2, 31, 64, 65, 100, 1000])), keep_first=int(rng.choice([0, 1, 4, 64, 70])))
        if owners and rng.random() < 0.45:
            j = int(rng.choice(owners))
            layer = copy.deepcopy(dict(type="attention", mixer=layers[j]["mixer"]))
            layer["mixer"].update(kv_from=j, scale=float(rng.choice([0.1, 0.3, 1.0])))
            layer["mixer"].pop("mask", None)
        else:
            kv = int(rng.choice([1, 2, 3]))
            dim = int(rng.choice([6, 8, 16, 24, 32, 64, 96]))
            rot = int(rng.choice([d for d in (2, 4, 6, 8, 16, 32, 64, 96) if d <= dim]))
            layer = attention(kv * int(rng.choice([1, 2, 3, 10])), kv, dim, int(rng.choice([6, 8, 16, 24, 64, 10])),
                              float(rng.choice([0.1, 0.3, 1.0])), rot, base=float(rng.choice([100.0, 10000.0, 500000.0])))
            owners.append(i)
        if mask is not None:
            layer["mixer"]["mask"] = mask
        layers.append(dict(layer, mlp=mlp))
    raw = dict(architecture="Dolutar", vocab=int(rng.choice([64, 300, 1000])), width=width,
               norm=dict(eps=float(rng.choice([1e-6, 1e-5]))), embedding=dict(scale=float(rng.choice([0.5, 1.0, 4.0]))), layers=layers)
    if rng.random() < 0.7:
        raw["embedding"]["bigram"] = dict(buckets=int(rng.choice([1, 50, 1009])), mul_prev=int(rng.choice([1, 127, 100003])),
                                          mul_cur=int(rng.choice([1, 7, 99991])))
    if rng.random() < 0.7:
        raw["logit_scale"] = float(rng.choice([0.1, 2.0, 5.0]))
    return raw
