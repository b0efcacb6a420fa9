"""A plain, slow implementation of the Dolutar decoder in numpy float64, one function per mechanism, written from
the design's equations and sharing no code with the product path.

The design: x = scale table[token] + pairs[row(previous token, token)]; every layer adds normed results to the stream,
x <- x + N1(attention(x)), x <- x + N2(ff(x)), with N the RMS norm; a layer without a feed-forward ends after the first
sum; the logits are a number times head(N(x)).
Attention: grouped-query softmax attention with biases on queries, keys and values, queries and keys normed per head
with shared gains and then turned in halves, a sliding window beside the sequence's first positions, and a sink per head
in the softmax's denominator; a layer with `kv_from` reads the keys and values of the layer it names.
A feed-forward is dense and clamped, or a mixture of silu experts whose router also knows experts that hand their input
on as it is.
"""
from __future__ import annotations

import json
import os
import struct

import numpy as np


# ------------------------------------------------------------------ file reading
def read_safetensors(path: str):
    """name -> float64 array: header length, JSON header, raw data."""
    with open(path, "rb") as f:
        n = struct.unpack("<Q", f.read(8))[0]
        head = json.loads(f.read(n))
        data = f.read()
    out = {}
    for name, e in head.items():
        if name == "__metadata__":
            continue
        lo, hi = e["data_offsets"]
        raw = data[lo:hi]
        if e["dtype"] == "BF16":
            a = (np.frombuffer(raw, dtype="<u2").astype(np.uint32) << 16).view(np.float32).astype(np.float64)
        elif e["dtype"] == "F32":
            a = np.frombuffer(raw, dtype="<f4").astype(np.float64)
        else:
            raise ValueError(f"{name}: dtype {e['dtype']}")
        out[name] = a.reshape(e["shape"])
    return out


# ------------------------------------------------------------------ small functions
def sigmoid(z):
    return 0.5 * (1.0 + np.tanh(0.5 * np.asarray(z, dtype=np.float64)))


def silu(z):
    return z * sigmoid(z)


def rms_norm(x, w, eps: float):
    return x / np.sqrt((x * x).mean(axis=-1, keepdims=True) + eps) * w


def rotate_halves(x, positions, base: float, dims: int):
    """Value i turns with value i + dims / 2, i < dims / 2, by position * base^(-2i/dims); the values from `dims`
    on pass.  x [tokens][heads][width]."""
    out = x.copy()
    half = dims // 2
    a = (np.asarray(positions, dtype=np.float64)[:, None] * (base ** (-2.0 * np.arange(half) / dims))[None, :])[:, None, :]
    u, v = x[..., :half], x[..., half:dims]
    out[..., :half] = u * np.cos(a) - v * np.sin(a)
    out[..., half:dims] = v * np.cos(a) + u * np.sin(a)
    return out


# ------------------------------------------------------------------ embedding
def pair_rows(tokens, buckets: int, mul_prev: int, mul_cur: int):
    """The row of the pair table for every token: (previous mul_prev + token mul_cur) mod buckets, and row `buckets`
    for a sequence's first token."""
    rows = [buckets]
    for i in range(1, len(tokens)):
        rows.append((int(tokens[i - 1]) * mul_prev + int(tokens[i]) * mul_cur) % buckets)
    return rows[:len(tokens)]


def embed(tokens, w, spec):
    x = w["embed"][np.asarray(tokens, dtype=np.int64)] * spec.get("scale", 1.0)
    pairs = spec.get("bigram")
    if pairs is not None:
        x = x + w["bigram"][pair_rows(tokens, pairs["buckets"], pairs["mul_prev"], pairs["mul_cur"])]
    return x


# ------------------------------------------------------------------ attention
def visible(i: int, j: int, mask) -> bool:
    """Whether position i sees position j."""
    if j > i:
        return False
    if mask is None:
        return True
    return i - j < mask["size"] or j < mask.get("keep_first", 0)


def sink_softmax(s, seen, sink):
    """Weights of the seen keys: e^s over the sum of e^s and e^sink.  s [heads][queries][keys], sink [heads]."""
    s = np.where(seen[None], s, -np.inf)
    m = np.maximum(s.max(axis=-1), sink[:, None])
    e = np.exp(s - m[..., None])
    return e / (e.sum(axis=-1) + np.exp(sink[:, None] - m))[..., None]


def keys_and_values(h, w, prefix: str, m, eps: float):
    """The layer's own keys (normed and turned) and values."""
    T, G = h.shape[0], m["kv_heads"]
    k = (h @ w[prefix + "k"].T + w[prefix + "k.b"]).reshape(T, G, m["dim"])
    v = (h @ w[prefix + "v"].T + w[prefix + "v.b"]).reshape(T, G, m["vdim"])
    k = rms_norm(k, w[prefix + "k.norm"], eps)
    if m.get("rot") is not None:
        k = rotate_halves(k, np.arange(T), m["rot"]["base"], m["rot"]["dims"])
    return k, v


def attention(h, kv, w, prefix: str, m, eps: float):
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]
    q = rms_norm((h @ w[prefix + "q"].T + w[prefix + "q.b"]).reshape(T, H, m["dim"]), w[prefix + "q.norm"], eps)
    if m.get("rot") is not None:
        q = rotate_halves(q, np.arange(T), m["rot"]["base"], m["rot"]["dims"])
    k, v = (np.repeat(a, H // G, axis=1) for a in kv)          # query head h reads head h // (H / G)
    s = np.einsum("ihd,jhd->hij", q, k) * m["scale"]
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    seen = j <= i
    mask = m.get("mask")
    if mask is not None:
        seen = seen & ((i - j < mask["size"]) | (j < mask.get("keep_first", 0)))
    p = sink_softmax(s, seen, w[prefix + "sink"])
    return np.einsum("hij,jhv->ihv", p, v).reshape(T, H * m["vdim"]) @ w[prefix + "o"].T


# ------------------------------------------------------------------ feed-forwards
def clamped_ff(h, w, prefix: str, limit: float):
    g = np.minimum(h @ w[prefix + "gate"].T, limit)
    u = np.clip(h @ w[prefix + "up"].T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ w[prefix + "down"].T


def route(h, w, prefix: str, top: int, forced=None):
    """(experts, weights, margins) of every token: scores are the softmax over all router outputs; chosen by score plus
    correction, weighed by the score as it is.  The margin is how far the last one chosen lies above the first one left
    out.  `forced` [tokens][top]: another's choice in its place (weighed by the scores here)."""
    z = h @ w[prefix + "router"].T
    e = np.exp(z - z.max(axis=-1, keepdims=True))
    s = e / e.sum(axis=-1, keepdims=True)
    choice = s + w[prefix + "correction"]
    order = np.argsort(-choice, axis=-1, kind="stable")
    ranked = np.take_along_axis(choice, order, axis=-1)
    margins = ranked[:, top - 1] - ranked[:, top] if top < choice.shape[1] else np.full(h.shape[0], np.inf)
    order = order[:, :top] if forced is None else np.asarray(forced)
    return order, np.take_along_axis(s, order, axis=-1), margins


def mixture(h, w, prefix: str, experts: int, top: int, forced=None, seen=None):
    """The weighted sum of the chosen experts; an expert number from `experts` on hands its input on.  `seen`, where
    given, gets (choices of the router here, margins)."""
    if seen is not None:
        own, _, margins = route(h, w, prefix, top)
        seen.append((own, margins))
    chosen, weight, _ = route(h, w, prefix, top, forced)
    out = np.zeros_like(h)
    for t in range(h.shape[0]):
        for e, a in zip(chosen[t], weight[t]):
            if e >= experts:
                out[t] += a * h[t]
            else:
                p = f"{prefix}e{e}."
                y = silu(w[p + "gate"] @ h[t]) * (w[p + "up"] @ h[t])
                out[t] += a * (w[p + "down"] @ y)
    return out


def feed_forward(h, w, prefix: str, mlp, forced=None, seen=None):
    if mlp["kind"] == "dense":
        return clamped_ff(h, w, prefix, mlp["limit"])
    return mixture(h, w, prefix, mlp["router"]["experts"], mlp["router"]["top"], forced, seen)


def greedy(logits) -> int:
    return int(np.argmax(logits))


# ------------------------------------------------------------------ the model
class PlainDolutar:
    def __init__(self, folder: str):
        with open(os.path.join(folder, "config.json")) as f:
            self.c = json.load(f)
        self.w = read_safetensors(os.path.join(folder, "model.safetensors"))

    def routed_layers(self):
        return [i for i, layer in enumerate(self.c["layers"]) if layer.get("mlp") and layer["mlp"]["kind"] == "moe"]

    def streams(self, tokens, forced=None, seen=None):
        """The residual stream behind every layer, [layers][tokens][width].  `forced`: {layer: another's choices of
        experts}; `seen` gets (choices, margins) of every routed layer."""
        c, w, eps = self.c, self.w, self.c["norm"]["eps"]
        x = embed(tokens, w, c.get("embedding") or {})
        kept, out = {}, []
        for i, layer in enumerate(c["layers"]):
            m, p = layer["mixer"], f"l{i}."
            j = m.get("kv_from")
            kept[i] = keys_and_values(x, w, p + "mix.", m, eps) if j is None else kept[j]
            x = x + rms_norm(attention(x, kept[i], w, p + "mix.", m, eps), w[p + "norm1"], eps)
            if layer.get("mlp") is not None:
                x = x + rms_norm(feed_forward(x, w, p + "mlp.", layer["mlp"], (forced or {}).get(i), seen), w[p + "norm2"], eps)
            out.append(x)
        return np.stack(out)

    def forward(self, tokens, forced=None, seen=None):
        """Logits of every position, [tokens][vocab]."""
        x = rms_norm(self.streams(tokens, forced, seen)[-1], self.w["final.norm"], self.c["norm"]["eps"])
        return x @ self.w["head"].T * self.c.get("logit_scale", 1.0)
