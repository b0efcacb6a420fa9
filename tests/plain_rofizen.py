"""A plain, slow implementation of the Rofizen decoder in numpy float64, one function per mechanism,
written from the design's equations and sharing no code with the product path.

The design: x = scale table[token]; a layer norms behind its sums, x <- L1(a x + mixer(x)), x <- L2(a x + ff(x)),
with L the layer norm (mean taken off, gain, no bias); a layer without a feed-forward ends after the first line.
A mixer is one of
  "gla":       linear attention whose state decays per key channel, by a low-rank gate of the token;
  "retention": linear attention with a fixed decay per head, queries and keys rotated in halves;
  "parallel":  half the sum of two normed results: causal softmax attention (queries and keys normed over the whole
               projection, capped scores less a slope times the distance, queries warmer with the position), and a
               matrix memory with exponential gates under a running maximum.
A feed-forward is dense with the square of relu, or a mixture of silu experts that a table picks by the token's id,
each weighing the same, beside a shared expert weighed by a sigmoid.
"""
from __future__ import annotations

import json
import math
import os
import struct

import numpy as np


# ------------------------------------------------------------------ file reading
def read_safetensors(path: str):
    """name -> float64 array (int32 stays): header length, JSON header, raw data."""
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
        elif e["dtype"] == "I32":
            a = np.frombuffer(raw, dtype="<i4").copy()
        else:
            raise ValueError(f"{name}: dtype {e['dtype']}")
        out[name] = a.reshape(e["shape"])
    return out


# ------------------------------------------------------------------ small functions
def sigmoid(z):
    return 0.5 * (1.0 + np.tanh(0.5 * np.asarray(z, dtype=np.float64)))


def log_sigmoid(z):
    z = np.asarray(z, dtype=np.float64)
    return np.minimum(z, 0.0) - np.log1p(np.exp(-np.abs(z)))


def silu(z):
    return z * sigmoid(z)


def unit_rms(x, eps: float):
    """x over its root mean square, eps inside the root."""
    return x / np.sqrt((x * x).mean(axis=-1, keepdims=True) + eps)


def layer_norm(x, w, eps: float):
    c = x - x.mean(axis=-1, keepdims=True)
    return c / np.sqrt((c * c).mean(axis=-1, keepdims=True) + eps) * w


def softmax_rows(s):
    """Softmax over the last axis; -inf entries weigh nothing."""
    e = np.exp(s - s.max(axis=-1, keepdims=True))
    return e / e.sum(axis=-1, keepdims=True)


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


# ------------------------------------------------------------------ mixers
def gla_decay(h, w, prefix: str, m):
    """The decay of every head and key channel, per token: sigmoid(A2 A1 h + b)^(1/tau)."""
    z = h @ w[prefix + "a1"].T @ w[prefix + "a2"].T + w[prefix + "a2.b"]
    return np.exp(log_sigmoid(z) / m["tau"]).reshape(h.shape[0], m["heads"], m["dim"])


def gated_linear_attention(h, w, prefix: str, m, eps: float):
    """"gla": S_t = diag(decay_t) S_(t-1) + k_t v_t^T, o_t = S_t^T q_t; o normed per head with a shared gain, times
    silu(Wg h)."""
    T, H, D, V = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = (h @ w[prefix + "q"].T).reshape(T, H, D) * D ** -0.5
    k = (h @ w[prefix + "k"].T).reshape(T, H, D)
    v = (h @ w[prefix + "v"].T).reshape(T, H, V)
    decay = gla_decay(h, w, prefix, m)
    o = np.zeros((T, H, V))
    for hd in range(H):
        S = np.zeros((D, V))
        for t in range(T):
            S = decay[t, hd][:, None] * S + np.outer(k[t, hd], v[t, hd])
            o[t, hd] = S.T @ q[t, hd]
    o = (unit_rms(o, eps) * w[prefix + "norm"]).reshape(T, H * V)
    return (o * silu(h @ w[prefix + "g"].T)) @ w[prefix + "o"].T


def retention(h, w, prefix: str, m, eps: float):
    """"retention": S_t = decay_h S_(t-1) + k_t v_t^T with rotated q and k (k times dim^-1/2); o over its root mean
    square per head, times silu(Wg h)."""
    T, H, D, V = h.shape[0], m["heads"], m["dim"], m["vdim"]
    pos = np.arange(T)
    q = rotate_halves((h @ w[prefix + "q"].T).reshape(T, H, D), pos, m["rot"]["base"], m["rot"]["dims"])
    k = rotate_halves((h @ w[prefix + "k"].T).reshape(T, H, D), pos, m["rot"]["base"], m["rot"]["dims"]) * D ** -0.5
    v = (h @ w[prefix + "v"].T).reshape(T, H, V)
    o = np.zeros((T, H, V))
    for hd in range(H):
        S = np.zeros((D, V))
        for t in range(T):
            S = m["decay"][hd] * S + np.outer(k[t, hd], v[t, hd])
            o[t, hd] = S.T @ q[t, hd]
    o = unit_rms(o, eps).reshape(T, H * V)
    return (o * silu(h @ w[prefix + "g"].T)) @ w[prefix + "o"].T


def query_temperature(positions, spec):
    return 1.0 + spec["coef"] * np.log(np.floor((np.asarray(positions) + 1) / spec["every"]) + 1.0)


def slopes(heads: int):
    return 2.0 ** (-8.0 * np.arange(1, heads + 1) / heads)


def sloped_attention(h, w, prefix: str, m, eps: float):
    """The left side of "parallel"."""
    T, H, G, D, V = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = unit_rms(h @ w[prefix + "q"].T + w[prefix + "q.b"], eps) * w[prefix + "q.norm"]      # over all heads at once
    k = unit_rms(h @ w[prefix + "k"].T + w[prefix + "k.b"], eps) * w[prefix + "k.norm"]
    v = (h @ w[prefix + "v"].T + w[prefix + "v.b"]).reshape(T, G, V)
    q, k = q.reshape(T, H, D), k.reshape(T, G, D)
    pos = np.arange(T)
    if m.get("q_temp") is not None:
        q = q * query_temperature(pos, m["q_temp"])[:, None, None]
    dist = pos[:, None] - pos[None, :]
    out = np.zeros((T, H, V))
    for hd in range(H):
        g = hd // (H // G)
        s = q[:, hd] @ k[:, g].T * m["scale"]
        if m.get("softcap") is not None:
            s = m["softcap"] * np.tanh(s / m["softcap"])
        s = s - slopes(H)[hd] * dist
        out[:, hd] = softmax_rows(np.where(dist >= 0, s, -np.inf)) @ v[:, g]
    return out.reshape(T, H * V) @ w[prefix + "o"].T + w[prefix + "o.b"]


def memory_gates(h, w, prefix: str, m):
    """(log input gate, log forget gate) [tokens][heads], both capped before anything else."""
    cap = m["gate_cap"]
    i = cap * np.tanh((h @ w[prefix + "i"].T + w[prefix + "i.b"]) / cap)
    f = log_sigmoid(cap * np.tanh((h @ w[prefix + "f"].T + w[prefix + "f.b"]) / cap))
    return i, f


def matrix_memory(h, w, prefix: str, m, eps: float):
    """The right side of "parallel": an outer-product memory with exponential gates under a running maximum that
    starts at 0, read with a denominator of its own."""
    T, H, D, V = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = (h @ w[prefix + "q"].T).reshape(T, H, D) * D ** -0.5
    k = (h @ w[prefix + "k"].T).reshape(T, H, D)
    v = (h @ w[prefix + "v"].T).reshape(T, H, V)
    i, f = memory_gates(h, w, prefix, m)
    o = np.zeros((T, H, V))
    for hd in range(H):
        S, n, top = np.zeros((D, V)), np.zeros(D), 0.0
        for t in range(T):
            new = max(f[t, hd] + top, i[t, hd])
            keep, take = math.exp(f[t, hd] + top - new), math.exp(i[t, hd] - new)
            S = keep * S + take * np.outer(k[t, hd], v[t, hd])
            n = keep * n + take * k[t, hd]
            top = new
            o[t, hd] = S.T @ q[t, hd] / (max(abs(n @ q[t, hd]), math.exp(-top)) + 1e-6)
    o = unit_rms(o, eps).reshape(T, H * V) * w[prefix + "norm"]
    return (o * sigmoid(h @ w[prefix + "g"].T)) @ w[prefix + "o"].T


def parallel(h, w, prefix: str, m, eps: float):
    left = sloped_attention(h, w, prefix + "left.", m["left"], eps)
    right = matrix_memory(h, w, prefix + "right.", m["right"], eps)
    return 0.5 * (unit_rms(left, eps) * w[prefix + "left.out"] + unit_rms(right, eps) * w[prefix + "right.out"])


# ------------------------------------------------------------------ feed-forward
def dense(h, w, prefix: str):
    return np.maximum(h @ w[prefix + "up"].T, 0.0) ** 2 @ w[prefix + "down"].T


def expert(h, w, stem: str):
    return (silu(h @ w[stem + ".gate"].T) * (h @ w[stem + ".up"].T)) @ w[stem + ".down"].T


def table_moe(h, tokens, w, prefix: str, mlp):
    """The experts a token's row of the table names, 1/top each, and the shared one where there is one."""
    top = mlp["router"]["top"]
    out = np.zeros((h.shape[0], w[prefix + "e0.down"].shape[0]))
    for t, token in enumerate(tokens):
        for e in w[prefix + "table"][token]:
            out[t] += expert(h[t:t + 1], w, f"{prefix}e{int(e)}")[0] / top
    if mlp.get("shared") is not None:
        out = out + sigmoid(h @ w[prefix + "shared.sg"].T) * expert(h, w, prefix + "shared")
    return out


# ------------------------------------------------------------------ the model
MIXERS = {"gla": gated_linear_attention, "retention": retention, "parallel": parallel}


def forward(cfg, w, tokens, keep_layers: bool = False):
    """Logits [tokens][vocab] of one whole sequence from position 0, and the streams after every layer."""
    eps, alpha = cfg["norm"]["eps"], cfg["postln_alpha"]
    x = w["embed"][np.asarray(tokens)] * cfg["embedding"]["scale"]
    streams = []
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        x = layer_norm(alpha * x + MIXERS[layer["type"]](x, w, p + "mix.", layer["mixer"], eps), w[p + "norm1"], eps)
        mlp = layer.get("mlp")
        if mlp is not None:
            y = dense(x, w, p + "mlp.") if mlp["kind"] == "dense" else table_moe(x, tokens, w, p + "mlp.", mlp)
            x = layer_norm(alpha * x + y, w[p + "norm2"], eps)
        if keep_layers:
            streams.append(x.copy())
    return layer_norm(x, w["final.norm"], eps) @ w["head"].T, streams


def load(folder: str):
    with open(os.path.join(folder, "config.json")) as f:
        cfg = json.load(f)
    return cfg, read_safetensors(os.path.join(folder, "model.safetensors"))


def greedy(row) -> int:
    return int(np.argmax(row))


class PlainRofizen:
    def __init__(self, cfg, w):
        self.cfg, self.w = cfg, w

    @classmethod
    def from_folder(cls, folder: str):
        return cls(*load(folder))

    def forward(self, tokens):
        """Logits [tokens][vocab]."""
        return forward(self.cfg, self.w, tokens)[0]
