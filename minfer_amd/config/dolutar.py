"""Dolutar: a decoder whose layers read the residual stream itself and norm their results on the way back into it,
x <- x + N1(attention(x)), x <- x + N2(ff(x)), with RMS norms.  The stream begins as the token's row of the embedding
table, scaled, plus a row of a second table picked by the token and the one before it; the logits may be scaled.
Attention is grouped-query softmax attention with biases on queries, keys and values, queries and keys RMS-normed per
head with shared gains and then rotated in halves, a sliding window beside the sequence's first positions, and a sink
per head; a layer with `kv_from` has no keys and values of its own and reads those of the layer it names.
A feed-forward is dense with clamped gates, or a mixture of silu experts whose router scores with a softmax over all
experts, chooses by score plus a correction, weighs by the score as it is, and counts among its experts some that hand
their input on.

config.json: `architecture` = "Dolutar"; `vocab`, `width`; `norm` = {eps}; `embedding` = {scale, bigram: {buckets,
mul_prev, mul_cur} or absent}; `logit_scale` or absent; `layers`, a list of {type: "attention", mixer: {...},
mlp: {...} or null}.
mixer: {heads, kv_heads, dim, vdim, scale, rot: {base, dims} or absent, mask: {size, keep_first} or absent, kv_from}.
mlp: {kind: "dense", ff, limit} or {kind: "moe", expert: {ff}, router: {experts, top, identity}}.
Tensors: embed, bigram, l<i>.norm1, l<i>.norm2, l<i>.mix.*, l<i>.mlp.*, final.norm, head.
"""
from __future__ import annotations

import copy
import math
from typing import Any, Dict, List, Optional

from .base import ConfigError, KeyReader
from ..parts.spec import BlockSpec, ModelSpec, PartSpec, RunEntry

ARCHITECTURE = "Dolutar"
MIXER_TYPES = ("attention",)
MLP_KINDS = ("dense", "moe")
MAX_POSITIONS = 1 << 20      # the design names no bound; rotation tables grow on demand up to here


def _mixer_sizes(raw: Any, where: str) -> Dict[str, Any]:
    r = KeyReader(raw, where)
    out: Dict[str, Any] = dict(heads=r.integer("heads"), kv_heads=r.integer("kv_heads"), dim=r.integer("dim"),
                               vdim=r.integer("vdim"), scale=r.number("scale", positive=False))
    if out["heads"] % out["kv_heads"]:
        raise ConfigError(f"{where}: 'heads' {out['heads']} is not a multiple of 'kv_heads' {out['kv_heads']}")
    out["rot"] = out["mask"] = None
    if r.raw_value("rot") is not None:
        k = KeyReader(r.raw_value("rot"), where + ".rot")
        dims = k.integer("dims")
        if dims % 2 or dims > out["dim"]:
            raise ConfigError(f"{where}.rot: 'dims' must be even and at most {out['dim']}, found {dims}")
        out["rot"] = dict(base=k.number("base"), dims=dims)
    if r.raw_value("mask") is not None:
        k = KeyReader(r.raw_value("mask"), where + ".mask")
        out["mask"] = dict(size=k.integer("size"), keep_first=k.integer("keep_first", default=0, minimum=0))
    out["kv_from"] = r.integer("kv_from", default=None, minimum=0)
    return out


def _mlp_sizes(raw: Any, where: str) -> Optional[Dict[str, Any]]:
    if raw is None:
        return None
    m = KeyReader(raw, where)
    kind = m.string("kind")
    if kind == "dense":
        return dict(kind=kind, ff=m.integer("ff"), limit=m.number("limit"))
    if kind != "moe":
        raise ConfigError(f"{where}: kind {kind!r} is not one of {list(MLP_KINDS)}")
    e = KeyReader(m.raw_value("expert") or {}, where + ".expert")
    r = KeyReader(m.raw_value("router") or {}, where + ".router")
    router = dict(experts=r.integer("experts"), top=r.integer("top"), identity=r.integer("identity", default=0, minimum=0))
    if router["top"] > router["experts"] + router["identity"]:
        raise ConfigError(f"{where}.router: {router['top']} experts cannot be chosen from {router['experts']} and "
                          f"{router['identity']} that hand their input on")
    return dict(kind=kind, expert=dict(ff=e.integer("ff")), router=router)


class DolutarConfig:
    architecture = ARCHITECTURE

    def __init__(self, vocab: int, width: int, eps: float, layers: List[Dict[str, Any]], embedding_scale: float = 1.0,
                 bigram: Optional[Dict[str, int]] = None, logit_scale: float = 1.0, init_std: Optional[float] = None):
        self.vocab, self.width, self.eps, self.layers = vocab, width, eps, layers
        self.embedding_scale, self.bigram, self.logit_scale = embedding_scale, bigram, logit_scale
        self.init_std = init_std
        self._fan_in: Optional[Dict[str, int]] = None

    # ---------------------------------------------------------------- reading
    @classmethod
    def from_dict(cls, raw: Dict[str, Any]) -> "DolutarConfig":
        r = KeyReader(raw)
        vocab, width = r.integer("vocab"), r.integer("width")
        eps = KeyReader(r.raw_value("norm") or {}, "config.json: norm").number("eps")
        emb = KeyReader(r.raw_value("embedding") or {}, "config.json: embedding")
        bigram = None
        if emb.raw_value("bigram") is not None:
            b = KeyReader(emb.raw_value("bigram"), "config.json: embedding.bigram")
            bigram = dict(buckets=b.integer("buckets"), mul_prev=b.integer("mul_prev", minimum=None),
                          mul_cur=b.integer("mul_cur", minimum=None))
        raw_layers = r.raw_value("layers")
        if not isinstance(raw_layers, list) or not raw_layers:
            raise ConfigError(f"config.json: 'layers' must be a non-empty list, found {raw_layers!r}")
        layers: List[Dict[str, Any]] = []
        for i, entry in enumerate(raw_layers):
            where = f"config.json: layers[{i}]"
            e = KeyReader(entry, where)
            kind = e.string("type")
            if kind not in MIXER_TYPES:
                raise ConfigError(f"{where}: type {kind!r} is not one of {list(MIXER_TYPES)}")
            layers.append(dict(type=kind, mixer=_mixer_sizes(e.raw_value("mixer"), where + ".mixer"),
                               mlp=_mlp_sizes(e.raw_value("mlp"), where + ".mlp")))
        for i, layer in enumerate(layers):
            j = layer["mixer"]["kv_from"]
            if j is None:
                continue
            where = f"config.json: layers[{i}].mixer"
            if j >= i or layers[j]["mixer"]["kv_from"] is not None:
                raise ConfigError(f"{where}: 'kv_from' {j} must name an earlier layer with keys and values of its own")
            mine, theirs = layer["mixer"], layers[j]["mixer"]
            for key in ("heads", "kv_heads", "dim", "vdim", "rot"):
                if mine[key] != theirs[key]:
                    raise ConfigError(f"{where}: '{key}' {mine[key]} differs from that of layer {j} ({theirs[key]}), "
                                      "whose keys and values this layer reads")
        return cls(vocab, width, eps, layers, embedding_scale=emb.number("scale", default=1.0, positive=False), bigram=bigram,
                   logit_scale=r.number("logit_scale", default=1.0, positive=False), init_std=raw.get("init_std"))

    def to_dict(self) -> Dict[str, Any]:
        """A config.json that reads back to this configuration."""
        embedding: Dict[str, Any] = dict(scale=self.embedding_scale)
        if self.bigram is not None:
            embedding["bigram"] = dict(self.bigram)
        d = dict(architecture=ARCHITECTURE, vocab=self.vocab, width=self.width, norm=dict(eps=self.eps), embedding=embedding,
                 logit_scale=self.logit_scale, layers=copy.deepcopy(self.layers))
        if self.init_std is not None:
            d["init_std"] = self.init_std
        return d

    # ---------------------------------------------------------------- description
    def _norm(self, name: str, **more: Any) -> PartSpec:
        return PartSpec("group_rmsnorm", dict(size=self.width, eps=self.eps, groups=1, weight=name, **more))

    def _mixer(self, m: Dict[str, Any]) -> PartSpec:
        mask, rot = m["mask"] or {}, m["rot"]
        position = None if rot is None else PartSpec("rope_half", dict(dims=rot["dims"], base=rot["base"], scaling=None,
                                                                       max_positions=MAX_POSITIONS))
        return PartSpec("normed_attention", dict(
            hidden_size=self.width, n_heads=m["heads"], n_kv_heads=m["kv_heads"], dim=m["dim"], v_dim=m["vdim"],
            scale=m["scale"], eps=self.eps, biases=True, out_bias=False, qk_norm=True, qk_gains=True, position=position,
            window=mask.get("size"), keep_first=mask.get("keep_first") or None, shared_kv=m["kv_from"] is not None,
            sink="mix.sink", q="mix.q", k="mix.k", v="mix.v", o="mix.o", q_norm="mix.q.norm", k_norm="mix.k.norm"))

    def _feed_forward(self, mlp: Dict[str, Any]) -> PartSpec:
        if mlp["kind"] == "dense":
            return PartSpec("swiglu", dict(hidden_size=self.width, intermediate_size=mlp["ff"], gate="mlp.gate", up="mlp.up",
                                           down="mlp.down", suffix="", limit=mlp["limit"]))
        r = mlp["router"]
        return PartSpec("grouped_moe", dict(
            hidden_size=self.width, intermediate_size=mlp["expert"]["ff"], n_experts=r["experts"], identity=r["identity"],
            top=r["top"], act="silu", score="softmax", normalize=False, correction="mlp.correction", router="mlp.router",
            expert="mlp.e{}"))

    def model_spec(self) -> ModelSpec:
        blocks, schedule = [], []
        for i, layer in enumerate(self.layers):
            norms = {"mixer_out": self._norm("norm1")}
            if layer["mlp"] is not None:
                norms["feed_forward_out"] = self._norm("norm2")
            blocks.append(BlockSpec(kind="branch_norm", prefix=f"l{i}.", mixer=self._mixer(layer["mixer"]),
                                    feed_forward=None if layer["mlp"] is None else self._feed_forward(layer["mlp"]),
                                    norms=norms))
            # a layer that reads another layer's keys and values runs on that layer's cache entry and writes nothing
            j = layer["mixer"]["kv_from"]
            schedule.append(RunEntry(block=i, cache=i if j is None else j, writes_cache=j is None))
        table = dict(name="embed", vocab_size=self.vocab, hidden_size=self.width, scale=self.embedding_scale)
        embedding = PartSpec("token_embedding", table) if self.bigram is None else \
            PartSpec("token_pair_embedding", dict(table, pairs="bigram", **self.bigram))
        # the logits' scale is a factor of the last norm's gain
        return ModelSpec(hidden_size=self.width, vocab_size=self.vocab, embedding=embedding, head_name="head",
                         final_norm=self._norm("final.norm", gain_scale=self.logit_scale), blocks=tuple(blocks),
                         schedule=tuple(schedule), max_positions=MAX_POSITIONS, stop_tokens=())

    def random_init_std(self, tensor_name: str) -> float:
        """Standard deviation for random weights: `init_std` where the configuration gives one, else
        1/sqrt(inputs) for matrices, 1 for the tables' rows and 0.3 for everything else."""
        if self.init_std is not None:
            return float(self.init_std)
        if tensor_name in ("embed", "bigram"):
            return 1.0
        if self._fan_in is None:
            from ..engine.model import expected_tensors
            self._fan_in = {n: (ts.shape[1] if len(ts.shape) == 2 else 0)
                            for n, ts in expected_tensors(self.model_spec()).items()}
        fan = self._fan_in.get(tensor_name, 0)
        return 1.0 / math.sqrt(fan) if fan else 0.3
