"""Rofizen: a decoder whose stream is layer-normed behind every sum, x <- L1(a x + mixer(x)), x <- L2(a x + ff(x)) (the
gain times the deviations over their root mean square; no bias), with the token's table row times a scale in front.
A mixer is
  "gla":       gated linear attention: a state with a decay per key channel, sigmoid(A2 A1 x + b)^(1/tau);
  "retention": linear attention with a fixed decay per head, queries and keys rotated in halves;
  "parallel":  half the sum of two results, each RMS-normed with a gain of its own: "left", causal grouped-query
               softmax attention (biases, q and k normed over their whole projections, a query temperature that grows
               with the position, capped scores less a slope 2^(-8 (h + 1) / heads) times the distance), and "right",
               a matrix memory with capped exponential gates under a running maximum.
A feed-forward is dense with the square of relu, or silu experts that a table picks by the token's id beside a shared
expert weighed by a sigmoid, or absent.

config.json: `architecture` = "Rofizen"; `vocab`, `width`; `embedding` = {scale}; `postln_alpha`; `norm` = {eps};
`layers`, a list of {type, mixer: {...}, mlp: {...} or null}.
Mixer sizes: gla {heads, dim, vdim, tau}; retention {heads, dim, vdim, decay: one number per head, rot: {base, dims}};
parallel {left: {heads, kv_heads, dim, vdim, scale, softcap, q_temp: {coef, every}}, right: {heads, dim, vdim,
gate_cap}} (softcap and q_temp may be absent).
mlp: {kind: "dense", ff} or {kind: "moe", expert: {ff}, router: {experts, top}, shared: {ff} or absent}.
The rank of a gla layer's decay is the first size of its tensor `l<i>.mix.a1` (`rank` in a configuration that is
written without a file).
Tensors: embed, l<i>.norm1, l<i>.norm2, l<i>.mix.*, l<i>.mlp.*, final.norm, head.
"""
from __future__ import annotations

import copy
import math
from typing import Any, Dict, List, Mapping, Optional, Sequence, Tuple

from .base import ConfigError, KeyReader
from ..parts.spec import BlockSpec, ModelSpec, PartSpec, straight_schedule

ARCHITECTURE = "Rofizen"
MIXER_TYPES = ("parallel", "gla", "retention")
MAX_POSITIONS = 1 << 20      # the design names no bound; rotation tables grow on demand up to here
PAIR_SCALE = 0.5             # of the two normed results of a "parallel" mixer


def _gla(raw: Any, where: str) -> Dict[str, Any]:
    r = KeyReader(raw, where)
    return dict(heads=r.integer("heads"), dim=r.integer("dim"), vdim=r.integer("vdim"), tau=r.number("tau"),
                rank=r.integer("rank", default=None))


def _retention(raw: Any, where: str) -> Dict[str, Any]:
    r = KeyReader(raw, where)
    out = dict(heads=r.integer("heads"), dim=r.integer("dim"), vdim=r.integer("vdim"))
    decay = r.raw_value("decay")
    if not isinstance(decay, list) or len(decay) != out["heads"] or \
            any(isinstance(d, bool) or not isinstance(d, (int, float)) or not 0.0 < d <= 1.0 for d in decay):
        raise ConfigError(f"{where}: 'decay' must hold {out['heads']} numbers above 0 and at most 1, found {decay!r}")
    out["decay"] = [float(d) for d in decay]
    k = KeyReader(r.raw_value("rot") or {}, where + ".rot")
    dims = k.integer("dims")
    if dims % 2 or dims > out["dim"]:
        raise ConfigError(f"{where}.rot: 'dims' must be even and at most {out['dim']}, found {dims}")
    out["rot"] = dict(base=k.number("base"), dims=dims)
    return out


def _parallel(raw: Any, where: str) -> Dict[str, Any]:
    p = KeyReader(raw, where)
    left = KeyReader(p.raw_value("left") or {}, where + ".left")
    right = KeyReader(p.raw_value("right") or {}, where + ".right")
    lf = dict(heads=left.integer("heads"), kv_heads=left.integer("kv_heads"), dim=left.integer("dim"), vdim=left.integer("vdim"),
              scale=left.number("scale"), softcap=None, q_temp=None)
    if lf["heads"] % lf["kv_heads"]:
        raise ConfigError(f"{where}.left: 'heads' {lf['heads']} is not a multiple of 'kv_heads' {lf['kv_heads']}")
    if left.raw_value("softcap") is not None:
        lf["softcap"] = left.number("softcap")
    if left.raw_value("q_temp") is not None:
        t = KeyReader(left.raw_value("q_temp"), where + ".left.q_temp")
        lf["q_temp"] = dict(coef=t.number("coef", positive=False), every=t.integer("every"))
    return dict(left=lf, right=dict(heads=right.integer("heads"), dim=right.integer("dim"), vdim=right.integer("vdim"),
                                    gate_cap=right.number("gate_cap")))


_MIXERS = {"gla": _gla, "retention": _retention, "parallel": _parallel}


def _mlp_sizes(raw: Any, where: str) -> Optional[Dict[str, Any]]:
    if raw is None:
        return None
    m = KeyReader(raw, where)
    kind = m.string("kind")
    if kind == "dense":
        return dict(kind="dense", ff=m.integer("ff"))
    if kind != "moe":
        raise ConfigError(f"{where}: kind {kind!r} is not one of ['dense', 'moe']")
    e = KeyReader(m.raw_value("expert") or {}, where + ".expert")
    r = KeyReader(m.raw_value("router") or {}, where + ".router")
    out = dict(kind="moe", expert=dict(ff=e.integer("ff")), router=dict(experts=r.integer("experts"), top=r.integer("top")))
    if out["router"]["top"] > out["router"]["experts"]:
        raise ConfigError(f"{where}.router: 'top' {out['router']['top']} of {out['router']['experts']} experts")
    if m.raw_value("shared") is not None:
        out["shared"] = dict(ff=KeyReader(m.raw_value("shared"), where + ".shared").integer("ff"))
    return out


class RofizenConfig:
    architecture = ARCHITECTURE

    def __init__(self, vocab: int, width: int, eps: float, alpha: float, layers: List[Dict[str, Any]],
                 embedding_scale: float = 1.0, init_std: Optional[float] = None):
        self.vocab, self.width, self.eps, self.alpha = vocab, width, eps, alpha
        self.layers, self.embedding_scale, self.init_std = layers, embedding_scale, init_std
        self._fan_in: Optional[Dict[str, int]] = None

    # ---------------------------------------------------------------- reading
    @classmethod
    def from_dict(cls, raw: Dict[str, Any]) -> "RofizenConfig":
        r = KeyReader(raw)
        vocab, width = r.integer("vocab"), r.integer("width")
        eps = KeyReader(r.raw_value("norm") or {}, "config.json: norm").number("eps")
        scale = KeyReader(r.raw_value("embedding") or {}, "config.json: embedding").number("scale", default=1.0)
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
            layers.append(dict(type=kind, mixer=_MIXERS[kind](e.raw_value("mixer") or {}, where + ".mixer"),
                               mlp=_mlp_sizes(e.raw_value("mlp"), where + ".mlp")))
        return cls(vocab, width, eps, r.number("postln_alpha"), layers, embedding_scale=scale, init_std=raw.get("init_std"))

    def adopt_tensor_shapes(self, shapes: Mapping[str, Sequence[int]]) -> None:
        """Sizes that only the tensors give: the rank of every gla layer's decay."""
        for i, layer in enumerate(self.layers):
            if layer["type"] != "gla" or layer["mixer"].get("rank") is not None:
                continue
            shape = shapes.get(f"l{i}.mix.a1")
            if shape is None or len(shape) != 2 or shape[0] < 1:
                raise ConfigError(f"config.json: layers[{i}].mixer: the first size of l{i}.mix.a1 gives the rank of the decay; "
                                  f"found shape {None if shape is None else list(shape)}")
            layer["mixer"]["rank"] = int(shape[0])

    def to_dict(self) -> Dict[str, Any]:
        """A config.json that reads back to this configuration."""
        d = dict(architecture=ARCHITECTURE, vocab=self.vocab, width=self.width, norm=dict(eps=self.eps),
                 embedding=dict(scale=self.embedding_scale), postln_alpha=self.alpha, layers=copy.deepcopy(self.layers))
        if self.init_std is not None:
            d["init_std"] = self.init_std
        return d

    # ---------------------------------------------------------------- description
    def _norm(self, name: str) -> PartSpec:
        return PartSpec("layernorm", dict(size=self.width, eps=self.eps, weight=name))

    def _mixer(self, i: int, layer: Dict[str, Any]) -> PartSpec:
        m, kind = layer["mixer"], layer["type"]
        common = dict(hidden_size=self.width, eps=self.eps)
        if kind == "gla":
            if m.get("rank") is None:
                raise ConfigError(f"config.json: layers[{i}].mixer: the rank of the decay is the first size of l{i}.mix.a1; "
                                  "without a file, give 'rank'")
            return PartSpec("gated_linear_attention", dict(
                common, n_heads=m["heads"], dim=m["dim"], v_dim=m["vdim"], tau=m["tau"], rank=m["rank"],
                a2_bias="mix.a2.b", **{k: "mix." + k for k in ("q", "k", "v", "g", "o", "a1", "a2", "norm")}))
        if kind == "retention":
            return PartSpec("retention", dict(
                common, n_heads=m["heads"], dim=m["dim"], v_dim=m["vdim"], decays=tuple(m["decay"]),
                position=PartSpec("rope_half", dict(dims=m["rot"]["dims"], base=m["rot"]["base"], scaling=None,
                                                    max_positions=MAX_POSITIONS)),
                **{k: "mix." + k for k in ("q", "k", "v", "g", "o")}))
        lf, rg = m["left"], m["right"]
        H = lf["heads"]
        left = PartSpec("normed_attention", dict(
            common, n_heads=H, n_kv_heads=lf["kv_heads"], dim=lf["dim"], v_dim=lf["vdim"], scale=lf["scale"],
            biases=True, row_norm=True, cap=lf["softcap"], q_temperature=lf["q_temp"],
            slopes=tuple(2.0 ** (-8.0 * (h + 1) / H) for h in range(H)),
            q="q", k="k", v="v", o="o", q_norm="q.norm", k_norm="k.norm"))
        right = PartSpec("matrix_memory", dict(
            common, n_heads=rg["heads"], dim=rg["dim"], v_dim=rg["vdim"], gate_cap=rg["gate_cap"], i_bias="i.b", f_bias="f.b",
            **{k: k for k in ("q", "k", "v", "g", "i", "f", "norm", "o")}))
        return PartSpec("side_by_side_normed", dict(
            common, left=left, right=right, left_prefix="mix.left.", right_prefix="mix.right.", left_norm="mix.left.out",
            right_norm="mix.right.out", scale=PAIR_SCALE))

    def _feed_forward(self, mlp: Dict[str, Any]) -> PartSpec:
        if mlp["kind"] == "dense":
            return PartSpec("dense_relu2", dict(hidden_size=self.width, intermediate_size=mlp["ff"], up="mlp.up", down="mlp.down"))
        shared = None
        if mlp.get("shared") is not None:
            shared = dict(stem="mlp.shared", weight="mlp.shared.sg", intermediate_size=mlp["shared"]["ff"])
        return PartSpec("table_moe", dict(
            hidden_size=self.width, intermediate_size=mlp["expert"]["ff"], n_experts=mlp["router"]["experts"],
            top=mlp["router"]["top"], act="silu", expert="mlp.e{}", shared=shared, table="mlp.table", vocab_size=self.vocab))

    def model_spec(self) -> ModelSpec:
        blocks = []
        for i, layer in enumerate(self.layers):
            norms = {"mixer_out": self._norm("norm1")}
            ffn = None
            if layer["mlp"] is not None:
                ffn = self._feed_forward(layer["mlp"])
                norms["feed_forward_out"] = self._norm("norm2")
            blocks.append(BlockSpec(kind="postnorm", prefix=f"l{i}.", mixer=self._mixer(i, layer), feed_forward=ffn,
                                    norms=norms, params=dict(stream_scale=self.alpha)))
        embedding = PartSpec("token_embedding", dict(name="embed", vocab_size=self.vocab, hidden_size=self.width,
                                                     scale=self.embedding_scale))
        return ModelSpec(hidden_size=self.width, vocab_size=self.vocab, embedding=embedding, head_name="head",
                         final_norm=self._norm("final.norm"), blocks=tuple(blocks), schedule=straight_schedule(len(blocks)),
                         max_positions=MAX_POSITIONS, stop_tokens=())

    def ignored_tensors(self) -> Tuple[str, ...]:
        """What a file may hold without the configuration having a use for it: the norm behind a feed-forward that a
        layer does not have."""
        return tuple(f"l{i}.norm2" for i, layer in enumerate(self.layers) if layer["mlp"] is None)

    def random_init_std(self, tensor_name: str) -> float:
        """Standard deviation for random weights: `init_std` where the configuration gives one, else
        1/sqrt(inputs) for matrices, 1 over the embedding's scale for the table's rows and 0.3 for everything else."""
        if self.init_std is not None:
            return float(self.init_std)
        if self._fan_in is None:
            from ..engine.model import expected_tensors
            self._fan_in = {n: (ts.shape[1] if len(ts.shape) == 2 else 0)
                            for n, ts in expected_tensors(self.model_spec()).items()}
        if tensor_name == "embed":
            return 1.0 / self.embedding_scale
        fan = self._fan_in.get(tensor_name, 0)
        return 1.0 / math.sqrt(fan) if fan else 0.3
