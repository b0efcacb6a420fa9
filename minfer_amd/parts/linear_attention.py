"""Linear attention with a decay per head: a fixed-size matrix state per sequence and head instead of keys and
values, in three designs.

"Lightning" attention:
q = silu(Wq x), k = silu(Wk x) (heads x dim), v = silu(Wv x) (heads x v_dim); per head
S_t = decay_h S_(t-1) + k_t v_t^T from S = 0 at a sequence's start, o_t = S_t^T q_t, no other scale;
the heads side by side are RMS-normed together with a gain vector, multiplied by sigmoid(Wg x) and
projected by Wo.  The state is float32 `[heads][dim][v_dim]` per cache slot; state, decays, products
and sums are 32-bit in both run types.

Retention: q = Wq x and k = Wk x (heads x dim) turned by the token's position (a rotation in halves), k further times
dim^(-1/2), v = Wv x; S_t = decay_h S_(t-1) + k_t v_t^T, o_t = S_t^T q_t; every head's o over its root mean square
(no gain), times silu(Wg x), projected by Wo.

Matrix memory (mLSTM): q = Wq x dim^(-1/2), k = Wk x, v = Wv x, and per head two gates from the token, a log input
gate i = cap tanh((wi x + bi) / cap) and a log forget gate f = logsigmoid(cap tanh((wf x + bf) / cap)).  With a running
maximum m from 0, m_t = max(f + m_(t-1), i): S_t = exp(f + m_(t-1) - m_t) S_(t-1) + exp(i - m_t) k_t v_t^T, n_t likewise
with k alone, o_t = S_t^T q_t / (max(|n_t . q_t|, exp(-m_t)) + 1e-6); every head's o over its root mean square, times a
gain vector as long as the heads side by side, times sigmoid(Wg x), projected by Wo.  S, n and m are the slot's state.
"""
from __future__ import annotations

import torch

from ..cache.paged import StateRequest
from ..kernels import ops
from ..weights.loader import TensorSpec
from .base import Mixer, POSITIONS, make_part, register_mixer
from .linear import Linear

# a step whose longest sequence brings more tokens than this walks its sequences in chunks side by side
CHUNKED_FROM = ops.LA_CHUNK


def la_chunks_of(ctx, dim: int):
    """The step's chunk table on the device and its number of chunks (made once a step), or None where every
    sequence is walked in one."""
    if ctx.all_decode or ctx.max_new <= CHUNKED_FROM or dim > ops.LA_CHUNKED_MAX_DIM:
        return None
    key = ("la_chunks",)
    if key not in ctx._memo:
        table, count = ops.la_chunks(ctx.host_new)
        ctx._memo[key] = (table.to(ctx.cu_seqlens.device), count)
    return ctx._memo[key]


@register_mixer("lightning_attention")
class LightningAttention(Mixer):
    """params: hidden_size, n_heads, dim, v_dim, decays (one number per head), eps (of the norm over
    the heads), q, k, v, g, o, norm (tensor names)."""

    takes_normed = True
    can_overwrite = True

    def __init__(self, spec, rt):
        super().__init__(spec, rt)
        p = spec.params
        self.hidden, self.nh, self.dim, self.vdim = (int(p[k]) for k in ("hidden_size", "n_heads", "dim", "v_dim"))
        self.eps = float(p["eps"])
        self.decay_values = [float(d) for d in p["decays"]]
        if len(self.decay_values) != self.nh:
            raise ValueError(f"lightning_attention: {len(self.decay_values)} decays for {self.nh} heads")
        if self.dim > 256:
            raise ValueError(f"lightning_attention: key width {self.dim} is beyond what the kernels take (256)")
        self.names = {k: p[k] for k in ("q", "k", "v", "g", "o", "norm")}
        self.proj = self.o = self.norm_weight = self.decays = None

    def tensor_specs(self):
        n, H = self.names, self.nh
        return {n["q"]: TensorSpec((H * self.dim, self.hidden)), n["k"]: TensorSpec((H * self.dim, self.hidden)),
                n["v"]: TensorSpec((H * self.vdim, self.hidden)), n["g"]: TensorSpec((H * self.vdim, self.hidden)),
                n["o"]: TensorSpec((self.hidden, H * self.vdim)), n["norm"]: TensorSpec((H * self.vdim,), init="ones")}

    def load(self, get):
        n = self.names
        self.proj = Linear.stacked([get(n["q"]), get(n["k"]), get(n["v"]), get(n["g"])])     # one product
        self.o = Linear(get(n["o"]))
        self.norm_weight = get(n["norm"]).to(torch.float32).contiguous()
        self.decays = torch.tensor(self.decay_values, dtype=torch.float32, device=self.norm_weight.device)

    def cache_request(self):
        return StateRequest((self.nh, self.dim, self.vdim), torch.float32)

    def decode_copies(self, make: bool, min_row_length: int = 0) -> int:
        return self.proj.decode_copy(make, min_row_length) + self.o.decode_copy(make, min_row_length)

    def forward(self, x, h, ctx, entry: int, writes_cache: bool, accumulate: bool = True) -> None:
        state = ctx.cache.state(entry)
        proj = self.proj(x, out_dtype=torch.float32)
        n, hv = proj.shape[0], self.nh * self.vdim
        o = torch.empty((n, hv), dtype=torch.float32, device=proj.device)
        ops.lightning_scan(proj, ctx.cu_seqlens, ctx.slot_ids, self.decays, state, o, self.nh, self.dim, self.vdim,
                           la_chunks_of(ctx, self.dim))
        y = torch.empty((n, hv), dtype=self.rt.dtype, device=proj.device)
        ops.gated_rmsnorm(o, proj, 2 * self.nh * self.dim + hv, self.norm_weight, self.eps, y)
        self.o(y, out=h, accumulate=accumulate)


@register_mixer("retention")
class Retention(Mixer):
    """params: hidden_size, n_heads, dim, v_dim, decays (one number per head), eps (of the norm over a head), position
    (PartSpec of a rotation in halves with `half_tables`, or None), q, k, v, g, o (tensor names)."""

    can_overwrite = True

    def __init__(self, spec, rt):
        super().__init__(spec, rt)
        p = spec.params
        self.hidden, self.nh, self.dim, self.vdim = (int(p[k]) for k in ("hidden_size", "n_heads", "dim", "v_dim"))
        self.eps = float(p["eps"])
        self.decay_values = [float(d) for d in p["decays"]]
        if len(self.decay_values) != self.nh:
            raise ValueError(f"retention: {len(self.decay_values)} decays for {self.nh} heads")
        if self.dim > 256:
            raise ValueError(f"retention: key width {self.dim} is beyond what the kernels take (256)")
        self.position = None
        if p.get("position") is not None:
            self.position = make_part(POSITIONS, p["position"], rt, "position encoding")
            if not hasattr(self.position, "half_tables") or self.position.dims > self.dim:
                raise ValueError(f"retention: the position encoding must be a rotation in halves over at most {self.dim} values")
        self.names = {k: p[k] for k in ("q", "k", "v", "g", "o")}
        self.proj = self.o = self.decays = None

    def tensor_specs(self):
        n, C, O = self.names, self.nh * self.dim, self.nh * self.vdim
        return {n["q"]: TensorSpec((C, self.hidden)), n["k"]: TensorSpec((C, self.hidden)), n["v"]: TensorSpec((O, self.hidden)),
                n["g"]: TensorSpec((O, self.hidden)), n["o"]: TensorSpec((self.hidden, O))}

    def load(self, get):
        n = self.names
        self.proj = Linear.stacked([get(n[k]) for k in ("q", "k", "v", "g")])     # one product
        self.o = Linear(get(n["o"]))
        self.decays = torch.tensor(self.decay_values, dtype=torch.float32, device=self.o.weight.device)

    def cache_request(self):
        return StateRequest((self.nh, self.dim, self.vdim), torch.float32)

    def decode_copies(self, make: bool, min_row_length: int = 0) -> int:
        return self.proj.decode_copy(make, min_row_length) + self.o.decode_copy(make, min_row_length)

    def prepare(self, max_len: int) -> None:
        if self.position is not None:
            self.position.prepare(max_len)

    def forward(self, x, h, ctx, entry: int, writes_cache: bool, accumulate: bool = True) -> None:
        state = ctx.cache.state(entry)
        proj = self.proj(x, out_dtype=torch.float32)
        n, C, O = proj.shape[0], self.nh * self.dim, self.nh * self.vdim
        o = torch.empty((n, O), dtype=torch.float32, device=proj.device)
        tables = None if self.position is None else self.position.half_tables(ctx.max_len)
        ops.retention_scan(proj, ctx.cu_seqlens, ctx.slot_ids, self.decays, tables, ctx.positions, 1.0, self.dim ** -0.5, state, o,
                           self.nh, self.dim, self.vdim, la_chunks_of(ctx, self.dim))
        y = torch.empty((n, O), dtype=self.rt.dtype, device=proj.device)
        ops.gated_head_norm(o, proj, 2 * C + O, None, self.eps, y, self.nh, "silu")
        self.o(y, out=h, accumulate=accumulate)


@register_mixer("matrix_memory")
class MatrixMemory(Mixer):
    """params: hidden_size, n_heads, dim, v_dim, gate_cap, eps (of the norm over a head), q, k, v, g, i, i_bias, f, f_bias,
    norm, o (tensor names)."""

    can_overwrite = True

    def __init__(self, spec, rt):
        super().__init__(spec, rt)
        p = spec.params
        self.hidden, self.nh, self.dim, self.vdim = (int(p[k]) for k in ("hidden_size", "n_heads", "dim", "v_dim"))
        self.cap, self.eps = float(p["gate_cap"]), float(p["eps"])
        if self.dim > 256 or not self.cap > 0:
            raise ValueError(f"matrix_memory: key width {self.dim} (at most 256), gate cap {self.cap} (above 0)")
        self.names = {k: p[k] for k in ("q", "k", "v", "g", "i", "i_bias", "f", "f_bias", "norm", "o")}
        self.proj = self.o = self.norm_weight = None

    def tensor_specs(self):
        n, C, O = self.names, self.nh * self.dim, self.nh * self.vdim
        return {n["q"]: TensorSpec((C, self.hidden)), n["k"]: TensorSpec((C, self.hidden)), n["v"]: TensorSpec((O, self.hidden)),
                n["g"]: TensorSpec((O, self.hidden)), n["o"]: TensorSpec((self.hidden, O)),
                n["norm"]: TensorSpec((O,), init="ones"),
                n["i"]: TensorSpec((self.nh, self.hidden)), n["i_bias"]: TensorSpec((self.nh,)),
                n["f"]: TensorSpec((self.nh, self.hidden)), n["f_bias"]: TensorSpec((self.nh,))}

    def load(self, get):
        n = self.names
        self.proj = Linear.stacked([get(n[k]) for k in ("q", "k", "v", "g", "i", "f")],
                                   [None, None, None, None, get(n["i_bias"]), get(n["f_bias"])])      # one product
        self.o = Linear(get(n["o"]))
        self.norm_weight = get(n["norm"]).to(torch.float32).contiguous()

    def cache_request(self):
        return StateRequest((ops.memory_state_len(self.nh, self.dim, self.vdim),), torch.float32)

    def decode_copies(self, make: bool, min_row_length: int = 0) -> int:
        return self.proj.decode_copy(make, min_row_length) + self.o.decode_copy(make, min_row_length)

    def forward(self, x, h, ctx, entry: int, writes_cache: bool, accumulate: bool = True) -> None:
        state = ctx.cache.state(entry)
        proj = self.proj(x, out_dtype=torch.float32)
        n, C, O = proj.shape[0], self.nh * self.dim, self.nh * self.vdim
        o = torch.empty((n, O), dtype=torch.float32, device=proj.device)
        den = torch.empty((n, self.nh), dtype=torch.float32, device=proj.device)
        floor = torch.empty_like(den)
        ops.memory_scan(proj, 2 * C + 2 * O, 2 * C + 2 * O + self.nh, self.cap, self.dim ** -0.5, ctx.cu_seqlens, ctx.slot_ids,
                        state, o, den, floor, self.nh, self.dim, self.vdim, la_chunks_of(ctx, self.dim))
        y = torch.empty((n, O), dtype=self.rt.dtype, device=proj.device)
        ops.gated_head_norm(o, proj, 2 * C + O, self.norm_weight, self.eps, y, self.nh, "sigmoid", den=den, floor=floor)
        self.o(y, out=h, accumulate=accumulate)
