"""Linear attention with a decay per key channel and token, in two designs.

Linear attention whose forget gate a sets the input gate as well, 1 - a (HGRN2): a fixed-size matrix
state per sequence and head instead of keys and values.

q = silu(Wq x) (heads x dim), v = Wv x (heads x v_dim), a = l + (1 - l) sigmoid(Wf x + b) per head and key
channel, with learned lower bounds l; per head S_t = diag(a_t) S_(t-1) + (1 - a_t) v_t^T from S = 0 at a
sequence's start, o_t = S_t^T q_t, no key and no other scale; every head's o is RMS-normed over its v_dim
values with a gain vector shared by the heads, the heads side by side are multiplied by `out_scale` and
projected by Wo.  The state is float32 `[heads][dim][v_dim]` per cache slot; gates, state, products and sums
are 32-bit in both run types.

Gated linear attention: q = Wq x, k = Wk x (heads x dim), v = Wv x (heads x v_dim), a = sigmoid(A2 A1 x + b)^(1/tau)
per head and key channel; per head S_t = diag(a_t) S_(t-1) + k_t v_t^T, o_t = S_t^T q_t dim^(-1/2); every head's o is
RMS-normed over its v_dim values with a gain vector shared by the heads, multiplied by silu(Wg x) and projected by
Wo.  q | k | v | g and A1 x come from one product; A2's part is taken in 32-bit behind it.
"""
from __future__ import annotations

import torch

from ..cache.paged import StateRequest
from ..kernels import ops
from ..weights.loader import TensorSpec
from .base import Mixer, register_mixer
from .linear import Linear

# a step whose longest sequence brings more tokens than this walks its sequences in chunks side by side
CHUNKED_FROM = ops.GR_CHUNK


def gr_chunks_of(ctx):
    """The step's chunk table on the device and its number of chunks (made once a step), or None where every
    sequence is walked in one."""
    if ctx.all_decode or ctx.max_new <= CHUNKED_FROM:
        return None
    key = ("gr_chunks",)
    if key not in ctx._memo:
        table, count = ops.gr_chunks(ctx.host_new)
        ctx._memo[key] = (table.to(ctx.cu_seqlens.device), count)
    return ctx._memo[key]


@register_mixer("gated_recurrence")
class GatedRecurrence(Mixer):
    """params: hidden_size, n_heads, dim, v_dim, eps (of the norm over a head), out_scale, q, f, f_bias, lower, v,
    norm, o (tensor names)."""

    takes_normed = True
    can_overwrite = True

    def __init__(self, spec, rt):
        super().__init__(spec, rt)
        p = spec.params
        self.hidden, self.nh, self.dim, self.vdim = (int(p[k]) for k in ("hidden_size", "n_heads", "dim", "v_dim"))
        self.eps = float(p["eps"])
        self.out_scale = float(p.get("out_scale", 1.0))
        if self.dim > 256:
            raise ValueError(f"gated_recurrence: key width {self.dim} is beyond what the kernels take (256)")
        self.names = {k: p[k] for k in ("q", "f", "f_bias", "lower", "v", "norm", "o")}
        self.proj = self.o = self.norm_weight = self.lower = None

    def tensor_specs(self):
        n, H = self.names, self.nh
        return {n["q"]: TensorSpec((H * self.dim, self.hidden)), n["f"]: TensorSpec((H * self.dim, self.hidden)),
                n["f_bias"]: TensorSpec((H * self.dim,)), n["lower"]: TensorSpec((H * self.dim,), init="halves"),
                n["v"]: TensorSpec((H * self.vdim, self.hidden)), n["norm"]: TensorSpec((self.vdim,), init="ones"),
                n["o"]: TensorSpec((self.hidden, H * self.vdim))}

    def load(self, get):
        n = self.names
        self.proj = Linear.stacked([get(n["q"]), get(n["f"]), get(n["v"])], [None, get(n["f_bias"]), None])   # one product
        self.o = Linear(get(n["o"]))
        self.norm_weight = get(n["norm"]).to(torch.float32).contiguous()
        self.lower = get(n["lower"]).to(torch.float32).contiguous()

    def cache_request(self):
        return StateRequest((self.nh, self.dim, self.vdim), torch.float32)

    def decode_copies(self, make: bool, min_row_length: int = 0) -> int:
        return self.proj.decode_copy(make, min_row_length) + self.o.decode_copy(make, min_row_length)

    def forward(self, x, h, ctx, entry: int, writes_cache: bool, accumulate: bool = True) -> None:
        state = ctx.cache.state(entry)
        proj = self.proj(x, out_dtype=torch.float32)
        n, hv = proj.shape[0], self.nh * self.vdim
        o = torch.empty((n, hv), dtype=torch.float32, device=proj.device)
        ops.gated_scan(proj, self.lower, ctx.cu_seqlens, ctx.slot_ids, state, o, self.nh, self.dim, self.vdim, gr_chunks_of(ctx))
        y = torch.empty((n, hv), dtype=self.rt.dtype, device=proj.device)
        ops.head_rmsnorm(o, self.norm_weight, self.eps, y, self.nh, self.out_scale)
        self.o(y, out=h, accumulate=accumulate)


@register_mixer("gated_linear_attention")
class GatedLinearAttention(Mixer):
    """params: hidden_size, n_heads, dim, v_dim, rank (of the decay's product), tau, eps (of the norm over a head), q, k,
    v, g, a1, a2, a2_bias, norm, o (tensor names)."""

    can_overwrite = True

    def __init__(self, spec, rt):
        super().__init__(spec, rt)
        p = spec.params
        self.hidden, self.nh, self.dim, self.vdim, self.rank = (
            int(p[k]) for k in ("hidden_size", "n_heads", "dim", "v_dim", "rank"))
        self.tau, self.eps = float(p["tau"]), float(p["eps"])
        if self.dim > 256:
            raise ValueError(f"gated_linear_attention: key width {self.dim} is beyond what the kernels take (256)")
        self.names = {k: p[k] for k in ("q", "k", "v", "g", "a1", "a2", "a2_bias", "norm", "o")}
        self.proj = self.o = self.norm_weight = self.a2 = self.a2_bias = None

    def tensor_specs(self):
        n, C, O = self.names, self.nh * self.dim, self.nh * self.vdim
        return {n["q"]: TensorSpec((C, self.hidden)), n["k"]: TensorSpec((C, self.hidden)), n["v"]: TensorSpec((O, self.hidden)),
                n["g"]: TensorSpec((O, self.hidden)), n["o"]: TensorSpec((self.hidden, O)),
                n["norm"]: TensorSpec((self.vdim,), init="ones"), n["a1"]: TensorSpec((self.rank, self.hidden)),
                n["a2"]: TensorSpec((C, self.rank)), n["a2_bias"]: TensorSpec((C,))}

    def load(self, get):
        n = self.names
        self.proj = Linear.stacked([get(n[k]) for k in ("q", "k", "v", "g", "a1")])      # one product
        self.o = Linear(get(n["o"]))
        self.norm_weight = get(n["norm"]).to(torch.float32).contiguous()
        self.a2 = get(n["a2"]).to(torch.float32).t().contiguous()      # [rank][heads dim], as the kernels read it
        self.a2_bias = get(n["a2_bias"]).to(torch.float32).contiguous()

    def cache_request(self):
        return StateRequest((self.nh, self.dim, self.vdim), torch.float32)

    def decode_copies(self, make: bool, min_row_length: int = 0) -> int:
        return self.proj.decode_copy(make, min_row_length) + self.o.decode_copy(make, min_row_length)

    def forward(self, x, h, ctx, entry: int, writes_cache: bool, accumulate: bool = True) -> None:
        state = ctx.cache.state(entry)
        proj = self.proj(x, out_dtype=torch.float32)
        n, C, O = proj.shape[0], self.nh * self.dim, self.nh * self.vdim
        o = torch.empty((n, O), dtype=torch.float32, device=proj.device)
        ops.low_rank_scan(proj, self.a2, self.a2_bias, 2 * C + 2 * O, self.tau, self.dim ** -0.5, ctx.cu_seqlens, ctx.slot_ids,
                          state, o, self.nh, self.dim, self.vdim, gr_chunks_of(ctx))
        y = torch.empty((n, O), dtype=self.rt.dtype, device=proj.device)
        ops.gated_head_norm(o, proj, 2 * C + O, self.norm_weight, self.eps, y, self.nh, "silu")
        self.o(y, out=h, accumulate=accumulate)
