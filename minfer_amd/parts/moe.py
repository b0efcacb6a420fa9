"""Mixture-of-experts feed-forwards: with a router that first keeps the best groups of experts, or with a table in
the router's place; and an expert that every token takes besides, where a design has one.

Router: z = Wr x in 32-bit, scores = softmax(z) over all experts; the experts form `groups` equal
groups of neighbours, a group's score is its best expert's, and only experts of the `keep` best groups
can be among the `top` chosen; the chosen experts' scores over their sum are the weights.
With one group (and so all of it kept) the weights are the softmax over the chosen logits alone.  A router may
add a bias per expert to its logits.  A router may also score with sigmoid(z) instead of the softmax, choose
groups and experts by score plus a correction per expert while weighing by the scores themselves, count a group
by the sum of its `group_top` best (corrected) scores, multiply the weights by a scale, and weigh by the chosen
scores as they are, not over their sum.
Experts that hand their input on (`identity` of them, behind the others in the router's order) have no matrices: the
router scores and chooses them like any other, and their output is the token's input.
Expert (no biases): g = min(Wg x, limit), u = clamp(Wu x, -limit, limit), y = g sigmoid(1.702 g) (u + 1),
output Wd y; or, with `act` "silu", the plain gated form y = silu(Wg x) (Wu x).  The result is the weighted sum
of the chosen experts' outputs.

Table: the token's id picks its experts from a table `[vocab][top]` of expert numbers, each weighing 1 / top; the
stream plays no part in the choice, so the host knows it too and a prompt's step waits for nothing.

Shared expert: silu(Wg x) (Wu x) times one number per token, sigmoid(w x), then Wd; added to the chosen experts'
sum.  The gate, the up matrix and w are one product.

Two forms, both of which read or multiply only what was chosen.  Steps of few tokens and decode steps (which
may be captured, so nothing may wait for the host): `ops.moe_sparse`, up to 16 tokens a launch, reads every
chosen expert's matrices once.  Steps of many tokens: the (token, choice) pairs are grouped by expert
(`ops.moe_group`; the host reads the experts' counts, the one wait of the step), the tokens' rows are put side by
side expert by expert, the experts' two products run over their rows (all experts in one launch where the sizes
allow it, `ops.linear_grouped`, else an expert at a time), and the rows' results are
added into the stream with the tokens' weights, a token's choices in their order.  (With a table nothing waits:
the host counts the experts' pairs itself.)

A step whose context carries a list under `_memo["route_log"]` gets every routed layer's choices
(`[rows][top]` expert numbers, on the device) appended to it, in run order.
"""
from __future__ import annotations

import numpy as np
import torch

from ..kernels import ops
from ..weights.loader import TensorSpec, WeightError
from .base import FeedForward, register_feed_forward
from .linear import Linear

# steps of at most this many tokens read only the chosen experts' matrices
SPARSE_UP_TO = ops.MOE_SPARSE_TOKENS


class SharedExpert:
    """The expert every token takes, weighed by a sigmoid of its own (plain silu form; widths of its own).
    `spec`: dict(stem, weight, intermediate_size); the matrices are stem + ".gate", ".up", ".down"."""

    PAD = 16        # the product's rows are filled up to a multiple of this

    def __init__(self, spec, hidden: int, rt):
        self.hidden, self.rt = hidden, rt
        self.inter, self.stem, self.weight_name = int(spec["intermediate_size"]), spec["stem"], spec["weight"]
        self.up = self.down = None

    def tensor_specs(self):
        return {self.stem + ".gate": TensorSpec((self.inter, self.hidden)), self.stem + ".up": TensorSpec((self.inter, self.hidden)),
                self.stem + ".down": TensorSpec((self.hidden, self.inter)), self.weight_name: TensorSpec((1, self.hidden))}

    def load(self, get):
        rows = [get(self.stem + ".gate"), get(self.stem + ".up"), get(self.weight_name)]
        fill = -(2 * self.inter + 1) % self.PAD
        if fill:
            rows.append(torch.zeros((fill, self.hidden), dtype=rows[0].dtype, device=rows[0].device))
        self.up = Linear.stacked(rows)
        self.down = Linear(get(self.stem + ".down"))

    def decode_copies(self, make: bool, min_row_length: int = 0) -> int:
        return self.up.decode_copy(make, min_row_length) + self.down.decode_copy(make, min_row_length)

    def forward(self, x, h, accumulate: bool) -> None:
        gu = self.up(x, out_dtype=torch.float32)
        y = torch.empty((x.shape[0], self.inter), dtype=self.rt.dtype, device=x.device)
        ops.gated_expert_act(gu, y)
        self.down(y, out=h, accumulate=accumulate)


class Experts(FeedForward):
    """The experts and their two forms; who takes which is a subclass's `choose`.  params: hidden_size,
    intermediate_size (of one expert), n_experts, top, act ("clamped_swish", the default, with `limit`; or "silu"),
    expert (format of an expert's tensor stem, e.g. "mlp.e{}"; its matrices are stem + ".gate", ".up", ".down"),
    shared (None, or dict(stem, weight, intermediate_size): the expert every token takes), identity (how many expert
    numbers from n_experts on stand for experts that hand their input on; default 0)."""

    can_overwrite = True

    def __init__(self, spec, rt):
        super().__init__(spec, rt)
        p = spec.params
        self.hidden, self.inter, self.ne, self.top = (
            int(p[k]) for k in ("hidden_size", "intermediate_size", "n_experts", "top"))
        act = p.get("act", "clamped_swish")
        if act not in ops.MOE_ACTS:
            raise ValueError(f"{spec.kind}: activation {act!r} is not one of {sorted(ops.MOE_ACTS)}")
        self.act = ops.MOE_ACTS[act]
        self.limit = float(p["limit"]) if act == "clamped_swish" else 0.0
        self.expert_name = p["expert"]
        self.shared = None if p.get("shared") is None else SharedExpert(p["shared"], self.hidden, rt)
        self.identity = int(p.get("identity") or 0)
        self.choices = self.ne + self.identity             # expert numbers that can be chosen
        if self.ne < 1 or self.identity < 0 or not 1 <= self.top <= min(64, self.choices) or self.choices > ops.MOE_MAX_EXPERTS:
            raise ValueError(f"{spec.kind}: {self.top} of {self.ne} + {self.identity} experts chosen (at most 64 of at most "
                             f"{ops.MOE_MAX_EXPERTS})")
        self.gate_up = self.down = None

    def tensor_specs(self):
        s = {}
        for e in range(self.ne):
            stem = self.expert_name.format(e)
            s[stem + ".gate"] = TensorSpec((self.inter, self.hidden))
            s[stem + ".up"] = TensorSpec((self.inter, self.hidden))
            s[stem + ".down"] = TensorSpec((self.hidden, self.inter))
        if self.shared is not None:
            s.update(self.shared.tensor_specs())
        return s

    def load(self, get):
        stems = [self.expert_name.format(e) for e in range(self.ne)]
        # [experts][gate | up][hidden] and [experts][hidden][inter]: an expert's matrices are contiguous slices
        self.gate_up = torch.stack([torch.cat([get(s + ".gate"), get(s + ".up")], dim=0) for s in stems]).contiguous()
        self.down = torch.stack([get(s + ".down") for s in stems]).contiguous()
        self.experts = [(Linear(self.gate_up[e]), Linear(self.down[e])) for e in range(self.ne)]
        if self.shared is not None:
            self.shared.load(get)

    def decode_copies(self, make: bool, min_row_length: int = 0) -> int:
        return 0 if self.shared is None else self.shared.decode_copies(make, min_row_length)

    def choose(self, x, ctx, chosen: torch.Tensor, weights: torch.Tensor) -> None:
        """Fills `chosen` (int32) and `weights` (float32), `[rows][top]`, for the rows x."""
        raise NotImplementedError

    def host_counts(self, ctx):
        """How many of the rows' choices fall on each expert, where the host knows it without waiting, else None."""
        return None

    def forward(self, x, h, ctx, accumulate: bool = True) -> None:
        n, dev = x.shape[0], x.device
        chosen = torch.empty((n, self.top), dtype=torch.int32, device=dev)
        weights = torch.empty((n, self.top), dtype=torch.float32, device=dev)
        self.choose(x, ctx, chosen, weights)
        log = ctx._memo.get("route_log") if ctx is not None else None
        if log is not None:                  # a caller that wants to know: every routed layer's choices, in run order
            log.append(chosen)
        if n == 0:
            return
        if self.shared is not None:
            self.shared.forward(x, h, accumulate)
            accumulate = True
        few = min(SPARSE_UP_TO, max(1, ops.MOE_SPARSE_PAIRS // self.top))
        if (n <= few or (ctx is not None and ctx.all_decode)) and x.dtype == self.gate_up.dtype:
            for t0 in range(0, n, few):      # (slices of a contiguous tensor's rows are contiguous)
                ops.moe_sparse(x[t0:t0 + few], self.gate_up, self.down, chosen[t0:t0 + few], weights[t0:t0 + few],
                               h[t0:t0 + few], self.ne, self.limit, self.act, accumulate=accumulate, hands_on=self.identity > 0)
            return
        rank = torch.empty_like(chosen)
        counts = torch.empty(self.choices, dtype=torch.int32, device=dev)
        ops.moe_group(chosen, self.choices, rank, counts)
        per_expert = self.host_counts(ctx)
        if per_expert is None:
            per_expert = [int(c) for c in counts.cpu()[:self.ne]]      # the step waits for the host here
        starts = [0]
        for c in per_expert:
            starts.append(starts[-1] + c)
        pairs = starts[-1]                   # of experts with matrices; the others' stand nowhere
        handed = dict(x=x, n_real=self.ne) if self.identity else {}
        # one product over all experts' rows where its kernel takes the sizes, else a product an expert
        grouped = pairs > 0 and x.dtype == self.gate_up.dtype and ops.grouped_takes(x.dtype, 2 * self.inter, self.hidden) \
            and ops.grouped_takes(x.dtype, self.hidden, self.inter)
        plans = [ops.grouped_plan(per_expert, 2 * self.inter, self.hidden), ops.grouped_plan(per_expert, self.hidden, self.inter)] \
            if grouped else []
        tables = [ops.row_groups(per_expert, v) for v in plans]
        flat = starts[:-1] + [0] * (-self.ne % 4) + [v for t in tables for row in t for v in row]
        # from pinned memory the copy does not wait for what the stream still has to do
        meta = torch.tensor(flat, dtype=torch.int32, pin_memory=dev.type == "cuda").to(dev, non_blocking=True)
        offsets, at = meta[:self.ne], (self.ne + 3) // 4 * 4
        xs = torch.empty((pairs, self.hidden), dtype=x.dtype, device=dev)
        ops.moe_gather(x, chosen, rank, offsets, xs, n_real=self.ne if self.identity else None)
        gu = torch.empty((pairs, 2 * self.inter), dtype=torch.float32, device=dev)
        y = torch.empty((pairs, self.inter), dtype=self.rt.dtype, device=dev)
        rows = torch.empty((pairs, self.hidden), dtype=torch.float32, device=dev)
        if pairs == 0:
            pass                             # every token's choices hand their input on
        elif grouped:
            sizes = [4 * len(t) for t in tables]
            up_groups, down_groups = (meta[at + o:at + o + s].view(-1, 4) for o, s in zip((0, sizes[0]), sizes))
            ops.linear_grouped(xs, self.gate_up, up_groups, plans[0], gu)
            ops.moe_act(gu, self._ones(pairs, dev), y, self.limit, self.act)
            ops.linear_grouped(y, self.down, down_groups, plans[1], rows)
        else:
            for e, (gate_up, _) in enumerate(self.experts):
                if per_expert[e]:
                    gate_up(xs[starts[e]:starts[e + 1]], out=gu[starts[e]:starts[e + 1]])
            ops.moe_act(gu, self._ones(pairs, dev), y, self.limit, self.act)
            for e, (_, down) in enumerate(self.experts):
                if per_expert[e]:
                    down(y[starts[e]:starts[e + 1]], out=rows[starts[e]:starts[e + 1]])
        ops.moe_combine(rows, chosen, rank, offsets, weights, h, accumulate=accumulate, **handed)

    def _ones(self, n: int, dev) -> torch.Tensor:
        """[n][1] ones: the activation kernel's weights where the weighting happens later."""
        have = getattr(self, "_ones_buf", None)
        if have is None or have.shape[0] < n:
            have = self._ones_buf = torch.ones((max(n, 4096), 1), dtype=torch.float32, device=dev)
        return have[:n]


@register_feed_forward("grouped_moe")
class GroupedMoE(Experts):
    """params: those of `Experts`, and groups and keep (default 1: no groups), router (tensor name), router_bias
    (tensor name, or None), score ("softmax", the default, or "sigmoid"), correction (tensor name, or None),
    group_top (default 1), weight_scale (default 1.0), normalize (default True: the weights are the chosen scores over
    their sum; False: the scores as they are).  The router has a row for each of the n_experts + identity experts."""

    def __init__(self, spec, rt):
        super().__init__(spec, rt)
        p = spec.params
        self.groups, self.keep = int(p.get("groups", 1)), int(p.get("keep", p.get("groups", 1)))
        self.router_name = p["router"]
        self.bias_name = p.get("router_bias")
        self.correction_name = p.get("correction")
        self.score, self.group_top = p.get("score", "softmax"), int(p.get("group_top", 1))
        self.weight_scale = float(p.get("weight_scale", 1.0))
        if self.score not in ops.MOE_SCORES or self.group_top < 1:
            raise ValueError(f"grouped_moe: scores {self.score!r} (one of {sorted(ops.MOE_SCORES)}), group_top {self.group_top}")
        self.normalize = bool(p.get("normalize", True))
        per = self.choices // max(1, self.groups)
        if self.choices % self.groups or not 1 <= self.keep <= self.groups or not self.top <= self.keep * per:
            raise ValueError(f"grouped_moe: {self.choices} experts in {self.groups} groups, {self.keep} kept, {self.top} chosen")
        self.router = self.router_bias = self.correction = None

    def tensor_specs(self):
        s = {self.router_name: TensorSpec((self.choices, self.hidden))}
        if self.bias_name is not None:
            s[self.bias_name] = TensorSpec((self.choices,))
        if self.correction_name is not None:
            s[self.correction_name] = TensorSpec((self.choices,))
        s.update(super().tensor_specs())
        return s

    def load(self, get):
        self.router = get(self.router_name).to(torch.float32).contiguous()   # the router's product is 32-bit
        if self.bias_name is not None:
            self.router_bias = get(self.bias_name).to(torch.float32).contiguous()
        if self.correction_name is not None:
            self.correction = get(self.correction_name).to(torch.float32).contiguous()
        super().load(get)

    def choose(self, x, ctx, chosen, weights) -> None:
        ops.moe_route(x, self.router, None, chosen, weights, self.groups, self.keep, bias=self.router_bias,
                      score=self.score, correction=self.correction, group_top=self.group_top,
                      weight_scale=self.weight_scale, normalize=self.normalize)


@register_feed_forward("table_moe")
class TableMoE(Experts):
    """Experts that a table picks by the token's id, each weighing 1 / top.  params: those of `Experts`, and table
    (tensor name of int32 `[vocab_size][top]`), vocab_size."""

    def __init__(self, spec, rt):
        super().__init__(spec, rt)
        if self.identity:
            raise ValueError("table_moe: a table picks among experts with matrices")
        self.table_name, self.vocab = spec.params["table"], int(spec.params["vocab_size"])
        self.table = self.host_table = None

    def tensor_specs(self):
        return dict(super().tensor_specs(), **{self.table_name: TensorSpec((self.vocab, self.top), below=self.ne)})

    def load(self, get):
        self.table = get(self.table_name).to(torch.int32).contiguous()
        self.host_table = self.table.cpu().numpy()
        ranked = np.sort(self.host_table, axis=1)
        if ranked.size and (ranked.min() < 0 or ranked.max() >= self.ne):
            raise WeightError(f"{self.table_name}: expert numbers {ranked.min()}..{ranked.max()}, the layer has {self.ne}")
        if (ranked[:, 1:] == ranked[:, :-1]).any():
            raise WeightError(f"{self.table_name}: a row names an expert twice")
        super().load(get)

    def choose(self, x, ctx, chosen, weights) -> None:
        ops.moe_table(self.table, ctx.token_ids, ctx.kept_rows, chosen, weights, 1.0 / self.top)

    def host_counts(self, ctx):
        if ctx.host_tokens is None:
            return None
        tokens = ctx.host_tokens if ctx.kept_rows is None else ctx.host_tokens[ctx.host_rows]
        return np.bincount(self.host_table[tokens].reshape(-1), minlength=self.ne).tolist()
