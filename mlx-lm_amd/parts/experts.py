"""A feed-forward of many small gated experts of which every token uses a few."""

import torch

from ..ops import kernels
from .base import FeedForward, TensorSpec, register_feed_forward


class GatedExperts(FeedForward):
    """``sum over a token's chosen experts of s_e * expert_e(x)  (+ shared(x))`` with

    * ``expert(x) = Wdown (silu(Wgate x) * (Wup x))``, no biases; ``n_experts`` of them with tensors
      ``e<i>.gate``, ``e<i>.up`` (``[inner, width]``) and ``e<i>.down`` (``[width, inner]``);
    * ``s = softmax(Wrouter x)`` over all ``n_experts + n_identity`` router outputs (32-bit sums
      of the products of the compute dtype's operands); the ``top`` largest of ``s + correction``
      are chosen (``correction``: a tensor, or none), and weigh in with ``s`` itself; with
      ``renormalize`` divided by the chosen ones' sum (+ 1e-20); times ``weight_scale``;
    * ``scores = "sigmoid"``: ``s`` is the logistic function of each output instead; ``groups = (count,
      keep)``: only experts of the ``keep`` best of ``count`` equal groups of neighbours can be chosen, a
      group counting the sum of its two largest choice scores;
    * the last ``n_identity`` router outputs stand for experts that give their input back;
    * ``shared_inner > 0``: one more expert of that inner size (``shared.gate`` ...) that every
      token uses with weight one;
    * ``activation = "clamped"``: an expert is ``Wdown (g sigmoid(1.702 g) (u + 1))`` with ``g = min(Wgate
      x, limit)`` and ``u = Wup x`` clamped to ``[-limit, limit]`` (not the shared expert).

    (``renormalize`` without a correction is the softmax over the chosen outputs alone.)

    The choice runs on the device (csrc/experts.hip), so a step launches kernels only.  For few
    tokens the chosen experts' weights are read straight from the stacked tensors, a wave four
    features, by kernels that touch nothing else; for many tokens the picks are sorted by expert on
    the device and go to the matrix cores in tiles of 32 to 128 picks of one expert.  The shared
    expert goes through the framework's products.  No counterpart in
    mlx_lm/models/gpt2.py, whose feed-forward (:71-84) is dense.
    """

    graph_safe = True  # launches kernels only: a step of such parts can be recorded
    can_overwrite = True
    MERGED_UP_TO = 16  # up to this many tokens the router's and the shared expert's first products are one
    # From TILES_FROM tokens in a step, or in bfloat16 from TILES_MIN tokens if every expert has TILES_EACH
    # picks on average, the picks are sorted and go to the matrix cores in tiles.
    TILES_FROM, TILES_MIN, TILES_EACH = 64, 8, 3

    def __init__(self, width, n_experts, inner, top, n_identity=0, shared_inner=0, correction=True, renormalize=False,
                 weight_scale=1.0, activation="silu", limit=0.0, scores="softmax", groups=None, prefix=""):
        super().__init__(prefix)
        if activation not in kernels.EXPERT_ACTIVATIONS:
            raise ValueError(f"experts' activation {activation!r} (known: {sorted(kernels.EXPERT_ACTIVATIONS)})")
        if activation == "clamped" and limit <= 0:
            raise ValueError(f"clamped activations need a positive limit, got {limit}")
        self.activation, self.limit = activation, float(limit)
        self.projection_given = False  # the router's outputs come out of a product that another part makes
        self.renormalize, self.weight_scale, self.scores = bool(renormalize), float(weight_scale), scores
        self.groups = tuple(groups) if groups is not None else None
        if n_experts < 0 or n_identity < 0 or n_experts + n_identity <= 0:
            raise ValueError(f"{n_experts} experts and {n_identity} identity experts")
        if not 0 < top <= n_experts + n_identity:
            raise ValueError(f"{top} of {n_experts + n_identity} experts a token")
        if width % 8:
            raise ValueError(f"the feed-forward's width must be a multiple of 8, got {width}")
        if n_experts and inner <= 0:
            raise ValueError(f"the experts' inner size must be positive, got {inner}")
        self.width, self.n_experts, self.inner, self.top = width, n_experts, inner, top
        self.n_identity, self.shared_inner, self.has_correction = n_identity, int(shared_inner or 0), bool(correction)
        self.n_out = n_experts + n_identity
        self.shared_padded = (self.shared_inner + 7) // 8 * 8  # zero weights beyond: silu(0) * 0 = 0 meets zero columns
        self.overwrite = False
        if scores not in kernels.ROUTER_SCORES:
            raise ValueError(f"router scores {scores!r} (known: {kernels.ROUTER_SCORES})")
        if self.groups is not None:
            count, keep = self.groups
            if count <= 0 or self.n_out % count or not 0 < keep <= count or top > keep * (self.n_out // count):
                raise ValueError(f"{top} picks out of {keep} of {count} groups of {self.n_out} experts")

    def tensors(self):
        n, t = self._name, {}
        for e in range(self.n_experts):
            t[n(f"e{e}.gate")] = TensorSpec((self.inner, self.width), "matrix")
            t[n(f"e{e}.up")] = TensorSpec((self.inner, self.width), "matrix")
            t[n(f"e{e}.down")] = TensorSpec((self.width, self.inner), "matrix")
        t[n("router")] = TensorSpec((self.n_out, self.width), "matrix")
        if self.has_correction:
            t[n("correction")] = TensorSpec((self.n_out,), "vector")
        if self.shared_inner:
            t[n("shared.gate")] = TensorSpec((self.shared_inner, self.width), "matrix")
            t[n("shared.up")] = TensorSpec((self.shared_inner, self.width), "matrix")
            t[n("shared.down")] = TensorSpec((self.width, self.shared_inner), "matrix")
        return t

    def input_names(self):
        """The tensor whose rows are the projection that ``forward`` starts with."""
        return [self._name("router")]

    def load(self, tensors):
        n = self._name
        self.w_gate = self.w_up = self.w_down = None
        if self.n_experts:
            self.w_gate = torch.stack([tensors[n(f"e{e}.gate")] for e in range(self.n_experts)]).contiguous()
            self.w_up = torch.stack([tensors[n(f"e{e}.up")] for e in range(self.n_experts)]).contiguous()
            self.w_down = torch.stack([tensors[n(f"e{e}.down")] for e in range(self.n_experts)]).contiguous()
        if not self.projection_given:
            self.router_rows = tensors[n("router")].contiguous()  # (an arrangement may take its product along: ``rows``)
            self.router_w = kernels.for_decode(self.router_rows)
            self.first_weight = self.router_w
        self.correction = tensors[n("correction")] if self.has_correction else None
        self.choice = dict(renormalize=self.renormalize, weight_scale=self.weight_scale, scores=self.scores, groups=self.groups)
        self.route = kernels.Route(self.correction, **self.choice)
        self.shared_in = self.shared_out = None
        if self.shared_inner:
            g, u, d = tensors[n("shared.gate")], tensors[n("shared.up")], tensors[n("shared.down")]
            pad = self.shared_padded - self.shared_inner
            if pad:
                g = torch.cat([g, g.new_zeros(pad, self.width)])
                u = torch.cat([u, u.new_zeros(pad, self.width)])
                d = torch.cat([d, d.new_zeros(self.width, pad)], 1)
            self.shared_in = kernels.for_decode(torch.cat([g, u]).contiguous())
            self.shared_out = kernels.for_decode(d.contiguous())
            # for steps of few tokens: router, gate and up in one product (float32 rows)
            if not self.projection_given:
                self.merged_in = kernels.for_decode(torch.cat([tensors[n("router")], g, u]).contiguous())

    def forward(self, ctx, x, residual, rows=None, after=None):
        """``rows``: the router's float32 outputs, where the caller has made them already.  ``after``:
        ``(out, norm operands)`` of a dynamic tanh over the rows that this completes, for the layer
        behind (made by the last kernel here)."""
        T = x.shape[0]
        merged = self.shared_inner and T <= self.MERGED_UP_TO and rows is None
        mark = ctx.scratch_mark()
        many = T >= self.TILES_FROM or (x.dtype == torch.bfloat16 and T >= self.TILES_MIN and T * self.top >= self.TILES_EACH * self.n_experts)
        tiles = self.n_experts and many and kernels.expert_tiles_takes(self.inner, self.width, x.dtype)
        route = None
        idx = ctx.scratch((T, self.top), torch.int32)
        weight = ctx.scratch((T, self.top), torch.float32)
        accumulate = not self.overwrite
        if merged:
            # few tokens: what a launch costs counts for more than what it computes
            zu = ctx.scratch((T, self.n_out + 2 * self.shared_padded), torch.float32)
            kernels.linear(zu, x, self.merged_in)
            act = ctx.scratch((T, self.shared_padded), ctx.dtype)
            kernels.route_and_gate(idx, weight, act, zu, self.correction, self.top, self.n_out, **self.choice)
            kernels.linear(residual, act, self.shared_out, accumulate=accumulate)
            accumulate = True
        else:
            z = rows
            if z is None:
                z = ctx.scratch((T, self.n_out), torch.float32)
                kernels.linear(z, x, self.router_w, splits=kernels.splits_alone(T))
            if not tiles and self.n_experts and self.top <= kernels.ROUTED_MOST:
                route = (z, self.route)  # (chosen by the kernel that reads the experts)
            else:
                kernels.router_choice(idx, weight, z, self.correction, self.top, **self.choice)
        if self.shared_inner and not merged:
            gu = ctx.scratch((T, 2 * self.shared_padded), ctx.dtype)
            kernels.linear(gu, x, self.shared_in, splits=kernels.splits_alone(T))
            act = ctx.scratch((T, self.shared_padded), ctx.dtype)
            kernels.silu_mul(act, gu)
            kernels.linear(residual, act, self.shared_out, accumulate=accumulate, splits=kernels.splits_alone(T))
            accumulate = True
        if tiles:
            kernels.expert_tiles(residual, x, self.w_gate, self.w_up, self.w_down, idx, weight, self.top, ctx.scratch,
                                 accumulate=accumulate, activation=self.activation, limit=self.limit, after=after)
        else:
            act = ctx.scratch((T * self.top, self.inner), ctx.dtype) if self.n_experts else None
            kernels.expert_rows(residual, x, self.w_gate, self.w_up, self.w_down, idx, weight, self.top, act,
                                accumulate=accumulate, activation=self.activation, limit=self.limit, route=route, after=after)
        ctx.scratch_release(mark)


register_feed_forward("gated_experts", GatedExperts)
