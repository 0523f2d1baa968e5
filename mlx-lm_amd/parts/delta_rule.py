"""Linear attention that corrects what its state already answers for a key (the gated delta rule)."""

import torch

from ..config.plan import StateNeed
from ..ops import kernels
from .base import Mixer, OutputProduct, ProjectsFirst, TensorSpec, register_mixer
from .linear_state import _SequenceArrays, _matrix, _padded_columns, _rows_for


class GatedDeltaRule(ProjectsFirst, _SequenceArrays, Mixer):
    """The gated delta rule, per head with a matrix state ``S`` (``key_dim x value_dim``):

        ``d_t = beta_t (v_t - g_t S_(t-1)^T k_t)``,   ``S_t = g_t S_(t-1) + k_t d_t^T``,   ``o_t = S_t^T q_t``

    ``q = Wq x``, ``k = Wk x`` (``n_key_heads x key_dim``; head ``h`` reads key head ``h // (n_heads /
    n_key_heads)``) and ``v = Wv x`` (``n_heads x value_dim``) each pass a short causal convolution per
    channel (``q.conv``, ``k.conv``, ``v.conv``, ``[channels, taps]``, the last tap for the current token,
    zeros before a request's start, no bias) and a silu; q and k are then unit vectors per head (``x /
    sqrt(sum x^2 + 1e-6)``), q times ``key_dim^(-1/2)``.  ``beta = sigmoid(Wb x)`` and ``g =
    exp(-exp(A_log) softplus(Wa x + dt_bias))``, one a head.  Each head's ``o`` is divided by its root
    mean square (``eps``), times ``norm`` (``value_dim`` values for all heads) and ``silu(Wg x)``; then
    ``Wo``.

    A request's state row is ``S`` of every head, float32, then the convolution's last inputs as a
    ring of ``taps`` rows (none for one tap).  One product gives ``[q | k | v | g | b | a]`` as float32
    rows; all up to the normed output is 32-bit.  A step in which every request brings one token is one
    kernel behind the product (csrc/state_step.hip); portions are prepared by a kernel of their own and
    go through the same recurrence, from ``CHUNKS_FROM`` tokens on in chunks (csrc/delta_chunks.hip).
    No counterpart in mlx_lm/models/gpt2.py.
    """

    graph_safe = True  # launches kernels only: a step of such parts can be recorded

    def __init__(self, width, n_heads, n_key_heads, key_dim, value_dim, taps, eps, prefix=""):
        super().__init__(prefix)
        if n_heads <= 0 or n_key_heads <= 0 or n_heads % n_key_heads:
            raise ValueError(f"{n_heads} heads cannot be grouped over {n_key_heads} key heads")
        if not 0 < value_dim <= 256 or not 0 < key_dim <= 256 or taps < 1:
            raise ValueError(f"keys of {key_dim} and values of {value_dim} (at most 256 each), {taps} taps")
        if width % 8:
            raise ValueError(f"width {width} must be a multiple of 8")
        self.width, self.n_heads, self.n_key_heads, self.key_dim, self.value_dim = width, n_heads, n_key_heads, key_dim, value_dim
        self.taps, self.eps = int(taps), float(eps)
        self.qk_width, self.v_width = n_key_heads * key_dim, n_heads * value_dim
        self.channels = 2 * self.qk_width + self.v_width
        self.state_floats = n_heads * key_dim * value_dim

    def cache_need(self):
        floats = self.state_floats + (self.taps * self.channels if self.taps > 1 else 0)
        return StateNeed(((floats + 3) // 4 * 4,), "float32")  # (whole pieces of 16 bytes: every row starts on one)

    def tensors(self):
        n, H = self._name, self.n_heads
        t = {n("b"): TensorSpec((H, self.width), "matrix"), n("a"): TensorSpec((H, self.width), "matrix"),
             n("A_log"): TensorSpec((H,), "vector"), n("dt_bias"): TensorSpec((H,), "vector"),
             n("norm"): TensorSpec((self.value_dim,), "vector"), n("g"): TensorSpec((self.v_width, self.width), "matrix"),
             n("o"): TensorSpec((self.width, self.v_width), "matrix")}
        for x, rows in (("q", self.qk_width), ("k", self.qk_width), ("v", self.v_width)):
            t[n(x)], t[n(x + ".conv")] = TensorSpec((rows, self.width), "matrix"), TensorSpec((rows, self.taps), "vector")
        return t

    def input_names(self):
        """The tensors whose rows, in this order, are the projection that ``forward`` starts with."""
        return [self._name(x) for x in ("q", "k", "v", "g", "b", "a")]

    def load(self, tensors):
        n = self._name
        self.load_projection(tensors)
        self.out_w = _matrix(_padded_columns(tensors[n("o")]))
        self.norm_w = tensors[n("norm")].contiguous()
        conv_w = torch.cat([tensors[n(x + ".conv")] for x in ("q", "k", "v")]).contiguous()
        self.raw = kernels.DeltaRaw(conv_w, self.state_floats, tensors[n("A_log")].contiguous(), tensors[n("dt_bias")].contiguous(),
                                    self.key_dim**-0.5)

    def forward(self, ctx, x, residual, cache, writes_cache=True, rows=None):
        """``rows``: the projection's float32 rows, where the caller has made them already."""
        T, H, G, N, P = x.shape[0], self.n_heads, self.n_key_heads, self.key_dim, self.value_dim
        mark = ctx.scratch_mark()
        u = rows if rows is not None else self.own_rows(ctx, x)
        a, v0, g0 = self.qk_width, 2 * self.qk_width, self.channels
        b0 = g0 + self.v_width
        gate = u[:, g0:b0]
        starts, lens, longest = ctx.array("sequences.starts"), ctx.array("sequences.lens"), ctx.array("sequences.longest")
        out, whole = _rows_for(ctx, T, self.v_width, -(-self.v_width // 8) * 8)
        common = (cache.state, cache.offset)
        if longest == 1:
            kernels.state_step(out, u[:, :a], u[:, a:v0], u[:, v0:g0], *common, starts, lens, ctx.slot_ids, ctx.n_requests, H, G, N, P,
                               self.norm_w, self.eps, gate=gate, beta=u[:, b0 : b0 + H], log_g=u[:, b0 + H : b0 + 2 * H], raw=self.raw,
                               positions=ctx.positions)
        else:
            ops = kernels.delta_prepare(ctx.scratch, u, b0, b0 + H, H, G, N, P, self.raw, cache.state, ctx.token_req, ctx.positions,
                                        starts, lens, ctx.slot_ids)
            if self._chunked(ctx) and kernels.delta_chunks_takes(N, P):
                spans = tuple(ctx.array("sequences." + s) for s in ("n_spans", "span_req", "span_start", "span_first"))
                kernels.delta_chunks(out, ops, *common, spans, starts, lens, ctx.slot_ids, ctx.n_requests, H, G, N, P, self.norm_w,
                                     self.eps, gate, ctx.scratch)
            else:
                q, k, v, log_g, beta = ops
                kernels.state_step(out, q, k, v, *common, starts, lens, ctx.slot_ids, ctx.n_requests, H, G, N, P, self.norm_w, self.eps,
                                   gate=gate, qk_stride=q.shape[1] // G, v_stride=v.shape[1] // H, log_g=log_g, beta=beta)
        kernels.linear(residual, out if whole is None else whole, self.out_w, accumulate=True, splits=kernels.splits_alone(T))
        ctx.scratch_release(mark)


class ChannelDeltaRule(OutputProduct, _SequenceArrays, Mixer):
    """The gated delta rule with a decay of its own for every key channel (the rows of ``S``):

        ``d_t = beta_t (v_t - (G_t S_(t-1))^T k_t)``,   ``S_t = G_t S_(t-1) + k_t d_t^T``,   ``o_t = S_t^T q_t``

    with ``G = diag(g)`` and ``g = exp(-exp(A_log) softplus(Wa2 (Wa1 x) + dt_bias))``, laid out ``n_heads x
    key_dim`` (``A_log`` one a head).  Queries, keys, values, their convolutions and unit vectors and ``beta`` are
    ``GatedDeltaRule``'s.  Each head's ``o`` is divided by its root mean square (``eps``), times ``norm``
    (``value_dim`` values for all heads) and ``sigmoid(Wg2 (Wg1 x))``, ``n_heads x value_dim``; then ``Wo``.
    ``decay_rank`` and ``gate_rank`` are the widths of the two narrow middles.

    A request's state row is ``S`` of every head, float32, then the convolution's last inputs as a ring of
    ``taps`` rows (none for one tap).  One product gives ``[q | k | v | b | Wa1 x | Wg1 x]`` as float32 rows; all up to
    the normed output is 32-bit.  A step in which every request brings one token is one kernel behind the
    product, which takes the narrow matrices too (csrc/state_step.hip); portions go through chunks of 64
    tokens (csrc/delta_chunks.hip).  No counterpart in mlx_lm/models/gpt2.py.
    """

    graph_safe = True  # launches kernels only: a step of such parts can be recorded

    def __init__(self, width, n_heads, n_key_heads, key_dim, value_dim, taps, eps, decay_rank, gate_rank, prefix=""):
        super().__init__(prefix)
        if n_heads <= 0 or n_key_heads <= 0 or n_heads % n_key_heads:
            raise ValueError(f"{n_heads} heads cannot be grouped over {n_key_heads} key heads")
        if not 0 < value_dim <= 256 or not 0 < key_dim <= 256 or taps < 1:
            raise ValueError(f"keys of {key_dim} and values of {value_dim} (at most 256 each), {taps} taps")
        if not 0 < decay_rank <= 2048 or not 0 < gate_rank <= 2048:
            raise ValueError(f"middles of {decay_rank} and {gate_rank} columns (1 to 2048)")
        if width % 8:
            raise ValueError(f"width {width} must be a multiple of 8")
        self.width, self.n_heads, self.n_key_heads, self.key_dim, self.value_dim = width, n_heads, n_key_heads, key_dim, value_dim
        self.taps, self.eps, self.decay_rank, self.gate_rank = int(taps), float(eps), int(decay_rank), int(gate_rank)
        self.qk_width, self.v_width = n_key_heads * key_dim, n_heads * value_dim
        self.channels = 2 * self.qk_width + self.v_width
        self.state_floats = n_heads * key_dim * value_dim

    def cache_need(self):
        floats = self.state_floats + (self.taps * self.channels if self.taps > 1 else 0)
        return StateNeed(((floats + 3) // 4 * 4,), "float32")  # (whole pieces of 16 bytes: every row starts on one)

    def tensors(self):
        n, H = self._name, self.n_heads
        t = {n("b"): TensorSpec((H, self.width), "matrix"), n("A_log"): TensorSpec((H,), "vector"),
             n("a1"): TensorSpec((self.decay_rank, self.width), "matrix"), n("a2"): TensorSpec((H * self.key_dim, self.decay_rank), "matrix"),
             n("dt_bias"): TensorSpec((H * self.key_dim,), "vector"), n("norm"): TensorSpec((self.value_dim,), "vector"),
             n("g1"): TensorSpec((self.gate_rank, self.width), "matrix"), n("g2"): TensorSpec((self.v_width, self.gate_rank), "matrix"),
             n("o"): TensorSpec((self.width, self.v_width), "matrix")}
        for x, rows in (("q", self.qk_width), ("k", self.qk_width), ("v", self.v_width)):
            t[n(x)], t[n(x + ".conv")] = TensorSpec((rows, self.width), "matrix"), TensorSpec((rows, self.taps), "vector")
        return t

    def load(self, tensors):
        n = self._name
        # the middles start at multiples of four columns of the projection and are padded to multiples of eight
        parts, at = [tensors[n(x)] for x in ("q", "k", "v", "b")], self.channels + self.n_heads
        zeros = lambda rows: parts[0].new_zeros(rows, self.width)  # noqa: E731
        parts.append(zeros(-at % 4))
        a_col = at + -at % 4
        parts += [tensors[n("a1")], zeros(-self.decay_rank % 8)]
        g_col = a_col + (self.decay_rank + 7) // 8 * 8
        parts += [tensors[n("g1")], zeros(-self.gate_rank % 8)]
        self.in_w = _matrix(torch.cat(parts))
        self.first_weight = self.in_w
        self.narrow = kernels.NarrowMiddle(_padded_columns(tensors[n("a2")]).contiguous(), a_col, _padded_columns(tensors[n("g2")]).contiguous(), g_col)
        self.out_w = _matrix(_padded_columns(tensors[n("o")]))
        self.norm_w = tensors[n("norm")].contiguous()
        conv_w = torch.cat([tensors[n(x + ".conv")] for x in ("q", "k", "v")]).contiguous()
        self.raw = kernels.DeltaRaw(conv_w, self.state_floats, tensors[n("A_log")].contiguous(), tensors[n("dt_bias")].contiguous(),
                                    self.key_dim**-0.5)
        # (a state that a block cannot hold in registers takes the chunks for single tokens too)
        self.has_step = kernels.state_step_takes(self.key_dim, self.value_dim)

    def forward(self, ctx, x, residual, cache, writes_cache=True):
        T, H, G, N, P = x.shape[0], self.n_heads, self.n_key_heads, self.key_dim, self.value_dim
        mark = ctx.scratch_mark()
        u = ctx.scratch((T, self.in_w.shape[0]), torch.float32)
        kernels.linear(u, x, self.in_w, splits=kernels.splits_alone(T))
        a, v0, b0 = self.qk_width, 2 * self.qk_width, self.channels
        starts, lens = ctx.array("sequences.starts"), ctx.array("sequences.lens")
        out, whole = _rows_for(ctx, T, self.v_width, -(-self.v_width // 8) * 8)
        if ctx.array("sequences.longest") == 1 and self.has_step:
            kernels.state_step(out, u[:, :a], u[:, a:v0], u[:, v0:b0], cache.state, cache.offset, starts, lens, ctx.slot_ids, ctx.n_requests,
                               H, G, N, P, self.norm_w, self.eps, beta=u[:, b0 : b0 + H], raw=self.raw, positions=ctx.positions,
                               narrow=(u, self.narrow), gate_activation="sigmoid")
        else:
            *ops, gate = kernels.delta_prepare(ctx.scratch, u, b0, 0, H, G, N, P, self.raw, cache.state, ctx.token_req, ctx.positions,
                                               starts, lens, ctx.slot_ids, narrow=self.narrow)
            spans = tuple(ctx.array("sequences." + s) for s in ("n_spans", "span_req", "span_start", "span_first"))
            kernels.delta_chunks(out, ops, cache.state, cache.offset, spans, starts, lens, ctx.slot_ids, ctx.n_requests, H, G, N, P,
                                 self.norm_w, self.eps, gate, ctx.scratch, by_channel=True, gate_activation="sigmoid")
        self.output(residual, out if whole is None else whole, self.out_w)
        ctx.scratch_release(mark)


register_mixer("delta_rule", GatedDeltaRule)
register_mixer("channel_delta_rule", ChannelDeltaRule)
