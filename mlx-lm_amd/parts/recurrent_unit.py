"""A gated linear recurrent unit: a state of one number per channel."""

import torch

from ..config.plan import StateNeed
from ..ops import kernels
from .base import Mixer, OutputProduct, TensorSpec, register_mixer
from .linear_state import _matrix, _padded_columns, _rows_for, _SequenceArrays


class RecurrentUnit(OutputProduct, _SequenceArrays, Mixer):
    """The recurrent block with a real-gated linear recurrent unit (Griffin): two branches of ``inner`` channels,

        ``y = gelu_tanh(Wy x + by)``,   ``u = conv(Wx x + bx)``,   ``out = Wo (S * y)``

    with a causal convolution per channel (``conv`` ``[inner, taps]``, the last tap for the current token, zeros
    before a request's start, shift ``conv.b``), and over ``u`` in ``blocks`` equal parts

        ``r = sigmoid(ra[b] u_b + ra.b[b])``,   ``i = sigmoid(ri[b] u_b + ri.b[b])``,
        ``a = exp(-decay r softplus(lam))``,   ``S_t = a S_(t-1) + sqrt(1 - a^2) i u``.

    A request's state row is ``S`` (``inner`` floats), then the convolution's last inputs as a ring of ``taps``
    rows (none for one tap).  One product gives ``[x | y]`` as float32 rows with their shifts; convolution, gates,
    recurrence and the gelu are 32-bit (csrc/rglru.hip): one kernel for a step of single tokens, two for
    portions.  No counterpart in mlx_lm/models/gpt2.py.
    """

    graph_safe = True  # launches kernels only: a step of such parts can be recorded

    def __init__(self, width, inner, blocks, taps, decay=8.0, prefix=""):
        super().__init__(prefix)
        if inner <= 0 or blocks <= 0 or inner % blocks or taps < 1:
            raise ValueError(f"{inner} channels in {blocks} equal parts, {taps} taps")
        if width % 8:
            raise ValueError(f"width {width} must be a multiple of 8")
        if decay <= 0:
            raise ValueError(f"the decay's constant must be positive, got {decay}")
        self.width, self.inner, self.blocks, self.taps, self.decay = width, int(inner), int(blocks), int(taps), float(decay)

    def cache_need(self):
        return StateNeed((self.inner * (1 + (self.taps if self.taps > 1 else 0)),), "float32")

    def tensors(self):
        n, C, w = self._name, self.inner, self.inner // self.blocks
        t = {n("conv"): TensorSpec((C, self.taps), "vector"), n("conv.b"): TensorSpec((C,), "vector"), n("lam"): TensorSpec((C,), "vector"),
             n("o"): TensorSpec((self.width, C), "matrix")}
        for x in ("y", "x"):
            t[n(x)], t[n(x + ".b")] = TensorSpec((C, self.width), "matrix"), TensorSpec((C,), "vector")
        for x in ("ra", "ri"):
            t[n(x)], t[n(x + ".b")] = TensorSpec((self.blocks, w, w), "matrix"), TensorSpec((self.blocks, w), "vector")
        return t

    def load(self, tensors):
        n = self._name
        if not kernels.rglru_takes(self.inner // self.blocks):
            raise ValueError(f"gate matrices of {self.inner // self.blocks} channels are wider than the kernels take")
        self.in_w = _matrix(torch.cat([tensors[n("x")], tensors[n("y")]]))
        self.in_b = torch.cat([tensors[n("x.b")], tensors[n("y.b")]]).contiguous()
        self.first_weight = self.in_w
        self.unit = kernels.RglruWeights(tensors[n("conv")], tensors[n("conv.b")].contiguous(), tensors[n("ra")], tensors[n("ra.b")],
                                         tensors[n("ri")], tensors[n("ri.b")], tensors[n("lam")], self.decay)
        self.out_w = _matrix(_padded_columns(tensors[n("o")]))

    def forward(self, ctx, x, residual, cache, writes_cache=True):
        T, C = x.shape[0], self.inner
        mark = ctx.scratch_mark()
        u = ctx.scratch((T, 2 * C), torch.float32)
        kernels.linear(u, x, self.in_w, bias=self.in_b, splits=kernels.splits_alone(T))
        out, whole = _rows_for(ctx, T, C, -(-C // 8) * 8)
        spans = None
        if ctx.array("sequences.longest") > 1:
            spans = tuple(ctx.array("sequences." + s) for s in ("n_spans", "span_req", "span_start", "span_first"))
        kernels.rglru(out, u[:, :C], u[:, C:], self.unit, cache.state, cache.offset, cache.offset + C, ctx.positions,
                      ctx.array("sequences.starts"), ctx.array("sequences.lens"), ctx.slot_ids, ctx.n_requests, spans, ctx.scratch)
        self.output(residual, out if whole is None else whole, self.out_w)
        ctx.scratch_release(mark)


register_mixer("recurrent_unit", RecurrentUnit)
