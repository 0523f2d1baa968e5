"""Linear attention over mixes of a token with the one before it, with a bonus for the current token."""

import torch

from ..config.plan import StateNeed
from ..ops import kernels
from .base import Mixer, TensorSpec, register_mixer
from .linear_state import _SequenceArrays, _matrix, _padded_columns, _rows_for


class TimeMix(_SequenceArrays, Mixer):
    """Time mixing in the manner of RWKV.  With ``h'`` the ``h`` of the token before (zeros ahead of a
    request's first), every projection reads a mix of its own, ``m_s = h + (h' - h) * mu_s``: ``r``, ``k``, ``v``
    (``n_heads x head_dim``), a gate ``silu(Wg m_g)`` and the decay, per head and key channel, through a
    narrow middle of ``decay_rank``, ``w = exp(-exp(W2 tanh(W1 m_w) + w0))``.  Per head

        ``o_t = S_(t-1)^T r_t + (r_t . (u * k_t)) v_t``,   ``S_t = diag(w_t) S_(t-1) + k_t v_t^T``

    with the bonus ``u`` for the current token only.  Each head's ``o`` is divided by its root mean
    square (``eps``), the heads side by side times ``norm`` (``n_heads * head_dim`` values) and the
    gate; then ``Wo``.

    A request's state row is ``S`` of every head and, behind it, the last ``h``, float32.  The layer's
    norm has to be one that needs no statistics (``dynamic_tanh``): norm, shift and the five mixes are
    one kernel (csrc/dynamic_tanh.hip), the products with them one launch for steps of few tokens
    (``kernels.GroupedWeight``), decay, recurrence, norm and gate one kernel for steps of few tokens
    (csrc/state_step.hip); portions go in chunks and spans through ``state_scan`` with a decay per key
    channel (csrc/linear_state.hip).  Everything up to the normed output is 32-bit.  No counterpart in
    mlx_lm/models/gpt2.py.
    """

    graph_safe = True  # launches kernels only: a step of such parts can be recorded
    MIXES = ("r", "k", "v", "g", "w")
    more_names = ()  # tensors of another part that reads the norm itself; its product rides along

    def __init__(self, width, n_heads, head_dim, decay_rank, eps, prefix=""):
        super().__init__(prefix)
        if n_heads <= 0 or not 0 < head_dim <= 256 or decay_rank <= 0:
            raise ValueError(f"{n_heads} heads of {head_dim} (at most 256), a middle of {decay_rank}")
        if width % 8:
            raise ValueError(f"width {width} must be a multiple of 8")
        self.width, self.n_heads, self.head_dim, self.decay_rank, self.eps = width, n_heads, head_dim, int(decay_rank), float(eps)
        self.inner = n_heads * head_dim
        self.state_floats = n_heads * head_dim * head_dim

    def cache_need(self):
        return StateNeed(((self.state_floats + self.width + 3) // 4 * 4,), "float32")

    def tensors(self):
        n = self._name
        t = {n("mu." + s): TensorSpec((self.width,), "vector") for s in self.MIXES}
        t.update({n(s): TensorSpec((self.inner, self.width), "matrix") for s in ("r", "k", "v", "g")})
        t.update({n("w1"): TensorSpec((self.decay_rank, self.width), "matrix"), n("w2"): TensorSpec((self.inner, self.decay_rank), "matrix"),
                  n("w0"): TensorSpec((self.inner,), "vector"), n("u"): TensorSpec((self.n_heads, self.head_dim), "vector"),
                  n("norm"): TensorSpec((self.inner,), "vector"), n("o"): TensorSpec((self.width, self.inner), "matrix")})
        return t

    def load(self, tensors):
        n = self._name
        self.mu = torch.stack([tensors[n("mu." + s)] for s in self.MIXES]).contiguous()
        # plane 0 is the normed row itself, plane 1 + i the i-th mix
        groups = [(tensors[n(s)], 1 + i) for i, s in enumerate(("r", "k", "v", "g"))] + [(tensors[n("w1")], 5)]
        if self.more_names:
            groups.append((torch.cat([tensors[x] for x in self.more_names]), 0))
        self.in_w = kernels.GroupedWeight(groups)
        self.decay = kernels.LowRankDecay(tensors[n("w2")].t().contiguous(), tensors[n("w0")].contiguous())
        self.bonus, self.norm_w = tensors[n("u")].reshape(-1).contiguous(), tensors[n("norm")].contiguous()
        self.out_w = _matrix(_padded_columns(tensors[n("o")]))

    def project(self, ctx, h, norm, cache):
        """``(normed rows, the float32 columns [r, k, v, g, middle], the other part's columns or None)``."""
        if not hasattr(norm, "operands"):
            raise ValueError(f"a token shift fuses a dynamic tanh, not a {type(norm).__name__}")
        planes = ctx.scratch((1 + len(self.MIXES), h.shape[0], self.width), ctx.dtype)
        kernels.token_mix(planes, h, norm.operands, self.mu, cache.state, cache.offset + self.state_floats, ctx.token_req,
                          ctx.array("sequences.starts"), ctx.array("sequences.lens"), ctx.slot_ids)
        columns = kernels.linear_groups(ctx.scratch, planes, self.in_w)
        return planes[0], columns[:5], columns[5] if self.more_names else None

    def forward(self, ctx, x, residual, cache, writes_cache=True, rows=None):
        """``rows``: what ``project`` gave (an arrangement that calls it hands it on)."""
        if rows is None:
            raise ValueError("a token shift starts from the stream and its norm: the arrangement calls project first")
        T, H, N = x.shape[0], self.n_heads, self.head_dim
        mark = ctx.scratch_mark()
        r, k, v, g, z = rows
        starts, lens = ctx.array("sequences.starts"), ctx.array("sequences.lens")
        out, whole = _rows_for(ctx, T, self.inner, -(-self.inner // 8) * 8)
        if self._chunked(ctx) and kernels.state_chunks_takes(N, N):
            log_w = ctx.scratch((T, self.inner), torch.float32)
            kernels.lowrank_decay(log_w, z, self.decay)
            kernels.state_scan(out, r, k, v, cache.state, cache.offset, starts, lens, ctx.slot_ids, ctx.n_requests, H, H, N, N,
                               channel_decay=log_w, bonus=self.bonus, unit_rms=True, eps=self.eps, norm_weight=self.norm_w, gate=g,
                               chunked=True, spans=self._spans(ctx))
        else:
            kernels.state_step(out, r, k, v, cache.state, cache.offset, starts, lens, ctx.slot_ids, ctx.n_requests, H, H, N, N,
                               self.norm_w, self.eps, gate=g, z=z, decay=self.decay, bonus=self.bonus)
        kernels.linear(residual, out if whole is None else whole, self.out_w, accumulate=True, splits=kernels.splits_alone(T))
        ctx.scratch_release(mark)


register_mixer("time_mix", TimeMix)
