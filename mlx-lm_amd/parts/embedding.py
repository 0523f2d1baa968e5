"""Token embedding: a row of the table for each token, written to the residual stream."""

import ctypes

from ..ops import kernels, native
from .base import NORMS, Part, TensorSpec, build_part, register_embedding


class TokenEmbedding(Part):
    """``h[t] = table[ids[t]] * scale``, plus a position term (not scaled) if the model has one.

    mlx_lm/models/gpt2.py:119-120,132 (where ``scale`` is 1).
    """

    graph_safe = True  # launches kernels only: a step of such parts can be recorded

    def __init__(self, vocab_size, width, weight_name="weight", scale=1.0, prefix=""):
        super().__init__(prefix)
        self.scale = float(scale)
        if vocab_size <= 0 or width <= 0:
            raise ValueError(f"embedding sizes must be positive, got {vocab_size} x {width}")
        self.vocab_size, self.width = vocab_size, width
        self.weight_name = self._name(weight_name)
        self.table = None

    def tensors(self):
        return {self.weight_name: TensorSpec((self.vocab_size, self.width), "matrix")}

    def load(self, tensors):
        self.table = tensors[self.weight_name]

    def reads_rows_of(self):
        """Tensors of which a step reads a row per token, not all."""
        return (self.weight_name,)

    native_kind = native.EMBEDDING

    def make_native(self):
        return native.made(native.lib().eng_make_token_embedding(
            self.table.data_ptr(), self.vocab_size, self.width, native.DT[self.table.dtype], self.scale), "token embedding")

    def forward(self, ctx, out, add=None):
        """Fill float32 ``out [tokens, width]``; ``add`` is ``(table, index)`` or ``None``."""
        if add is None:
            kernels.embed_gather_add(out, self.table, ctx.token_ids, scale=self.scale)
        else:
            kernels.embed_gather_add(out, self.table, ctx.token_ids, add[0], add[1], scale=self.scale)
        return out


class NormedTokenEmbedding(TokenEmbedding):
    """``h[t] = norm(table[ids[t]] * scale)``: the token's row passes a norm on its way into the stream,
    in one launch (csrc/dynamic_tanh.hip).  ``norm`` (a ``PartSpec``) is a ``dynamic_tanh``; there is no
    position term.  No counterpart in mlx_lm/models/gpt2.py."""

    def __init__(self, vocab_size, width, norm, weight_name="weight", scale=1.0, prefix=""):
        super().__init__(vocab_size, width, weight_name, scale, prefix)
        self.norm = build_part(NORMS, "norm", norm)
        if not hasattr(self.norm, "operands"):
            raise ValueError(f"a normed embedding fuses a dynamic tanh, not a {type(self.norm).__name__}")

    def tensors(self):
        return {**super().tensors(), **self.norm.tensors()}

    def load(self, tensors):
        super().load(tensors)
        self.norm.load(tensors)

    def make_native(self):
        P = ctypes.c_void_p
        L = native.part_library("dynamic_tanh", {"make_normed_tokens": [P, ctypes.c_int, ctypes.c_int, ctypes.c_float, P, P, P]})
        return native.made(L.make_normed_tokens(native.host(), self.table.data_ptr(), self.width, native.DT[self.table.dtype],
                                                self.scale, *(native.ptr(t) for t in self.norm.operands)), "normed token embedding")

    def forward(self, ctx, out, add=None):
        if add is not None:
            raise ValueError("a normed embedding takes no position term")
        return kernels.embed_dynamic_tanh(out, self.table, ctx.token_ids, self.scale, self.norm.operands)


register_embedding("token", TokenEmbedding)
register_embedding("normed_token", NormedTokenEmbedding)
