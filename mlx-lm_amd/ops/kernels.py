"""Python faces of the HIP kernels: argument checks, pointers, launch.

Each function takes torch tensors that live on the GPU, checks on the host
what the kernel assumes about them (shape, dtype, contiguity) and launches on
torch's current stream.  Nothing here computes on the CPU or through a torch
operator; a missing library raises.  A model's step does not come through
here: the native host (``csrc/engine.hip``) issues its launches itself.  These
faces are for a kernel alone (tests), for parts written in Python, and for
sampling; ``linear`` and ``PendingSum`` call the native host's own product
routine, so there is one place that chooses among the product kernels.
"""

import ctypes
import weakref

import torch

from . import build, native

_c_int = ctypes.c_int
_c_float = ctypes.c_float
_c_size_t = ctypes.c_size_t
_vp = ctypes.c_void_p

DT = {torch.float32: 0, torch.bfloat16: 1}

GEMM_GELU = 1
GEMM_ACCUMULATE = 2
GEMM_OUT_F32 = 4
GEMM_KV = 8

# Up to this many rows a bfloat16 product goes to the decode kernels, which stream the weights
# once and fuse the norm and the cache scatter; more rows go to the tile kernels.
DECODE_MAX_ROWS = 16


# torch's current stream as a raw handle.  torch.cuda.current_stream() builds a Stream object
# through several Python layers (some 4 us a call, once per launch); the binding below is what
# that ends in.
_raw_stream = getattr(torch._C, "_cuda_getCurrentRawStream", None)
_current_device = getattr(torch._C, "_cuda_getDevice", None)


def raw_stream():
    """The handle of the stream that torch launches on now, as an integer."""
    if _raw_stream is not None and _current_device is not None:
        return _raw_stream(_current_device())
    return torch.cuda.current_stream().cuda_stream


def _stream():
    return _vp(raw_stream())


def n_compute_units():
    """Compute units of the current device (asked of the device once)."""
    return native.lib().eng_compute_units()


_BARE = {}


def bare_context():
    """A native context outside any step: the stream, the split workspace, no scratch memory."""
    dev = torch.cuda.current_device()
    c = _BARE.get(dev)
    if c is None:
        c = _BARE[dev] = native.EngCtx()
        ws = split_workspace(torch.device("cuda", dev))
        c.split_ws, c.split_ws_floats = ws.data_ptr(), ws.numel()
        c.n_compute_units = n_compute_units()
        c.dtype = 1
    c.stream = raw_stream()
    c.force_splits = force_splits
    return c


def _ptr(t):
    return _vp(t.data_ptr()) if t is not None else _vp(0)


def _need(cond, msg):
    if not cond:
        raise ValueError(msg)


def _fail(msg):
    """``cond or _fail(f"...")``: the message is put together only when the check fails."""
    raise ValueError(msg)


def _dev(t, name, dtype=None):
    t.is_cuda or _fail(f"{name} must be on the GPU")
    t.is_contiguous() or _fail(f"{name} must be contiguous")
    if dtype is not None:
        t.dtype == dtype or _fail(f"{name} must be {dtype}, is {t.dtype}")


def _rows2d(t, name):
    """A 2-D tensor whose rows are contiguous; returns its row stride."""
    t.is_cuda or _fail(f"{name} must be on the GPU")
    (t.dim() == 2 and t.stride(1) == 1) or _fail(f"{name} must be 2-D with contiguous rows")
    return t.stride(0)


# ---------------------------------------------------------------------------


def embed_gather_add(out, table, ids, add_table=None, add_ids=None, scale=1.0):
    """``out[t] = table[ids[t]] * scale (+ add_table[add_ids[t]])`` into float32 ``out``."""
    lib = build.load("embed")
    n, width = out.shape
    _dev(out, "out", torch.float32)
    _dev(table, "table")
    _dev(ids, "ids", torch.int32)
    table.dtype in DT or _fail(f"table dtype {table.dtype} not supported")
    _need(table.shape[1] == width and ids.numel() >= n, "embed_gather_add: shapes disagree")
    if add_table is not None:
        _dev(add_table, "add_table", table.dtype)
        _dev(add_ids, "add_ids", torch.int32)
        _need(add_table.shape[1] == width and add_ids.numel() >= n, "embed_gather_add: shapes disagree")
    rc = lib.embed_scale_add(
        _ptr(out), _ptr(table), _ptr(ids), _ptr(add_table), _ptr(add_ids),
        _c_int(n), _c_int(width), _c_int(DT[table.dtype]), ctypes.c_float(scale), _stream(),
    )
    build.check(lib, rc, "embed_gather_add")
    return out


def feed_tokens(ids, src, index, vocab):
    """``ids[t] = src[index[t]]`` where ``index[t] >= 0``: sampled tokens that are still on the device."""
    lib = build.load("embed")
    for name, t in (("ids", ids), ("src", src), ("index", index)):
        _dev(t, name, torch.int32)
    _need(index.numel() >= ids.numel(), "feed_tokens: an index for every id")
    rc = lib.feed_tokens(_ptr(ids), _ptr(src), _ptr(index), _c_int(ids.numel()), _c_int(vocab), _stream())
    build.check(lib, rc, "feed_tokens")
    return ids


def layernorm(out, x, gamma, beta, eps, rows=None):
    """LayerNorm of float32 rows of ``x`` (all, or those listed in ``rows``) into ``out``."""
    lib = build.load("norm")
    n, width = out.shape
    _dev(out, "out")
    _dev(x, "x", torch.float32)
    out.dtype in DT or _fail(f"out dtype {out.dtype} not supported")
    _need(x.shape[-1] == width, "layernorm: widths disagree")
    if rows is None:
        _need(x.shape[0] >= n, "layernorm: fewer input rows than output rows")
    else:
        _dev(rows, "rows", torch.int32)
        _need(rows.numel() >= n, "layernorm: fewer row indices than output rows")
    for name, v in (("gamma", gamma), ("beta", beta)):
        if v is not None:
            _dev(v, name, torch.float32)
            v.numel() == width or _fail(f"layernorm: {name} has {v.numel()} elements, width is {width}")
    rc = lib.layernorm(
        _ptr(out), _ptr(x), _ptr(rows), _ptr(gamma), _ptr(beta), _c_float(eps),
        _c_int(n), _c_int(width), _c_int(DT[out.dtype]), _stream(),
    )
    build.check(lib, rc, "layernorm")
    return out


class NormedInput:
    """The LayerNorm of float32 rows (``rms``: their root-mean-square norm, no mean taken off and
    no shift), not computed yet.

    ``linear`` takes it as its input and, where its kernel can, norms the rows
    itself while the first weights are on their way; anything else calls
    ``materialize()`` and gets the tensor.
    """

    def __init__(self, alloc, x, gamma, beta, eps, dtype, rms=False):
        self.alloc, self.x, self.gamma, self.beta, self.eps, self.dtype = alloc, x, gamma, beta, eps, dtype
        self.rms = bool(rms)
        self.shape = tuple(x.shape)
        self._out = None

    def materialize(self):
        if self._out is None:
            self._out = self.alloc(self.shape, self.dtype)
            if self.rms:
                rmsnorm(self._out, self.x, self.gamma, self.eps)
            else:
                layernorm(self._out, self.x, self.gamma, self.beta, self.eps)
        return self._out


def normed(x):
    """``x`` as a tensor: a ``NormedInput`` is computed (once), a tensor is itself."""
    return x.materialize() if isinstance(x, NormedInput) else x


def rmsnorm(out, x, weight, eps):
    """``out = x / sqrt(mean(x^2) + eps) * weight`` over float32 rows ``x``; ``out`` float32 or bfloat16."""
    lib = build.load("rmsnorm")
    ldx = _f32_rows(x, "x", out.shape[1])
    _dev(weight, "weight", torch.float32)
    _need(out.is_contiguous() and out.dtype in DT and weight.numel() == out.shape[1] and x.shape[0] >= out.shape[0], "rmsnorm: shapes")
    rc = lib.rmsnorm(_ptr(out), _ptr(x), _c_int(ldx), None, _ptr(weight), _c_float(eps), _c_int(out.shape[0]),
                     _c_int(out.shape[1]), _c_int(DT[out.dtype]), _stream())
    build.check(lib, rc, "rmsnorm")
    return out


class KVScatter:
    """Where the key and value columns of a fused q/k/v projection go: the
    pages of ``kv``, for each token at its request's position."""

    def __init__(self, kv, block_table, token_req, positions, q_width):
        self.kv, self.block_table, self.token_req, self.positions = kv, block_table, token_req, positions
        self.q_width = q_width
        self.kv_width = kv.n_kv_heads * kv.head_dim


class PackedWeight:
    """A bfloat16 weight matrix ``[N, K]`` in the order the decode kernel's lanes read it.

    Tiles of 16 features by 64 k, zero padded; tile ``(b, c)`` holds, for lane
    ``l`` (feature ``l % 16``, k group ``l // 16``), first the 8 values
    ``k = 64 c + 16 (l // 16) + 0..7`` of all lanes, then the 8 values ``+ 8..15``.
    A wave's load is then 1 KB of consecutive bytes.  The kernels that take
    many rows read this order too, so the row-major matrix need not be kept
    (``keep_rows=False`` lets it go: one copy of the weights on the device).
    """

    def __init__(self, w, keep_rows=True):
        _need(w.dtype == torch.bfloat16 and w.dim() == 2, "PackedWeight: a 2-D bfloat16 matrix")
        self.w = w if keep_rows else None
        self.shape, self.dtype, self.device = tuple(w.shape), w.dtype, w.device
        N, K = w.shape
        Np, Kp = (N + 15) // 16 * 16, (K + 63) // 64 * 64
        padded = torch.zeros((Np, Kp), dtype=w.dtype, device=w.device)
        padded[:N, :K] = w
        # (block, feature, k-block, k group, half, 8) -> (block, k-block, half, k group, feature, 8)
        t = padded.view(Np // 16, 16, Kp // 64, 4, 2, 8).permute(0, 2, 4, 3, 1, 5)
        self.packed = t.contiguous().view(-1)
        # what one block of the decode kernel reads (16 features, all of K) and how many there are
        self.chunk_bytes, self.n_chunks = Kp * 16 * 2, Np // 16
        self.c = native.EngWeight(w.data_ptr() if keep_rows else None, self.packed.data_ptr(), N, K,
                                  w.stride(0) if keep_rows else 0, DT[w.dtype], self.chunk_bytes, self.n_chunks, 0)


class PackedRows:
    """bfloat16 activations ``[M, K]`` in the order in which the product of 17 to 64 rows reads them
    fastest: tiles of 16 rows by 64 columns, each laid out like a tile of ``PackedWeight``.  What
    lies beyond row ``M`` or column ``K`` in the last tiles is never used.

    ``PackedRows.empty(M, K, device)`` makes room for a kernel to write into
    (``sum_partials_norm(..., out=...)``, ``attn_decode``, ``linear(out=...)``);
    ``PackedRows.of(a)`` packs a row-major matrix and ``.rows()`` gives it back (tests)."""

    def __init__(self, data, shape):
        self.data, self.shape = data, tuple(shape)
        self.dtype, self.device = data.dtype, data.device

    @classmethod
    def empty(cls, M, K, device):
        n = (M + 15) // 16 * ((K + 63) // 64) * 1024
        return cls(torch.zeros(n, dtype=torch.bfloat16, device=device), (M, K))

    @classmethod
    def of(cls, a):
        _need(a.dtype == torch.bfloat16 and a.dim() == 2, "PackedRows: a 2-D bfloat16 matrix")
        M, K = a.shape
        Mp, Kp = (M + 15) // 16 * 16, (K + 63) // 64 * 64
        padded = torch.zeros((Mp, Kp), dtype=a.dtype, device=a.device)
        padded[:M, :K] = a
        t = padded.view(Mp // 16, 16, Kp // 64, 4, 2, 8).permute(0, 2, 4, 3, 1, 5)
        return cls(t.contiguous().view(-1), (M, K))

    def rows(self):
        M, K = self.shape
        Mp, Kp = (M + 15) // 16 * 16, (K + 63) // 64 * 64
        t = self.data.view(Mp // 16, Kp // 64, 2, 4, 16, 8).permute(0, 4, 1, 3, 2, 5)
        return t.reshape(Mp, Kp)[:M, :K].contiguous()

    def data_ptr(self):
        return self.data.data_ptr()


def wants_packed_rows(w, n_rows):
    """Whether the product of ``n_rows`` rows with ``w`` (a ``PackedWeight``) reads its rows fastest
    as ``PackedRows``: the kernel that holds a block's weights in registers takes it."""
    if not isinstance(w, PackedWeight):
        return False
    return bool(native.lib().eng_wants_packed_rows(ctypes.byref(bare_context()), ctypes.byref(w.c), int(n_rows)))


def weight_struct(w):
    """The native description of a weight matrix (a ``PackedWeight`` or a 2-D tensor ``[N, K]``)."""
    if isinstance(w, PackedWeight):
        return w.c
    ld = _rows2d(w, "w")
    w.dtype in DT or _fail(f"weight dtype {w.dtype} not supported")
    return native.EngWeight(w.data_ptr(), None, w.shape[0], w.shape[1], ld, DT[w.dtype], 0, 0, 0)


def read_ahead_pays(w, n_rows, with_norm=False):
    """Whether the rows' next product should have ``w`` read ahead by the kernel before it: a
    ``PackedWeight`` that the decode kernel takes whole, 16 features a block (then block ``j``
    reads chunk ``j``, on die ``j % 8``), for few enough rows that most CUs have none."""
    if not isinstance(w, PackedWeight):
        return False
    return bool(native.lib().eng_read_ahead_pays(ctypes.byref(bare_context()), ctypes.byref(w.c), int(n_rows),
                                                 1 if with_norm else 0))


def for_decode(w, keep_rows=False):
    """``w`` in the packed order where the product kernels can use it (bfloat16 on the GPU),
    instead of the row-major matrix unless ``keep_rows``; anything else is returned as it is."""
    if isinstance(w, torch.Tensor) and w.is_cuda and w.dtype == torch.bfloat16 and w.dim() == 2:
        return PackedWeight(w, keep_rows=keep_rows)
    return w


_SPLIT_WS = {}
SPLIT_WS_FLOATS = 8 << 20  # 32 MB: sixteen splits of 64 rows by 8192 features

# Tests set this to split K wherever the kernels can, also at sizes where the
# launch would fill the GPU without (tiny models): 0 leaves the choice to the library.
force_splits = 0


def splits_alone(n_rows):
    """``splits`` for a product of ``n_rows`` rows whose partial sums nobody else would add (a part
    written in Python has no norm behind it that takes them): 17 to 64 rows go unsplit, since the
    second kernel that adds the parts costs more there than the split saves (a decode step of 32
    rows, 1,024 wide: 1.92 ms against 2.08); otherwise the library chooses."""
    return 1 if DECODE_MAX_ROWS < n_rows <= 64 else None


def split_workspace(device):
    """Float32 room for the partial sums of projections that split K over blocks.

    One per device, made at first use and kept (before any step is recorded):
    launches on one stream follow each other, and at most one sum is pending.
    """
    device = torch.device(device)
    key = (device.type, device.index if device.index is not None else torch.cuda.current_device())
    ws = _SPLIT_WS.get(key)
    if ws is None:
        ws = torch.empty(SPLIT_WS_FLOATS, dtype=torch.float32, device=device)
        _SPLIT_WS[key] = ws
    return ws


class PendingSum:
    """Partial products that still have to be added into the residual stream.

    A projection that splits K leaves ``n_splits`` partial sums in the
    workspace; with a ``PendingSum`` given, ``linear(accumulate=True)`` may
    stop there.  Whoever reads the stream next either adds them and norms the
    rows in one kernel (``settle_normed``) or just adds them (``settle``).
    ``allowed`` is set by a caller that promises to do so.  The state is a
    struct of the native host's (a step's own lies in its context).
    """

    def __init__(self, c=None, ctx=None):
        self.c = c if c is not None else native.EngPending()
        # the step whose pending sum this is, if any (weakly: the step holds this object)
        self._ctx = weakref.proxy(ctx) if ctx is not None else None

    allowed = property(lambda self: bool(self.c.allowed),
                       lambda self, v: setattr(self.c, "allowed", 1 if v else 0))
    target = property(lambda self: self.c.target)  # the address that the sum goes to, or None
    n_splits = property(lambda self: self.c.n_splits)

    def _native(self):
        if self._ctx is None:
            return bare_context()
        self._ctx.c.stream = raw_stream()
        return self._ctx.c

    def waits_on(self, x):
        c = self.c
        return bool(c.target) and c.target == x.data_ptr() and (c.rows, c.cols) == tuple(x.shape)

    def settle(self):
        """Add what is pending (if anything) into its target."""
        native.check(native.lib().eng_pending_settle(ctypes.byref(self._native()), ctypes.byref(self.c)))

    def settle_normed(self, out, gamma, beta, eps, ahead=None):
        """Add what is pending into its target and write the LayerNorm of the new rows to ``out``.

        ``ahead``: the weights of the product that reads ``out`` (see ``sum_partials_norm``);
        ``out`` may be a ``PackedRows`` where that product reads its rows fastest so."""
        packed = isinstance(out, PackedRows)
        if packed:
            m = native.EngMat(out.data_ptr(), out.shape[0], out.shape[1], 0, DT[out.dtype])
        else:
            _need(out.is_contiguous(), "settle_normed: out must be contiguous")
            m = native.mat(out)
        native.check(native.lib().eng_pending_settle_normed(
            ctypes.byref(self._native()), ctypes.byref(self.c), ctypes.byref(m), native.ptr(gamma),
            native.ptr(beta), float(eps), ctypes.byref(ahead.c) if ahead is not None else None, 1 if packed else 0))

    def can_norm(self, x):
        if not self.waits_on(x) or x.stride(1) != 1:
            return False
        m = native.mat(x)
        return bool(native.lib().eng_pending_can_norm(ctypes.byref(self.c), ctypes.byref(m)))


def _scatter_args(sc):
    return (
        _ptr(sc.kv.k if sc else None), _ptr(sc.kv.v if sc else None),
        _c_size_t(sc.kv.page_stride if sc else 0), _ptr(sc.block_table if sc else None),
        _c_int(sc.block_table.shape[1] if sc else 0), _ptr(sc.token_req if sc else None),
        _ptr(sc.positions if sc else None), _c_int(sc.q_width if sc else 0),
        _c_int(sc.kv_width if sc else 0), _c_int(sc.kv.head_dim if sc else 0),
        _c_int(sc.kv.page_size if sc else 0),
    )


def sum_partials(out, ws, n_splits, bias=None, gelu=False, accumulate=False, scatter=None):
    """``out = epilogue(sum of the partial products ws[:n_splits] + bias)``: the
    second step of a projection that split K (``linear`` runs it itself unless
    the sum stays pending)."""
    lib = build.load("gemm_bf16_decode")
    M, N = out.shape
    _dev(out, "out")
    _dev(ws, "ws", torch.float32)
    _need(ws.numel() >= n_splits * M * N, "sum_partials: workspace too small")
    flags = (GEMM_GELU if gelu else 0) | (GEMM_ACCUMULATE if accumulate else 0)
    if out.dtype == torch.float32:
        flags |= 0 if accumulate else GEMM_OUT_F32
    else:
        _need(out.dtype == torch.bfloat16 and not accumulate, "sum_partials: out must be float32 or bfloat16")
    if scatter is not None:
        flags |= GEMM_KV
    rc = lib.sum_partials(_ptr(out), _ptr(ws), _c_int(n_splits), _ptr(bias), _c_int(M), _c_int(N),
                          _c_int(_rows2d(out, "out")), _c_int(flags), *_scatter_args(scatter), _stream())
    build.check(lib, rc, "sum_partials")
    return out


def sum_partials_norm(h, ws, n_splits, bias, gamma, beta, eps, out, ahead=None):
    """``h += bias + sum of the partial products``; ``out = LayerNorm(h)`` (rows of ``h``, all of them).

    ``ahead``: the ``PackedWeight`` of the product that comes next; CUs that have no row read it
    meanwhile, each the chunks that a block on its own die will ask for."""
    lib = build.load("gemm_bf16_decode")
    M, N = h.shape
    _dev(h, "h", torch.float32)
    _dev(ws, "ws", torch.float32)
    packed = isinstance(out, PackedRows)
    if packed:
        _need(out.shape == (M, N), "sum_partials_norm: out's shape")
    else:
        _dev(out, "out")
        _need(out.dtype in DT and tuple(out.shape) == (M, N) and out.is_contiguous(), "sum_partials_norm: out")
    _need(ws.numel() >= n_splits * M * N, "sum_partials_norm: workspace too small")
    for name, v in (("bias", bias), ("gamma", gamma), ("beta", beta)):
        if v is not None:
            _dev(v, name, torch.float32)
            v.numel() == N or _fail(f"sum_partials_norm: {name} has {v.numel()} elements, width is {N}")
    rc = lib.sum_partials_norm(_ptr(h), _c_int(_rows2d(h, "h")), _ptr(ws), _c_int(n_splits), _ptr(bias),
                               _ptr(gamma), _ptr(beta), _c_float(eps), _ptr(out.data if packed else out),
                               _c_int(DT[out.dtype]), _c_int(1 if packed else 0),
                               _c_int(M), _c_int(N), _ptr(ahead.packed if ahead is not None else None),
                               _c_size_t(ahead.chunk_bytes if ahead is not None else 0),
                               _c_int(ahead.n_chunks if ahead is not None else 0), _stream())
    build.check(lib, rc, "sum_partials_norm")
    return out


ACTIVATIONS = {None: 0, "gelu_tanh": 1, "relu2": 2}  # the product kernels' epilogue activations, by code


def linear(out, a, w, bias=None, gelu=False, accumulate=False, variant=0, scatter=None, splits=None,
           pending=None, activation=None):
    """``out = epilogue(a @ w.T + bias)``.

    ``gelu`` asks for the tanh GELU in the epilogue; ``activation`` names any of ``ACTIVATIONS``
    (``"relu2"``: the square of the ReLU) instead.

    ``a`` is ``[M, K]`` (or a ``NormedInput``), ``w`` is ``[N, K]`` (or a
    ``PackedWeight``, whose packed copy the decode kernel reads), both
    float32 or both bfloat16; ``bias`` float32.  ``accumulate`` adds into a
    float32 ``out`` (the residual stream); otherwise ``out`` is float32 or the
    operands' dtype.  With ``scatter`` (a ``KVScatter``) the columns from
    ``scatter.q_width`` on are also written to the key/value pages.  Up to 16
    bfloat16 rows go to the decode kernels, which fuse the norm and the
    scatter; 17 to 48 rows of packed weights to the kernel that holds a
    block's weights in registers; more go to the tile kernels.  Where the launch
    would not fill the GPU, both split K over ``splits`` blocks and add the
    partial sums in a second kernel; with ``accumulate`` and a ``pending``
    that allows it, that second step is left to the next reader of ``out``.
    The choices are the native host's (``linear`` in csrc/engine.hip), which
    a model's step uses too.
    """
    L = native.lib()
    ctx = pending._native() if pending is not None else bare_context()
    call = native.EngLinear()
    call.w = weight_struct(w)
    N, K = call.w.N, call.w.K
    if isinstance(a, NormedInput):
        M = a.shape[0]
        fused = variant == 0 and L.eng_linear_norms_itself(ctypes.byref(ctx), M, N, K, DT[a.dtype], splits or 0)
        if not fused:
            a = a.materialize()
    if isinstance(a, NormedInput):
        _dev(a.x, "x", torch.float32)
        call.a.lazy, call.a.ldx = 2 if a.rms else 1, a.x.stride(0)
        call.a.m = native.EngMat(None, a.shape[0], a.shape[1], a.shape[1], DT[a.dtype])
        call.a.x, call.a.gamma, call.a.beta, call.a.eps = a.x.data_ptr(), native.ptr(a.gamma), native.ptr(a.beta), a.eps
    elif isinstance(a, PackedRows):
        call.a.m = native.EngMat(a.data_ptr(), a.shape[0], a.shape[1], 0, DT[a.dtype])
        call.a.packed = 1
    else:
        call.a.m = native.mat(a)
    if isinstance(out, PackedRows):
        call.out = native.EngMat(out.data_ptr(), out.shape[0], out.shape[1], 0, DT[out.dtype])
        call.out_packed = 1
    else:
        call.out = native.mat(out)
    if bias is not None:
        _dev(bias, "bias", torch.float32)
        _need(bias.numel() == N, "linear: bias length")
        call.bias = bias.data_ptr()
    sc = None
    if scatter is not None:
        kv = scatter.kv
        _attn_common(out, kv, scatter.block_table, scatter.token_req, scatter.positions)
        sc = native.EngScatter(kv.k.data_ptr(), kv.v.data_ptr(), kv.page_stride, kv.n_kv_heads, kv.head_dim,
                               kv.page_size, DT[kv.k.dtype], scatter.block_table.data_ptr(),
                               scatter.token_req.data_ptr(), scatter.positions.data_ptr(),
                               scatter.block_table.shape[1], scatter.q_width, scatter.kv_width, 0)
        call.scatter = ctypes.pointer(sc)
    if activation not in ACTIVATIONS:
        _fail(f"linear: unknown activation {activation!r} (known: {sorted(k for k in ACTIVATIONS if k)})")
    code = ACTIVATIONS[activation] or int(bool(gelu))
    call.gelu, call.accumulate, call.variant, call.splits = code, int(accumulate), int(variant), int(splits or 0)
    rc = L.eng_linear(ctypes.byref(ctx), ctypes.byref(call), ctypes.byref(pending.c) if pending is not None else None)
    native.check(rc, "linear")
    return out


class GroupedWeight:
    """Several weight matrices ``[n_i, K]`` that read different inputs of one shape (``planes``), for one
    product: ``groups`` is a list of ``(weight, plane)``.  The matrices lie one after the other, each
    padded with zero rows to whole blocks of ``BLOCK`` features, so that a block of a product kernel
    reads one plane only; ``columns`` are each one's first column and width in the product's rows."""

    BLOCK = 32

    def __init__(self, groups):
        K = groups[0][0].shape[1]
        parts, self.columns, self.planes, at = [], [], [], 0
        for w, plane in groups:
            _need(w.dim() == 2 and w.shape[1] == K and w.dtype == groups[0][0].dtype, "GroupedWeight: matrices of one width and dtype")
            n = w.shape[0]
            pad = -n % self.BLOCK
            parts += [w, w.new_zeros(pad, K)] if pad else [w]
            self.columns.append((at, n))
            self.planes.append(int(plane))
            at += n + pad
        whole = torch.cat(parts).contiguous()
        self.N, self.K, self.dtype = at, K, whole.dtype
        self.w = for_decode(whole)
        ends = [a + (n + self.BLOCK - 1) // self.BLOCK * self.BLOCK for a, n in self.columns]
        self.c_ends, self.c_planes = (_c_int * len(ends))(*ends), (_c_int * len(ends))(*self.planes)
        # each group by itself, over the same memory: whole blocks of sixteen features of the packed order
        self.parts = [self._slice(start, (n + 15) // 16 * 16 if isinstance(self.w, PackedWeight) else n, n) for start, n in self.columns]

    def _slice(self, start, padded, n):
        if not isinstance(self.w, PackedWeight):
            return self.w[start : start + n]
        part = PackedWeight.__new__(PackedWeight)
        tile_row = (self.K + 63) // 64 * 1024  # elements of sixteen features
        part.w, part.shape, part.dtype, part.device = None, (n, self.K), self.w.dtype, self.w.device
        part.packed = self.w.packed[start // 16 * tile_row : (start + padded) // 16 * tile_row]
        part.chunk_bytes, part.n_chunks = self.w.chunk_bytes, padded // 16
        part.c = native.EngWeight(None, part.packed.data_ptr(), n, self.K, 0, DT[part.dtype], part.chunk_bytes, part.n_chunks, 0)
        return part


def linear_groups(alloc, planes, w):
    """The products of a ``GroupedWeight``: for every group its float32 rows ``planes[plane] @ weight.T``.
    ``planes`` is contiguous ``[n, rows, K]``; the rows lie in memory that ``alloc(shape, dtype)`` gives."""
    T = planes.shape[1]
    _need(planes.is_contiguous() and planes.shape[2] == w.K and planes.dtype == w.dtype, "linear_groups: shapes")
    rows = alloc((T, w.N), torch.float32)
    out = [rows[:, a : a + n] for a, n in w.columns]
    if isinstance(w.w, PackedWeight) and 0 < T <= 64:  # few rows: one launch for all
        lib = build.load("gemm_bf16_decode")
        ws = split_workspace(planes.device)
        rc = lib.gemm_bf16_groups(_ptr(rows), _ptr(planes), _c_int(w.K), _c_size_t(T * w.K), w.c_ends, w.c_planes, _c_int(len(w.planes)),
                                  _ptr(w.w.packed), _c_int(T), _c_int(w.N), _c_int(w.K), _c_int(w.N), _ptr(ws), _c_size_t(ws.numel()),
                                  _stream())
        if rc != 2:
            build.check(lib, rc, "linear_groups")
            return out
    for view, plane, part in zip(out, w.planes, w.parts):
        linear(view, planes[plane], part, splits=splits_alone(T))
    return out


# ---------------------------------------------------------------------------


class PagedKV:
    """Keys and values of one cache slot: two views ``[n_pages, Hkv, page, hd]``."""

    __slots__ = ("k", "v", "page_stride", "n_kv_heads", "head_dim", "page_size")

    def __init__(self, k, v):
        _need(k.shape == v.shape and k.dim() == 4, "PagedKV: k and v must be [pages, heads, page, dim]")
        _need(k.dtype == v.dtype and k.dtype in DT, "PagedKV: dtype")
        for t in (k, v):
            _need(t.is_cuda and t.stride(3) == 1 and t.stride(2) == t.shape[3]
                  and t.stride(1) == t.shape[2] * t.shape[3], "PagedKV: a page must be contiguous")
        _need(k.stride(0) == v.stride(0), "PagedKV: k and v page strides differ")
        self.k, self.v = k, v
        self.page_stride = k.stride(0)
        _, self.n_kv_heads, self.page_size, self.head_dim = k.shape


def _attn_common(qkv_like, kv, block_table, token_req, positions):
    _dev(block_table, "block_table", torch.int32)
    _dev(token_req, "token_req", torch.int32)
    _dev(positions, "positions", torch.int32)
    _need(block_table.dim() == 2, "block_table must be [requests, max_blocks]")
    _need(qkv_like.dtype == kv.k.dtype, "queries and cache must share a dtype")


def kv_write(k_src, v_src, kv, block_table, token_req, positions):
    """Scatter rows of ``k_src``/``v_src`` ``[T, Hkv*hd]`` into their pages."""
    lib = build.load("attention")
    ld = _rows2d(k_src, "k_src")
    _need(_rows2d(v_src, "v_src") == ld, "kv_write: k and v row strides differ")
    n = k_src.shape[0]
    _need(k_src.shape == v_src.shape and k_src.shape[1] == kv.n_kv_heads * kv.head_dim,
          "kv_write: source width must be n_kv_heads*head_dim")
    _attn_common(k_src, kv, block_table, token_req, positions)
    _need(token_req.numel() >= n and positions.numel() >= n, "kv_write: per-token arrays too short")
    rc = lib.kv_write(
        _ptr(k_src), _ptr(v_src), _c_int(ld), _ptr(kv.k), _ptr(kv.v), _c_size_t(kv.page_stride),
        _ptr(block_table), _c_int(block_table.shape[1]), _ptr(token_req), _ptr(positions),
        _c_int(n), _c_int(kv.n_kv_heads), _c_int(kv.head_dim), _c_int(kv.page_size),
        _c_int(DT[k_src.dtype]), _stream(),
    )
    build.check(lib, rc, "kv_write")


class AttnTerms(ctypes.Structure):
    """Mirror of ``AttnTerms`` in csrc/attention_tiles.h."""

    _fields_ = [("head_scale", _vp), ("slopes", _vp), ("gate", _vp), ("ldg", _c_int), ("keep_first", _c_int),
                ("softcap", _c_float), ("dist_bias", _vp), ("n_dist", _c_int), ("sinks", _vp), ("head_gate", _vp), ("ldhg", _c_int)]


class ScoreTerms:
    """Optional terms that the four attention kernels take beside the plain causal scores:
    ``head_scale`` (float32 ``[n_heads]``, instead of ``scale``), ``slopes`` (float32 ``[n_heads]``:
    ``slope * (query position - key position)`` is taken off a score), ``gate`` (``[tokens,
    n_heads * head_dim]`` of the queries' dtype: the output is multiplied by its sigmoid),
    ``keep_first`` (with a window, the first so many keys stay visible), ``softcap`` (a scaled
    score ``s`` becomes ``softcap * tanh(s / softcap)``) and ``distance_bias`` (float32 ``[n_heads,
    n]``: entry ``min(distance, n - 1)`` of the head's row is added to a score).  A score takes
    them in this order: scale, cap, slope, table.  ``sinks`` (float32 ``[n_heads]``): the softmax's
    denominator holds ``exp(sinks[h])`` too, which brings no value.  ``head_gate`` (float32 rows of at least
    ``n_heads`` columns): head ``h``'s output is multiplied by the sigmoid of its column."""

    def __init__(self, head_scale=None, slopes=None, gate=None, keep_first=0, softcap=0.0, distance_bias=None, sinks=None,
                 head_gate=None):
        self.sinks, self.head_gate = sinks, head_gate
        self.head_scale, self.slopes, self.gate, self.keep_first = head_scale, slopes, gate, int(keep_first)
        self.softcap, self.distance_bias = float(softcap), distance_bias

    def struct(self, q, n_heads):
        """The terms as the kernels' ``_terms`` entry points and the native host take them."""
        a = self.args(q, n_heads)
        t = AttnTerms()
        t.head_scale, t.slopes, t.gate = _ptr(self.head_scale), _ptr(self.slopes), _ptr(self.gate)
        t.ldg, t.keep_first, t.softcap = a[3].value, self.keep_first, self.softcap
        _need(self.softcap >= 0.0, "softcap must not be negative")
        if self.distance_bias is not None:
            _dev(self.distance_bias, "distance_bias", torch.float32)
            _need(self.distance_bias.dim() == 2 and self.distance_bias.shape[0] == n_heads and self.distance_bias.is_contiguous(),
                  "distance_bias: a contiguous row a head")
            t.dist_bias, t.n_dist = _ptr(self.distance_bias), self.distance_bias.shape[1]
        if self.sinks is not None:
            _dev(self.sinks, "sinks", torch.float32)
            _need(self.sinks.numel() == n_heads, "sinks: one value a head")
            t.sinks = _ptr(self.sinks)
        if self.head_gate is not None:
            t.ldhg = _f32_rows(self.head_gate, "head_gate", n_heads)
            _need(self.head_gate.shape[0] >= q.shape[0], "head_gate: fewer rows than queries")
            t.head_gate = _ptr(self.head_gate)
        return t

    def args(self, q, n_heads):
        for name in ("head_scale", "slopes"):
            t = getattr(self, name)
            if t is not None:
                _dev(t, name, torch.float32)
                _need(t.numel() == n_heads, f"{name}: one value a head")
        ldg = 0
        if self.gate is not None:
            ldg = _rows2d(self.gate, "gate")
            _need(self.gate.dtype == q.dtype and self.gate.shape == q.shape, "gate: the queries' shape and dtype")
        return [_ptr(self.head_scale), _ptr(self.slopes), _ptr(self.gate), _c_int(ldg), _c_int(self.keep_first)]


def _terms(terms, q, n_heads):
    """The terms as the one argument that the kernels' ``_terms`` entry points take."""
    return [ctypes.byref((terms or ScoreTerms()).struct(q, n_heads))]


def attn_tile(out, q, kv, block_table, token_req, positions, tiles, n_tiles, n_heads, scale, window=0, terms=None):
    """Attention for tiles of up to 16 consecutive queries of one request each.

    ``tiles`` is int32 ``[n_tiles, 2]``: first flat row and number of rows.  ``terms``: ``ScoreTerms``.
    """
    lib = build.load("attention")
    ldq, ldo = _rows2d(q, "q"), _rows2d(out, "out")
    _need(q.shape[1] == n_heads * kv.head_dim, "attn_tile: q width must be n_heads*head_dim")
    _need(out.shape[1] == n_heads * kv.head_dim and out.dtype == q.dtype, "attn_tile: out shape/dtype")
    _attn_common(q, kv, block_table, token_req, positions)
    _dev(tiles, "tiles", torch.int32)
    _need(tiles.numel() >= 2 * n_tiles, "attn_tile: tile list too short")
    rc = lib.attn_tile_terms(
        _ptr(out), _ptr(q), _c_int(ldq), _c_int(ldo), _ptr(kv.k), _ptr(kv.v),
        _c_size_t(kv.page_stride), _ptr(block_table), _c_int(block_table.shape[1]),
        _ptr(token_req), _ptr(positions), _ptr(tiles), _c_int(n_tiles), _c_int(n_heads),
        _c_int(kv.n_kv_heads), _c_int(kv.head_dim), _c_int(kv.page_size), _c_int(window),
        _c_float(scale), _c_int(DT[q.dtype]), *_terms(terms, q, n_heads), _stream(),
    )
    build.check(lib, rc, "attn_tile")
    return out


ATTN_ROW_MAX_HEAD_DIM = 144  # beyond this the per-wave key tiles do not fit in LDS


def attn_row(out, q, kv, block_table, token_req, positions, rows, n_rows, n_heads, scale,
             window=0, n_splits=1, part_o=None, part_ml=None, terms=None):
    """Attention for single query rows, keys split ``n_splits`` ways."""
    lib = build.load("attention")
    ldq, ldo = _rows2d(q, "q"), _rows2d(out, "out")
    _need(q.shape[1] == n_heads * kv.head_dim, "attn_row: q width must be n_heads*head_dim")
    _need(out.shape[1] == n_heads * kv.head_dim and out.dtype == q.dtype, "attn_row: out shape/dtype")
    _need(kv.head_dim <= ATTN_ROW_MAX_HEAD_DIM,
          f"attn_row: head_dim {kv.head_dim} above {ATTN_ROW_MAX_HEAD_DIM}; use attn_tile")
    _attn_common(q, kv, block_table, token_req, positions)
    _dev(rows, "rows", torch.int32)
    _need(rows.numel() >= n_rows, "attn_row: row list too short")
    if n_splits > 1:
        _dev(part_o, "part_o", torch.float32)
        _dev(part_ml, "part_ml", torch.float32)
        _need(part_o.numel() >= n_rows * n_heads * n_splits * kv.head_dim, "attn_row: part_o too small")
        _need(part_ml.numel() >= n_rows * n_heads * n_splits * 2, "attn_row: part_ml too small")
    rc = lib.attn_row_terms(
        _ptr(out), _ptr(q), _c_int(ldq), _c_int(ldo), _ptr(kv.k), _ptr(kv.v),
        _c_size_t(kv.page_stride), _ptr(block_table), _c_int(block_table.shape[1]),
        _ptr(token_req), _ptr(positions), _ptr(rows), _c_int(n_rows), _c_int(n_heads),
        _c_int(kv.n_kv_heads), _c_int(kv.head_dim), _c_int(kv.page_size), _c_int(window),
        _c_float(scale), _c_int(n_splits), _ptr(part_o), _ptr(part_ml), _c_int(DT[q.dtype]),
        *_terms(terms, q, n_heads), _stream(),
    )
    build.check(lib, rc, "attn_row")
    return out


_TILE_SIZES = None


def attn_tile_sizes():
    """``(queries a tile of attn_tile, queries a tile of attn_prefill)``: what the kernels are
    compiled with (``csrc/attention_tiles.h``, the one place these sizes are written), asked of
    the native host, which includes the same header."""
    global _TILE_SIZES
    if _TILE_SIZES is None:
        a, b = ctypes.c_int(), ctypes.c_int()
        native.lib().eng_attn_tile_sizes(ctypes.byref(a), ctypes.byref(b))
        _TILE_SIZES = (a.value, b.value)
    return _TILE_SIZES


def rows_split_from():
    """The context length from which a decode step may split a row's keys over blocks (the native
    host's policy; recorded decode steps are kept apart by it)."""
    return int(native.lib().eng_rows_split_from())


def attn_prefill_takes(q_dtype, kv):
    """Whether the matrix-core prefill kernel takes this cache geometry."""
    return q_dtype == torch.bfloat16 and kv.head_dim in (32, 64, 128, 256)


def attn_prefill(out, q, kv, block_table, token_req, positions, tiles, n_tiles, n_heads, scale, window=0, terms=None):
    """``attn_tile`` on the matrix cores: bfloat16, head_dim 32/64/128/256, tiles of up to 128 queries."""
    lib = build.load("attention_prefill")
    ldq, ldo = _rows2d(q, "q"), _rows2d(out, "out")
    _need(q.dtype == torch.bfloat16, "attn_prefill: bfloat16 only")
    _need(q.shape[1] == n_heads * kv.head_dim, "attn_prefill: q width must be n_heads*head_dim")
    _need(out.shape[1] == n_heads * kv.head_dim and out.dtype == q.dtype, "attn_prefill: out shape/dtype")
    _attn_common(q, kv, block_table, token_req, positions)
    _dev(tiles, "tiles", torch.int32)
    _need(tiles.numel() >= 2 * n_tiles, "attn_prefill: tile list too short")
    rc = lib.attn_prefill_terms(
        _ptr(out), _ptr(q), _c_int(ldq), _c_int(ldo), _ptr(kv.k), _ptr(kv.v),
        _c_size_t(kv.page_stride), _ptr(block_table), _c_int(block_table.shape[1]),
        _ptr(token_req), _ptr(positions), _ptr(tiles), _c_int(n_tiles), _c_int(n_heads),
        _c_int(kv.n_kv_heads), _c_int(kv.head_dim), _c_int(kv.page_size), _c_int(window),
        _c_float(scale), *_terms(terms, q, n_heads), _stream(),
    )
    build.check(lib, rc, "attn_prefill")
    return out


def attn_decode_takes(q_dtype, kv):
    """Whether the register-streaming decode kernel takes this cache geometry."""
    if q_dtype not in (torch.bfloat16, torch.float32):
        return False
    key_bytes = kv.head_dim * q_dtype.itemsize
    return key_bytes in (64, 128, 256, 512) and kv.page_size % (1024 // key_bytes) == 0


def attn_decode(out, q, kv, block_table, token_req, positions, rows, n_rows, n_heads, scale,
                window=0, n_splits=1, part_o=None, part_ml=None, n_waves=4, ahead=None, ahead_chunks=0,
                rows_are_requests=False, key_tile=32, join_in_kernel=0, terms=None):
    """``attn_row`` for keys of 64 to 512 bytes (bfloat16 with head_dim 32, 64, 128 or 256, float32
    with 16, 32, 64 or 128): keys stream into registers.

    ``ahead``: a ``PackedWeight`` whose first ``ahead_chunks`` chunks the CUs without a row read
    meanwhile, each the chunks that a block on its own die will ask for (``sum_partials_norm``).
    ``rows_are_requests``: item ``i`` of ``rows`` is row ``i`` of request ``i`` (the caller says so).
    ``key_tile``: 32 or 64 keys a wave at a time.  ``join_in_kernel``: 0, a second kernel joins
    the ``n_splits`` parts of a (row, head); 1, the block that finishes it last does; 2, the same,
    and a short row takes fewer than ``n_splits`` by its own length."""
    lib = build.load("attention_decode")
    packed_out = isinstance(out, PackedRows)  # (the order that the product after attention reads fastest)
    ldq, ldo = _rows2d(q, "q"), 0 if packed_out else _rows2d(out, "out")
    _need(q.dtype in (torch.bfloat16, torch.float32), "attn_decode: bfloat16 or float32")
    _need(q.shape[1] == n_heads * kv.head_dim, "attn_decode: q width must be n_heads*head_dim")
    _need(out.shape[1] == n_heads * kv.head_dim and out.dtype == q.dtype, "attn_decode: out shape/dtype")
    if packed_out:
        _need(out.shape[0] >= q.shape[0], "attn_decode: out has fewer rows than q")
    _attn_common(q, kv, block_table, token_req, positions)
    _dev(rows, "rows", torch.int32)
    _need(rows.numel() >= n_rows, "attn_decode: row list too short")
    if n_splits > 1:
        _dev(part_o, "part_o", torch.float32)
        _dev(part_ml, "part_ml", torch.float32)
        _need(part_o.numel() >= n_rows * n_heads * n_splits * kv.head_dim, "attn_decode: part_o too small")
        _need(part_ml.numel() >= n_rows * n_heads * n_splits * 2, "attn_decode: part_ml too small")
    if rows_are_requests:
        _need(n_rows <= block_table.shape[0], "attn_decode: more rows than requests")
    rc = lib.attn_decode_rows_terms(
        _ptr(out.data if packed_out else out), _ptr(q), _c_int(ldq), _c_int(ldo), _ptr(kv.k), _ptr(kv.v),
        _c_size_t(kv.page_stride), _ptr(block_table), _c_int(block_table.shape[1]),
        _ptr(token_req), _ptr(positions), _ptr(rows), _c_int(n_rows), _c_int(n_heads),
        _c_int(kv.n_kv_heads), _c_int(kv.head_dim), _c_int(kv.page_size), _c_int(window),
        _c_float(scale), _c_int(n_splits), _ptr(part_o), _ptr(part_ml), _c_int(n_waves),
        _ptr(ahead.packed if ahead is not None else None),
        _c_size_t(ahead.chunk_bytes if ahead is not None else 0),
        _c_int(min(ahead_chunks, ahead.n_chunks) if ahead is not None else 0),
        _c_int(1 if rows_are_requests else 0), _c_int(DT[q.dtype]), _c_int(key_tile),
        _c_int(int(join_in_kernel)), *_terms(terms, q, n_heads), _stream(),
    )
    build.check(lib, rc, "attn_decode")
    return out


def attn_decode_group(out, q, kv, block_table, token_req, positions, rows, n_rows, n_heads, scale, window=0, n_splits=1,
                      part_o=None, part_ml=None, rows_are_requests=False, terms=None):
    """``attn_row`` for bfloat16 caches with head_dim 64, 128 or 256 where many query heads share a key
    head: a block takes sixteen query heads of a key head at once, on the matrix cores, so a key is
    read once for all of them.  ``n_splits`` parts of a row's keys, joined by a second kernel.  Of the
    ``terms`` only sinks and the heads' gate."""
    lib = build.load("attention_decode")
    ldq, ldo = _rows2d(q, "q"), _rows2d(out, "out")
    _need(q.dtype == torch.bfloat16 and out.dtype == q.dtype, "attn_decode_group: bfloat16 only")
    _need(q.shape[1] == n_heads * kv.head_dim and out.shape[1] == q.shape[1], "attn_decode_group: rows of n_heads*head_dim")
    _attn_common(q, kv, block_table, token_req, positions)
    _dev(rows, "rows", torch.int32)
    _need(rows.numel() >= n_rows, "attn_decode_group: row list too short")
    if n_splits > 1:
        _dev(part_o, "part_o", torch.float32)
        _dev(part_ml, "part_ml", torch.float32)
        _need(part_o.numel() >= n_rows * n_heads * n_splits * kv.head_dim, "attn_decode_group: part_o too small")
        _need(part_ml.numel() >= n_rows * n_heads * n_splits * 2, "attn_decode_group: part_ml too small")
    if rows_are_requests:
        _need(n_rows <= block_table.shape[0], "attn_decode_group: more rows than requests")
    rc = lib.attn_decode_group(
        _ptr(out), _ptr(q), _c_int(ldq), _c_int(ldo), _ptr(kv.k), _ptr(kv.v), _c_size_t(kv.page_stride), _ptr(block_table),
        _c_int(block_table.shape[1]), _ptr(token_req), _ptr(positions), _ptr(rows), _c_int(n_rows), _c_int(n_heads),
        _c_int(kv.n_kv_heads), _c_int(kv.head_dim), _c_int(kv.page_size), _c_int(window), _c_float(scale), _c_int(n_splits),
        _ptr(part_o), _ptr(part_ml), _c_int(1 if rows_are_requests else 0), *_terms(terms, q, n_heads), _stream())
    build.check(lib, rc, "attn_decode_group")
    return out


# ---------------------------------------------------------------------------


def sample_rows(tokens, token_logprob, logits, temp, top_p, min_p, min_keep, top_k, xtc_prob,
                xtc_thr, seed, counter, xtc_special=None, logprobs=None):
    """Sample one token from each row of float32 ``logits``; see csrc/sampling.hip."""
    lib = build.load("sampling")
    ld = _rows2d(logits, "logits")
    n, vocab = logits.shape
    _need(logits.dtype == torch.float32, "sample_rows: logits must be float32")
    _dev(tokens, "tokens", torch.int32)
    _dev(token_logprob, "token_logprob", torch.float32)
    for name, t, dt in (("temp", temp, torch.float32), ("top_p", top_p, torch.float32),
                        ("min_p", min_p, torch.float32), ("min_keep", min_keep, torch.int32),
                        ("top_k", top_k, torch.int32), ("xtc_prob", xtc_prob, torch.float32),
                        ("xtc_thr", xtc_thr, torch.float32), ("seed", seed, torch.int64),
                        ("counter", counter, torch.int32)):
        _dev(t, name, dt)
        t.numel() >= n or _fail(f"sample_rows: {name} shorter than the rows")
    _need(tokens.numel() >= n and token_logprob.numel() >= n, "sample_rows: outputs too short")
    n_special = 0
    if xtc_special is not None and xtc_special.numel() > 0:
        _dev(xtc_special, "xtc_special", torch.int32)
        n_special = xtc_special.numel()
    ld_lp = 0
    if logprobs is not None:
        ld_lp = _rows2d(logprobs, "logprobs")
        _need(logprobs.dtype == torch.float32 and logprobs.shape[0] >= n and logprobs.shape[1] >= vocab,
              "sample_rows: logprobs shape/dtype")
    rc = lib.sample_rows(
        _ptr(tokens), _ptr(token_logprob), _ptr(logprobs), _c_int(ld_lp), _ptr(logits), _c_int(ld),
        _c_int(n), _c_int(vocab), _ptr(temp), _ptr(top_p), _ptr(min_p), _ptr(min_keep), _ptr(top_k),
        _ptr(xtc_prob), _ptr(xtc_thr), _ptr(seed), _ptr(counter),
        _ptr(xtc_special if n_special else None), _c_int(n_special), _stream(),
    )
    build.check(lib, rc, "sample_rows")


def apply_logit_bias(logits, offsets, idx, val):
    lib = build.load("sampling")
    ld = _rows2d(logits, "logits")
    _need(logits.dtype == torch.float32, "apply_logit_bias: logits must be float32")
    _dev(offsets, "offsets", torch.int32)
    _dev(idx, "idx", torch.int32)
    _dev(val, "val", torch.float32)
    _need(offsets.numel() == logits.shape[0] + 1, "apply_logit_bias: offsets length")
    rc = lib.apply_logit_bias(_ptr(logits), _c_int(ld), _c_int(logits.shape[0]), _ptr(offsets),
                              _ptr(idx), _ptr(val), _stream())
    build.check(lib, rc, "apply_logit_bias")


def apply_penalties(logits, offsets, hist, rep, rep_ctx, pres, pres_ctx, freq, freq_ctx):
    lib = build.load("sampling")
    ld = _rows2d(logits, "logits")
    n = logits.shape[0]
    _need(logits.dtype == torch.float32, "apply_penalties: logits must be float32")
    _dev(offsets, "offsets", torch.int32)
    _dev(hist, "hist", torch.int32)
    _need(offsets.numel() == n + 1, "apply_penalties: offsets length")
    for name, t, dt in (("rep", rep, torch.float32), ("pres", pres, torch.float32),
                        ("freq", freq, torch.float32), ("rep_ctx", rep_ctx, torch.int32),
                        ("pres_ctx", pres_ctx, torch.int32), ("freq_ctx", freq_ctx, torch.int32)):
        _dev(t, name, dt)
        t.numel() >= n or _fail(f"apply_penalties: {name} shorter than the rows")
    rc = lib.apply_penalties(_ptr(logits), _c_int(ld), _c_int(n), _ptr(offsets), _ptr(hist),
                             _ptr(rep), _ptr(rep_ctx), _ptr(pres), _ptr(pres_ctx), _ptr(freq),
                             _ptr(freq_ctx), _c_int(logits.shape[1]), _stream())
    build.check(lib, rc, "apply_penalties")


# ---------------------------------------------------------------------------
# layers normed on both sides of their sublayers; heads normed one by one


def add_normed(h, y, w_post, mult, eps, w_next=None, out=None):
    """``h += mult * LN(y; w_post)`` on float32 rows, and ``out = LN(h; w_next)`` of the new rows
    where ``w_next`` is given (csrc/sandwich_block.hip)."""
    lib = build.load("sandwich_block")
    ldh, ldy = _rows2d(h, "h"), _rows2d(y, "y")
    _need(h.dtype == torch.float32 and y.dtype == torch.float32 and h.shape == y.shape, "add_normed: float32 rows of one shape")
    n, width = h.shape
    _dev(w_post, "w_post", torch.float32)
    _need(w_post.numel() == width, "add_normed: w_post length")
    if w_next is not None:
        _dev(w_next, "w_next", torch.float32)
        _dev(out, "out")
        _need(w_next.numel() == width and tuple(out.shape) == (n, width) and out.dtype in DT, "add_normed: w_next / out")
    rc = lib.add_normed(_ptr(h), _c_int(ldh), _ptr(y), _c_int(ldy), _ptr(w_post), _c_float(mult), _c_float(eps),
                        _ptr(w_next), _ptr(out if w_next is not None else None), _c_int(n), _c_int(width),
                        _c_int(DT[out.dtype] if w_next is not None else 0), _stream())
    build.check(lib, rc, "add_normed")
    return h


def scaled_pair_sum(y, a, ya, b, yb, accumulate=False):
    """``y = a * ya + b * yb`` (``+= `` with ``accumulate``) on float32 rows of one shape."""
    lib = build.load("sandwich_block")
    for name, t in (("y", y), ("ya", ya), ("yb", yb)):
        _dev(t, name, torch.float32)
        _need(t.shape == y.shape, "scaled_pair_sum: shapes differ")
    rc = lib.scaled_pair_sum(_ptr(y), _c_float(a), _ptr(ya), _c_float(b), _ptr(yb), ctypes.c_long(y.numel()),
                             _c_int(int(bool(accumulate))), _stream())
    build.check(lib, rc, "scaled_pair_sum")
    return y


def head_rmsnorm(x, n_heads, head_stride, dim, weight, eps):
    """RMS norm of the first ``dim`` columns of each of ``n_heads`` heads, ``head_stride`` columns
    apart, of every row of ``x``, in place (csrc/head_norm.hip)."""
    lib = build.load("head_norm")
    ld = _rows2d(x, "x")
    _need(x.dtype in DT, "head_rmsnorm: float32 or bfloat16")
    _need(0 < dim <= head_stride and (n_heads - 1) * head_stride + dim <= x.shape[1], "head_rmsnorm: heads do not fit the rows")
    if weight is not None:
        _dev(weight, "weight", torch.float32)
        _need(weight.numel() == dim, "head_rmsnorm: weight length")
    rc = lib.head_rmsnorm(_ptr(x), _c_int(ld), _c_int(x.shape[0]), _c_int(n_heads), _c_int(head_stride), _c_int(dim),
                          _ptr(weight), _c_float(eps), _c_int(DT[x.dtype]), _stream())
    build.check(lib, rc, "head_rmsnorm")
    return x


# ---------------------------------------------------------------------------
# mixers with a decaying matrix state per head (csrc/linear_state.hip)


class ScanArgs(ctypes.Structure):
    """Mirror of ``ScanArgs`` in csrc/linear_state.hip."""

    _fields_ = [("q", _vp), ("k", _vp), ("v", _vp), ("ldq", _c_int), ("ldk", _c_int), ("ldv", _c_int),
                ("log_a", _vp), ("decay", _vp), ("k_scale", _vp), ("k_mult", _c_float), ("skip", _vp),
                ("rot_dims", _c_int), ("inv_freq", _vp), ("positions", _vp), ("unit_rms", _c_int), ("eps", _c_float),
                ("gate", _vp), ("ldg", _c_int), ("out", _vp), ("ldo", _c_int), ("out_dtype", _c_int),
                ("state", _vp), ("state_stride", _c_size_t), ("state_offset", _c_size_t), ("seq_start", _vp),
                ("seq_len", _vp), ("slot_ids", _vp), ("n_requests", _c_int), ("H", _c_int), ("Hk", _c_int),
                ("N", _c_int), ("P", _c_int), ("n_tokens_hint", _c_int), ("chan_a", _vp), ("ldca", _c_int),
                ("chan_logit", _c_int), ("chan_mult", _c_float), ("norm_w", _vp), ("norm_stride", _c_int), ("bonus", _vp)]


def _f32_rows(t, name, min_cols):
    ld = _rows2d(t, name)
    _need(t.dtype == torch.float32, f"{name} must be float32")
    _need(t.shape[1] >= min_cols, f"{name}: rows of {t.shape[1]} columns, {min_cols} needed")
    return ld


def state_scan(out, q, k, v, state, state_offset, seq_start, seq_len, slot_ids, n_requests, n_heads, n_key_heads,
               key_dim, value_dim, log_a=None, decay=None, k_scale=None, k_mult=1.0, skip=None, rot_dims=0,
               inv_freq=None, positions=None, unit_rms=False, eps=0.0, gate=None, chunked=False, spans=None,
               channel_decay=None, channel_logit_mult=None, norm_weight=None, bonus=None):
    """``S = a S + k v^T; o = S^T q`` token by token for every (request, head), from and into the
    requests' rows of ``state`` (float32 ``[slots, floats a request]``, head ``h``'s matrix
    ``[key_dim, value_dim]`` at ``state_offset + h * key_dim * value_dim``).  ``q``, ``k``
    (``[tokens, >= n_key_heads * key_dim]``), ``v`` (``[tokens, >= n_heads * value_dim]``) and
    ``gate`` are float32 rows (column views of a projection's output are fine; with ``chunked`` and
    ``rot_dims`` the rows of ``q`` and ``k`` are turned in place, so they are work memory); ``out`` is
    ``[tokens, n_heads * value_dim]`` in float32 or bfloat16.  ``chunked``: the kernel that takes
    up to 64 tokens of a request at a time (for steps in which a request brings many); otherwise
    token by token.  ``spans``: ``(tokens a span, number of spans, span_req, span_start,
    span_first, alloc)`` cuts long portions into spans that run side by side (int32 device arrays:
    the request and the first token of every span, counted from the request's first token of
    this step, and every request's first span; ``alloc(shape, dtype)`` gives the work memory).
    ``channel_decay`` (float32 ``[tokens, >= n_heads * key_dim]``): a decay for every key channel
    instead of one a head, given as its logarithm, or, with ``channel_logit_mult = m``, as a logit
    ``z`` with ``log a = m * log sigmoid(z)``.  ``norm_weight`` (float32 ``[value_dim]``): with
    ``unit_rms``, the normed output times this weight, the same for every head (``[n_heads *
    value_dim]``: a weight of its own for every head).  ``bonus`` (float32 ``[n_heads * key_dim]``,
    with ``channel_decay`` and ``chunked``): ``o_t = (S_(t-1) + diag(bonus) k_t v_t^T)^T q_t``.
    See csrc/linear_state.hip for the options."""
    lib = build.load("linear_state")
    a = ScanArgs()
    T = out.shape[0]
    a.ldq, a.ldk = _f32_rows(q, "q", n_key_heads * key_dim), _f32_rows(k, "k", n_key_heads * key_dim)
    a.ldv = _f32_rows(v, "v", n_heads * value_dim)
    _need(q.shape[0] >= T and k.shape[0] >= T and v.shape[0] >= T, "state_scan: fewer operand rows than output rows")
    a.q, a.k, a.v = q.data_ptr(), k.data_ptr(), v.data_ptr()
    for name, t in (("log_a", log_a), ("k_scale", k_scale)):
        if t is not None:
            _dev(t, name, torch.float32)
            _need(t.numel() >= T * n_heads, f"state_scan: {name} is [tokens, heads]")
            setattr(a, name, t.data_ptr())
    for name, t in (("decay", decay), ("skip", skip)):
        if t is not None:
            _dev(t, name, torch.float32)
            _need(t.numel() == n_heads, f"state_scan: {name} has one value a head")
            setattr(a, name, t.data_ptr())
    _need(log_a is not None or decay is not None or channel_decay is not None,
          "state_scan: a decay per token, per head or per key channel is needed")
    if channel_decay is not None:
        _need(n_key_heads == n_heads, "state_scan: decays per key channel need a key head for every head")
        a.ldca, a.chan_a = _f32_rows(channel_decay, "channel_decay", n_heads * key_dim), channel_decay.data_ptr()
        _need(channel_decay.shape[0] >= T, "state_scan: fewer decay rows than output rows")
        if channel_logit_mult is not None:
            a.chan_logit, a.chan_mult = 1, float(channel_logit_mult)
    if norm_weight is not None:
        _dev(norm_weight, "norm_weight", torch.float32)
        _need(unit_rms and norm_weight.numel() in (value_dim, n_heads * value_dim), "state_scan: norm_weight has value_dim values (a head) and goes with unit_rms")
        a.norm_w, a.norm_stride = norm_weight.data_ptr(), value_dim if norm_weight.numel() != value_dim else 0
    if bonus is not None:
        _dev(bonus, "bonus", torch.float32)
        _need(channel_decay is not None and chunked and bonus.numel() == n_heads * key_dim, "state_scan: a bonus for every key channel")
        a.bonus = bonus.data_ptr()
    a.k_mult = float(k_mult)
    if rot_dims:
        _dev(inv_freq, "inv_freq", torch.float32)
        _dev(positions, "positions", torch.int32)
        _need(inv_freq.numel() == rot_dims // 2 and positions.numel() >= T, "state_scan: inv_freq / positions")
        a.rot_dims, a.inv_freq, a.positions = int(rot_dims), inv_freq.data_ptr(), positions.data_ptr()
    a.unit_rms, a.eps = int(bool(unit_rms)), float(eps)
    if gate is not None:
        a.ldg, a.gate = _f32_rows(gate, "gate", n_heads * value_dim), gate.data_ptr()
    a.ldo = _rows2d(out, "out")
    _need(out.dtype in DT and out.shape[1] == n_heads * value_dim, "state_scan: out is [tokens, heads * value_dim]")
    a.out, a.out_dtype = out.data_ptr(), DT[out.dtype]
    _dev(state, "state", torch.float32)
    _need(state.dim() == 2 and state_offset + n_heads * key_dim * value_dim <= state.shape[1], "state_scan: the state rows are too short")
    a.state, a.state_stride, a.state_offset = state.data_ptr(), state.stride(0), int(state_offset)
    for name, t in (("seq_start", seq_start), ("seq_len", seq_len), ("slot_ids", slot_ids)):
        _dev(t, name, torch.int32)
        _need(t.numel() >= n_requests, f"state_scan: {name} is shorter than the requests")
        setattr(a, name, t.data_ptr())
    a.n_requests, a.H, a.Hk, a.N, a.P = int(n_requests), int(n_heads), int(n_key_heads), int(key_dim), int(value_dim)
    a.n_tokens_hint = int(T)
    if spans is not None and chunked:
        span, n_spans, span_req, span_start, span_first, alloc = spans
        for name, t, n in (("span_req", span_req, n_spans), ("span_start", span_start, n_spans), ("span_first", span_first, n_requests)):
            _dev(t, name, torch.int32)
            _need(t.numel() >= n, f"state_scan: {name} too short")
        ws_state = alloc((n_spans * n_heads * key_dim * value_dim,), torch.float32)
        ws_decay = alloc((n_spans * n_heads * (key_dim if channel_decay is not None else 1),), torch.float32)
        rc = lib.state_scan(ctypes.byref(a), _c_int(2), _c_int(span), _c_int(n_spans), _ptr(span_req), _ptr(span_start),
                            _ptr(span_first), _ptr(ws_state), _ptr(ws_decay), _stream())
    else:
        rc = lib.state_scan(ctypes.byref(a), _c_int(int(bool(chunked))), _c_int(0), _c_int(0), None, None, None, None, None,
                            _stream())
    build.check(lib, rc, "state_scan")
    return out


# ---------------------------------------------------------------------------
# between a projection and the attention that reads its heads, and behind it (csrc/head_prepare.hip)


class PrepareArgs(ctypes.Structure):
    """Mirror of ``PrepareArgs`` in csrc/head_prepare.hip."""

    _fields_ = [("src", _vp), ("lds", _c_int), ("src_col", _c_int), ("src_stride", _c_int), ("n_rows", _c_int),
                ("n_heads", _c_int), ("dim", _c_int), ("norm_dim", _c_int), ("norm_w", _vp), ("eps", _c_float),
                ("rot_off", _c_int), ("rot_dims", _c_int), ("interleaved", _c_int), ("inv_freq", _vp),
                ("rot_mult", _c_float), ("positions", _vp), ("dst", _vp), ("ldd", _c_int), ("dst_stride", _c_int),
                ("dst_fill", _c_int), ("copies", _c_int), ("dst_head", _vp),
                ("conv_w", _vp), ("taps", _c_int), ("conv_channels", _c_int), ("conv_single", _c_int), ("conv_state", _vp),
                ("conv_state_stride", _c_size_t), ("conv_offset", _c_size_t), ("seq_start", _vp), ("slot_ids", _vp),
                ("token_req", _vp), ("block_table", _vp), ("max_blocks", _c_int), ("page_size", _c_int),
                ("page_stride", _c_size_t), ("norm_whole", _c_int)]


class ConvolutionAhead:
    """A causal convolution that ``head_prepare`` runs over its source's columns on their way in:
    ``y[t, c] = sum_j weight[c, j] * u[t - taps + 1 + j, c]`` over each request's own tokens (column
    ``c`` of ``u`` is channel ``c``); the inputs of earlier steps come from the request's row of
    ``state`` (``[taps - 1, channels]`` at ``offset``, the latest last).  With ``single`` (every
    request brings one token) the kernel also moves these up by one; otherwise ``conv_state_update``
    does afterwards."""

    def __init__(self, weight, state, offset, token_req, seq_start, slot_ids, single):
        _dev(weight, "weight", torch.float32)
        _dev(state, "state", torch.float32)
        for name, t in (("token_req", token_req), ("seq_start", seq_start), ("slot_ids", slot_ids)):
            _dev(t, name, torch.int32)
        channels, taps = weight.shape
        _need(weight.is_contiguous() and state.dim() == 2 and offset + (taps - 1) * channels <= state.shape[1],
              "a convolution's weight is [channels, taps] and its state rows hold taps - 1 inputs of every channel")
        self.weight, self.state, self.offset, self.single = weight, state, int(offset), bool(single)
        self.token_req, self.seq_start, self.slot_ids = token_req, seq_start, slot_ids


class PagesOut:
    """The keys' (or values') pages of a cache view as the place ``head_prepare`` writes to: a row goes
    where its request's block table and its position say, as ``kv_write`` has it."""

    def __init__(self, kv, values, block_table, token_req, positions):
        self.pages = kv.v if values else kv.k
        self.kv, self.block_table, self.token_req, self.positions = kv, block_table, token_req, positions
        for name, t in (("block_table", block_table), ("token_req", token_req), ("positions", positions)):
            _dev(t, name, torch.int32)
        self.dtype, self.shape = self.pages.dtype, None


def head_prepare(dst, src, src_col, n_heads, dim, **options):
    """Heads of a float32 projection row on their way to an attention: head ``h`` is ``dim`` columns
    of ``src`` from ``src_col + h * src_stride``; RMS norm over its first ``norm_dim`` columns
    (times ``norm_weight``, shared by the heads); rotation of ``rot_dims`` columns from ``rot_off``
    by ``position * inv_freq[i]`` (pairs ``(2i, 2i + 1)`` with ``interleaved``, else ``(i, i +
    rot_dims / 2)``; cos and sin times ``rot_mult``); written to ``dst`` (float32 or bfloat16) at
    column ``dst_head[c, h] * dst_stride`` for each of ``copies`` copies (``h * dst_stride`` without
    a table), with zeros from ``dim`` up to ``dst_fill`` columns.  ``norm_whole = n``: the norm runs over
    the ``n`` columns from ``src_col`` on, all heads at once, with ``norm_weight`` of ``n`` values, and
    every column of a head is normed.  ``conv`` (a ``ConvolutionAhead``):
    the source's columns pass a causal convolution first.  ``dst`` may be a ``PagesOut``."""
    lib = build.load("head_prepare")
    a = _prepare_args(dst, src, src_col, n_heads, dim, **options)
    rc = lib.head_prepare(ctypes.byref(a), _c_int(DT[dst.dtype]), _stream())
    build.check(lib, rc, "head_prepare")
    return dst


def head_prepare_many(*calls):
    """Several ``head_prepare`` calls in one launch: each of ``calls`` is ``(dst, src, src_col,
    n_heads, dim, options)``; at most four, their ``dst`` (a matrix or a ``PagesOut``) of one dtype."""
    lib = build.load("head_prepare")
    _need(1 <= len(calls) <= 4 and len({c[0].dtype for c in calls}) == 1, "head_prepare_many: one to four calls, outputs of one dtype")
    args = (PrepareArgs * len(calls))(*[_prepare_args(*c[:5], **c[5]) for c in calls])
    rc = lib.head_prepare_many(args, _c_int(len(calls)), _c_int(DT[calls[0][0].dtype]), _stream())
    build.check(lib, rc, "head_prepare_many")


def _prepare_args(dst, src, src_col, n_heads, dim, src_stride=None, dst_stride=None, dst_fill=None, norm_dim=0,
                  norm_weight=None, eps=0.0, rot_off=0, rot_dims=0, inv_freq=None, rot_mult=1.0, interleaved=True,
                  positions=None, dst_head=None, copies=1, conv=None, norm_whole=0):
    a = PrepareArgs()
    src_stride = dim if src_stride is None else src_stride
    n_rows = src.shape[0] if isinstance(dst, PagesOut) else dst.shape[0]
    dst_stride = dim if dst_stride is None else dst_stride
    a.lds = _f32_rows(src, "src", src_col + (n_heads - 1) * src_stride + dim)
    a.src, a.src_col, a.src_stride = src.data_ptr(), int(src_col), int(src_stride)
    a.n_rows, a.n_heads, a.dim = n_rows, int(n_heads), int(dim)
    _need(src.shape[0] >= n_rows, "head_prepare: fewer source rows than rows of dst")
    a.norm_dim, a.eps, a.norm_whole = int(norm_dim), float(eps), int(norm_whole)
    if norm_weight is not None:
        _dev(norm_weight, "norm_weight", torch.float32)
        _need(norm_weight.numel() == (norm_whole or norm_dim), "head_prepare: norm_weight has norm_dim values (norm_whole, for a norm over all heads)")
        a.norm_w = norm_weight.data_ptr()
    if rot_dims:
        _dev(inv_freq, "inv_freq", torch.float32)
        _dev(positions, "positions", torch.int32)
        _need(inv_freq.numel() == rot_dims // 2 and positions.numel() >= n_rows, "head_prepare: inv_freq / positions")
        a.rot_off, a.rot_dims, a.interleaved = int(rot_off), int(rot_dims), int(bool(interleaved))
        a.inv_freq, a.rot_mult, a.positions = inv_freq.data_ptr(), float(rot_mult), positions.data_ptr()
    _need(dst.dtype in DT, "head_prepare: dst is float32 or bfloat16")
    a.dst_stride, a.dst_fill, a.copies = int(dst_stride), int(dst_fill or dim), int(copies)
    if dst_head is not None:
        _dev(dst_head, "dst_head", torch.int32)
        _need(dst_head.numel() == copies * n_heads, "head_prepare: dst_head is [copies, heads]")
        a.dst_head = dst_head.data_ptr()
    if isinstance(dst, PagesOut):
        kv = dst.kv
        _need(kv.head_dim == dst_stride and n_heads * copies <= kv.n_kv_heads and dst.token_req.numel() >= n_rows
              and dst.positions.numel() >= n_rows, "head_prepare: the heads do not fit the cache's pages")
        a.dst, a.block_table, a.max_blocks = dst.pages.data_ptr(), dst.block_table.data_ptr(), dst.block_table.shape[1]
        a.page_size, a.page_stride = kv.page_size, kv.page_stride
        a.token_req, a.positions = dst.token_req.data_ptr(), dst.positions.data_ptr()
    else:
        a.ldd, a.dst = _rows2d(dst, "dst"), dst.data_ptr()
        _need(dst.shape[1] >= (n_heads * copies - 1) * dst_stride + a.dst_fill, "head_prepare: dst rows are too short for the heads")
    if conv is not None:
        channels, taps = conv.weight.shape
        _need(src.shape[1] >= channels and conv.token_req.numel() >= n_rows, "head_prepare: the convolution's channels are the source's columns")
        a.conv_w, a.taps, a.conv_channels, a.conv_single = conv.weight.data_ptr(), taps, channels, int(conv.single)
        a.conv_state, a.conv_state_stride, a.conv_offset = conv.state.data_ptr(), conv.state.stride(0), conv.offset
        a.seq_start, a.slot_ids, a.token_req = conv.seq_start.data_ptr(), conv.slot_ids.data_ptr(), conv.token_req.data_ptr()
    return a


def diff_combine(out, att, head_stride, first, second, lam, mult, eps, vdim):
    """``out[t, h] = mult * unit_rms(att[t, first[h]] - lam * att[t, second[h]])`` over the first
    ``vdim`` columns of heads that lie ``head_stride`` apart in ``att``."""
    lib = build.load("head_prepare")
    lda, ldo = _rows2d(att, "att"), _rows2d(out, "out")
    _dev(first, "first", torch.int32)
    _dev(second, "second", torch.int32)
    n_heads = first.numel()
    _need(second.numel() == n_heads and out.dtype == att.dtype and att.dtype in DT and att.shape[0] >= out.shape[0], "diff_combine: shapes")
    rc = lib.diff_combine(_ptr(att), _c_int(lda), _c_int(head_stride), _ptr(first), _ptr(second), _c_float(lam), _c_float(mult),
                          _c_float(eps), _c_int(out.shape[0]), _c_int(n_heads), _c_int(vdim), _ptr(out), _c_int(ldo),
                          _c_int(DT[out.dtype]), _stream())
    build.check(lib, rc, "diff_combine")
    return out


def head_gate(x, head_stride, n_heads, gate):
    """``x[t, h, :] *= sigmoid(gate[t, h])`` in place; ``gate`` float32 rows of at least ``n_heads`` columns."""
    lib = build.load("head_prepare")
    ldx, ldg = _rows2d(x, "x"), _f32_rows(gate, "gate", n_heads)
    _need(x.dtype in DT and x.shape[1] >= n_heads * head_stride and gate.shape[0] >= x.shape[0], "head_gate: shapes")
    rc = lib.head_gate(_ptr(x), _c_int(ldx), _c_int(head_stride), _c_int(n_heads), _ptr(gate), _c_int(ldg),
                       _c_int(x.shape[0]), _c_int(DT[x.dtype]), _stream())
    build.check(lib, rc, "head_gate")
    return x


FAST_HEAD_DIMS = (16, 32, 64, 128, 256)
WIDE_HEAD_DIM = 1024  # the widest head that the general tile kernel takes (it stages 256 columns at a time)


def attention_head_dim(columns):
    """The head size under which a mixer with heads of ``columns`` columns keeps its pages: the
    next size that the matrix-core and the streaming attention kernels take (the columns beyond
    the head's own are zeros in queries, keys and values)."""
    for n in FAST_HEAD_DIMS:
        if columns <= n:
            return n
    raise ValueError(f"heads of {columns} columns: the attention kernels take at most {FAST_HEAD_DIMS[-1]}")


def attend(ctx, out, q, cache, n_heads, n_kv_heads, head_dim, scale, window=0, terms=None):
    """Causal attention of the step's queries ``q`` ``[tokens, n_heads * head_dim]`` over the pages
    of ``cache`` (a ``CacheView``), into ``out``: the native host chooses among the attention kernels
    as it does for the built-in attention part (single rows to the decode kernels, portions to the
    tile kernels), by the step arrays that part declares (``parts.attention.CausalSelfAttention``:
    a mixer that calls this names the same ``step_arrays_key``).  ``terms``: ``ScoreTerms``."""
    from ..parts.attention import CausalSelfAttention as A

    base = native.array_ids(A.step_arrays_key, A.step_array_names)
    qm, om = native.mat(q), native.mat(out)
    t = terms.struct(q, n_heads) if terms is not None else None
    with ctx.enter():
        if t is None:
            rc = native.lib().eng_attend(ctypes.byref(ctx.c), ctypes.byref(om), ctypes.byref(qm), cache.slot, int(n_heads),
                                         int(n_kv_heads), int(head_dim), int(window), float(scale), base)
        else:
            rc = native.lib().eng_attend_terms(ctypes.byref(ctx.c), ctypes.byref(om), ctypes.byref(qm), cache.slot,
                                               int(n_heads), int(n_kv_heads), int(head_dim), int(window), float(scale),
                                               base, ctypes.byref(t))
    native.check(rc, "attend")
    return out


def ssm_prepare(xbc, dt, log_a, u, conv_col, dt_col, conv_w, conv_b, dt_bias, a_log, state, conv_offset, token_req,
                seq_start, slot_ids, single_tokens=False):
    """The causal convolution (with the requests' last inputs from ``state``), bias and silu of
    columns ``conv_col ..`` of the float32 rows ``u`` into ``xbc``; ``dt = softplus(u[:, dt_col + h]
    + dt_bias[h])`` and ``log_a = -exp(a_log[h]) * dt`` (csrc/linear_state.hip).  ``single_tokens``:
    every request brings one token, and the kernel also does what ``conv_state_update`` would."""
    lib = build.load("linear_state")
    ldu = _f32_rows(u, "u", 1)
    T, C = xbc.shape
    H = dt.shape[1]
    taps = conv_w.shape[1]
    for name, t in (("xbc", xbc), ("dt", dt), ("log_a", log_a), ("conv_w", conv_w), ("dt_bias", dt_bias),
                    ("a_log", a_log), ("state", state)):
        _dev(t, name, torch.float32)
    if conv_b is not None:
        _dev(conv_b, "conv_b", torch.float32)
        _need(conv_b.numel() == C, "ssm_prepare: conv_b length")
    _need(tuple(conv_w.shape) == (C, taps) and dt.shape == log_a.shape and dt.shape[0] == T, "ssm_prepare: shapes")
    _need(dt_bias.numel() == H and a_log.numel() == H and u.shape[0] >= T, "ssm_prepare: per-head vectors")
    _need(conv_col + C <= u.shape[1] and dt_col + H <= u.shape[1], "ssm_prepare: columns beyond the rows")
    _need(state.dim() == 2 and conv_offset + (taps - 1) * C <= state.shape[1], "ssm_prepare: the state rows are too short")
    for name, t in (("token_req", token_req), ("seq_start", seq_start), ("slot_ids", slot_ids)):
        _dev(t, name, torch.int32)
    rc = lib.ssm_prepare(_ptr(u), _c_int(ldu), _c_int(conv_col), _c_int(dt_col), _ptr(conv_w), _ptr(conv_b),
                         _c_int(taps), _c_int(C), _c_int(H), _ptr(dt_bias), _ptr(a_log), _ptr(state),
                         _c_size_t(state.stride(0)), _c_size_t(conv_offset), _ptr(token_req), _ptr(seq_start),
                         _ptr(slot_ids), _ptr(xbc), _ptr(dt), _ptr(log_a), _c_int(T), _c_int(int(bool(single_tokens))),
                         _stream())
    build.check(lib, rc, "ssm_prepare")


def conv_state_update(u, conv_col, taps, n_channels, state, conv_offset, seq_start, seq_len, slot_ids, n_requests):
    """Each request's last ``taps - 1`` inputs (columns ``conv_col ..`` of ``u``) into its state row."""
    lib = build.load("linear_state")
    ldu = _f32_rows(u, "u", conv_col + n_channels)
    _dev(state, "state", torch.float32)
    _need(state.dim() == 2 and conv_offset + (taps - 1) * n_channels <= state.shape[1], "conv_state_update: the state rows are too short")
    for name, t in (("seq_start", seq_start), ("seq_len", seq_len), ("slot_ids", slot_ids)):
        _dev(t, name, torch.int32)
        _need(t.numel() >= n_requests, f"conv_state_update: {name} is shorter than the requests")
    rc = lib.conv_state_update(_ptr(u), _c_int(ldu), _c_int(conv_col), _c_int(taps), _c_int(n_channels), _ptr(state),
                               _c_size_t(state.stride(0)), _c_size_t(conv_offset), _ptr(seq_start), _ptr(seq_len),
                               _ptr(slot_ids), _c_int(n_requests), _stream())
    build.check(lib, rc, "conv_state_update")


def gated_group_rmsnorm(out, y, z, weight, groups, eps):
    """``out = RMSnorm(y * silu(z))`` in ``groups`` equal parts of a row, times ``weight``."""
    lib = build.load("linear_state")
    T, width = out.shape
    ldy, ldz, ldo = _f32_rows(y, "y", width), _f32_rows(z, "z", width), _rows2d(out, "out")
    _dev(weight, "weight", torch.float32)
    _need(weight.numel() == width and out.dtype in DT and y.shape[0] >= T and z.shape[0] >= T, "gated_group_rmsnorm: shapes")
    rc = lib.gated_group_rmsnorm(_ptr(y), _c_int(ldy), _ptr(z), _c_int(ldz), _ptr(weight), _c_float(eps), _c_int(T),
                                 _c_int(width), _c_int(groups), _ptr(out), _c_int(ldo), _c_int(DT[out.dtype]), _stream())
    build.check(lib, rc, "gated_group_rmsnorm")
    return out


# ---------------------------------------------------------------------------
# experts chosen per token (csrc/experts.hip)


class RouteArgs(ctypes.Structure):
    """Mirror of ``RouteArgs`` in csrc/experts.hip."""

    _fields_ = [("z", _vp), ("ldz", _c_int), ("correction", _vp), ("n_out", _c_int), ("renorm", _c_int), ("mult", _c_float),
                ("sigmoid", _c_int), ("groups", _c_int), ("keep", _c_int)]


ROUTER_SCORES = ("softmax", "sigmoid")


class Route:
    """How experts are chosen from router outputs: a score is the ``softmax`` over all outputs or the
    ``sigmoid`` of each; the ``top`` largest of score + ``correction`` (float32 ``[outputs]`` or None) are
    chosen, with ``groups = (count, keep)`` only out of the ``keep`` best of ``count`` equal groups of
    neighbours (a group counts the sum of its two largest choice scores); a pick's weight is its score,
    with ``renormalize`` divided by the picks' sum (+ 1e-20), times ``weight_scale``."""

    def __init__(self, correction=None, renormalize=False, weight_scale=1.0, scores="softmax", groups=None):
        _need(scores in ROUTER_SCORES, f"router scores {scores!r} (known: {ROUTER_SCORES})")
        self.correction, self.renormalize, self.weight_scale, self.scores = correction, bool(renormalize), float(weight_scale), scores
        self.groups = tuple(int(n) for n in groups) if groups is not None else (1, 1)

    def struct(self, z, n_out, n_tokens):
        a = RouteArgs()
        a.ldz, a.z, a.n_out = _f32_rows(z, "z", n_out), z.data_ptr(), int(n_out)
        _need(z.shape[0] >= n_tokens, "router: fewer rows of outputs than tokens")
        if self.correction is not None:
            _dev(self.correction, "correction", torch.float32)
            _need(self.correction.numel() == n_out, "router: correction length")
            a.correction = self.correction.data_ptr()
        a.renorm, a.mult, a.sigmoid = int(self.renormalize), self.weight_scale, int(self.scores == "sigmoid")
        a.groups, a.keep = self.groups
        return a


def _picks(idx, weight, T, top):
    _dev(idx, "idx", torch.int32)
    _dev(weight, "weight", torch.float32)
    _need(idx.numel() >= T * top and weight.numel() >= T * top, "router: idx / weight too short")


def router_choice(idx, weight, z, correction, top, renormalize=False, weight_scale=1.0, scores="softmax", groups=None):
    """From float32 router outputs ``z`` ``[tokens, outputs]`` every token's experts into ``idx`` (int32
    ``[tokens, top]``) and their weights into ``weight`` (``Route``)."""
    lib = build.load("experts")
    T, n_out = z.shape
    _picks(idx, weight, T, top)
    a = Route(correction, renormalize, weight_scale, scores, groups).struct(z, n_out, T)
    rc = lib.router_choice(ctypes.byref(a), _c_int(T), _c_int(top), _ptr(idx), _ptr(weight), _stream())
    build.check(lib, rc, "router_choice")


def route_and_gate(idx, weight, act, zu, correction, top, n_out, renormalize=False, weight_scale=1.0, scores="softmax", groups=None):
    """``router_choice`` on the first ``n_out`` columns of the float32 rows ``zu`` and ``silu_mul`` on
    the ``2 * act.shape[1]`` columns behind them, in one launch (for steps of few tokens)."""
    lib = build.load("experts")
    ldo = _rows2d(act, "act")
    T, F = act.shape
    _need(zu.shape[0] >= T and zu.shape[1] == n_out + 2 * F and act.dtype in DT, "route_and_gate: shapes")
    _picks(idx, weight, T, top)
    a = Route(correction, renormalize, weight_scale, scores, groups).struct(zu, n_out, T)
    rc = lib.route_and_gate(ctypes.byref(a), _c_int(T), _c_int(top), _c_int(F), _ptr(idx), _ptr(weight), _ptr(act), _c_int(ldo),
                            _c_int(DT[act.dtype]), _stream())
    build.check(lib, rc, "route_and_gate")


GATE_ACTIVATIONS = {"silu": 0, "gelu_tanh": 1}


def silu_mul(out, gate_up, activation="silu"):
    """``out = act(gate_up[:, :F]) * gate_up[:, F:2F]`` with ``F = out.shape[1]``; ``activation``:
    ``silu``, or ``gelu_tanh`` (``0.5 z (1 + tanh(sqrt(2 / pi) (z + 0.044715 z^3)))``)."""
    lib = build.load("experts")
    ld, ldo = _rows2d(gate_up, "gate_up"), _rows2d(out, "out")
    T, F = out.shape
    _need(gate_up.dtype == out.dtype and out.dtype in DT and gate_up.shape[1] == 2 * F and gate_up.shape[0] >= T, "silu_mul: shapes")
    _need(activation in GATE_ACTIVATIONS, f"silu_mul: activation {activation!r} (known: {sorted(GATE_ACTIVATIONS)})")
    rc = lib.act_mul(_ptr(gate_up), _c_int(ld), _ptr(out), _c_int(ldo), _c_int(T), _c_int(F), _c_int(DT[out.dtype]),
                     _c_int(GATE_ACTIVATIONS[activation]), _stream())
    build.check(lib, rc, "silu_mul")
    return out


EXPERT_ACTIVATIONS = {"silu": 0, "clamped": 1}


def _expert_activation(activation, limit):
    _need(activation in EXPERT_ACTIVATIONS, f"experts: activation {activation!r} (known: {sorted(EXPERT_ACTIVATIONS)})")
    return _c_int(EXPERT_ACTIVATIONS[activation]), _c_float(limit)


class NextNorm(ctypes.Structure):
    """Mirror of ``NextNorm`` in csrc/experts.hip."""

    _fields_ = [("alpha", _vp), ("w", _vp), ("b", _vp), ("out", _vp)]


def _next_norm(after, x, accumulate):
    out, norm = after
    _need(out.is_contiguous() and out.dtype == x.dtype and out.shape == x.shape and accumulate, "experts: after goes with rows that are complete here")
    nn = NextNorm()
    nn.alpha, nn.w, nn.b = (p.value for p in _tanh_norm(norm, x.shape[1]))
    nn.out = out.data_ptr()
    return nn


ROUTED_MOST = 64  # up to this many picks a token, ``expert_rows`` makes the choice itself


def expert_rows(y, x, w_gate, w_up, w_down, idx, weight, top, act, accumulate=True, activation="silu", limit=0.0, route=None, after=None):
    """``y (+)= sum over a token's picks of weight * expert(x)``, reading only the picked experts'
    weights (``w_gate``, ``w_up``: ``[experts, F, width]``, ``w_down``: ``[experts, width, F]``); a
    pick at or beyond the number of experts gives ``weight * x``.  ``act``: room for ``[tokens *
    top, F]`` of ``x``'s dtype.  ``activation``: ``silu(g) * u``, or ``clamped``: ``g sigmoid(1.702 g) (u
    + 1)`` with ``g`` at most ``limit`` and ``u`` within ``[-limit, limit]``.  ``route = (z, Route)``:
    the choice is made here (``router_choice``), into ``idx`` and ``weight``.
    ``after = (out, norm)``: the rows that this completes (``accumulate``) pass ``dynamic_tanh`` with
    ``norm`` into ``out`` (``x``'s dtype) too."""
    lib = build.load("experts")
    ldx, ldy = _rows2d(x, "x"), _rows2d(y, "y")
    T, width = x.shape
    n_experts = 0 if w_gate is None else w_gate.shape[0]
    F = 1 if w_gate is None else w_gate.shape[1]
    _need(y.dtype == torch.float32 and tuple(y.shape) == (T, width) and x.dtype in DT, "expert_rows: x / y")
    if n_experts:
        for name, t, shape in (("w_gate", w_gate, (n_experts, F, width)), ("w_up", w_up, (n_experts, F, width)),
                               ("w_down", w_down, (n_experts, width, F))):
            _dev(t, name, x.dtype)
            _need(tuple(t.shape) == shape, f"expert_rows: {name} is {tuple(t.shape)}, want {shape}")
        _dev(act, "act", x.dtype)
        _need(act.numel() >= T * top * F, "expert_rows: act too small")
    _dev(idx, "idx", torch.int32)
    _dev(weight, "weight", torch.float32)
    _need(idx.numel() >= T * top and weight.numel() >= T * top, "expert_rows: idx / weight too short")
    rt, nn = None, None
    if route is not None:
        rt = route[1].struct(route[0], route[0].shape[1], T)
    if after is not None:
        nn = _next_norm(after, x, accumulate)
    rc = lib.expert_rows(_ptr(x), _c_int(ldx), _ptr(w_gate), _ptr(w_up), _ptr(w_down), _ptr(idx), _ptr(weight),
                         _c_int(T), _c_int(n_experts), _c_int(top), _c_int(F), _c_int(width), _ptr(act), _ptr(y),
                         _c_int(ldy), _c_int(int(bool(accumulate))), _c_int(DT[x.dtype]),
                         *_expert_activation(activation, limit), ctypes.byref(rt) if rt is not None else None,
                         ctypes.byref(nn) if nn is not None else None, _stream())
    build.check(lib, rc, "expert_rows")
    return y


def expert_tiles_takes(inner, width, dtype):
    """Whether ``expert_tiles`` takes experts of this inner size at this width."""
    return bool(build.load("experts").expert_tiles_takes(_c_int(inner), _c_int(width), _c_int(DT[dtype])))


def expert_tiles(y, x, w_gate, w_up, w_down, idx, weight, top, alloc, accumulate=True, activation="silu", limit=0.0, after=None):
    """What ``expert_rows`` computes, for many tokens: the picks are sorted by expert on the device
    and every tile of 32 to 128 picks of one expert is a small product on the matrix cores.
    ``alloc(shape, dtype)`` gives the work memory (the sorted list, the tiles, the activations
    and a float32 row for every pick)."""
    lib = build.load("experts")
    ldx, ldy = _rows2d(x, "x"), _rows2d(y, "y")
    T, width = x.shape
    n_experts, F = w_gate.shape[0], w_gate.shape[1]
    _need(y.dtype == torch.float32 and tuple(y.shape) == (T, width) and x.dtype in DT, "expert_tiles: x / y")
    for name, t, shape in (("w_gate", w_gate, (n_experts, F, width)), ("w_up", w_up, (n_experts, F, width)),
                           ("w_down", w_down, (n_experts, width, F))):
        _dev(t, name, x.dtype)
        _need(tuple(t.shape) == shape, f"expert_tiles: {name} is {tuple(t.shape)}, want {shape}")
    _dev(idx, "idx", torch.int32)
    _dev(weight, "weight", torch.float32)
    _need(idx.numel() >= T * top and weight.numel() >= T * top, "expert_tiles: idx / weight too short")
    most = lib.expert_tiles_most(_c_int(T * top), _c_int(n_experts))
    order, tiles, n_tiles = alloc((T * top,), torch.int32), alloc((3 * most,), torch.int32), alloc((1,), torch.int32)
    act, out = alloc((T * top, F), x.dtype), alloc((T * top, width), torch.float32)
    rc = lib.expert_tiles(_ptr(x), _c_int(ldx), _ptr(w_gate), _ptr(w_up), _ptr(w_down), _ptr(idx), _ptr(weight), _c_int(T),
                          _c_int(n_experts), _c_int(top), _c_int(F), _c_int(width), _ptr(order), _ptr(tiles), _ptr(n_tiles),
                          _ptr(act), _ptr(out), _ptr(y), _c_int(ldy), _c_int(int(bool(accumulate))), _c_int(DT[x.dtype]),
                          *_expert_activation(activation, limit),
                          ctypes.byref(_next_norm(after, x, accumulate)) if after is not None else None, _stream())
    build.check(lib, rc, "expert_tiles")
    return y


# ---------------------------------------------------------------------------
# a layer whose sublayers share one norm and whose outgoing stream is a sum over depth (csrc/parallel_block.hip)


class CanonArgs(ctypes.Structure):
    """Mirror of ``CanonArgs`` in csrc/parallel_block.hip."""

    _fields_ = [("w", _vp), ("taps", _c_int), ("state", _vp), ("state_stride", _c_size_t), ("state_offset", _c_size_t),
                ("token_req", _vp), ("seq_start", _vp), ("slot_ids", _vp), ("mixed", _vp)]


class InputConvolution:
    """A causal convolution over time on a mixer's input, added to it: ``m_t = h_t + sum_j weight[:, j]
    h_(t - taps + 1 + j)`` per channel over a request's own rows (``weight`` float32 ``[width, taps]``);
    rows of earlier steps come from the request's row of ``state`` (``[taps - 1, width]`` from
    ``offset`` on, the latest last).  ``mixed``: where ``m`` goes, ``[rows, width]`` in the compute dtype."""

    def __init__(self, weight, state, offset, token_req, seq_start, slot_ids, mixed):
        _dev(weight, "weight", torch.float32)
        _dev(state, "state", torch.float32)
        for name, t in (("token_req", token_req), ("seq_start", seq_start), ("slot_ids", slot_ids)):
            _dev(t, name, torch.int32)
        width, taps = weight.shape
        _need(state.dim() == 2 and offset + (taps - 1) * width <= state.shape[1], "a convolution's state rows hold taps - 1 inputs of every channel")
        _need(mixed.is_contiguous() and mixed.dtype in DT and mixed.shape[1] == width and token_req.numel() >= mixed.shape[0],
              "the convolution's output is contiguous [rows, width]")
        self.mixed, self.width = mixed, width
        self._keep = (weight, state, token_req, seq_start, slot_ids)
        c = self.c = CanonArgs()
        c.w, c.taps, c.state, c.state_stride, c.state_offset = weight.data_ptr(), taps, state.data_ptr(), state.stride(0), int(offset)
        c.token_req, c.seq_start, c.slot_ids, c.mixed = token_req.data_ptr(), seq_start.data_ptr(), slot_ids.data_ptr(), mixed.data_ptr()


CANON_FUSED_MAX_WIDTH = 8192  # up to this width the norm's kernel keeps a row in registers and can run the convolution too


def canon_rows(h, canon):
    """``canon`` (an ``InputConvolution``) over the float32 rows ``h`` of a step of any shape; the
    requests' state rows are not touched (``conv_state_update`` keeps the last inputs afterwards)."""
    lib = build.load("parallel_block")
    _dev(h, "h", torch.float32)
    _need(h.dim() == 2 and h.shape[1] == canon.width and h.shape[0] >= canon.mixed.shape[0], "canon_rows: shapes")
    rc = lib.canon_rows(_ptr(h), _c_int(canon.mixed.shape[0]), _c_int(canon.width), _c_int(DT[canon.mixed.dtype]),
                        ctypes.byref(canon.c), _stream())
    build.check(lib, rc, "canon_rows")
    return canon.mixed


def norm_fanout(out, x, weight, eps, out32=None, copy_a=None, copy_b=None, canon=None):
    """``out = x / sqrt(mean(x^2) + eps) * weight`` over the float32 rows ``x`` (``out``: float32 or
    bfloat16, contiguous); the same as float32 into ``out32``, and ``x`` itself into ``copy_a`` and
    ``copy_b`` (contiguous float32 ``[rows, width]``), each where given.  ``canon`` (an
    ``InputConvolution``, for a step in which every request brings one token): the convolution runs
    here too, and every request's state row moves up by one."""
    lib = build.load("parallel_block")
    n, width = out.shape
    ldx = _f32_rows(x, "x", width)
    _dev(weight, "weight", torch.float32)
    _need(out.is_contiguous() and out.dtype in DT and weight.numel() == width and x.shape[0] >= n, "norm_fanout: shapes")
    for name, t in (("out32", out32), ("copy_a", copy_a), ("copy_b", copy_b)):
        if t is not None:
            _dev(t, name, torch.float32)
            _need(t.is_contiguous() and tuple(t.shape) == (n, width), f"norm_fanout: {name} is contiguous [rows, width]")
    if canon is not None:
        _need(canon.width == width and canon.mixed.shape[0] == n and canon.mixed.dtype == out.dtype and width <= CANON_FUSED_MAX_WIDTH,
              "norm_fanout: the convolution's rows are the norm's")
    rc = lib.norm_fanout(_ptr(x), _c_int(ldx), _ptr(weight), _c_float(eps), _c_int(n), _c_int(width), _ptr(out),
                         _c_int(DT[out.dtype]), _ptr(out32), _ptr(copy_a), _ptr(copy_b),
                         ctypes.byref(canon.c) if canon is not None else None, _stream())
    build.check(lib, rc, "norm_fanout")
    return out


def depth_average(out, kept, weights, n):
    """``out[t] = sum over j < n of weights[j] * kept[j, t]``: ``kept`` float32 ``[>= n, rows, width]``,
    ``weights`` float32 on the device, ``out`` contiguous float32 ``[rows, width]``."""
    lib = build.load("parallel_block")
    _dev(out, "out", torch.float32)
    _dev(kept, "kept", torch.float32)
    _dev(weights, "weights", torch.float32)
    _need(kept.dim() == 3 and kept.shape[0] >= n and kept.is_contiguous() and out.is_contiguous()
          and tuple(kept.shape[1:]) == tuple(out.shape) and weights.numel() >= n, "depth_average: shapes")
    rc = lib.depth_average(_ptr(out), _ptr(kept), _c_size_t(kept.stride(0)), _ptr(weights), _c_int(n), _c_int(out.shape[0]),
                           _c_int(out.shape[1]), _stream())
    build.check(lib, rc, "depth_average")
    return out


# ---------------------------------------------------------------------------
# between a projection's float rows and a recurrence, and behind it (csrc/state_gates.hip)


def silu_columns(u, col, n):
    """``u[:, col:col + n] <- silu(...)`` in place on float32 rows."""
    lib = build.load("state_gates")
    ld = _f32_rows(u, "u", col + n)
    rc = lib.silu_columns(_ptr(u), _c_int(ld), _c_int(u.shape[0]), _c_int(col), _c_int(n), _stream())
    build.check(lib, rc, "silu_columns")
    return u


def forget_gate(u, q_col, z_col, n, lower, keys):
    """A forget gate with a floor, ``f = lower + (1 - lower) * sigmoid(z)``, for ``S <- diag(f) S +
    (1 - f) v^T``: the logits ``u[:, z_col:z_col + n]`` become ``log f`` in place, ``1 - f`` goes to
    ``keys`` (float32 ``[rows, >= n]``), and the queries ``u[:, q_col:q_col + n]`` pass a silu in place."""
    lib = build.load("state_gates")
    ld, ldk = _f32_rows(u, "u", max(q_col, z_col) + n), _f32_rows(keys, "keys", n)
    _dev(lower, "lower", torch.float32)
    _need(lower.numel() == n and keys.shape[0] >= u.shape[0], "forget_gate: a floor a channel, a row of keys a row")
    rc = lib.forget_gate(_ptr(u), _c_int(ld), _c_int(u.shape[0]), _c_int(q_col), _c_int(z_col), _c_int(n), _ptr(lower),
                         _ptr(keys), _c_int(ldk), _stream())
    build.check(lib, rc, "forget_gate")
    return keys


def normed_gate(out, y, gate, weight, eps):
    """``out = y / sqrt(mean(y^2) + eps) * weight * sigmoid(gate)`` over whole float32 rows; ``out``
    float32 or bfloat16 ``[rows, width]`` (its rows may be wider apart)."""
    lib = build.load("state_gates")
    n, width = out.shape
    ldy, ldg, ldo = _f32_rows(y, "y", width), _f32_rows(gate, "gate", width), _rows2d(out, "out")
    _dev(weight, "weight", torch.float32)
    _need(out.dtype in DT and weight.numel() == width and y.shape[0] >= n and gate.shape[0] >= n, "normed_gate: shapes")
    rc = lib.normed_gate(_ptr(y), _c_int(ldy), _ptr(gate), _c_int(ldg), _ptr(weight), _c_float(eps), _c_int(n), _c_int(width),
                         _ptr(out), _c_int(ldo), _c_int(DT[out.dtype]), _stream())
    build.check(lib, rc, "normed_gate")
    return out


# ---------------------------------------------------------------------------
# a norm without statistics, and the token shift behind it (csrc/dynamic_tanh.hip)


class TokenMixArgs(ctypes.Structure):
    """Mirror of ``TokenMixArgs`` in csrc/dynamic_tanh.hip."""

    _fields_ = [("x", _vp), ("ldx", _c_int), ("n_rows", _c_int), ("width", _c_int), ("alpha", _vp), ("w", _vp), ("b", _vp),
                ("mu", _vp), ("n_mix", _c_int), ("out", _vp), ("state", _vp), ("state_stride", _c_size_t),
                ("state_offset", _c_size_t), ("token_req", _vp), ("seq_start", _vp), ("seq_len", _vp), ("slot_ids", _vp)]


def _tanh_norm(norm, width):
    """The device pointers of a norm given as ``(alpha, weight, shift)``, float32."""
    for name, t, n in zip(("alpha", "weight", "shift"), norm, (1, width, width)):
        _dev(t, name, torch.float32)
        t.numel() == n or _fail(f"dynamic_tanh: {name} has {t.numel()} values, want {n}")
    return [_ptr(t) for t in norm]


def dynamic_tanh(out, x, norm):
    """``out = tanh(alpha * x) * weight + shift`` over float32 rows; ``norm = (alpha, weight, shift)``;
    ``out`` float32 or bfloat16, contiguous."""
    lib = build.load("dynamic_tanh")
    n, width = out.shape
    ldx = _f32_rows(x, "x", width)
    _need(out.is_contiguous() and out.dtype in DT and x.shape[0] >= n, "dynamic_tanh: shapes")
    rc = lib.dynamic_tanh(_ptr(out), _ptr(x), _c_int(ldx), None, *_tanh_norm(norm, width), _c_int(n), _c_int(width),
                          _c_int(DT[out.dtype]), _stream())
    build.check(lib, rc, "dynamic_tanh")
    return out


def embed_dynamic_tanh(out, table, ids, scale, norm):
    """``out[t] = tanh(alpha * scale * table[ids[t]]) * weight + shift`` into float32 ``out``."""
    lib = build.load("dynamic_tanh")
    n, width = out.shape
    _dev(out, "out", torch.float32)
    _dev(table, "table")
    _dev(ids, "ids", torch.int32)
    _need(table.dtype in DT and table.shape[1] == width and ids.numel() >= n, "embed_dynamic_tanh: shapes")
    rc = lib.embed_dynamic_tanh(_ptr(out), _ptr(table), _c_int(DT[table.dtype]), _ptr(ids), _c_float(scale),
                                *_tanh_norm(norm, width), _c_int(n), _c_int(width), _stream())
    build.check(lib, rc, "embed_dynamic_tanh")
    return out


def token_mix(out, x, norm, mu, state, state_offset, token_req, seq_start, seq_len, slot_ids):
    """The rows ``h`` of a dynamic-tanh norm over the float32 stream ``x`` into ``out[0]`` and ``h + (h' -
    h) * mu[m]`` into ``out[1 + m]``, where ``h'`` is the row before in the same sequence (zeros ahead
    of the first; from the request's row of ``state`` at ``state_offset`` where it came in an earlier
    step).  ``out`` contiguous ``[1 + n_mix, rows, width]``, float32 or bfloat16; ``mu`` float32
    ``[n_mix, width]``.  The requests' last normed rows are left in ``state``."""
    lib = build.load("dynamic_tanh")
    planes, n, width = out.shape
    a = TokenMixArgs()
    a.ldx, a.x = _f32_rows(x, "x", width), x.data_ptr()
    _need(out.is_contiguous() and out.dtype in DT and x.shape[0] >= n and token_req.numel() >= n, "token_mix: shapes")
    a.n_rows, a.width, a.n_mix, a.out = n, width, planes - 1, out.data_ptr()
    _dev(mu, "mu", torch.float32)
    _need(tuple(mu.shape) == (planes - 1, width), "token_mix: a row of mu a mix")
    a.mu = mu.data_ptr()
    a.alpha, a.w, a.b = (p.value for p in _tanh_norm(norm, width))
    _dev(state, "state", torch.float32)
    _need(state.dim() == 2 and state_offset + width <= state.shape[1], "token_mix: the state rows are too short")
    a.state, a.state_stride, a.state_offset = state.data_ptr(), state.stride(0), int(state_offset)
    for name, t in (("token_req", token_req), ("seq_start", seq_start), ("seq_len", seq_len), ("slot_ids", slot_ids)):
        _dev(t, name, torch.int32)
        setattr(a, name, t.data_ptr())
    rc = lib.token_mix(ctypes.byref(a), _c_int(DT[out.dtype]), _stream())
    build.check(lib, rc, "token_mix")
    return out


# ---------------------------------------------------------------------------
# recurrences over a matrix state for steps of few tokens (csrc/state_step.hip)


class StepArgs(ctypes.Structure):
    """Mirror of ``StepArgs`` in csrc/state_step.hip."""

    _fields_ = [("q", _vp), ("k", _vp), ("v", _vp), ("ldq", _c_int), ("ldk", _c_int), ("ldv", _c_int), ("qk_stride", _c_int),
                ("v_stride", _c_int), ("gate", _vp), ("ldg", _c_int), ("norm_w", _vp), ("norm_stride", _c_int), ("eps", _c_float),
                ("out", _vp), ("ldo", _c_int), ("out_dtype", _c_int), ("state", _vp), ("state_stride", _c_size_t),
                ("state_offset", _c_size_t), ("seq_start", _vp), ("seq_len", _vp), ("slot_ids", _vp), ("n_requests", _c_int),
                ("H", _c_int), ("Hk", _c_int), ("N", _c_int), ("P", _c_int), ("mode", _c_int), ("log_g", _vp), ("beta", _vp),
                ("ld_gb", _c_int), ("A_log", _vp), ("dt_bias", _vp), ("conv_w", _vp), ("taps", _c_int), ("ring_offset", _c_size_t),
                ("positions", _vp), ("q_scale", _c_float), ("z", _vp), ("ldz", _c_int), ("rank", _c_int), ("w2_dtype", _c_int),
                ("w2t", _vp), ("w0", _vp), ("bonus", _vp), ("gate_sigmoid", _c_int), ("a2", _vp), ("y", _vp), ("ldy", _c_int), ("g_rank", _c_int),
                ("g2", _vp)]


STEP_DELTA, STEP_DELTA_RAW, STEP_BONUS, STEP_CHANNEL_RAW = 0, 1, 2, 3


class DeltaRaw:
    """What ``state_step`` needs to make the delta rule's operands from the projection's own columns:
    the convolution's weights (float32 ``[channels, taps]``, channels of queries, keys and values in
    this order), where its ring of inputs starts in a request's state row (``[taps, channels]``,
    position ``p`` in row ``p % taps``), ``A_log`` a head and ``dt_bias`` a head (or a key channel of every
    head), the queries' factor."""

    def __init__(self, conv_w, ring_offset, a_log, dt_bias, q_scale):
        for name, t in (("conv_w", conv_w), ("a_log", a_log), ("dt_bias", dt_bias)):
            _dev(t, name, torch.float32)
        self.conv_w, self.ring_offset, self.a_log, self.dt_bias, self.q_scale = conv_w, int(ring_offset), a_log, dt_bias, float(q_scale)


class NarrowMiddle:
    """Gates of a recurrence through narrow middles, ``logits = W2 m`` with the middle ``m`` in columns of a
    projection's float32 rows: ``a2`` ``[heads * key_dim, rank]`` for a decay per key channel, ``g2`` ``[heads
    * value_dim, rank]`` for an output gate.  Ranks are multiples of 8 (zero columns beyond the middle's
    own), the middles start at multiples of 4 columns (``a_col``, ``g_col``)."""

    def __init__(self, a2, a_col, g2, g_col):
        for name, t in (("a2", a2), ("g2", g2)):
            _dev(t, name)
            _need(t.dtype in DT and t.dim() == 2 and t.is_contiguous() and t.shape[1] % 8 == 0, f"{name}: rows of a multiple of 8 columns")
        _need(a2.dtype == g2.dtype and a_col % 4 == 0 and g_col % 4 == 0, "a2 and g2 share a dtype, their middles start at multiples of 4")
        self.a2, self.a_col, self.g2, self.g_col = a2, int(a_col), g2, int(g_col)


class LowRankDecay:
    """A decay per key channel through a narrow middle, ``log w = -exp(w0 + W2 tanh(z))``: ``w2t`` is
    ``W2`` transposed, ``[rank, channels]`` (float32 or bfloat16), ``w0`` float32 a channel."""

    def __init__(self, w2t, w0):
        _dev(w2t, "w2t")
        _dev(w0, "w0", torch.float32)
        _need(w2t.dtype in DT and w2t.dim() == 2 and w0.numel() == w2t.shape[1], "LowRankDecay: a row a middle column")
        self.w2t, self.w0, self.rank, self.width = w2t, w0, w2t.shape[0], w2t.shape[1]


def lowrank_decay(log_w, z, decay):
    """``log_w[t] = -exp(w0 + W2 tanh(z[t]))`` (float32 ``[rows, channels]``)."""
    lib = build.load("state_step")
    ldz = _f32_rows(z, "z", decay.rank)
    _dev(log_w, "log_w", torch.float32)
    _need(log_w.shape[1] == decay.width and z.shape[0] >= log_w.shape[0], "lowrank_decay: shapes")
    rc = lib.lowrank_decay(_ptr(z), _c_int(ldz), _c_int(decay.rank), _ptr(decay.w2t), _c_int(DT[decay.w2t.dtype]), _ptr(decay.w0),
                           _c_int(decay.width), _ptr(log_w), _c_int(log_w.shape[0]), _stream())
    build.check(lib, rc, "lowrank_decay")
    return log_w


def state_step_takes(key_dim, value_dim):
    """Whether ``state_step`` holds a head's state of these sizes in a block's registers."""
    return bool(build.load("state_step").state_step_takes(_c_int(key_dim), _c_int(value_dim)))


def state_step(out, q, k, v, state, state_offset, seq_start, seq_len, slot_ids, n_requests, n_heads, n_key_heads, key_dim,
               value_dim, norm_weight, eps, gate=None, qk_stride=None, v_stride=None, log_g=None, beta=None, raw=None,
               positions=None, z=None, decay=None, bonus=None, narrow=None, gate_activation="silu"):
    """A recurrence over a matrix state token by token, a block a (head, request), the state in
    registers; the heads' output divided by its root mean square, times ``norm_weight`` (``value_dim``
    values, or that many a head) and ``silu(gate)`` (``gate_activation``: or ``sigmoid``).

    * the gated delta rule ``u = beta (v - g S^T k); S <- g S + k u^T; o = S^T q`` on prepared
      rows: ``log_g``, ``beta`` float32 ``[rows, n_heads]``;
    * with ``raw`` (a ``DeltaRaw``; every request brings one token) the same from the projection's
      columns, ``beta`` and ``log_g`` the columns that become them (convolution, silu, unit vectors,
      ``beta = sigmoid(.)``, ``g = exp(-exp(A_log) softplus(. + dt_bias))``);
    * with ``raw`` and ``narrow = (u, NarrowMiddle)`` the same with a decay per key channel, ``g[n] =
      exp(-exp(A_log) softplus(a2 m + dt_bias))``, and the gate's logits from their middle, both columns of ``u``;
    * with ``decay`` (a ``LowRankDecay`` over ``z``, float32 ``[rows, >= rank]``) and ``bonus``: ``o =
      (S + diag(bonus) k v^T)^T q; S <- diag(w) S + k v^T``.

    Key head ``h`` at column ``h * qk_stride``, value head at ``h * v_stride`` (default: side by side)."""
    lib = build.load("state_step")
    a = StepArgs()
    T = out.shape[0]
    qs, vstr = key_dim if qk_stride is None else qk_stride, value_dim if v_stride is None else v_stride
    a.ldq, a.ldk = (_f32_rows(t, n, (n_key_heads - 1) * qs + key_dim) for t, n in ((q, "q"), (k, "k")))
    a.ldv = _f32_rows(v, "v", (n_heads - 1) * vstr + value_dim)
    _need(q.shape[0] >= T and k.shape[0] >= T and v.shape[0] >= T, "state_step: fewer operand rows than output rows")
    a.q, a.k, a.v, a.qk_stride, a.v_stride = q.data_ptr(), k.data_ptr(), v.data_ptr(), int(qs), int(vstr)
    if gate is not None:
        a.ldg, a.gate = _f32_rows(gate, "gate", n_heads * value_dim), gate.data_ptr()
    _dev(norm_weight, "norm_weight", torch.float32)
    _need(norm_weight.numel() in (value_dim, n_heads * value_dim), "state_step: norm_weight has value_dim values (a head)")
    a.norm_w, a.norm_stride, a.eps = norm_weight.data_ptr(), value_dim if norm_weight.numel() != value_dim else 0, float(eps)
    a.ldo = _rows2d(out, "out")
    _need(out.dtype in DT and out.shape[1] == n_heads * value_dim, "state_step: out is [tokens, heads * value_dim]")
    a.out, a.out_dtype = out.data_ptr(), DT[out.dtype]
    _dev(state, "state", torch.float32)
    _need(state.dim() == 2 and state_offset + n_heads * key_dim * value_dim <= state.shape[1], "state_step: the state rows are too short")
    a.state, a.state_stride, a.state_offset = state.data_ptr(), state.stride(0), int(state_offset)
    for name, t in (("seq_start", seq_start), ("seq_len", seq_len), ("slot_ids", slot_ids)):
        _dev(t, name, torch.int32)
        _need(t.numel() >= n_requests, f"state_step: {name} is shorter than the requests")
        setattr(a, name, t.data_ptr())
    a.n_requests, a.H, a.Hk, a.N, a.P = int(n_requests), int(n_heads), int(n_key_heads), int(key_dim), int(value_dim)
    if decay is not None:
        a.mode = STEP_BONUS
        _need(decay.width == n_heads * key_dim and n_key_heads == n_heads, "state_step: a decay for every key channel")
        a.ldz, a.z = _f32_rows(z, "z", decay.rank), z.data_ptr()
        a.rank, a.w2_dtype, a.w2t, a.w0 = decay.rank, DT[decay.w2t.dtype], decay.w2t.data_ptr(), decay.w0.data_ptr()
        _dev(bonus, "bonus", torch.float32)
        _need(bonus.numel() == n_heads * key_dim and z.shape[0] >= T, "state_step: a bonus for every key channel")
        a.bonus = bonus.data_ptr()
    else:
        ld = _f32_rows(beta, "beta", n_heads)
        _need(beta.shape[0] >= T, "state_step: fewer rows of beta than of out")
        a.beta, a.ld_gb, a.mode = beta.data_ptr(), ld, STEP_DELTA
        if narrow is None:
            _need(_f32_rows(log_g, "log_g", n_heads) == ld and log_g.shape[0] >= T, "state_step: log_g and beta are rows of one stride")
            a.log_g = log_g.data_ptr()
        if raw is not None:
            channels, taps = raw.conv_w.shape
            _dev(positions, "positions", torch.int32)
            _need(channels == 2 * n_key_heads * key_dim + n_heads * value_dim and raw.a_log.numel() == n_heads
                  and raw.dt_bias.numel() == n_heads * (key_dim if narrow is not None else 1) and positions.numel() >= T,
                  "state_step: the convolution's channels, gates a head")
            _need(taps == 1 or raw.ring_offset + taps * channels <= state.shape[1], "state_step: the state rows are too short")
            a.mode, a.conv_w, a.taps, a.ring_offset = STEP_DELTA_RAW, raw.conv_w.data_ptr(), taps, raw.ring_offset
            a.A_log, a.dt_bias, a.positions, a.q_scale = raw.a_log.data_ptr(), raw.dt_bias.data_ptr(), positions.data_ptr(), raw.q_scale
        if narrow is not None:
            u, nm = narrow
            ldu = _f32_rows(u, "u", max(nm.a_col + nm.a2.shape[1], nm.g_col + nm.g2.shape[1]))
            _need(raw is not None and gate is None and u.shape[0] >= T and nm.a2.shape[0] == n_heads * key_dim
                  and nm.g2.shape[0] == n_heads * value_dim, "state_step: a row of a2 a key channel, of g2 a value column")
            a.mode, a.ldz, a.ldy, a.rank, a.g_rank, a.w2_dtype = STEP_CHANNEL_RAW, ldu, ldu, nm.a2.shape[1], nm.g2.shape[1], DT[nm.a2.dtype]
            a.z, a.y, a.a2, a.g2 = u.data_ptr() + 4 * nm.a_col, u.data_ptr() + 4 * nm.g_col, nm.a2.data_ptr(), nm.g2.data_ptr()
    _need(gate_activation in ("silu", "sigmoid"), f"state_step: gate activation {gate_activation!r}")
    a.gate_sigmoid = int(gate_activation == "sigmoid")
    rc = lib.state_step(ctypes.byref(a), _stream())
    build.check(lib, rc, "state_step")
    return out


def state_chunks_takes(key_dim, value_dim, by_channel=True):
    """Whether ``state_scan``'s kernels that take chunks of tokens hold a state of these sizes."""
    return bool(build.load("linear_state").state_chunks_takes(_c_int(key_dim), _c_int(value_dim), _c_int(int(by_channel))))


# ---------------------------------------------------------------------------
# the gated delta rule for portions of many tokens (csrc/delta_chunks.hip)


class DeltaPrepareArgs(ctypes.Structure):
    """Mirror of ``DeltaPrepareArgs`` in csrc/delta_chunks.hip."""

    _fields_ = [("u", _vp), ("ldu", _c_int), ("b_col", _c_int), ("a_col", _c_int), ("n_rows", _c_int), ("H", _c_int), ("Hk", _c_int),
                ("N", _c_int), ("P", _c_int), ("conv_w", _vp), ("taps", _c_int), ("A_log", _vp), ("dt_bias", _vp), ("q_scale", _c_float),
                ("state", _vp), ("state_stride", _c_size_t), ("ring_offset", _c_size_t), ("token_req", _vp), ("positions", _vp),
                ("seq_start", _vp), ("seq_len", _vp), ("slot_ids", _vp), ("q", _vp), ("k", _vp), ("v", _vp), ("log_g", _vp), ("beta", _vp)]


class DeltaChunkArgs(ctypes.Structure):
    """Mirror of ``DeltaChunkArgs`` in csrc/delta_chunks.hip."""

    _fields_ = [("q", _vp), ("k", _vp), ("v", _vp), ("log_g", _vp), ("beta", _vp), ("cum", _vp), ("w", _vp), ("u", _vp), ("states", _vp),
                ("state", _vp), ("state_stride", _c_size_t), ("state_offset", _c_size_t), ("span_req", _vp), ("span_start", _vp),
                ("span_first", _vp), ("seq_start", _vp), ("seq_len", _vp), ("slot_ids", _vp), ("n_chunks", _c_int), ("n_requests", _c_int),
                ("H", _c_int), ("Hk", _c_int), ("N", _c_int), ("P", _c_int), ("norm_w", _vp), ("norm_stride", _c_int), ("eps", _c_float),
                ("gate", _vp), ("ldg", _c_int), ("out", _vp), ("ldo", _c_int), ("out_dtype", _c_int), ("gate_sigmoid", _c_int), ("k_end", _vp),
                ("q_hat", _vp), ("scores", _vp), ("shrink", _vp)]


class LowRankGates(ctypes.Structure):
    """Mirror of ``LowRankGates`` in csrc/delta_chunks.hip."""

    _fields_ = [("u", _vp), ("ldu", _c_int), ("n_rows", _c_int), ("a_col", _c_int), ("a_rank", _c_int), ("a2", _vp), ("A_log", _vp),
                ("dt_bias", _vp), ("log_g", _vp), ("g_col", _c_int), ("g_rank", _c_int), ("g2", _vp), ("gate", _vp), ("H", _c_int),
                ("N", _c_int), ("P", _c_int), ("dtype", _c_int)]


DELTA_CHUNK = 64  # tokens a chunk


def _sixteens(n):
    return (n + 15) // 16 * 16


def delta_prepare(alloc, u, b_col, a_col, n_heads, n_key_heads, key_dim, value_dim, raw, state, token_req, positions, seq_start,
                  seq_len, slot_ids, narrow=None):
    """The delta rule's operands from the projection's float32 rows ``u`` (queries, keys and values from
    column 0 on, the columns that become ``beta`` and ``g`` from ``b_col`` and ``a_col``): ``(q, k, v,
    log_g, beta)`` in memory that ``alloc(shape, dtype)`` gives, heads padded by zeros to multiples of
    sixteen columns.  ``raw``: a ``DeltaRaw``.  The requests' last inputs go to their rings.  With ``narrow`` (a
    ``NarrowMiddle``; ``a_col`` is not used) ``log_g`` has a column for every (padded) key channel of a head, and the
    output gate's logits, float32 ``[rows, heads * value_dim]``, come sixth."""
    lib = build.load("delta_chunks")
    T = u.shape[0]
    channels, taps = raw.conv_w.shape
    a = DeltaPrepareArgs()
    a_col = 0 if narrow is not None else a_col
    a.ldu, a.u = _f32_rows(u, "u", max(channels, b_col + n_heads, a_col + n_heads)), u.data_ptr()
    _need(channels == 2 * n_key_heads * key_dim + n_heads * value_dim and raw.a_log.numel() == n_heads
          and raw.dt_bias.numel() == n_heads * (key_dim if narrow is not None else 1), "delta_prepare: the convolution's channels, gates a head")
    _dev(state, "state", torch.float32)
    _need(state.dim() == 2 and (taps == 1 or raw.ring_offset + taps * channels <= state.shape[1]), "delta_prepare: the state rows are too short")
    a.b_col, a.a_col, a.n_rows, a.H, a.Hk, a.N, a.P = int(b_col), int(a_col), T, int(n_heads), int(n_key_heads), int(key_dim), int(value_dim)
    a.conv_w, a.taps, a.A_log, a.dt_bias, a.q_scale = raw.conv_w.data_ptr(), taps, raw.a_log.data_ptr(), raw.dt_bias.data_ptr(), raw.q_scale
    a.state, a.state_stride, a.ring_offset = state.data_ptr(), state.stride(0), raw.ring_offset
    for name, t, n in (("token_req", token_req, T), ("positions", positions, T), ("seq_start", seq_start, 1), ("seq_len", seq_len, 1),
                       ("slot_ids", slot_ids, 1)):
        _dev(t, name, torch.int32)
        _need(t.numel() >= n, f"delta_prepare: {name} too short")
        setattr(a, name, t.data_ptr())
    q, k = (alloc((T, n_key_heads * _sixteens(key_dim)), torch.float32) for _ in range(2))
    v = alloc((T, n_heads * _sixteens(value_dim)), torch.float32)
    log_g = alloc((T, n_heads * (_sixteens(key_dim) if narrow is not None else 1)), torch.float32)
    beta = alloc((T, n_heads), torch.float32)
    a.q, a.k, a.v, a.beta = (t.data_ptr() for t in (q, k, v, beta))
    a.log_g = log_g.data_ptr() if narrow is None else None
    rc = lib.delta_prepare(ctypes.byref(a), _stream())
    build.check(lib, rc, "delta_prepare")
    if narrow is None:
        return q, k, v, log_g, beta
    gate = alloc((T, n_heads * value_dim), torch.float32)
    g = LowRankGates()
    g.ldu = _f32_rows(u, "u", max(narrow.a_col + narrow.a2.shape[1], narrow.g_col + narrow.g2.shape[1]))
    _need(narrow.a2.shape[0] == n_heads * key_dim and narrow.g2.shape[0] == n_heads * value_dim, "delta_prepare: a row of a2 a key channel, of g2 a value column")
    g.u, g.n_rows, g.a_col, g.a_rank, g.a2 = u.data_ptr(), T, narrow.a_col, narrow.a2.shape[1], narrow.a2.data_ptr()
    g.A_log, g.dt_bias, g.log_g = raw.a_log.data_ptr(), raw.dt_bias.data_ptr(), log_g.data_ptr()
    g.g_col, g.g_rank, g.g2, g.gate = narrow.g_col, narrow.g2.shape[1], narrow.g2.data_ptr(), gate.data_ptr()
    g.H, g.N, g.P, g.dtype = a.H, a.N, a.P, DT[narrow.a2.dtype]
    rc = lib.lowrank_gates(ctypes.byref(g), _stream())
    build.check(lib, rc, "lowrank_gates")
    return q, k, v, log_g, beta, gate


def delta_chunks_takes(key_dim, value_dim):
    return bool(build.load("delta_chunks").delta_chunks_takes(_c_int(key_dim), _c_int(value_dim)))


def delta_chunks(out, operands, state, state_offset, spans, seq_start, seq_len, slot_ids, n_requests, n_heads, n_key_heads, key_dim,
                 value_dim, norm_weight, eps, gate, alloc, by_channel=False, gate_activation="silu"):
    """The gated delta rule over ``operands`` (what ``delta_prepare`` returned) in chunks of 64 tokens;
    the rest as in ``state_step``.  ``spans``: ``(number of chunks, request of each, its first token
    counted from the request's first of this step, every request's first chunk)``, int32 on the device.  ``by_channel``: ``log_g`` has
    a column for every padded key channel of a head; ``gate_activation``: ``silu`` or ``sigmoid``."""
    lib = build.load("delta_chunks")
    q, k, v, log_g, beta = operands
    n_chunks, span_req, span_start, span_first = spans
    T, Np, Pp = out.shape[0], _sixteens(key_dim), _sixteens(value_dim)
    a = DeltaChunkArgs()
    for name, t, shape in (("q", q, (T, n_key_heads * Np)), ("k", k, (T, n_key_heads * Np)), ("v", v, (T, n_heads * Pp)),
                           ("log_g", log_g, (T, n_heads * Np if by_channel else n_heads)), ("beta", beta, (T, n_heads))):
        _dev(t, name, torch.float32)
        _need(tuple(t.shape) == shape, f"delta_chunks: {name} is {tuple(t.shape)}, want {shape}")
        setattr(a, name, t.data_ptr())
    work = {"w": alloc((T, n_heads * Np), torch.float32),
            "u": alloc((T, n_heads * Pp), torch.float32), "states": alloc((n_chunks, n_heads, Np, Pp), torch.float32)}
    if by_channel:
        work.update(k_end=alloc((T, n_heads * Np), torch.float32), q_hat=alloc((T, n_heads * Np), torch.float32),
                    scores=alloc((n_chunks, n_heads, DELTA_CHUNK, DELTA_CHUNK), torch.float32), shrink=alloc((n_chunks, n_heads, Np), torch.float32))
    else:
        work["cum"] = alloc((T, n_heads), torch.float32)
    for name, t in work.items():
        setattr(a, name, t.data_ptr())
    _need(gate_activation in ("silu", "sigmoid"), f"delta_chunks: gate activation {gate_activation!r}")
    a.gate_sigmoid = int(gate_activation == "sigmoid")
    _dev(state, "state", torch.float32)
    _need(state.dim() == 2 and state_offset + n_heads * key_dim * value_dim <= state.shape[1], "delta_chunks: the state rows are too short")
    a.state, a.state_stride, a.state_offset = state.data_ptr(), state.stride(0), int(state_offset)
    for name, t, n in (("span_req", span_req, n_chunks), ("span_start", span_start, n_chunks), ("span_first", span_first, n_requests),
                       ("seq_start", seq_start, n_requests), ("seq_len", seq_len, n_requests), ("slot_ids", slot_ids, n_requests)):
        _dev(t, name, torch.int32)
        _need(t.numel() >= n, f"delta_chunks: {name} too short")
        setattr(a, name, t.data_ptr())
    a.n_chunks, a.n_requests, a.H, a.Hk, a.N, a.P = int(n_chunks), int(n_requests), int(n_heads), int(n_key_heads), int(key_dim), int(value_dim)
    _dev(norm_weight, "norm_weight", torch.float32)
    _need(norm_weight.numel() in (value_dim, n_heads * value_dim), "delta_chunks: norm_weight has value_dim values (a head)")
    a.norm_w, a.norm_stride, a.eps = norm_weight.data_ptr(), value_dim if norm_weight.numel() != value_dim else 0, float(eps)
    if gate is not None:
        a.ldg, a.gate = _f32_rows(gate, "gate", n_heads * value_dim), gate.data_ptr()
        _need(gate.shape[0] >= T, "delta_chunks: fewer gate rows than output rows")
    a.ldo = _rows2d(out, "out")
    _need(out.dtype in DT and out.shape[1] == n_heads * value_dim, "delta_chunks: out is [tokens, heads * value_dim]")
    a.out, a.out_dtype = out.data_ptr(), DT[out.dtype]
    rc = lib.delta_chunks(ctypes.byref(a), _stream())
    build.check(lib, rc, "delta_chunks")
    return out


# ---------------------------------------------------------------------------
# a residual stream kept as several streams (csrc/hyper.hip)


class HyperArgs(ctypes.Structure):
    """Mirror of ``HyperArgs`` in csrc/hyper.hip."""

    _fields_ = [("xs", _vp), ("first", _vp), ("ld_first", _c_int), ("xs_out", _vp), ("y", _vp), ("ldy", _c_int), ("n_parts", _c_int),
                ("y_part", _c_size_t), ("bias", _vp), ("mix", _vp), ("out", _vp), ("in_", _vp), ("gamma", _vp), ("beta", _vp),
                ("eps", _c_float), ("norm_out", _vp), ("norm_dtype", _c_int), ("sum_out", _vp), ("ld_sum", _c_int), ("T", _c_int),
                ("D", _c_int), ("S", _c_int), ("w", _vp), ("rows_out", _vp), ("n_rows", _c_int)]


HYPER_MAX_STREAMS, HYPER_MAX_WIDTH = 8, 32768
HYPER_MAX_ROWS = 128  # of the small matrix whose product with the norm rides along


class HyperWrite:
    """A sublayer's output on its way into the streams: ``x_t <- sum_s mix[s, t] x_s + out[t] y``.  ``y`` float32
    ``[tokens, width]``; where ``pending`` (a ``PendingSum``) waits on it, its value still lies in that sum's parts."""

    def __init__(self, y, mix, out, pending=None):
        self.y, self.mix, self.out, self.pending = y, mix, out, pending


def hyper_step(n_streams, width, xs=None, first=None, xs_out=None, write=None, read=None, norm_out=None, gamma=None, beta=None, eps=0.0,
               sum_out=None, rows=None):
    """One pass over the streams ``xs`` (float32 ``[tokens, streams, width]``; all of them are ``first``, ``[tokens,
    width]``, where ``xs`` is None): ``write`` (a ``HyperWrite``) first, the new streams into ``xs_out`` (may be
    ``xs``), then ``u = sum_s read[s] x_s`` (``read`` None: the plain sum), its LayerNorm into ``norm_out`` and ``u``
    itself into ``sum_out``.  ``rows = (w, out)``: the norm's product with a small matrix ``w`` ``[n, width]`` of its dtype into
    float32 ``out`` ``[tokens, n]``."""
    lib = build.load("hyper")
    a = HyperArgs()
    src = xs if xs is not None else first
    T = src.shape[0]
    for name, t, shape in (("xs", xs, (T, n_streams, width)), ("xs_out", xs_out, (T, n_streams, width))):
        if t is not None:
            _dev(t, name, torch.float32)
            _need(tuple(t.shape) == shape and t.is_contiguous(), f"hyper_step: {name} is {tuple(t.shape)}, want {shape}")
            setattr(a, name, t.data_ptr())
    if xs is None:
        a.ld_first, a.first = _f32_rows(first, "first", width), first.data_ptr()
    if write is not None:
        y = write.y
        _need(tuple(y.shape) == (T, width), "hyper_step: y")
        a.ldy, a.n_parts, a.y = _f32_rows(y, "y", width), 1, y.data_ptr()
        if write.pending is not None and write.pending.waits_on(y):
            c = write.pending.c
            a.y, a.ldy, a.n_parts, a.y_part, a.bias = c.ws, width, c.n_splits, T * width, c.bias
            c.target = None  # (this adds the parts; nobody else has to)
        for name, t, n in (("mix", write.mix, n_streams * n_streams), ("out", write.out, n_streams)):
            _dev(t, name, torch.float32)
            _need(t.numel() == n and t.is_contiguous(), f"hyper_step: {name} has {n} values")
            setattr(a, name, t.data_ptr())
    for field, name, t, n in (("in_", "read", read, n_streams), ("gamma", "gamma", gamma, width), ("beta", "beta", beta, width)):
        if t is not None:
            _dev(t, name, torch.float32)
            _need(t.numel() == n, f"hyper_step: {name} has {n} values")
            setattr(a, field, t.data_ptr())
    if norm_out is not None:
        _need(tuple(norm_out.shape) == (T, width) and norm_out.is_contiguous() and norm_out.dtype in DT, "hyper_step: norm_out")
        a.norm_out, a.norm_dtype, a.eps = norm_out.data_ptr(), DT[norm_out.dtype], float(eps)
    if sum_out is not None:
        _need(sum_out.shape[0] >= T, "hyper_step: sum_out")
        a.ld_sum, a.sum_out = _f32_rows(sum_out, "sum_out", width), sum_out.data_ptr()
    if rows is not None:
        w, out = rows
        _dev(w, "w", norm_out.dtype)
        _dev(out, "rows", torch.float32)
        _need(w.dim() == 2 and w.shape[1] == width and w.is_contiguous() and tuple(out.shape) == (T, w.shape[0]) and out.is_contiguous(), "hyper_step: rows")
        a.w, a.rows_out, a.n_rows = w.data_ptr(), out.data_ptr(), w.shape[0]
    a.T, a.D, a.S = T, int(width), int(n_streams)
    rc = lib.hyper_step(ctypes.byref(a), _stream())
    build.check(lib, rc, "hyper_step")


# ---------------------------------------------------------------------------
# the real-gated linear recurrent unit (csrc/rglru.hip)


class RglruArgs(ctypes.Structure):
    """Mirror of ``RglruArgs`` in csrc/rglru.hip."""

    _fields_ = [("x", _vp), ("y", _vp), ("ldx", _c_int), ("conv_w", _vp), ("conv_b", _vp), ("taps", _c_int), ("ra", _vp), ("ri", _vp),
                ("ra_b", _vp), ("ri_b", _vp), ("lam", _vp), ("state", _vp), ("state_stride", _c_size_t), ("state_offset", _c_size_t),
                ("ring_offset", _c_size_t), ("positions", _vp), ("seq_start", _vp), ("seq_len", _vp),
                ("slot_ids", _vp), ("span_req", _vp), ("span_start", _vp), ("span_first", _vp), ("a", _vp), ("b", _vp), ("does", _vp),
                ("s0", _vp), ("out", _vp), ("ldo", _c_int), ("dtype", _c_int), ("n_requests", _c_int), ("n_spans", _c_int),
                ("W", _c_int), ("B", _c_int), ("w", _c_int), ("wp", _c_int), ("decay", _c_float)]


def rglru_takes(part):
    """Whether the unit's kernels take gate matrices of ``part`` channels."""
    return bool(build.load("rglru").rglru_takes(_c_int(int(part))))


class RglruWeights:
    """The unit's weights: ``conv_w`` float32 ``[width, taps]``, ``conv_b`` ``[width]`` or None; the gates'
    matrices ``[blocks, part, part]`` of the compute dtype (kept padded by zero columns to a multiple of 8), their
    shifts and ``lam`` float32 ``[width]``; ``decay``: the constant of ``log a = -decay r softplus(lam)``."""

    def __init__(self, conv_w, conv_b, ra, ra_b, ri, ri_b, lam, decay):
        self.blocks, self.part = ra.shape[0], ra.shape[1]
        self.width, self.taps = conv_w.shape
        _need(tuple(ra.shape) == tuple(ri.shape) == (self.blocks, self.part, self.part) and self.blocks * self.part == self.width
              and ra.dtype == ri.dtype and ra.dtype in DT, "rglru: square gate matrices, one a block")
        pad = -self.part % 8
        self.ra, self.ri = (torch.cat([t, t.new_zeros(self.blocks, self.part, pad)], 2).contiguous() if pad else t.contiguous() for t in (ra, ri))
        self.conv_w, self.conv_b, self.decay = conv_w.contiguous(), conv_b, float(decay)
        self.ra_b, self.ri_b, self.lam = ra_b.reshape(-1).contiguous(), ri_b.reshape(-1).contiguous(), lam.contiguous()
        for name, t in (("conv_w", self.conv_w), ("ra_b", self.ra_b), ("ri_b", self.ri_b), ("lam", self.lam)):
            _dev(t, name, torch.float32)
            _need(t.numel() == self.width * (self.taps if name == "conv_w" else 1), f"rglru: {name}")


def rglru(out, x, y, weights, state, state_offset, ring_offset, positions, seq_start, seq_len, slot_ids, n_requests, spans, alloc):
    """``out = S * gelu_tanh(y)`` with ``S`` the unit's state over ``conv(x)``, for every token: ``x`` and ``y``
    float32 columns of the same rows, ``out`` of the gates' dtype.  A request's row of ``state`` holds ``S`` (``width``
    floats at ``state_offset``) and the convolution's inputs (a ring ``[taps, width]`` at ``ring_offset``, position
    ``p`` in row ``p % taps``; none for one tap).  ``spans``: None where every request brings one token, otherwise
    ``(number of spans of 64 tokens, request of each, its first token counted from the request's first of this
    step, every request's first span)``."""
    lib = build.load("rglru")
    w, a = weights, RglruArgs()
    T = out.shape[0]
    a.ldx, a.x, a.y = _f32_rows(x, "x", w.width), x.data_ptr(), y.data_ptr()
    _need(_f32_rows(y, "y", w.width) == a.ldx and x.shape[0] >= T and y.shape[0] >= T, "rglru: x and y are columns of the same rows")
    a.conv_w, a.conv_b, a.taps = w.conv_w.data_ptr(), native.ptr(w.conv_b), w.taps
    a.ra, a.ri, a.ra_b, a.ri_b, a.lam = (t.data_ptr() for t in (w.ra, w.ri, w.ra_b, w.ri_b, w.lam))
    _dev(state, "state", torch.float32)
    _need(state.dim() == 2 and state_offset + w.width <= state.shape[1]
          and (w.taps == 1 or ring_offset + w.taps * w.width <= state.shape[1]), "rglru: the state rows are too short")
    a.state, a.state_stride, a.state_offset, a.ring_offset = state.data_ptr(), state.stride(0), int(state_offset), int(ring_offset)
    for name, t, n in (("positions", positions, T), ("seq_start", seq_start, n_requests), ("seq_len", seq_len, n_requests),
                       ("slot_ids", slot_ids, n_requests)):
        _dev(t, name, torch.int32)
        _need(t.numel() >= n, f"rglru: {name} too short")
        setattr(a, name, t.data_ptr())
    a.ldo, a.out, a.dtype = _rows2d(out, "out"), out.data_ptr(), DT[out.dtype]
    _need(out.dtype == w.ra.dtype and out.shape[1] >= w.width, "rglru: out has the gates' dtype and a column a channel")
    a.n_requests, a.W, a.B, a.w, a.wp, a.decay = int(n_requests), w.width, w.blocks, w.part, w.ra.shape[2], w.decay
    if spans is None:
        rc = lib.rglru_step(ctypes.byref(a), _stream())
        build.check(lib, rc, "rglru_step")
        return out
    n_spans, span_req, span_start, span_first = spans
    for name, t, n in (("span_req", span_req, n_spans), ("span_start", span_start, n_spans), ("span_first", span_first, n_requests)):
        _dev(t, name, torch.int32)
        _need(t.numel() >= n, f"rglru: {name} too short")
        setattr(a, name, t.data_ptr())
    a.n_spans = int(n_spans)
    work = [alloc((T, w.width), torch.float32), alloc((T, w.width), torch.float32), alloc((n_spans, w.width, 2), torch.float32),
            alloc((n_requests, w.width), torch.float32)]
    a.a, a.b, a.does, a.s0 = (t.data_ptr() for t in work)
    rc = lib.rglru_portions(ctypes.byref(a), _stream())
    build.check(lib, rc, "rglru_portions")
    return out
