"""Lutodra in the engine against the plain implementation (plain_lutodra.py): each mechanism's kernels,
each mixer alone in a one-layer model, whole prompts, decoding, portions, mixed batches, reused pages
and state rows, far tokens, sinks, loops, generation through the entry points."""

import copy
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import helpers
import plain_lutodra as plain
from test_lutodra import SMALL, _attention, _config, _delta, _dense, _lru, _moe

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))

# max |engine - plain| over max |plain logits|: float32 sums where the plain side has float64;
# bfloat16 rounds activations between the products (the plain side gets the rounded matrices)
TOL = {"float32": 5e-5, "bfloat16": 6e-2}

CONFIGS = {
    "A": SMALL,
    # corners: one stream, one head, one key head for all heads, a key head a head, one tap, seven taps, one
    # part of the unit and parts of odd sizes, one expert of one, every expert chosen, one group, a group an expert,
    # no rotation, every column turning, values wider and narrower than keys and no multiples of four, a loop of
    # one layer
    "B": _config(72, 97, [
        _moe(_delta(4, 1, 12, 20, 1), 10, 1, 1),
        _dense(_attention(1, 1, 24, 20, 0), 28),
        _moe(_lru(33, 3, 7), 12, 6, 6, (1, 1), 3.0),
        _moe(_attention(3, 1, 10, 28, 10, 50.0, (2.0, 1.0, 1.0, 30), scale=0.5), 9, 5, 2, (5, 3)),
        _delta(3, 3, 20, 10, 7),
        _lru(20, 1, 1),
        _moe(_attention(6, 6, 6, 44, 2, 9.0), 16, 4, 2, (2, 2))],
        streams=1, loop=(4, 5, 3), eps=1e-3, logit_scale=1.7),
    # wider, for bfloat16: heads of 64 and 128
    "C": _config(128, 300, [
        _dense(_lru(96, 2, 4), 96),
        _moe(_attention(8, 2, 64, 64, 32, 1e5, (8.0, 1.0, 4.0, 128)), 64, 8, 3, (4, 2), 1.2),
        _moe(_delta(4, 2, 64, 48, 4), 72, 6, 2, (2, 1)),
        _dense(_attention(2, 1, 128, 96, 128, 1e5), 40),
        _moe(_delta(2, 1, 32, 128, 2), 64, 8, 4, (2, 2), 0.7)], streams=5, loop=(0, 3, 2), logit_scale=0.3),
}
SEEDS = {"A": 3, "B": 4, "C": 5}
RANKS = {"A": 4, "B": 3, "C": 16}


def _folder(path, config, weights):
    from safetensors.torch import save_file

    os.makedirs(path, exist_ok=True)
    json.dump(config, open(os.path.join(path, "config.json"), "w"))
    save_file({k: v.contiguous() for k, v in weights.items()}, os.path.join(path, "model.safetensors"))
    return path


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    """By (name, dtype).  The bfloat16 models use all their experts: a choice between two of nearly equal
    score may rightly fall the other way after rounding, and the states carry that on to later tokens; and
    their norms' eps is large: a head whose few columns nearly vanish would otherwise turn rounding into
    errors of any size (the plain side with rounded norms then differs from itself by a tenth of the scale)."""
    out = {}
    for name, dtype in [(n, d) for n in CONFIGS for d in ("float32", "bfloat16")]:
        config = copy.deepcopy(CONFIGS[name])
        for entry in config["layers"]:
            if entry["mlp"] is not None and entry["mlp"]["kind"] == "moe" and dtype == "bfloat16":
                router = entry["mlp"]["router"]
                router["top"], router["groups"]["keep"] = router["experts"], router["groups"]["count"]
        if dtype == "bfloat16":
            config["norm"]["eps"] = 1e-2
        weights = plain.random_weights(config, SEEDS[name], sharp=2.0 if dtype == "float32" else 1.0, rank=RANKS[name])
        out[name, dtype] = (_folder(str(tmp_path_factory.mktemp("lut" + name)), config, weights), config, weights)
    return out


def _engine(folder, dtype, n_pages, page_size=16, max_requests=4, **kw):
    from mlx_lm_amd.engine import Engine
    from mlx_lm_amd.utils import load_model

    model, _ = load_model(folder, dtype=dtype)
    return Engine(model, dtype=dtype, page_size=page_size, n_pages=n_pages, max_requests=max_requests, **kw)


def _rounded(weights):
    """What the engine's bfloat16 path holds: the products' matrices rounded; connections, convolutions, shifts
    and norms as they are."""
    kept = (".conv", ".in", ".out", ".mix", ".b")
    return {k: v if v.dim() < 2 or k.endswith(kept) and not k.endswith("mix.b") else v.to(torch.bfloat16).float() for k, v in weights.items()}


def _plain(weights, config, tokens, dtype):
    return plain.model(_rounded(weights) if dtype == "bfloat16" else weights, config, tokens)


def _close(got, want, dtype, what="", strict=True):
    """Every position within the tolerance.  Not ``strict`` (bfloat16 where some of the experts are
    chosen): nine positions in ten, and none far off."""
    scale = want.abs().max().item()
    err = (got.double().cpu() - want).abs().amax(-1) / scale
    if strict or dtype == "float32":
        assert err.max().item() <= TOL[dtype], f"{what}: max error {err.max().item():.3e} of the scale at {int(err.argmax())}"
    else:
        n = int((err > TOL[dtype]).sum())
        assert n <= max(1, err.numel() // 10) and err.max().item() < 0.5, \
            f"{what}: {n} of {err.numel()} positions beyond the tolerance, worst {err.max().item():.3e} at {int(err.argmax())}"


def _run(engine, rid, tokens, cuts):
    from mlx_lm_amd.engine import StepEntry

    engine.add_request(rid)
    rows, i = [], 0
    for n in cuts:
        part = tokens[i : i + n]
        rows.append(engine.step([StepEntry(rid, part, list(range(len(part))))]).clone())
        i += n
    assert i == len(tokens)
    engine.end_request(rid)
    return torch.cat(rows)


def _ints(values):
    return torch.tensor(values, dtype=torch.int32).cuda()


def _alloc(shape, dtype):
    return torch.empty(shape, dtype=dtype, device="cuda")


def _spans(lens):
    """The chunks of 64 tokens that the step's requests fall into, as the packer lists them."""
    req, lo, first = [], [], []
    for r, n in enumerate(lens):
        first.append(len(req))
        for at in range(0, n, 64):
            req.append(r)
            lo.append(at)
    return len(req), _ints(req), _ints(lo), _ints(first)


# -- kernels -------------------------------------------------------------------------------


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("streams,width,T", [(1, 64, 3), (2, 72, 1), (3, 1028, 5), (4, 2048, 9), (5, 4100, 2), (6, 200, 4), (7, 8196, 2), (8, 24, 70)])
def test_the_streams_written_read_and_normed_in_one_pass(streams, width, T, dtype):
    """First reads of streams that are all the same; a write of an output that lies in one piece or in
    parts; streams updated in place; a small matrix's product with the norm; the sum at the end."""
    from mlx_lm_amd.ops import kernels

    g = torch.Generator().manual_seed(width)
    rnd = lambda *s: torch.randn(*s, generator=g)  # noqa: E731
    S, D = streams, width
    first, read, mix, out = rnd(T, D) * 3 + 1, rnd(S), rnd(S, S), rnd(S)
    w = {"n": rnd(D) + 1, "n.b": rnd(D), "c.in": read, "c.mix": mix, "c.out": out}
    wd = {k: v.double() for k, v in w.items()}
    tol = 2e-5 if dtype == torch.float32 else 1e-2
    dev = {k: v.cuda() for k, v in w.items()}
    xs = first.double().expand(S, T, D)
    u = torch.empty(T, D, dtype=dtype, device="cuda")
    small = rnd(1 + width % 70, D).to(dtype)
    z = torch.empty(T, small.shape[0], device="cuda")
    norm = dict(norm_out=u, gamma=dev["n"], beta=dev["n.b"], eps=1e-3, read=dev["c.in"], rows=(small.cuda(), z))

    def check():
        want = plain.layer_norm(plain.hyper_read(xs, wd, "c."), wd, "n", 1e-3)
        assert (u.double().cpu() - want).abs().max() <= tol * want.abs().max()
        rows = u.double().cpu() @ small.double().t()  # (the row as it was written)
        assert (z.double().cpu() - rows).abs().max() <= 2e-5 * rows.abs().max()

    kernels.hyper_step(S, D, first=first.cuda(), **norm)
    check()
    buf = torch.full((T, S, D), float("nan"), device="cuda")
    for i, parts in enumerate((1, 3, 6)):
        y = rnd(parts, T, D)
        pending = kernels.PendingSum()
        yd = torch.full((T, D), float("nan"), device="cuda") if parts > 1 else y[0].cuda()
        ws = y.cuda()
        if parts > 1:
            c = pending.c
            c.target, c.rows, c.cols, c.ws, c.n_splits = yd.data_ptr(), T, D, ws.data_ptr(), parts
        write = kernels.HyperWrite(yd, dev["c.mix"], dev["c.out"], pending)
        kernels.hyper_step(S, D, xs=buf if i else None, first=None if i else first.cuda(), xs_out=buf, write=write, **norm)
        assert pending.target is None
        xs = plain.hyper_write(xs, y.double().sum(0), wd, "c.")
        check()
        assert (buf.double().cpu() - xs.transpose(0, 1)).abs().max() <= 2e-5 * xs.abs().max()
    h, y = torch.full((T, D), float("nan"), device="cuda"), rnd(T, D)
    kernels.hyper_step(S, D, xs=buf, write=kernels.HyperWrite(y.cuda(), dev["c.mix"], dev["c.out"]), sum_out=h)
    want = plain.hyper_write(xs, y.double(), wd, "c.").sum(0)
    assert (h.double().cpu() - want).abs().max() <= 2e-5 * want.abs().max()


def _delta_operands(n, C, H, rank, g, far):
    """The projection's rows ``[q | k | v | b | .. | middle | .. | middle of the gate]``."""
    return torch.randn(n, C + H, generator=g), torch.randn(n, rank, generator=g) * far, torch.randn(n, rank + 3, generator=g)


def _delta_plain(u, za, zg, conv_w, a2, g2, a_log, dt_bias, norm_w, H, G, N, P, eps):
    u, C = u.double(), 2 * G * N + H * P
    x = plain.silu(plain.causal_conv(u[:, :C], conv_w.double()))
    q = plain.unit_length(x[:, : G * N].view(-1, G, N)) * N ** -0.5
    k, v = plain.unit_length(x[:, G * N : 2 * G * N].view(-1, G, N)), x[:, 2 * G * N :].view(-1, H, P)
    beta = plain.sigmoid(u[:, C:])
    step = plain.softplus(za.double() @ a2.double().t() + dt_bias.double()).view(-1, H, N)
    decay = torch.exp(-torch.exp(a_log.double())[:, None] * step)
    o = torch.stack([plain.delta_recurrence(q[:, h // (H // G)], k[:, h // (H // G)], v[:, h], decay[:, h], beta[:, h]) for h in range(H)], 1)
    o = plain.unit_rms(o, eps) * norm_w.double()
    return (o * plain.sigmoid(zg.double() @ g2.double().t()).view(-1, H, P)).flatten(1)


@pytest.mark.parametrize("H,G,N,P,taps,rank,far", [
    (4, 2, 16, 32, 4, 8, 1.0), (3, 3, 8, 8, 1, 5, 1.0), (2, 1, 64, 64, 4, 24, 1.0), (4, 1, 5, 6, 3, 3, 1.0), (2, 2, 128, 128, 4, 128, 1.0),
    (1, 1, 40, 20, 7, 1, 1.0), (2, 1, 200, 100, 2, 33, 1.0), (1, 1, 17, 33, 4, 9, 1.0), (2, 1, 256, 256, 2, 16, 1.0),
    (2, 1, 64, 64, 4, 16, 12.0), (2, 2, 24, 16, 3, 8, 30.0)])
def test_the_delta_rule_by_channel_in_portions_of_two_requests(H, G, N, P, taps, rank, far):
    """Two requests side by side: single tokens (all in the step's own kernel), portions in chunks, cut at
    and around a chunk's edge; the convolution's inputs and the states carried over, other rows untouched.
    ``far``: how widely the decays differ; with 12 and 30 some channels forget all within a token, others nothing, so
    tiles take the way pair by pair."""
    from mlx_lm_amd.ops import kernels

    if not kernels.state_step_takes(N, P) or not kernels.delta_chunks_takes(N, P):
        pytest.fail("these sizes have kernels")
    g = torch.Generator().manual_seed(N + P)
    C, eps = 2 * G * N + H * P, 1e-4
    lens = [(1, 1), (2, 1), (70, 3), (1, 1), (1, 64), (5, 7), (65, 1), (1, 1), (63, 129)]
    total = [sum(x[r] for x in lens) for r in range(2)]
    ops = [_delta_operands(n, C, H, rank, g, far) for n in total]
    conv_w, norm_w = torch.randn(C, taps, generator=g), 1 + 0.3 * torch.randn(P, generator=g)
    a_log, dt_bias = torch.randn(H, generator=g) - 1.0, torch.randn(H * N, generator=g) * 1.5 - 2.0
    a2, g2 = torch.randn(H * N, rank, generator=g) * rank ** -0.5, torch.randn(H * P, rank + 3, generator=g) * rank ** -0.5
    want = [_delta_plain(*x, conv_w, a2, g2, a_log, dt_bias, norm_w, H, G, N, P, eps) for x in ops]
    # rows as the mixer lays them out: the middles start at multiples of four, padded to multiples of eight
    pad8 = lambda n: (n + 7) // 8 * 8  # noqa: E731
    a_col = (C + H + 3) // 4 * 4
    g_col = a_col + pad8(rank)
    rows_of = []
    for u, za, zg in ops:
        r = torch.zeros(u.shape[0], g_col + pad8(rank + 3))
        r[:, : C + H], r[:, a_col : a_col + rank], r[:, g_col : g_col + rank + 3] = u, za, zg
        rows_of.append(r)
    wide = lambda w: torch.nn.functional.pad(w, (0, pad8(w.shape[1]) - w.shape[1])).contiguous().cuda()  # noqa: E731
    narrow = kernels.NarrowMiddle(wide(a2), a_col, wide(g2), g_col)
    S0 = 8  # the matrices' place in a state row
    ring = S0 + H * N * P
    floats = (ring + taps * C + 3) // 4 * 4
    state = torch.full((4, floats), 5.0).cuda()
    state[[3, 1], S0:] = 0.0
    raw = kernels.DeltaRaw(conv_w.cuda(), ring, a_log.cuda(), dt_bias.cuda(), N ** -0.5)
    slots = _ints([3, 1])
    at, got = [0, 0], [[], []]
    for step in lens:
        rows = torch.cat([rows_of[r][at[r] : at[r] + step[r]] for r in range(2)]).cuda()
        starts, ns = _ints([0, step[0]]), _ints(step)
        pos = _ints([at[0] + i for i in range(step[0])] + [at[1] + i for i in range(step[1])])
        out = torch.empty(sum(step), H * P, device="cuda")
        if max(step) == 1:
            kernels.state_step(out, rows[:, : G * N], rows[:, G * N : 2 * G * N], rows[:, 2 * G * N : C], state, S0, starts, ns, slots, 2, H, G, N, P,
                               norm_w.cuda(), eps, beta=rows[:, C : C + H], raw=raw, positions=pos, narrow=(rows, narrow), gate_activation="sigmoid")
        else:
            *prepared, gate = kernels.delta_prepare(_alloc, rows, C, 0, H, G, N, P, raw, state, _ints([0] * step[0] + [1] * step[1]), pos, starts,
                                                    ns, slots, narrow=narrow)
            kernels.delta_chunks(out, prepared, state, S0, _spans(step), starts, ns, slots, 2, H, G, N, P, norm_w.cuda(), eps, gate, _alloc,
                                 by_channel=True, gate_activation="sigmoid")
        got[0].append(out[: step[0]].cpu()), got[1].append(out[step[0] :].cpu())
        at = [at[0] + step[0], at[1] + step[1]]
    for r in range(2):
        err = (torch.cat(got[r]).double() - want[r]).abs().amax(-1) / want[r].abs().max()
        assert err.max() <= 5e-5, (r, int(err.argmax()), float(err.max()))
    assert (state[[0, 2]] == 5.0).all() and (state[:, :S0] == 5.0).all()


@pytest.mark.parametrize("cuts", [[900], [899, 1], [892, 8], [63, 1, 64, 65, 700, 7], [448, 2, 449, 1]])
def test_a_key_far_back_in_a_channel_that_keeps(cuts):
    """The key of token 3 lies along a channel that no other key touches and that hardly decays, among channels
    that forget everything within a token; the last of 900 queries lies along it too, so its output is token 3's
    value, decayed."""
    from mlx_lm_amd.ops import kernels

    n, N, P = 900, 16, 16
    g = torch.Generator().manual_seed(6)
    k, q, v = torch.randn(n, N, generator=g), torch.randn(n, N, generator=g), torch.randn(n, P, generator=g)
    k[:, 0] = 0.0
    k[3], q[n - 1] = 0.0, 0.0
    k[3, 0], q[n - 1, 0] = 1.0, 1.0
    k = torch.nn.functional.normalize(k, dim=-1)
    log_g, beta = torch.full((n, N), -1e-4), torch.rand(n, 1, generator=g)
    log_g[:, 5], log_g[:, 9] = -40.0, -7.0
    beta[3] = 1.0
    eps = 1e-6
    o = plain.delta_recurrence(q.double(), k.double(), v.double(), log_g.double().exp(), beta.double()[:, 0])
    assert torch.allclose(o[n - 1], v[3].double() * float(np.exp(-1e-4 * (n - 4))), atol=1e-6)
    want, ones = plain.unit_rms(o, eps), torch.ones(P).cuda()
    state, got, at = torch.zeros(1, N * P).cuda(), [], 0
    for m in cuts:
        part = [t[at : at + m].contiguous().cuda() for t in (q, k, v, log_g, beta)]
        out = torch.empty(m, P, device="cuda")
        kernels.delta_chunks(out, part, state, 0, _spans([m]), _ints([0]), _ints([m]), _ints([0]), 1, 1, 1, N, P, ones, eps, None, _alloc, by_channel=True)
        got.append(out.cpu())
        at += m
    assert (torch.cat(got).double() - want).abs().max() <= 1e-4 * want.abs().max()


def test_keys_that_repeat_with_decays_of_every_speed():
    """A sequence that writes one key again and again with a step size near one, its channels' decays from
    nothing to all within a token: the triangular systems and the exponents at their worst."""
    from mlx_lm_amd.ops import kernels

    n, N, P = 200, 32, 16
    g = torch.Generator().manual_seed(9)
    base = torch.nn.functional.normalize(torch.randn(3, N, generator=g), dim=-1)
    k = torch.nn.functional.normalize(base[torch.arange(n) % 3] + 0.01 * torch.randn(n, N, generator=g), dim=-1)
    q, v = torch.randn(n, N, generator=g), torch.randn(n, P, generator=g)
    log_g = -torch.logspace(-6, 2, N)[None].expand(n, N) * torch.rand(n, 1, generator=g)
    beta = torch.full((n, 1), 0.999)
    for speeds in (log_g.contiguous(), torch.zeros(n, N), (log_g * 0.05).contiguous()):
        want = plain.unit_rms(plain.delta_recurrence(q.double(), k.double(), v.double(), speeds.double().exp(), beta.double()[:, 0]), 1e-6)
        state, out = torch.zeros(1, N * P).cuda(), torch.empty(n, P, device="cuda")
        kernels.delta_chunks(out, [t.cuda() for t in (q, k, v, speeds, beta)], state, 0, _spans([n]), _ints([0]), _ints([n]), _ints([0]), 1, 1, 1, N, P,
                             torch.ones(P).cuda(), 1e-6, None, _alloc, by_channel=True)
        assert (out.double().cpu() - want).abs().max() <= 1e-4 * want.abs().max()


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("W,B,taps,decay", [(64, 2, 4, 8.0), (33, 3, 1, 8.0), (20, 1, 7, 2.0), (120, 5, 3, 8.0), (512, 2, 4, 8.0), (520, 1, 2, 8.0), (700, 1, 4, 8.0)])
def test_the_recurrent_unit_in_portions_of_two_requests(W, B, taps, decay, dtype):
    """Two requests side by side, then one alone, in single tokens and portions shorter than the taps and longer than
    a span; parts of few channels and of so many that sixteen tokens fill the LDS; states and inputs carried over."""
    from mlx_lm_amd.ops import kernels

    g = torch.Generator().manual_seed(W + taps)
    rnd = lambda *s: torch.randn(*s, generator=g)  # noqa: E731
    w = W // B
    lens = [(1, 1), (2, 1), (70, 3), (1, 1), (1, 64), (5, 7), (65, 1), (1, 1), (63, 129)]
    total = [sum(x[r] for x in lens) for r in range(2)]
    conv_w, conv_b, lam = rnd(W, taps), rnd(W), rnd(W) - 3.0
    ra, ri = ((rnd(B, w, w) * w ** -0.5).to(dtype) for _ in range(2))
    ra_b, ri_b = rnd(B, w), rnd(B, w)
    x, y = [rnd(n, W) for n in total], [rnd(n, W) for n in total]
    want = []
    for a, b in zip(x, y):
        u = plain.causal_conv(a.double(), conv_w.double()) + conv_b.double()
        parts = u.view(-1, B, w)
        r, i = (plain.sigmoid(torch.stack([parts[:, p] @ m[p].double().t() + s[p].double() for p in range(B)], 1)).reshape(-1, W)
                for m, s in ((ra, ra_b), (ri, ri_b)))
        step = torch.exp(-decay * r * plain.softplus(lam.double()))
        S, rows = torch.zeros(W).double(), []
        for t in range(u.shape[0]):
            S = step[t] * S + torch.sqrt(1 - step[t] ** 2) * i[t] * u[t]
            rows.append(S)
        if decay == 8.0:
            assert torch.allclose(torch.stack(rows), plain.lru_recurrence(u, r, i, lam.double()))
        want.append(torch.stack(rows) * plain.gelu_tanh(b.double()))
    weights = kernels.RglruWeights(conv_w.cuda(), conv_b.cuda(), ra.cuda(), ra_b.cuda(), ri.cuda(), ri_b.cuda(), lam.cuda(), decay)
    S0 = 5
    ring = S0 + W
    state = torch.full((4, ring + taps * W), 7.0).cuda()
    state[[3, 1], S0:] = 0.0
    at, got = [0, 0], [[], []]
    for step in lens:
        rows = torch.cat([torch.cat([x[r][at[r] : at[r] + step[r]], y[r][at[r] : at[r] + step[r]]], 1) for r in range(2)]).cuda()
        pos = _ints([at[0] + i for i in range(step[0])] + [at[1] + i for i in range(step[1])])
        out = torch.empty(sum(step), W, dtype=dtype, device="cuda")
        kernels.rglru(out, rows[:, :W], rows[:, W:], weights, state, S0, ring, pos, _ints([0, step[0]]), _ints(step), _ints([3, 1]), 2,
                      None if max(step) == 1 else _spans(step), _alloc)
        got[0].append(out[: step[0]].cpu()), got[1].append(out[step[0] :].cpu())
        at = [at[0] + step[0], at[1] + step[1]]
    for r in range(2):
        err = (torch.cat(got[r]).double() - want[r]).abs().amax(-1) / want[r].abs().max()
        assert err.max() <= (5e-5 if dtype == torch.float32 else 4e-3), (r, int(err.argmax()), float(err.max()))
    # (the state itself is 32-bit: the gates' products do not round the convolution's output)
    for r, slot in enumerate((3, 1)):
        S = want[r][-1] / plain.gelu_tanh(y[r][-1].double())
        assert ((state[slot, S0 : S0 + W].double().cpu() - S).abs() <= 5e-5 * S.abs().max()).all()
    assert (state[[0, 2]] == 7.0).all() and (state[:, :S0] == 7.0).all()


def test_forty_requests_step_the_recurrent_unit_together():
    from mlx_lm_amd.ops import kernels

    g = torch.Generator().manual_seed(2)
    rnd = lambda *s: torch.randn(*s, generator=g)  # noqa: E731
    R, W, B, taps = 40, 72, 3, 3
    w = W // B
    args = [rnd(W, taps), rnd(W), rnd(B, w, w) * w ** -0.5, rnd(B, w), rnd(B, w, w) * w ** -0.5, rnd(B, w), rnd(W) - 3.0]
    weights = kernels.RglruWeights(*[t.cuda() for t in args], 8.0)
    slots = torch.randperm(R, generator=g).tolist()
    state = torch.zeros(R, W + taps * W).cuda()
    x, y = rnd(6, R, W), rnd(6, R, W)
    got = []
    for t in range(6):
        rows = torch.cat([x[t], y[t]], 1).cuda()
        out = torch.empty(R, W, device="cuda")
        kernels.rglru(out, rows[:, :W], rows[:, W:], weights, state, 0, W, _ints([t] * R), _ints(list(range(R))), _ints([1] * R), _ints(slots), R, None, _alloc)
        got.append(out.cpu())
    got = torch.stack(got)
    conv_w, conv_b, ra, ra_b, ri, ri_b, lam = (t.double() for t in args)
    for r in range(R):
        u = plain.causal_conv(x[:, r].double(), conv_w) + conv_b
        parts = u.view(-1, B, w)
        gates = [plain.sigmoid(torch.stack([parts[:, p] @ m[p].t() + s[p] for p in range(B)], 1)).reshape(-1, W) for m, s in ((ra, ra_b), (ri, ri_b))]
        want = plain.lru_recurrence(u, *gates, lam) * plain.gelu_tanh(y[:, r].double())
        assert (got[:, r].double() - want).abs().max() <= 5e-5 * want.abs().max()


@pytest.mark.parametrize("kernel,dtype,d,H,G", [
    ("tile", torch.float32, 48, 4, 2), ("tile", torch.float32, 64, 4, 2), ("tile", torch.float32, 128, 2, 1), ("tile", torch.bfloat16, 24, 4, 2),
    ("tile", torch.float32, 272, 2, 1), ("row", torch.float32, 40, 4, 2), ("row", torch.bfloat16, 48, 3, 3), ("prefill", torch.bfloat16, 32, 4, 2),
    ("prefill", torch.bfloat16, 64, 4, 1), ("prefill", torch.bfloat16, 128, 4, 2), ("decode", torch.float32, 32, 4, 2), ("decode", torch.bfloat16, 64, 4, 2),
    ("decode", torch.bfloat16, 128, 8, 2), ("group", torch.bfloat16, 64, 16, 2), ("group", torch.bfloat16, 128, 40, 2)])
@pytest.mark.parametrize("splits", [1, 3])
def test_attention_kernels_with_a_sink_and_a_gate_a_head(kernel, dtype, d, H, G, splits):
    """Queries at positions 530 .. of a request: sinks far above the scores, among them and far below, a gate a
    head; a key that stands out far back among hundreds."""
    from mlx_lm_amd.ops import kernels
    from test_pafutar_gpu import _paged

    if splits > 1 and kernel in ("tile", "prefill"):
        pytest.skip("tiles are not split")
    offset = 530
    n_q = {"tile": 16, "row": 3, "prefill": 150, "decode": 3, "group": 3}[kernel]
    n = offset + n_q
    g = torch.Generator().manual_seed(d + H)
    q = torch.randn(n_q, H, d, generator=g).to(dtype)
    k = torch.randn(n, G, d, generator=g).to(dtype)
    v = torch.randn(n, G, d, generator=g).to(dtype)
    gate = torch.randn(n_q, H, generator=g) * 2
    sinks = torch.linspace(-30.0, 14.0, H)
    k[2, G - 1] = (q[0, H - 1].float() * 3.0).to(dtype)
    scale = 1.0 / d**0.5
    s = torch.einsum("ihd,jhd->hij", q.double(), k.double().repeat_interleave(H // G, dim=1)) * scale
    i, j = torch.arange(n_q)[:, None] + offset, torch.arange(n)[None, :]
    s = torch.cat([s.masked_fill((j > i).unsqueeze(0), float("-inf")), sinks.double().view(H, 1, 1).expand(H, n_q, 1)], 2)
    p = torch.softmax(s, -1)
    assert p[H - 1, 0, 2] > 0.02 and p[H - 1, 1, n] > 0.9 and p[0, 1, n] < 1e-9
    want = torch.einsum("hij,jhd->ihd", p[:, :, :n], v.double().repeat_interleave(H // G, dim=1))
    want = (want * torch.sigmoid(gate.double())[:, :, None]).reshape(n_q, H * d)

    kv, block_table = _paged(k, v, 16, dtype, seed=d)
    qd = q.reshape(n_q, H * d).cuda()
    out = torch.empty_like(qd)
    zeros = torch.zeros(n_q, dtype=torch.int32, device="cuda")
    positions = (torch.arange(n_q, dtype=torch.int32) + offset).cuda()
    wide = torch.full((n_q, H + 7), float("nan"))
    wide[:, 3 : 3 + H] = gate
    terms = kernels.ScoreTerms(sinks=sinks.cuda(), head_gate=wide.cuda()[:, 3 : 3 + H])
    items = torch.arange(n_q, dtype=torch.int32).cuda()
    part_o, part_ml = torch.empty(n_q * H * splits * d, device="cuda"), torch.empty(n_q * H * splits * 2, device="cuda")
    tables = (block_table, zeros, positions)
    if kernel == "tile":
        kernels.attn_tile(out, qd, kv, *tables, _ints([0, n_q]), 1, H, scale, 0, terms)
    elif kernel == "prefill":
        kernels.attn_prefill(out, qd, kv, *tables, _ints([128, n_q - 128, 0, 128]), 2, H, scale, 0, terms)
    elif kernel == "row":
        kernels.attn_row(out, qd, kv, *tables, items, n_q, H, scale, 0, splits, part_o, part_ml, terms)
    elif kernel == "group":
        kernels.attn_decode_group(out, qd, kv, *tables, items, n_q, H, scale, 0, splits, part_o, part_ml, terms=terms)
    else:
        outs = []
        for join in (0, 2):
            kernels.attn_decode(out, qd, kv, *tables, items, n_q, H, scale, 0, splits, part_o, part_ml, n_waves=4, join_in_kernel=join, terms=terms)
            outs.append(out.clone())
        assert (outs[0].float() - outs[1].float()).abs().max() <= 1e-2 * want.abs().max()
    err = (out.double().cpu() - want).abs().max().item()
    assert err <= (2e-5 if dtype == torch.float32 else 2.5e-2) * want.abs().max().item(), err


@pytest.mark.parametrize("n_out,top,groups", [(8, 3, (4, 2)), (5, 1, None), (12, 4, (3, 2)), (70, 6, (7, 3)), (64, 8, (8, 4)), (200, 40, (50, 25)),
                                              (9, 3, (9, 4)), (512, 8, (8, 3)), (6, 6, (2, 2))])
def test_the_choice_by_sigmoid_out_of_the_best_groups(n_out, top, groups):
    """Experts and weights as the plain side has them, ties included (rounded outputs: the lower index first, and
    two equal largest scores of a group both count); the same choice inside the experts' kernel."""
    from mlx_lm_amd.ops import kernels

    T = 40
    g = torch.Generator().manual_seed(n_out)
    z = torch.randn(T, n_out, generator=g) * 2
    z[T // 2 :] = torch.round(z[T // 2 :] * 2) / 2
    idx, weight = torch.empty(T, top, dtype=torch.int32, device="cuda"), torch.empty(T, top, device="cuda")
    kernels.router_choice(idx, weight, z.cuda(), None, top, renormalize=True, weight_scale=1.5, scores="sigmoid", groups=groups)
    router = {"experts": n_out, "top": top, "scale": 1.5, "groups": dict(zip(("count", "keep"), groups or (1, 1)))}
    for t in range(T):
        chosen, want = plain.choose(z[t].double(), router)
        if t < T // 2:
            assert idx[t].tolist() == chosen.tolist()
        # (tied scores may be told apart differently, the weights are the same)
        assert torch.allclose(weight[t].double().cpu(), want, rtol=1e-5, atol=1e-7)
        if groups and t >= T // 2:
            size, s = n_out // groups[0], torch.sigmoid(z[t].double())
            score = torch.stack([s[i * size : (i + 1) * size].topk(min(2, size)).values.sum() for i in range(groups[0])])
            least = score.topk(groups[1]).values.min()
            assert all(score[e // size] >= least - 1e-12 for e in idx[t].tolist())
    if top > kernels.ROUTED_MOST:
        return
    width, F, dtype = 16, 8, torch.float32
    x = torch.randn(3, width, generator=g).to(dtype).cuda()
    ws = [torch.randn(n_out, *s, generator=g).cuda() for s in ((F, width), (F, width), (width, F))]
    outs = []
    for route in (None, (z[:3].cuda(), kernels.Route(None, True, 1.5, "sigmoid", groups))):
        y = torch.empty(3, width, device="cuda")
        i2, w2 = (idx[:3].clone(), weight[:3].clone()) if route is None else (torch.zeros_like(idx[:3]), torch.zeros_like(weight[:3]))
        kernels.expert_rows(y, x, *ws, i2, w2, top, torch.empty(3 * top, F, device="cuda"), accumulate=False, route=route)
        outs.append(y)
        assert torch.equal(i2, idx[:3]) and torch.equal(w2, weight[:3])
    assert torch.equal(*outs)


# -- each mixer alone, in a model of one layer ----------------------------------------------


ALONE = {
    "delta": [_delta(4, 2, 16, 24, 4)],
    "delta, one tap": [_delta(2, 2, 24, 8, 1)],
    "delta, odd sizes": [_delta(3, 1, 7, 9, 3)],
    "delta with experts": [_moe(_delta(2, 1, 16, 16, 2), 20, 4, 2, (2, 1))],
    "lru": [_lru(48, 3, 4)],
    "lru, odd sizes": [_lru(35, 5, 3)],
    "lru, one part and one tap": [_dense(_lru(40, 1, 1), 12)],
    "attention": [_attention(3, 1, 16, 24, 8, 300.0)],
    "attention, scaled frequencies": [_attention(4, 2, 32, 32, 32, 100.0, (4.0, 1.0, 4.0, 40))],
    "attention, eight heads a key head": [_dense(_attention(16, 2, 64, 48, 16, 1e4, scale=0.3), 20)],
    "attention, nothing turns": [_attention(2, 2, 10, 6, 0)],
    "two passes": [_dense(_attention(2, 1, 16, 16, 4, 50.0), 16), _lru(16, 2, 2)],
}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(ALONE))
def test_a_mixer_alone(tmp_path, name, dtype):
    """Whole, the last tokens one by one, in portions of changing size and of two tokens; portions
    shorter than the convolution's taps among them."""
    config = _config(48, 61, copy.deepcopy(ALONE[name]), streams=1 + len(name) % 4, loop=(0, 2, 2) if name == "two passes" else None)
    weights = plain.random_weights(config, 7, sharp=2.0, rank=5)
    folder = _folder(str(tmp_path / "m"), config, weights)
    n = 100
    tokens = helpers.random_tokens(n, 61, seed=len(name))
    want = _plain(weights, config, tokens, dtype)
    strict = "experts" not in name
    eng = _engine(folder, dtype, n_pages=16)
    _close(_run(eng, "whole", tokens, [n]), want, dtype, name + " whole", strict)
    _close(_run(eng, "decoded", tokens, [n - 40] + [1] * 40), want, dtype, name + " decoded", strict)
    _close(_run(eng, "portions", tokens, helpers.cuts_changing(n)), want, dtype, name + " in portions", strict)
    _close(_run(eng, "twos", tokens[:40], [2] * 20), want[:40], dtype, name + " in twos", strict)
    _close(_run(eng, "ones", tokens[:20], [1] * 20), want[:20], dtype, name + " from the first token one by one", strict)
    eng.cache.check()


# -- whole, decoded, portions ----------------------------------------------------------


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name,n", [("A", 150), ("B", 130), ("C", 200)])
def test_whole_decoded_and_portions(models, dtype, name, n):
    folder, config, weights = models[name, dtype]
    tokens = helpers.random_tokens(n, config["vocab"], seed=n)
    want = _plain(weights, config, tokens, dtype)
    eng = _engine(folder, dtype, n_pages=(n + 15) // 16 + 2)
    _close(_run(eng, "whole", tokens, [n]), want, dtype, "whole")
    _close(_run(eng, "decoded", tokens, [n - 90] + [1] * 90), want, dtype, "last 90 one by one")
    _close(_run(eng, "portions", tokens, helpers.cuts_changing(n)), want, dtype, "portions of changing size")
    _close(_run(eng, "twos", tokens[:64], [2] * 32), want[:64], dtype, "portions of two tokens")
    eng.cache.check()
    assert eng.cache.free_pages() == eng.cache.n_pages


@pytest.mark.parametrize("page_size", [16, 64])
def test_portions_give_what_the_whole_prompt_gives(models, page_size):
    """However a prompt is cut (at a page's or a chunk's border, one token before and after it, token by
    token, shorter than the taps), the logits agree with the uncut prompt's to rounding: the engine against itself."""
    folder, config, _ = models["A", "float32"]
    tokens = helpers.random_tokens(150, config["vocab"], seed=8)
    eng = _engine(folder, "float32", n_pages=192 // page_size, page_size=page_size)
    whole = _run(eng, "w", tokens, [150])
    for cuts in (helpers.cuts_changing(150), [1] * 150, [16, 16, 1, 15, 17, 15, 2, 68], [15, 2, 3, 17, 27, 64, 22], [64, 64, 22], [63, 2, 63, 22], [147, 3],
                 [65, 64, 21]):
        got = _run(eng, "c", tokens, cuts)
        assert (got - whole).abs().max().item() <= 2e-5 * whole.abs().max().item(), cuts[:6]


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_first_tokens_and_long_decode(models, dtype):
    """Every token one by one from the first: 400 of them, recorded decode steps replayed, page after
    page taken, the states and the convolutions' inputs carried 400 times."""
    folder, config, weights = models["C", dtype]
    n = 400
    tokens = helpers.random_tokens(n, config["vocab"], seed=77)
    want = _plain(weights, config, tokens, dtype)
    eng = _engine(folder, dtype, n_pages=n // 16)
    got = _run(eng, "r", tokens, [1] * n)
    _close(got[:8], want[:8], dtype, "first tokens")
    _close(got, want, dtype, "decoding every token")


def test_a_key_far_back_found_over_a_sink(tmp_path):
    """A marked key 896 tokens back stands out for the last query among hundreds, over a sink that takes
    nearly all where nothing stands out; in a prompt, at a portion's end, and decoded alone."""
    config = _config(32, 40, [_attention(2, 1, 24, 16, 8, 1e4, scale=1.0)], streams=3, eps=1e-6)
    w = plain.random_weights(config, 11)
    # column 0 of the embedding marks the ids below 4 (keys), column 1 the ids 4 to 7 (queries); one column of a
    # head that does not turn answers the mark
    w["embed"][:8] *= 0.05
    w["embed"][:, :2] = 0.0
    w["embed"][:4, 0], w["embed"][4:8, 1] = 6.0, 6.0
    w["l0.norm1"][:2], w["l0.norm1.b"][:2] = 2.0, 0.0
    w["l0.mix.q"][:, :2], w["l0.mix.k"][:, :2] = 0.0, 0.0
    w["l0.mix.q"][20::24, 1], w["l0.mix.k"][20, 0] = 3.0, 3.0
    w["l0.mix.g"][:, :2] = 0.0
    w["l0.mix.o"] *= 4.0
    w["l0.mix.sink"][:] = torch.tensor([9.0, 11.0])
    folder = _folder(str(tmp_path / "m"), config, w)
    n, key = 920, 23
    tokens = [8 + t for t in helpers.random_tokens(n, 32, seed=5)]
    tokens[key], tokens[n - 1] = 2, 5
    want = plain.model(w, config, tokens)
    other, calm = list(tokens), dict(w)
    other[key] = 20
    moved = ((plain.model(w, config, other)[n - 1] - want[n - 1]).abs().max() / want.abs().max()).item()
    calm["l0.mix.sink"] = w["l0.mix.sink"] - 40.0
    sunk = ((plain.model(calm, config, tokens)[:200] - want[:200]).abs().max() / want.abs().max()).item()
    assert moved > 0.02 and sunk > 0.02, (moved, sunk)
    eng = _engine(folder, "float32", n_pages=60)
    for cuts in ([n], [n - 1, 1], [n - 6, 6], [key + 1, n - key - 2, 1], [n - 3, 1, 1, 1], [512, 402, 2, 4]):
        got = _run(eng, "r", tokens, cuts)
        _close(got[n - 1 :], want[n - 1 :], "float32", f"the last of {cuts}")
        _close(got, want, "float32", f"{cuts}")


def test_a_token_far_back_that_the_unit_still_holds(tmp_path):
    """One channel that hardly decays takes in a marked token alone; the logits 700 tokens later still lean on it."""
    config = _config(32, 40, [_lru(16, 2, 2)], streams=2)
    w = plain.random_weights(config, 12)
    w["embed"][:, 0] = 0.0
    w["embed"][2, 0] = 60.0
    w["l0.mix.x"][:, 0] = 0.0
    w["l0.mix.x"][5], w["l0.mix.x.b"][5] = 0.0, 0.0
    w["l0.mix.x"][5, 0] = 5.0
    w["l0.norm1"][0], w["l0.norm1.b"][0] = 1.0, 0.0
    w["l0.mix.lam"][5], w["l0.mix.conv.b"][5] = -9.0, 0.0
    w["l0.mix.y.b"][5], w["l0.mix.o"][:, 5] = 3.0, w["l0.mix.o"][:, 5] * 8.0
    folder = _folder(str(tmp_path / "m"), config, w)
    n, mark = 730, 23
    tokens = [8 + t for t in helpers.random_tokens(n, 32, seed=6)]
    tokens[mark] = 2
    want = plain.model(w, config, tokens)
    other = list(tokens)
    other[mark] = 20
    moved = ((plain.model(w, config, other)[n - 1] - want[n - 1]).abs().max() / want.abs().max()).item()
    assert moved > 0.01, moved
    eng = _engine(folder, "float32", n_pages=1)
    for cuts in ([n], [n - 1, 1], [mark + 1, n - mark - 2, 1], [mark, 2, 64, n - mark - 66], [n - 40] + [1] * 40):
        _close(_run(eng, "r", tokens, cuts), want, "float32", f"{cuts[:4]}")


# -- batches -------------------------------------------------------------------------------


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["A", "B", "C"])
def test_mixed_batches_equal_each_request_alone(models, dtype, name):
    """Up to four live requests of unequal lengths, portions beside single tokens, requests that sit a
    step out; state rows (the matrices, the units' states, the convolutions' inputs) and pages of finished
    requests are used again by later ones, and what freed pages hold is never read."""
    from mlx_lm_amd.engine import StepEntry

    folder, config, weights = models[name, dtype]
    lengths = [70, 9, 131, 40, 3, 97, 55]
    tokens, steps = helpers.mixed_trace({"vocab_size": config["vocab"]}, 21, lengths, n_live=4)
    eng = _engine(folder, dtype, n_pages=helpers.held(lengths, 4) // 16, max_requests=4)
    got = {rid: [] for rid in tokens}
    for s in steps:
        entries = []
        for e in s["entries"]:
            if not eng.has_request(e["id"]):
                eng.add_request(e["id"])
            entries.append(StepEntry(e["id"], e["tokens"], e["want"]))
        logits = eng.step(entries).clone()
        at = 0
        for e in entries:
            got[e.request_id].append(logits[at : at + len(e.want)])
            at += len(e.want)
        for rid in s["end"]:
            eng.end_request(rid)
        eng.cache.poison_free_pages()
    for rid, toks in tokens.items():
        _close(torch.cat(got[rid]), _plain(weights, config, toks, dtype), dtype, f"request {rid} in mixed batches")
    eng.cache.check()
    assert eng.cache.free_pages() == eng.cache.n_pages


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("n_requests", [20, 70])
def test_many_requests_decode_together(models, dtype, n_requests):
    from mlx_lm_amd.engine import StepEntry

    folder, config, weights = models["C", dtype]
    lengths = [5 + (7 * i) % 90 for i in range(n_requests)]
    steps = 12 if n_requests == 20 else 4
    tokens = [helpers.random_tokens(n + steps, config["vocab"], seed=200 + i) for i, n in enumerate(lengths)]
    eng = _engine(folder, dtype, n_pages=sum((n + steps + 15) // 16 for n in lengths), max_requests=n_requests)
    for i, (n, toks) in enumerate(zip(lengths, tokens)):
        eng.add_request(i)
        eng.step([StepEntry(i, toks[:n], [])])
    got = [[] for _ in lengths]
    for step in range(steps):
        logits = eng.step([StepEntry(i, [tokens[i][n + step]], [0]) for i, n in enumerate(lengths)]).clone()
        for i in range(len(lengths)):
            got[i].append(logits[i])
    for i, n in list(enumerate(lengths))[:: 1 if n_requests == 20 else 7]:
        _close(torch.stack(got[i]), _plain(weights, config, tokens[i], dtype)[n:], dtype, f"request {i} among {n_requests}")


def _drawn_config(seed):
    g = torch.Generator().manual_seed(1000 + seed)

    def pick(options):
        return options[int(torch.randint(0, len(options), (), generator=g))]

    layers = []
    for _ in range(pick([1, 2, 3, 4, 5])):
        kind = pick(["delta", "lru", "attention"])
        if kind == "delta":
            kv = pick([1, 2, 3])
            entry = _delta(kv * pick([1, 2, 4]), kv, pick([8, 12, 16, 32, 40, 64]), pick([8, 16, 24, 48, 80, 128]), pick([1, 2, 3, 4, 5]))
        elif kind == "lru":
            b = pick([1, 2, 3, 8])
            entry = _lru(b * pick([5, 8, 12, 32, 70]), b, pick([1, 2, 3, 4, 6]))
        else:
            kv, dim = pick([1, 2, 3]), pick([8, 16, 20, 48, 64, 128])
            scaling = pick([None, (4.0, 1.0, 4.0, 64), (2.5, 0.3, 9.0, 20)])
            entry = _attention(kv * pick([1, 2, 8]), kv, dim, pick([8, 24, 64, 128]), pick([0, 2, dim // 2, dim]), pick([10.0, 1e4, 1e6]), scaling,
                               scale=pick([None, 0.3]))
        mlp = pick(["none", "dense", "moe", "moe"])
        if mlp == "dense":
            entry = _dense(entry, pick([8, 20, 64]))
        elif mlp == "moe":
            count = pick([1, 2, 4])
            size, keep = pick([1, 2, 5]), pick(list(range(1, count + 1)))
            entry = _moe(entry, pick([4, 8, 20, 64]), count * size, pick(list(range(1, min(4, keep * size) + 1))), (count, keep), pick([0.5, 1.0, 2.5]))
        layers.append(entry)
    loop = None
    if pick([0, 1, 1]):
        a = pick(list(range(len(layers))))
        loop = (a, pick(list(range(a + 1, len(layers) + 1))), pick([1, 2, 3]))
    return _config(pick([16, 40, 64, 104, 256]), pick([17, 100, 257, 1000]), layers, streams=pick([1, 2, 3, 4, 6]), loop=loop, eps=pick([1e-6, 1e-5, 1e-2]),
                   logit_scale=pick([0.125, 1.0, 2.5]))


@pytest.mark.parametrize("seed", range(14))
def test_drawn_configurations(tmp_path, seed):
    """Every size, the layers' order, the loop and constants drawn: whole, in portions, and two requests
    side by side, in float32."""
    from mlx_lm_amd.engine import StepEntry

    config = _drawn_config(seed)
    weights = plain.random_weights(config, 100 + seed, sharp=2.0, rank=1 + seed % 7)
    folder = _folder(str(tmp_path / "m"), config, weights)
    a, b = helpers.random_tokens(120, config["vocab"], seed=seed), helpers.random_tokens(75, config["vocab"], seed=50 + seed)
    wa, wb = plain.model(weights, config, a), plain.model(weights, config, b)
    eng = _engine(folder, "float32", n_pages=16)
    _close(_run(eng, "whole", a, [120]), wa, "float32", f"seed {seed} whole: {json.dumps(config)}")
    eng.add_request("a"), eng.add_request("b")
    ga, gb, ia, ib = [], [], 0, 0
    for ca, cb in ((50, 2), (1, 40), (1, 1), (38, 1), (2, 30), (28, 1)):
        out = eng.step([StepEntry("a", a[ia : ia + ca], list(range(ca))), StepEntry("b", b[ib : ib + cb], list(range(cb)))]).clone()
        ga.append(out[:ca]), gb.append(out[ca:])
        ia, ib = ia + ca, ib + cb
    _close(torch.cat(ga), wa, "float32", f"seed {seed}, first of two")
    _close(torch.cat(gb), wb, "float32", f"seed {seed}, second of two")


def test_recorded_steps_equal_eager_steps(models):
    """Decode steps replayed from recorded graphs against the same steps run eagerly, bit for bit."""
    from mlx_lm_amd.engine import StepEntry

    folder, config, _ = models["A", "bfloat16"]
    seqs = {"a": helpers.random_tokens(60, config["vocab"], 1), "b": helpers.random_tokens(45, config["vocab"], 2)}
    results = {}
    for use_graphs in (True, False):
        eng = _engine(folder, "bfloat16", n_pages=10, use_graphs=use_graphs)
        assert eng.use_graphs == use_graphs  # every part launches kernels only
        for r in seqs:
            eng.add_request(r)
        out = [eng.step([StepEntry("a", seqs["a"][:20], [19]), StepEntry("b", seqs["b"][:5], [4])]).clone()]
        for i in range(40):
            out.append(eng.step([StepEntry("a", [seqs["a"][20 + i]], [0]), StepEntry("b", [seqs["b"][5 + i]], [0])]).clone())
        if use_graphs:
            assert helpers.decode_graphs(eng, 2)[0].graph is not None
        results[use_graphs] = torch.cat(out)
    assert torch.equal(results[True], results[False])


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_products_left_in_parts_for_the_next_pass(models, dtype):
    """K split wherever a product can be: sublayers leave their parts to the streams' kernel."""
    from mlx_lm_amd.ops import kernels

    folder, config, weights = models["C", dtype]
    tokens = helpers.random_tokens(90, config["vocab"], seed=31)
    want = _plain(weights, config, tokens, dtype)
    eng = _engine(folder, dtype, n_pages=8)
    kernels.force_splits = 2
    try:
        _close(_run(eng, "r", tokens, [40, 9, 2, 1, 1, 1, 30, 1, 1, 1, 1, 1, 1]), want, dtype, "with split products")
    finally:
        kernels.force_splits = 0


# -- generation through the entry points -----------------------------------------------------


def test_greedy_generation_through_the_scheduler(models):
    from mlx_lm_amd import batch_generate, load, stream_generate

    folder, config, weights = models["A", "float32"]
    model, tok = load(folder, dtype="float32")
    prompts = [helpers.random_tokens(n, config["vocab"], seed=n) for n in (23, 5, 61)]
    want = [plain.greedy(weights, config, p, 10) for p in prompts]
    got = [r.token for r in stream_generate(model, tok, prompts[0], max_tokens=10, prefill_step_size=7)]
    assert got == want[0]
    batch = batch_generate(model, tok, prompts, max_tokens=10)
    assert [[int(t) for t in text.split()] for text in batch.texts] == want


def test_command_line_and_trace_replay(tmp_path, models):
    """``python -m mlx_lm_amd generate`` on a folder of this design, and the replay program on that
    folder: a prompt in two steps beside a second request that starts later."""
    folder, config, weights = models["B", "float32"]
    prompt = [3, 1, 4, 1, 5, 9, 2, 6]
    want = plain.greedy(weights, config, prompt, 25)
    env = dict(os.environ, PYTHONPATH=ROOT)
    out = subprocess.run(
        [sys.executable, "-m", "mlx_lm_amd", "generate", "--model", folder, "--prompt-ids", ",".join(map(str, prompt)),
         "--max-tokens", "25", "--dtype", "float32", "--verbose", "F", "--num-pages", "8", "--prefill-step-size", "3"],
        capture_output=True, text=True, env=env, timeout=300)
    assert out.returncode == 0, out.stderr[-2000:]
    assert out.stdout.strip() == " ".join(map(str, want))
    a, b = helpers.random_tokens(50, config["vocab"], seed=9), helpers.random_tokens(20, config["vocab"], seed=10)
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": a[:31], "want": [30]}], "end": []},
             {"step": 1, "entries": [{"id": "x", "tokens": a[31:], "want": [0, 18]}, {"id": "y", "tokens": b, "want": [19]}], "end": ["x", "y"]}]
    proc = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", folder, "--dtype", "float32",
                           "--out", str(tmp_path / "out"), "--max-tokens", "128"],
                          input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True, timeout=300)
    assert proc.returncode == 0, proc.stderr[-2000:]
    assert "done 0" in proc.stdout and "done 1" in proc.stdout
    wa, wb = plain.model(weights, config, a), plain.model(weights, config, b)
    first = np.fromfile(tmp_path / "out" / "0.f32", dtype="<f4").reshape(-1, config["vocab"])
    second = np.fromfile(tmp_path / "out" / "1.f32", dtype="<f4").reshape(-1, config["vocab"])
    _close(torch.from_numpy(first), wa[30:31], "float32", "the replay's first step")
    _close(torch.from_numpy(second), torch.stack([wa[31], wa[49], wb[19]]), "float32", "the replay's second step")
