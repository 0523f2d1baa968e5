"""Gilidra in the engine against the plain implementation (plain_gilidra.py): each mechanism's
kernels, each mixer alone in a one-layer model, whole prompts, decoding, portions, mixed batches,
reused pages and state rows, window edges, far tokens, generation through the entry points."""

import copy
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import helpers
import plain_gilidra as plain
from test_gilidra import SMALL, _config, _delta, _latent, _moe, _wkv

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))

# max |engine - plain| over max |plain logits|: float32 sums where the plain side has float64;
# bfloat16 rounds activations between the products (the plain side gets the rounded matrices)
TOL = {"float32": 5e-5, "bfloat16": 6e-2}

CONFIGS = {
    "A": SMALL,
    # corners: one head, one key head for all heads, a key head for every head, one tap, seven taps,
    # one expert of one, every expert chosen, an inner size that is no multiple of eight, a window of one
    # and of everything, two readers of one layer's latents with a shorter and a longer window, values
    # wider and narrower than keys and no multiples of four, a logit scale above one
    "B": _config(72, 97, [
        _moe(_delta(4, 1, 12, 20, 1), 10, 1, 1, 0.5),
        _latent(1, 24, 4, 20, 8, 28, 1, base=50.0),
        _moe(_wkv(1, 20), 12, 6, 6, 3.0),
        _moe(_latent(3, 8, 4, 12, 16, 28, 25, base=50.0, kv_from=1, scale=0.5), 9, 5, 2),
        _delta(3, 3, 20, 10, 7),
        _latent(2, 16, 4, 8, 9, 28, 0, base=50.0, kv_from=1),
        _wkv(3, 10),
        _moe(_latent(1, 6, 2, 44, 20, 60, 33, base=9.0), 16, 3, 2)],
        eps=1e-3, logit_scale=1.7),
    # wider, for bfloat16: heads of 64
    "C": _config(128, 300, [
        _moe(_wkv(2, 64), 96, 8, 2, 1.7),
        _moe(_latent(8, 32, 16, 48, 48, 48, 70, base=1e5), 64, 8, 3),
        _moe(_delta(4, 2, 64, 48, 4), 72, 6, 2),
        _moe(_latent(8, 64, 16, 32, 40, 48, 45, base=1e5, kv_from=1), 96, 5, 2),
        _moe(_delta(2, 1, 32, 128, 2), 64, 8, 4)], logit_scale=0.3),
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
    score may rightly fall the other way after rounding, and the states carry that on to later tokens."""
    out = {}
    for name, dtype in [(n, d) for n in CONFIGS for d in ("float32", "bfloat16")]:
        config = copy.deepcopy(CONFIGS[name])
        for entry in config["layers"]:
            if entry["mlp"] is not None and dtype == "bfloat16":
                entry["mlp"]["router"]["top"] = entry["mlp"]["router"]["experts"]
        weights = plain.random_weights(config, SEEDS[name], sharp=2.0, decay_rank=RANKS[name])
        out[name, dtype] = (_folder(str(tmp_path_factory.mktemp("gil" + name)), config, weights), config, weights)
    return out


def _engine(folder, dtype, n_pages, page_size=16, max_requests=4, **kw):
    from mlx_lm_amd.engine import Engine
    from mlx_lm_amd.utils import load_model

    model, _ = load_model(folder, dtype=dtype)
    return Engine(model, dtype=dtype, page_size=page_size, n_pages=n_pages, max_requests=max_requests, **kw)


def _plain(weights, config, tokens, dtype):
    w = helpers.round_matrices_to_bf16(weights) if dtype == "bfloat16" else weights
    return plain.model(w, config, tokens)


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
        req += [r] * ((n + 63) // 64)
        lo += list(range(0, n, 64))
    return len(req), _ints(req), _ints(lo), _ints(first)


# -- each mechanism's kernels alone -------------------------------------------------------


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("width", [8, 100, 1500])
def test_dynamic_tanh_and_a_normed_embedding(dtype, width):
    from mlx_lm_amd.ops import kernels

    g = torch.Generator().manual_seed(width)
    x = torch.randn(5, width + 4, generator=g) * 20.0
    w = {"n": torch.randn(width, generator=g), "n.b": torch.randn(width, generator=g), "n.alpha": torch.tensor(0.37)}
    norm = tuple(t.cuda() for t in (w["n.alpha"].reshape(1), w["n"], w["n.b"]))
    w = {k: v.double() for k, v in w.items()}
    out = torch.empty(5, width, dtype=dtype, device="cuda")
    kernels.dynamic_tanh(out, x.cuda()[:, :width], norm)
    tol = 2e-6 if dtype == torch.float32 else 2e-2
    assert (out.double().cpu() - plain.dynamic_tanh(x[:, :width].double(), w, "n")).abs().max() <= tol
    table = torch.randn(9, width, generator=g).to(dtype)
    rows = torch.empty(4, width, device="cuda")
    kernels.embed_dynamic_tanh(rows, table.cuda(), _ints([8, 0, 3, 3]), 2.5, norm)
    want = plain.dynamic_tanh(table.double()[[8, 0, 3, 3]] * 2.5, w, "n")
    assert (rows.double().cpu() - want).abs().max() <= 2e-6


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_the_token_shift_over_portions_of_two_requests(dtype):
    """Portions of changing size of two requests side by side; the row before a portion's first comes
    from the state row, zeros before a request's start."""
    from mlx_lm_amd.ops import kernels

    g = torch.Generator().manual_seed(3)
    W, n, M = 40, 14, 3
    x = [torch.randn(n, W, generator=g) for _ in range(2)]
    w = {"n": torch.randn(W, generator=g), "n.b": torch.randn(W, generator=g), "n.alpha": torch.tensor(0.8)}
    norm = tuple(t.cuda() for t in (w["n.alpha"].reshape(1), w["n"], w["n.b"]))
    w = {k: v.double() for k, v in w.items()}
    mu = torch.rand(M, W, generator=g)
    state = torch.full((3, 5 + W), 9.0).cuda()
    state[[2, 0], 5:] = 0
    at, got = [0, 0], [[], []]
    for lens in ((2, 1), (1, 1), (1, 4), (7, 2), (1, 5), (2, 1)):
        rows = torch.cat([x[r][at[r] : at[r] + lens[r]] for r in range(2)]).cuda()
        out = torch.empty(1 + M, sum(lens), W, dtype=dtype, device="cuda")
        kernels.token_mix(out, rows, norm, mu.cuda(), state, 5, _ints([0] * lens[0] + [1] * lens[1]), _ints([0, lens[0]]), _ints(lens), _ints([2, 0]))
        got[0].append(out[:, : lens[0]].cpu()), got[1].append(out[:, lens[0] :].cpu())
        at = [at[0] + lens[0], at[1] + lens[1]]
    tol = 2e-6 if dtype == torch.float32 else 2e-2
    for r in range(2):
        h = plain.dynamic_tanh(x[r].double(), w, "n")
        before = torch.cat([torch.zeros_like(h[:1]), h[:-1]])
        want = torch.stack([h] + [h + (before - h) * m for m in mu.double()])
        assert (torch.cat(got[r], 1).double() - want).abs().max() <= tol
    assert (state[1] == 9.0).all() and (state[:, :5] == 9.0).all()


def _delta_operands(n, H, G, N, P, taps, g):
    """Random projection rows ``[q | k | v | gate | b | a]`` of one request and what they mean."""
    C = 2 * G * N + H * P
    return torch.randn(n, C + H * P + 2 * H, generator=g)


def _delta_plain(u, conv_w, a_log, dt_bias, norm_w, H, G, N, P, eps):
    u, C = u.double(), 2 * G * N + H * P
    x = plain.silu(plain.causal_conv(u[:, :C], conv_w.double()))
    q = plain.unit_length(x[:, : G * N].view(-1, G, N)) * N ** -0.5
    k, v = plain.unit_length(x[:, G * N : 2 * G * N].view(-1, G, N)), x[:, 2 * G * N :].view(-1, H, P)
    gate, b, a = u[:, C : C + H * P], u[:, C + H * P : C + H * P + H], u[:, C + H * P + H :]
    beta = plain.sigmoid(b)
    decay = torch.exp(-torch.exp(a_log.double()) * torch.log1p(torch.exp(a + dt_bias.double())))
    o = torch.stack([plain.delta_recurrence(q[:, h // (H // G)], k[:, h // (H // G)], v[:, h], decay[:, h], beta[:, h]) for h in range(H)], 1)
    o = plain.unit_rms(o, eps) * norm_w.double()
    return (o * plain.silu(gate).view(-1, H, P)).flatten(1)


@pytest.mark.parametrize("H,G,N,P,taps", [(4, 2, 16, 32, 4), (3, 3, 8, 8, 1), (2, 1, 64, 64, 4), (4, 1, 5, 6, 3), (2, 2, 128, 128, 4), (1, 1, 40, 20, 7),
                                          (2, 1, 200, 100, 2), (1, 1, 17, 33, 4), (2, 1, 256, 256, 2)])
def test_the_delta_rule_in_portions_of_two_requests(H, G, N, P, taps):
    """Two requests side by side: single tokens (operands made in the step's own kernel), portions of a
    few tokens (prepared, token by token) and of many (in chunks), cut at and around a chunk's edge;
    the convolution's inputs and the states carried over, other rows untouched."""
    from mlx_lm_amd.ops import kernels

    g = torch.Generator().manual_seed(N + P)
    C, eps = 2 * G * N + H * P, 1e-4
    lens = [(1, 1), (2, 1), (70, 3), (1, 1), (1, 64), (5, 7), (65, 1), (1, 1), (63, 129)]
    total = [sum(x[r] for x in lens) for r in range(2)]
    u = [_delta_operands(n, H, G, N, P, taps, g) for n in total]
    conv_w, norm_w = torch.randn(C, taps, generator=g), 1 + 0.3 * torch.randn(P, generator=g)
    a_log, dt_bias = torch.randn(H, generator=g) - 1.0, torch.randn(H, generator=g) - 1.0
    want = [_delta_plain(x, conv_w, a_log, dt_bias, norm_w, H, G, N, P, eps) for x in u]
    S0 = 8  # the matrices' place in a state row
    ring = S0 + H * N * P
    floats = (ring + taps * C + 3) // 4 * 4
    state = torch.full((4, floats), 5.0).cuda()
    state[[3, 1], S0:] = 0.0
    raw = kernels.DeltaRaw(conv_w.cuda(), ring, a_log.cuda(), dt_bias.cuda(), N ** -0.5)
    slots = _ints([3, 1])
    at, got = [0, 0], [[], []]
    for step in lens:
        rows = torch.cat([u[r][at[r] : at[r] + step[r]] for r in range(2)]).cuda()
        starts, ns = _ints([0, step[0]]), _ints(step)
        pos = _ints([at[0] + i for i in range(step[0])] + [at[1] + i for i in range(step[1])])
        out = torch.empty(sum(step), H * P, device="cuda")
        gate, b0 = rows[:, C : C + H * P], C + H * P
        if max(step) == 1:
            kernels.state_step(out, rows[:, : G * N], rows[:, G * N : 2 * G * N], rows[:, 2 * G * N : C], state, S0, starts, ns, slots, 2, H, G, N, P,
                               norm_w.cuda(), eps, gate=gate, beta=rows[:, b0 : b0 + H], log_g=rows[:, b0 + H :], raw=raw, positions=pos)
        else:
            ops = kernels.delta_prepare(_alloc, rows, b0, b0 + H, H, G, N, P, raw, state, _ints([0] * step[0] + [1] * step[1]), pos, starts, ns, slots)
            if max(step) >= 8:
                kernels.delta_chunks(out, ops, state, S0, _spans(step), starts, ns, slots, 2, H, G, N, P, norm_w.cuda(), eps, gate, _alloc)
            else:
                q, k, v, log_g, beta = ops
                kernels.state_step(out, q, k, v, state, S0, starts, ns, slots, 2, H, G, N, P, norm_w.cuda(), eps, gate=gate,
                                   qk_stride=q.shape[1] // G, v_stride=v.shape[1] // H, log_g=log_g, beta=beta)
        got[0].append(out[: step[0]].cpu()), got[1].append(out[step[0] :].cpu())
        at = [at[0] + step[0], at[1] + step[1]]
    for r in range(2):
        err = (torch.cat(got[r]).double() - want[r]).abs().amax(-1) / want[r].abs().max()
        assert err.max() <= 5e-5, (r, int(err.argmax()), float(err.max()))
    assert (state[[0, 2]] == 5.0).all() and (state[:, :S0] == 5.0).all()


@pytest.mark.parametrize("cuts", [[900], [899, 1], [892, 8], [63, 1, 64, 65, 700, 7], [448, 2, 449, 1]])
def test_a_key_far_back_in_the_delta_rules_state(cuts):
    """The key of token 3 lies along a column that no other key touches; the last of 900 queries lies
    along it too, so its output is token 3's value, decayed."""
    from mlx_lm_amd.ops import kernels

    n, N, P = 900, 16, 12
    g = torch.Generator().manual_seed(6)
    k, q, v = torch.randn(n, N, generator=g), torch.randn(n, N, generator=g), torch.randn(n, P, generator=g)
    k[:, 0] = 0.0
    k[3], q[n - 1] = 0.0, 0.0
    k[3, 0], q[n - 1, 0] = 1.0, 1.0
    k = torch.nn.functional.normalize(k, dim=-1)
    log_g, beta = torch.full((n, 1), -1e-4), torch.rand(n, 1, generator=g)
    beta[3] = 1.0
    eps = 1e-6
    o = plain.delta_recurrence(q.double(), k.double(), v.double(), log_g.double().exp()[:, 0], beta.double()[:, 0])
    assert torch.allclose(o[n - 1], v[3].double() * float(np.exp(-1e-4 * (n - 4))), atol=1e-6)
    want, ones = plain.unit_rms(o, eps), torch.ones(P).cuda()
    state, got, at = torch.zeros(1, N * P).cuda(), [], 0
    for m in cuts:
        part = [t[at : at + m].contiguous().cuda() for t in (q, k, torch.nn.functional.pad(v, (0, 4)), log_g, beta)]
        out = torch.empty(m, P, device="cuda")
        args = (_ints([0]), _ints([m]), _ints([0]), 1, 1, 1, N, P, ones, eps)
        if m >= 8:
            kernels.delta_chunks(out, part, state, 0, _spans([m]), *args, None, _alloc)
        else:
            kernels.state_step(out, *part[:3], state, 0, *args, v_stride=16, log_g=part[3], beta=part[4])
        got.append(out.cpu())
        at += m
    assert (torch.cat(got).double() - want).abs().max() <= 1e-4 * want.abs().max()


def test_keys_that_repeat_and_full_step_sizes():
    """A sequence that writes one key again and again with a step size near one (every write takes the
    last one's place), and one with no decay at all: the triangular systems at their worst."""
    from mlx_lm_amd.ops import kernels

    n, N, P = 200, 32, 16
    g = torch.Generator().manual_seed(9)
    base = torch.nn.functional.normalize(torch.randn(3, N, generator=g), dim=-1)
    k = base[torch.arange(n) % 3] + 0.01 * torch.randn(n, N, generator=g)
    k = torch.nn.functional.normalize(k, dim=-1)
    q, v = torch.randn(n, N, generator=g), torch.randn(n, P, generator=g)
    log_g, beta = torch.zeros(n, 1), torch.full((n, 1), 0.999)
    want = plain.unit_rms(plain.delta_recurrence(q.double(), k.double(), v.double(), torch.ones(n).double(), beta.double()[:, 0]), 1e-6)
    state, out = torch.zeros(1, N * P).cuda(), torch.empty(n, P, device="cuda")
    kernels.delta_chunks(out, [t.cuda() for t in (q, k, v, log_g, beta)], state, 0, _spans([n]), _ints([0]), _ints([n]), _ints([0]), 1, 1, 1, N, P,
                         torch.ones(P).cuda(), 1e-6, None, _alloc)
    assert (out.double().cpu() - want).abs().max() <= 1e-4 * want.abs().max()


@pytest.mark.parametrize("wide", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,N,rank", [(2, 64, 16), (3, 8, 1), (1, 20, 5), (2, 10, 70), (1, 128, 32), (4, 32, 8)])
def test_the_bonus_recurrence_in_portions_of_two_requests(H, N, rank, wide):
    """Single tokens and few tokens (decays made in the step's own kernel), and portions of many: chunks
    and spans with the decays as rows of their own.  Some channels forget within a token, some keep all."""
    from mlx_lm_amd.ops import kernels

    g = torch.Generator().manual_seed(N + rank)
    W, eps, S0 = H * N, 1e-4, 12
    lens = [(1, 1), (3, 1), (1, 1), (70, 2), (1, 129), (65, 7), (16, 17), (1, 1), (200, 15)]
    total = [sum(x[r] for x in lens) for r in range(2)]
    r_, k, v, gate = ([torch.randn(n, W, generator=g) for n in total] for _ in range(4))
    z = [torch.randn(n, rank, generator=g) for n in total]
    w2, w0 = (torch.randn(W, rank, generator=g) * rank ** -0.5).to(wide), torch.randn(W, generator=g) * 1.5 - 3.0
    w0[0], w0[W - 1] = 4.0, -14.0
    bonus, norm_w = torch.randn(W, generator=g), 1 + 0.3 * torch.randn(W, generator=g)
    want = []
    for i in range(2):
        decay = torch.exp(-torch.exp(torch.tanh(z[i].double()) @ w2.double().t() + w0.double()))
        heads = [plain.wkv_recurrence(*(t[i].double()[:, h * N : h * N + N] for t in (r_, k, v)), decay[:, h * N : h * N + N], bonus.double()[h * N : h * N + N])
                 for h in range(H)]
        want.append(plain.unit_rms(torch.stack(heads, 1), eps).flatten(1) * norm_w.double() * plain.silu(gate[i].double()))
    state = torch.full((3, S0 + H * N * N), 2.0).cuda()
    state[[2, 1], S0:] = 0.0
    decay = kernels.LowRankDecay(w2.t().contiguous().cuda(), w0.cuda())
    at, got = [0, 0], [[], []]
    for step in lens:
        rows = lambda xs: torch.cat([xs[i][at[i] : at[i] + step[i]] for i in range(2)]).cuda()  # noqa: E731, B023
        out = torch.empty(sum(step), W, device="cuda")
        common = (_ints([0, step[0]]), _ints(step), _ints([2, 1]), 2, H, H, N, N)
        if max(step) < 8:
            kernels.state_step(out, rows(r_), rows(k), rows(v), state, S0, *common, norm_w.cuda(), eps, gate=rows(gate), z=rows(z), decay=decay,
                               bonus=bonus.cuda())
        else:
            log_w = torch.empty(sum(step), W, device="cuda")
            kernels.lowrank_decay(log_w, rows(z), decay)
            spans = None
            if max(step) >= 128:
                n, req, lo, first = _spans(step)
                spans = (64, n, req, lo, first, _alloc)
            kernels.state_scan(out, rows(r_), rows(k), rows(v), state, S0, *common, channel_decay=log_w, bonus=bonus.cuda(), unit_rms=True, eps=eps,
                               norm_weight=norm_w.cuda(), gate=rows(gate), chunked=True, spans=spans)
        got[0].append(out[: step[0]].cpu()), got[1].append(out[step[0] :].cpu())
        at = [at[0] + step[0], at[1] + step[1]]
    for i in range(2):
        err = (torch.cat(got[i]).double() - want[i]).abs().amax(-1) / want[i].abs().max()
        assert err.max() <= 5e-5, (i, int(err.argmax()), float(err.max()))
    assert (state[0] == 2.0).all() and (state[:, :S0] == 2.0).all()


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("T", [3, 80, 300])
@pytest.mark.parametrize("F,top,W", [(24, 2, 48), (9, 1, 48), (64, 5, 48), (136, 3, 200)])
def test_clamped_experts_with_weights_over_the_chosen_alone(dtype, T, F, top, W):
    """A few tokens, and tiles of 32, 64 and 128 picks of an expert (one expert gets few picks)."""
    from mlx_lm_amd.ops import kernels

    g = torch.Generator().manual_seed(F + top)
    E, limit = 5, 0.6
    x = torch.randn(T, W, generator=g).to(dtype)
    gate, up, down = ((torch.randn(*s, generator=g) * s[-1] ** -0.5 * f).to(dtype) for s, f in (((E, F, W), 2.0), ((E, F, W), 2.0), ((E, W, F), 1.0)))
    z = torch.randn(T, E, generator=g) * 3
    z[:, 2] -= 4.0
    idx, weight = torch.empty(T, top, dtype=torch.int32, device="cuda"), torch.empty(T, top, device="cuda")
    kernels.router_choice(idx, weight, z.cuda(), None, top, renormalize=True)
    y = torch.full((T, W), 0.5, device="cuda")
    args = (y, x.cuda(), gate.cuda(), up.cuda(), down.cuda(), idx, weight, top)
    if T >= 64 and kernels.expert_tiles_takes(F, W, dtype):
        kernels.expert_tiles(*args, _alloc, activation="clamped", limit=limit)
    else:
        kernels.expert_rows(*args, torch.empty(T * top, F, dtype=dtype, device="cuda"), activation="clamped", limit=limit)
    w = {}
    for e in range(E):
        w[f"e{e}.gate"], w[f"e{e}.up"], w[f"e{e}.down"] = gate[e].double(), up[e].double(), down[e].double()
    want = torch.zeros(T, W).double()
    for t in range(T):
        chosen = torch.topk(z[t].double(), top).indices
        for e, s in zip(chosen.tolist(), torch.softmax(z[t].double()[chosen], 0)):
            want[t] += s * plain.expert(x[t].double(), w, f"e{e}.", limit)
    tol = 1e-5 if dtype == torch.float32 else 2e-2
    assert (y.double().cpu() - 0.5 - want).abs().max() <= tol * want.abs().max()


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("F,width,top,E", [(24, 48, 1, 5), (9, 44, 2, 70), (64, 96, 5, 5), (40, 24, 4, 130), (16, 8, 11, 12)])
def test_the_choice_and_the_next_norm_inside_the_experts_kernels(dtype, F, width, top, E):
    """The experts chosen by the kernel that reads them, and the next layer's norm left by the one that
    completes the rows, against the separate kernels: the same picks and weights, sums to rounding."""
    from mlx_lm_amd.ops import kernels

    g = torch.Generator().manual_seed(F + top)
    T = 7
    x = torch.randn(T, width, generator=g).to(dtype).cuda()
    gate, up, down = (torch.randn(*s, generator=g).to(dtype).cuda() * s[-1] ** -0.5 for s in ((E, F, width), (E, F, width), (E, width, F)))
    zs = torch.randn(T, E + 3, generator=g).cuda()
    z, correction = zs[:, :E], torch.randn(E, generator=g).cuda() * 0.1
    norm = tuple(t.cuda() for t in (torch.tensor([0.6]), torch.randn(width, generator=g), torch.randn(width, generator=g)))
    idx, weight = torch.empty(T, top, dtype=torch.int32, device="cuda"), torch.empty(T, top, device="cuda")
    kernels.router_choice(idx, weight, z, correction, top, renormalize=True, weight_scale=1.5)
    start = torch.randn(T, width, generator=g).cuda()
    act = torch.empty(T * top, F, dtype=dtype, device="cuda")
    y, y2, out = start.clone(), start.clone(), torch.empty(T, width, dtype=dtype, device="cuda")
    kernels.expert_rows(y, x, gate, up, down, idx, weight, top, act, activation="clamped", limit=0.8)
    idx2, weight2 = torch.full_like(idx, -1), torch.zeros_like(weight)
    kernels.expert_rows(y2, x, gate, up, down, idx2, weight2, top, act, activation="clamped", limit=0.8, route=(z, kernels.Route(correction, True, 1.5)),
                        after=(out, norm))
    assert torch.equal(idx, idx2) and torch.equal(weight, weight2) and torch.equal(y, y2)
    want = torch.empty_like(out)
    kernels.dynamic_tanh(want, y, norm)
    assert torch.equal(out, want)
    if kernels.expert_tiles_takes(F, width, dtype):
        y3 = start.clone()
        kernels.expert_tiles(y3, x, gate, up, down, idx, weight, top, _alloc, activation="clamped", limit=0.8, after=(out, norm))
        kernels.dynamic_tanh(want, y3, norm)
        assert torch.equal(out, want)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("T", [1, 5, 16, 17, 33, 64, 65, 200])
def test_products_that_read_planes_of_their_own(dtype, T):
    """Matrices of widths that are no multiples of a block, each over an input of its own, for one
    token and for hundreds."""
    from mlx_lm_amd.ops import kernels

    g = torch.Generator().manual_seed(T)
    K, widths, planes = 104, [70, 32, 5, 96, 33], [2, 0, 1, 2, 3]
    ws = [(torch.randn(n, K, generator=g) * K ** -0.5).to(dtype) for n in widths]
    x = torch.randn(4, T, K, generator=g).to(dtype)
    w = kernels.GroupedWeight([(m.cuda(), p) for m, p in zip(ws, planes)])
    out = kernels.linear_groups(_alloc, x.cuda(), w)
    for o, m, p in zip(out, ws, planes):
        want = x[p].double() @ m.double().t()
        assert o.shape == want.shape and o.dtype == torch.float32
        assert (o.double().cpu() - want).abs().max() <= 2e-5 * want.abs().max()


# -- each mixer alone, in a model of one layer ----------------------------------------------


ALONE = {
    "delta": [_delta(4, 2, 16, 24, 4)],
    "delta, one tap": [_delta(2, 2, 24, 8, 1)],
    "delta, odd sizes": [_delta(3, 1, 7, 9, 3)],
    "delta with experts": [_moe(_delta(2, 1, 16, 16, 2), 20, 4, 2)],
    "wkv": [_wkv(3, 16)],
    "wkv, odd sizes": [_wkv(2, 7)],
    "wkv with experts": [_moe(_wkv(2, 24), 12, 9, 3, 1.0)],
    "latent": [_latent(3, 16, 8, 24, 20, 40, 30, base=300.0)],
    "latent, eight heads, a window of a page": [_latent(8, 16, 8, 24, 20, 56, 16, base=300.0)],
    "latent and readers": [_latent(2, 8, 6, 12, 10, 18, 9, base=20.0, scale=0.9), _latent(4, 12, 6, 8, 14, 18, 40, base=20.0, kv_from=0),
                           _latent(1, 12, 6, 8, 14, 18, 2, base=20.0, kv_from=0)],
    "latent wider than a fast head": [_latent(2, 16, 32, 24, 20, 250, 50, base=300.0)],
}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(ALONE))
def test_a_mixer_alone(tmp_path, name, dtype):
    """Whole, the last tokens one by one, in portions of changing size and of two tokens; portions
    shorter than the convolution's taps among them."""
    config = _config(48, 61, copy.deepcopy(ALONE[name]))
    weights = plain.random_weights(config, 7, sharp=2.0, decay_rank=5)
    folder = _folder(str(tmp_path / "m"), config, weights)
    n = 100
    tokens = helpers.random_tokens(n, 61, seed=len(name))
    want = _plain(weights, config, tokens, dtype)
    strict = "experts" not in name
    eng = _engine(folder, dtype, n_pages=8)
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


def test_portions_give_what_the_whole_prompt_gives(models):
    """However a prompt is cut (at a page's, a window's or a chunk's border, one token before and after
    it, token by token), the logits agree with the uncut prompt's to rounding: the engine against itself."""
    folder, config, _ = models["A", "float32"]
    tokens = helpers.random_tokens(150, config["vocab"], seed=8)
    eng = _engine(folder, "float32", n_pages=12)
    whole = _run(eng, "w", tokens, [150])
    for cuts in (helpers.cuts_changing(150), [1] * 150, [16, 16, 1, 15, 17, 15, 2, 68], [15, 2, 3, 17, 27, 64, 22], [64, 64, 22], [63, 2, 63, 22], [147, 3]):
        got = _run(eng, "c", tokens, cuts)
        assert (got - whole).abs().max().item() <= 2e-5 * whole.abs().max().item(), cuts[:6]


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_first_tokens_and_long_decode(models, dtype):
    """Every token one by one from the first: 400 of them, recorded decode steps replayed, page after
    page taken and given back behind the windows, the states carried 400 times."""
    folder, config, weights = models["C", dtype]
    n = 400
    tokens = helpers.random_tokens(n, config["vocab"], seed=77)
    want = _plain(weights, config, tokens, dtype)
    eng = _engine(folder, dtype, n_pages=8)  # (the longest window is 70: far fewer pages than tokens)
    got = _run(eng, "r", tokens, [1] * n)
    _close(got[:8], want[:8], dtype, "first tokens")
    _close(got, want, dtype, "decoding every token")


def _marked(config, p, w):
    """Weights under which the latent attention of layer ``p`` reads marked tokens only: column 0 of the
    embedding marks the ids below 4 (keys), column 1 the ids 4 to 7 (queries)."""
    m = config["layers"][int(p[1:-5])]["mixer"]
    w["embed"][:8] *= 0.05
    w["embed"][:, :2] = 0.0
    w["embed"][:4, 0], w["embed"][4:8, 1] = 6.0, 6.0
    for name in ("embed.norm", "l0.norm1"):
        w[name][:2], w[name + ".b"][:2] = 2.0, 0.0
    if p + "dkv" in w:
        w[p + "dkv"][:, :2] = 0.0
        w[p + "dkv"][0, 0] = 6.0
    w[p + "dq"][:, :2] = 0.0
    w[p + "dq"][0, 1] = 6.0
    w[p + "uq"][:, 0], w[p + "uk"][:, 0] = 0.0, 0.0
    w[p + "uq"][0 :: m["dim"] + m["rot_dim"], 0], w[p + "uk"][0 :: m["dim"], 0] = 6.0, 6.0


@pytest.mark.parametrize("page_size", [16, 64])
@pytest.mark.parametrize("window", [33, 48, 129])
def test_a_key_just_inside_and_just_outside_a_window(tmp_path, window, page_size):
    """A marked key stands out for a marked query exactly ``window - 1`` and ``window`` tokens later: the
    first reads it, the second does not; in a prompt, at a portion's end, and decoded alone."""
    config = _config(32, 40, [_latent(2, 16, 4, 16, 12, 24, window, scale=1.0)])
    w = plain.random_weights(config, 11)
    _marked(config, "l0.mix.", w)
    folder = _folder(str(tmp_path / "m"), config, w)
    eng = _engine(folder, "float32", n_pages=512 // page_size, page_size=page_size)
    for gap, inside in ((window - 1, True), (window, False)):
        key = 21
        n = key + gap + 1
        tokens = [8 + t for t in helpers.random_tokens(n, 32, seed=window)]
        tokens[key], tokens[n - 1] = 2, 5
        want = plain.model(w, config, tokens)
        other = list(tokens)
        other[key] = 20
        moved = ((plain.model(w, config, other)[n - 1] - want[n - 1]).abs().max() / want.abs().max()).item()
        assert moved > 0.02 if inside else moved == 0.0, (gap, moved)
        for cuts in ([n], [n - 1, 1], [n - 6, 6], [key + 1, n - key - 2, 1], [n - 3, 1, 1, 1]):
            got = _run(eng, "r", tokens, cuts)
            _close(got[n - 1 :], want[n - 1 :], "float32", f"gap {gap}: the last of {cuts}")
            _close(got, want, "float32", f"gap {gap}: {cuts}")


@pytest.mark.parametrize("own,reader", [(8, 90), (90, 8), (8, 0)])
def test_a_reader_keeps_what_its_own_window_needs(tmp_path, own, reader):
    """A layer reads another's latents with a longer window (or none) than the layer that made them, or
    with a shorter one: the pages last for the longer, each layer sees its own.  Little but the needed pages is there."""
    config = _config(32, 40, [_latent(2, 16, 4, 16, 12, 24, own, scale=1.0), _latent(2, 16, 4, 16, 12, 24, reader, kv_from=0, scale=1.0)])
    w = plain.random_weights(config, 13, sharp=2.0)
    _marked(config, "l0.mix.", w)
    folder = _folder(str(tmp_path / "m"), config, w)
    n = 180
    tokens = [8 + t for t in helpers.random_tokens(n, 32, seed=3)]
    want = plain.model(w, config, tokens)
    eng = _engine(folder, "float32", n_pages=12)
    for cuts in ([n], [100] + [1] * 80, helpers.cuts_changing(n)):
        _close(_run(eng, "r", tokens, cuts), want, "float32", f"windows {own} and {reader}: {cuts[:5]}")
        eng.cache.poison_free_pages()


# -- batches -------------------------------------------------------------------------------


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["A", "B", "C"])
def test_mixed_batches_equal_each_request_alone(models, dtype, name):
    """Up to four live requests of unequal lengths, portions beside single tokens, requests that sit a
    step out; state rows (the matrices, the convolutions' inputs, the last normed rows) and pages of
    finished requests are used again by later ones, and what freed pages hold is never read."""
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

    layers, latents = [], []
    for i in range(pick([1, 2, 3, 4, 5])):
        kind = pick(["delta", "wkv", "latent"])
        if kind == "delta":
            kv = pick([1, 2, 3])
            entry = _delta(kv * pick([1, 2, 4]), kv, pick([8, 12, 16, 32, 40, 64]), pick([8, 16, 24, 48, 80, 128]), pick([1, 2, 3, 4, 5]))
        elif kind == "wkv":
            entry = _wkv(pick([1, 2, 4]), pick([8, 12, 16, 32, 48, 64]))
        else:
            reads = pick(latents + [None]) if latents else None
            window = pick([1, 2, 16, 17, 40, 64, 0])
            if reads is not None:
                src = layers[reads]["mixer"]
                entry = _latent(pick([1, 2, 8]), pick([8, 16, 24]), src["rot_dim"], pick([8, 16, 40]), pick([8, 12, 32]), src["kv_rank"], window,
                                base=src["rot"]["base"], kv_from=reads, scale=pick([None, 0.3]))
            else:
                entry = _latent(pick([1, 2, 8]), pick([8, 16, 24]), pick([2, 4, 8, 16]), pick([8, 16, 40]), pick([8, 12, 32]),
                                pick([8, 20, 48, 64, 120]), window, base=pick([10.0, 1e4, 1e6]), scale=pick([None, 0.3]))
                latents.append(i)
        if pick([0, 1, 1]):
            experts = pick([1, 3, 8, 20])
            entry = _moe(entry, pick([4, 8, 20, 64]), experts, min(experts, pick([1, 2, 4])), pick([0.5, 2.0, 7.0]))
        layers.append(entry)
    return _config(pick([16, 40, 64, 104, 256]), pick([17, 100, 257, 1000]), layers, eps=pick([1e-6, 1e-5, 1e-2]), logit_scale=pick([0.125, 1.0, 2.5]))


@pytest.mark.parametrize("seed", range(12))
def test_drawn_configurations(tmp_path, seed):
    """Every size, the layers' order and constants drawn: whole, in portions, and two requests side by
    side, in float32."""
    from mlx_lm_amd.engine import StepEntry

    config = _drawn_config(seed)
    weights = plain.random_weights(config, 100 + seed, sharp=2.0, decay_rank=1 + seed % 7)
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
