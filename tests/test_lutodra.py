"""Lutodra without a GPU: the registry, the plan run by run, refusals, sizes read from a checkpoint's
shapes, the frequency table, and properties of the plain implementation (plain_lutodra.py) that the GPU
tests lean on."""

import copy
import math

import pytest
import torch

import plain_lutodra as plain
from mlx_lm_amd.config import CacheNeed, StateNeed, get_model_classes
from mlx_lm_amd.parts.rotary import rotary_table


def _delta(heads, kv_heads, dim, vdim, conv):
    return {"type": "channel_delta", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}}


def _lru(width, blocks, conv):
    return {"type": "rglru", "mixer": {"width": width, "blocks": blocks, "conv": conv}}


def _attention(heads, kv_heads, dim, vdim, rot, base=10000.0, scaling=None, scale=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale or dim ** -0.5}
    if rot:
        m["rot"] = {"dims": rot, "base": base}
        if scaling:
            m["rot"]["scaling"] = dict(zip(("factor", "low", "high", "original"), scaling))
    return {"type": "attention", "mixer": m}


def _dense(entry, ff):
    return dict(entry, mlp={"kind": "dense", "ff": ff})


def _moe(entry, ff, experts, top, groups=(1, 1), scale=1.0):
    router = {"experts": experts, "top": top, "scale": scale, "groups": {"count": groups[0], "keep": groups[1]}}
    return dict(entry, mlp={"kind": "moe", "expert": {"ff": ff}, "router": router})


def _config(width, vocab, layers, streams=2, loop=None, eps=1e-5, logit_scale=0.7):
    for entry in layers:
        entry.setdefault("mlp", None)
    c = {"architecture": "Lutodra", "vocab": vocab, "width": width, "streams": streams, "norm": {"eps": eps}, "logit_scale": logit_scale, "layers": layers}
    if loop:
        c["loop"] = dict(zip(("start", "stop", "times"), loop))
    return c


SMALL = _config(64, 130, [
    _dense(_attention(6, 2, 24, 16, 12, 300.0, (3.0, 0.5, 6.0, 50)), 40),
    _moe(_delta(6, 3, 16, 24, 4), 24, 8, 3, (4, 2), 1.5),
    _lru(60, 3, 5),
    _moe(_attention(4, 4, 16, 32, 16, 1e4), 16, 6, 2, (2, 1), 0.8),
    _dense(_lru(32, 4, 2), 20),
    _moe(_delta(2, 2, 8, 12, 3), 20, 9, 4, (3, 2))], streams=4, loop=(1, 4, 2))


def _args(config, w=None):
    Model, Args = get_model_classes(config)
    w = w if w is not None else plain.random_weights(config, 0)
    return Model, Args.from_dict(Args.sizes_from_tensors(config, {k: tuple(v.shape) for k, v in w.items()}))


def test_the_registry_finds_the_design_by_its_architecture_key():
    Model, _ = get_model_classes(SMALL)
    assert Model.__module__.endswith("models.lutodra")
    with pytest.raises(ValueError):
        get_model_classes({"architecture": "Lutodro"})


def test_the_plan_run_by_run():
    """Layers 1 to 3 run twice, every run with a cache or state of its own."""
    Model, args = _args(SMALL)
    decoder = Model(args).decoder
    order = [0, 1, 2, 3, 1, 2, 3, 4, 5]
    assert [(r.layer, r.cache, r.writes_cache, r.state) for r in decoder.schedule] == [(i, s, True, None) for s, i in enumerate(order)]
    assert plain.run_order(SMALL) == order and all(b.n_runs == 9 for b in decoder.layers)
    needs = decoder.cache_needs()
    assert needs[0] == CacheNeed(2, 32, 0) and needs[3] == needs[6] == CacheNeed(4, 32, 0)
    assert needs[1] == needs[4] == StateNeed((6 * 16 * 24 + 4 * (2 * 3 * 16 + 6 * 24),), "float32")
    assert needs[2] == StateNeed((60 + 5 * 60,), "float32")
    assert needs[8] == StateNeed((2 * 8 * 12 + 3 * (2 * 2 * 8 + 2 * 12),), "float32")
    names = decoder.expected_tensors()
    assert "l2.norm2" not in names and "l2.hc2.in" not in names and "l2.hc1.mix" in names and names["l1.hc2.mix"].shape == (4, 4)


def test_without_a_loop_or_with_one_pass_the_layers_run_once():
    for loop in (None, (0, 6, 1), (2, 3, 1)):
        config = copy.deepcopy(SMALL)
        config.pop("loop")
        if loop:
            config["loop"] = dict(zip(("start", "stop", "times"), loop))
        _, args = _args(config)
        assert args.run_order() == list(range(6)) == plain.run_order(config)


def test_one_tap_keeps_no_inputs():
    Model, args = _args(_config(32, 20, [_delta(2, 1, 8, 8, 1), _lru(24, 2, 1)]))
    assert Model(args).decoder.cache_needs() == [StateNeed((2 * 8 * 8,), "float32"), StateNeed((24,), "float32")]


def test_the_plains_weights_carry_the_names_the_model_expects():
    w = plain.random_weights(SMALL, 0, rank=4)
    Model, args = _args(SMALL, w)
    assert args.layers[1]["mixer"]["decay_rank"] == 4 and args.layers[1]["mixer"]["gate_rank"] == 5
    names = Model(args).decoder.expected_tensors()
    assert set(names) == set(w) and all(tuple(names[k].shape) == tuple(w[k].shape) for k in w)
    random = Model.random_weights(args, 1, "b")
    assert {k: tuple(v.shape) for k, v in random.items()} == {k: tuple(v.shape) for k, v in w.items()}


def test_taps_come_from_the_tensors_where_the_configuration_has_none():
    config = copy.deepcopy(SMALL)
    w = plain.random_weights(config, 0)
    for entry in config["layers"]:
        entry["mixer"].pop("conv", None)
    Model, args = _args(config, w)
    layers = Model(args).decoder.layers
    assert layers[1].mixer.taps == 4 and layers[2].mixer.taps == 5


def test_a_sublayer_that_is_not_there_may_leave_its_norm_and_connections():
    w = plain.random_weights(SMALL, 0)
    Model, args = _args(SMALL, w)
    extra = {"l2.norm2": w["l1.norm2"], "l2.norm2.b": w["l1.norm2.b"], "l2.hc2.in": w["l1.hc2.in"]}
    assert set(Model(args).sanitize({**w, **extra})) == set(w)


def test_what_cannot_run_is_refused():
    Model, Args = get_model_classes(SMALL)
    for change in (lambda c: c["layers"][0].update(type="window"), lambda c: c["layers"][0]["mlp"].update(kind="wide"),
                   lambda c: c.update(streams=0), lambda c: c.update(streams=9), lambda c: c.pop("norm"),
                   lambda c: c["loop"].update(stop=7), lambda c: c["loop"].update(start=4), lambda c: c["loop"].update(times=0),
                   lambda c: c["layers"][1]["mlp"]["router"]["groups"].update(count=3), lambda c: c["layers"][1]["mlp"]["router"].update(top=5),
                   lambda c: c["layers"][2]["mixer"].update(blocks=7), lambda c: c["layers"][0]["mixer"]["rot"].update(dims=26),
                   lambda c: c["layers"][0]["mixer"].update(kv_heads=4)):
        c = copy.deepcopy(SMALL)
        change(c)
        with pytest.raises(ValueError):
            Model(Args.from_dict(c))


def test_the_frequency_table_against_its_definition():
    """Pairs within, between and beyond the two wavelengths; no scaling at all; both limits the same."""
    for base, dims, scaling in ((500.0, 16, (4.0, 1.0, 4.0, 300)), (1e4, 32, (8.0, 0.5, 2.0, 64)), (50.0, 6, None), (100.0, 8, (2.0, 3.0, 3.0, 40))):
        rot = {"dims": dims, "base": base}
        if scaling:
            rot["scaling"] = dict(zip(("factor", "low", "high", "original"), scaling))
        table, mult = rotary_table(dims, base, rot.get("scaling"))
        want = plain.rotary_frequencies(rot) if not scaling or scaling[1] != scaling[2] else [
            f if 2 * math.pi / f <= scaling[3] / scaling[2] else f / scaling[0] for f in (base ** (-2.0 * i / dims) for i in range(dims // 2))]
        assert mult == 1.0 and torch.allclose(table.double(), torch.tensor(want, dtype=torch.float64), rtol=1e-6)
    kinds = {f / (500.0 ** (-2.0 * i / 16)) for i, f in enumerate(plain.rotary_frequencies(
        {"dims": 16, "base": 500.0, "scaling": {"factor": 4.0, "low": 1.0, "high": 4.0, "original": 300}}))}
    assert 1.0 in kinds and min(kinds) == pytest.approx(0.25) and any(0.26 < k < 0.99 for k in kinds)


def test_the_plain_side_is_causal_and_leans_on_every_mechanism():
    w = {k: v.double() for k, v in plain.random_weights(SMALL, 3, sharp=2.0).items()}
    tokens = torch.randint(0, 130, (60,), generator=torch.Generator().manual_seed(1)).tolist()
    base = plain.forward(SMALL, w, tokens)
    other = plain.forward(SMALL, w, tokens[:25] + [(t + 1) % 130 for t in tokens[25:]])
    assert torch.equal(base[:25], other[:25]) and (base[25:] - other[25:]).abs().max() > 0.1
    scale = base.abs().max()

    def moved(change):
        c, ww = copy.deepcopy(SMALL), dict(w)
        change(c, ww)
        return ((plain.forward(c, ww, tokens) - base).abs().max() / scale).item()

    def with_tensor(name, f):
        return lambda c, ww: ww.update({name: f(ww[name])})

    # each of these is a fault that an engine could have; all move the logits by far more than a tolerance of 5e-5
    assert moved(lambda c, ww: c["loop"].update(times=1)) > 1e-2
    assert moved(lambda c, ww: c["layers"][0]["mixer"]["rot"].update(base=310.0)) > 1e-4
    assert moved(lambda c, ww: c["layers"][0]["mixer"]["rot"]["scaling"].update(factor=3.2)) > 1e-4
    assert moved(lambda c, ww: c["layers"][0]["mixer"]["rot"]["scaling"].update(low=0.6)) > 1e-5
    assert moved(lambda c, ww: c["layers"][1]["mlp"]["router"].update(top=2)) > 1e-3
    assert moved(lambda c, ww: c["layers"][1]["mlp"]["router"]["groups"].update(keep=3)) > 1e-3
    assert moved(lambda c, ww: c["layers"][1]["mlp"]["router"].update(scale=1.45)) > 1e-4
    for i, hc in ((1, "hc1"), (1, "hc2"), (4, "hc2")):
        assert moved(with_tensor(f"l{i}.{hc}.mix", lambda t: t.t())) > 1e-3
        assert moved(with_tensor(f"l{i}.{hc}.in", lambda t: t.flip(0))) > 1e-3
        assert moved(with_tensor(f"l{i}.{hc}.out", lambda t: t.flip(0))) > 1e-4
    assert moved(with_tensor("l0.mix.sink", lambda t: t - 50.0)) > 1e-3
    assert moved(with_tensor("l0.mix.sink", lambda t: t.flip(0))) > 1e-3
    assert moved(with_tensor("l0.mix.g", lambda t: 0 * t)) > 1e-3
    assert moved(with_tensor("l0.mix.q.norm", lambda t: t.flip(0))) > 1e-3
    assert moved(with_tensor("l1.mix.dt_bias", lambda t: t + 0.05)) > 1e-4
    assert moved(with_tensor("l1.mix.dt_bias", lambda t: t.view(6, 16).mean(1, keepdim=True).expand(6, 16).reshape(-1))) > 1e-3
    assert moved(with_tensor("l1.mix.A_log", lambda t: t + 0.05)) > 1e-4
    assert moved(with_tensor("l1.mix.k.conv", lambda t: t.flip(1))) > 1e-2
    assert moved(with_tensor("l1.mix.g2", lambda t: 0 * t)) > 1e-3
    assert moved(with_tensor("l2.mix.lam", lambda t: t + 0.1)) > 1e-4
    assert moved(with_tensor("l2.mix.conv", lambda t: t.flip(1))) > 1e-2
    assert moved(with_tensor("l2.mix.conv.b", lambda t: 0 * t)) > 1e-3
    assert moved(with_tensor("l2.mix.x.b", lambda t: 0 * t)) > 1e-3
    assert moved(with_tensor("l2.mix.ra", lambda t: t.transpose(1, 2))) > 1e-4
    assert moved(with_tensor("l2.mix.ri", lambda t: t.flip(0))) > 1e-3
    assert moved(with_tensor("final.norm.b", lambda t: 0 * t)) > 1e-3


def test_the_recurrences_against_sums_written_out():
    g = torch.Generator().manual_seed(0)
    T, N, P = 7, 4, 3
    q, k, v = (torch.randn(T, n, generator=g).double() for n in (N, N, P))
    k = plain.unit_length(k)
    decay, beta = torch.rand(T, N, generator=g).double(), torch.rand(T, generator=g).double()
    # the delta rule as a product of transitions (1 - beta_s k_s k_s^T) diag(g_s) on every write beta_j k_j v_j^T
    want = []
    for t in range(T):
        S = torch.zeros(N, P).double()
        for j in range(t + 1):
            piece = beta[j] * torch.outer(k[j], v[j])
            for s in range(j + 1, t + 1):
                piece = decay[s][:, None] * piece
                piece = piece - beta[s] * torch.outer(k[s], k[s] @ piece)
            S += piece
        want.append(S.t() @ q[t])
    assert torch.allclose(plain.delta_recurrence(q, k, v, decay, beta), torch.stack(want), atol=1e-12)
    # the unit: S_t = sum_j (prod_(j < s <= t) a_s) sqrt(1 - a_j^2) i_j u_j
    u, r, i = (torch.rand(T, N, generator=g).double() for _ in range(3))
    lam = torch.randn(N, generator=g).double()
    a = torch.exp(-8.0 * r * torch.log1p(torch.exp(lam)))
    want = torch.stack([sum(a[j + 1 : t + 1].prod(0) * torch.sqrt(1 - a[j] ** 2) * i[j] * u[j] for j in range(t + 1)) for t in range(T)])
    assert torch.allclose(plain.lru_recurrence(u, r, i, lam), want, atol=1e-12)


def test_a_sink_takes_its_share_and_counts_once():
    g = torch.Generator().manual_seed(4)
    q, k, v = (torch.randn(6, 5, generator=g).double() for _ in range(3))
    got = plain.sink_attention(q, k, v, 0.4, torch.tensor(0.3).double())
    for t in range(6):
        e = torch.exp((k[: t + 1] @ q[t]) * 0.4)
        assert torch.allclose(got[t], (e[:, None] * v[: t + 1]).sum(0) / (e.sum() + math.exp(0.3)))


def test_experts_outside_the_best_groups_are_never_chosen():
    """The largest score of all may stand in a group that two middling ones beat."""
    router = {"experts": 8, "top": 3, "scale": 2.0, "groups": {"count": 4, "keep": 2}}
    z = torch.tensor([9.0, -9.0, 2.0, 2.1, 1.0, 1.1, 1.9, 2.2]).double()
    chosen, weights = plain.choose(z, router)
    assert chosen.tolist() == [7, 3, 2] and abs(weights.sum().item() - 2.0) < 1e-9
    chosen, _ = plain.choose(z, dict(router, groups={"count": 1, "keep": 1}))
    assert chosen.tolist() == [0, 7, 3]
    chosen, _ = plain.choose(z, dict(router, groups={"count": 8, "keep": 3}))
    assert chosen.tolist() == [0, 7, 3]
