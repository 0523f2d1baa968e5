"""Gilidra without a GPU: the registry, the plan run by run, refusals, sizes read from a checkpoint's
shapes, and properties of the plain implementation (plain_gilidra.py) that the GPU tests lean on."""

import copy

import pytest
import torch

import plain_gilidra as plain
from mlx_lm_amd.config import CacheNeed, StateNeed, get_model_classes


def _delta(heads, kv_heads, dim, vdim, conv):
    return {"type": "delta", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}}


def _wkv(heads, dim):
    return {"type": "wkv", "mixer": {"heads": heads, "dim": dim}}


def _latent(heads, dim, rot_dim, vdim, q_rank, kv_rank, window, base=10000.0, kv_from=None, scale=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank,
         "scale": scale or (dim + rot_dim) ** -0.5, "rot": {"dims": rot_dim, "base": base}}
    if window:
        m["mask"] = {"size": window}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m}


def _moe(entry, ff, experts, top, limit=2.0):
    return dict(entry, mlp={"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": {"experts": experts, "top": top}})


def _config(width, vocab, layers, eps=1e-5, logit_scale=0.7):
    for entry in layers:
        entry.setdefault("mlp", None)
    return {"architecture": "Gilidra", "vocab": vocab, "width": width, "norm": {"eps": eps}, "logit_scale": logit_scale, "layers": layers}


SMALL = _config(64, 130, [
    _moe(_latent(3, 16, 8, 24, 20, 40, 20, base=300.0), 24, 5, 2, 1.2),
    _moe(_delta(6, 3, 16, 24, 4), 40, 7, 3),
    _wkv(3, 24),
    _moe(_latent(2, 8, 8, 16, 12, 40, 37, base=300.0, kv_from=0), 16, 3, 1, 0.8),
    _delta(2, 2, 8, 12, 3),
    _moe(_wkv(2, 12), 20, 4, 4)])


def _args(config, w=None):
    Model, Args = get_model_classes(config)
    w = w if w is not None else plain.random_weights(config, 0)
    return Model, Args.from_dict(Args.sizes_from_tensors(config, {k: tuple(v.shape) for k, v in w.items()}))


def test_the_registry_finds_the_design_by_its_architecture_key():
    Model, _ = get_model_classes(SMALL)
    assert Model.__module__.endswith("models.gilidra")
    with pytest.raises(ValueError):
        get_model_classes({"architecture": "Gilidro"})


def test_the_plan_run_by_run():
    Model, args = _args(SMALL)
    model = Model(args)
    # the fourth layer reads the first one's pages, which are kept for the longer of the two windows
    assert [(r.layer, r.cache, r.writes_cache, r.state) for r in model.decoder.schedule] == [
        (0, 0, True, None), (1, 1, True, None), (2, 2, True, None), (3, 0, False, None), (4, 3, True, None), (5, 4, True, None)]
    needs = model.decoder.cache_needs()
    assert needs[0] == CacheNeed(1, 64, 37)
    assert needs[1] == StateNeed((6 * 16 * 24 + 4 * (2 * 3 * 16 + 6 * 24),), "float32")
    assert needs[2] == StateNeed((3 * 24 * 24 + 64,), "float32")
    assert needs[3] == StateNeed((2 * 8 * 12 + 3 * (2 * 2 * 8 + 2 * 12),), "float32")
    assert model.decoder.layers[0].mixer.window == 20 and model.decoder.layers[3].mixer.window == 37
    names = model.decoder.expected_tensors()
    assert "l3.mix.dkv" not in names and "l0.mix.dkv" in names and "l0.mix.g" not in names and "l2.mlp.router" not in names
    assert names["embed.norm.alpha"].shape == () and names["l1.mix.v.conv"].shape == (144, 4)


def test_one_reader_without_a_window_keeps_every_page():
    config = copy.deepcopy(SMALL)
    del config["layers"][3]["mixer"]["mask"]
    Model, args = _args(config)
    assert Model(args).decoder.cache_needs()[0] == CacheNeed(1, 64, 0)
    config["layers"][0]["mixer"].pop("mask")
    config["layers"][3]["mixer"]["mask"] = {"size": 9}
    Model, args = _args(config)
    assert Model(args).decoder.cache_needs()[0] == CacheNeed(1, 64, 0)


def test_the_plains_weights_carry_the_names_the_model_expects():
    w = plain.random_weights(SMALL, 0, decay_rank=4)
    Model, args = _args(SMALL, w)
    assert args.layers[2]["mixer"]["decay_rank"] == 4
    names = Model(args).decoder.expected_tensors()
    assert set(names) == set(w) and all(tuple(names[k].shape) == tuple(w[k].shape) for k in w)
    random = Model.random_weights(args, 1, "b")
    assert {k: tuple(v.shape) for k, v in random.items()} == {k: tuple(v.shape) for k, v in w.items()}


def test_an_alpha_stored_as_a_vector_of_one_is_taken():
    w = plain.random_weights(SMALL, 0)
    Model, args = _args(SMALL, w)
    w["final.norm.alpha"] = w["final.norm.alpha"].reshape(1)
    assert Model(args).sanitize(w)["final.norm.alpha"].shape == ()


def test_what_cannot_run_is_refused():
    _, Args = get_model_classes(SMALL)
    for change in (lambda c: c["layers"][0].update(type="window"), lambda c: c["layers"][0]["mlp"].update(kind="dense"),
                   lambda c: c["layers"][3]["mixer"].update(kv_from=1), lambda c: c["layers"][3]["mixer"].update(kv_from=3),
                   lambda c: c["layers"][3]["mixer"].update(kv_rank=48), lambda c: c.pop("norm"),
                   lambda c: c["layers"][0]["mixer"]["rot"].update(dims=4), lambda c: c["layers"][0]["mixer"].update(mask={"size": 0})):
        c = copy.deepcopy(SMALL)
        change(c)
        with pytest.raises(ValueError):
            Args.from_dict(c)


def test_a_feed_forwards_router_rides_in_the_mixers_product():
    Model, args = _args(SMALL)
    layers = Model(args).decoder.layers
    for i in (0, 1, 3, 5):
        assert layers[i].mixer.more_names == (f"l{i}.mlp.router",) and layers[i].ffn.projection_given
    assert layers[2].mixer.more_names == () and layers[4].mixer.more_names == ()


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
    assert moved(lambda c, ww: c["layers"][0]["mixer"]["mask"].update(size=21)) > 1e-3
    assert moved(lambda c, ww: c["layers"][3]["mixer"]["mask"].update(size=36)) > 1e-3
    assert moved(lambda c, ww: c["layers"][0]["mixer"]["rot"].update(base=310.0)) > 1e-4
    assert moved(lambda c, ww: c["layers"][1]["mlp"]["router"].update(top=2)) > 1e-3
    assert moved(lambda c, ww: c["layers"][0]["mlp"]["expert"].update(limit=1.25)) > 1e-4
    assert moved(with_tensor("l1.mix.dt_bias", lambda t: t + 0.05)) > 1e-4
    assert moved(with_tensor("l1.mix.A_log", lambda t: t + 0.05)) > 1e-4
    assert moved(with_tensor("l1.mix.k.conv", lambda t: t.flip(1))) > 1e-2
    assert moved(with_tensor("l2.mix.u", lambda t: t.flip(0))) > 1e-3
    assert moved(with_tensor("l2.mix.w0", lambda t: t + 0.05)) > 1e-4
    assert moved(with_tensor("l2.mix.mu.w", lambda t: 0 * t)) > 1e-4
    assert moved(with_tensor("l5.mix.norm", lambda t: t.flip(0))) > 1e-3
    assert moved(with_tensor("embed.norm.alpha", lambda t: t * 1.01)) > 1e-4


def test_the_recurrences_against_sums_written_out():
    g = torch.Generator().manual_seed(0)
    T, N, P = 7, 4, 3
    q, k, v = (torch.randn(T, n, generator=g).double() for n in (N, N, P))
    k = plain.unit_length(k)
    decay, beta = torch.rand(T, generator=g).double(), torch.rand(T, generator=g).double()
    # the delta rule as a product of transitions: S_t = sum_j (prod_(j < s <= t) g_s (1 - beta_s k_s k_s^T)) beta_j k_j v_j^T
    want = []
    for t in range(T):
        S = torch.zeros(N, P).double()
        for j in range(t + 1):
            piece = beta[j] * torch.outer(k[j], v[j])
            for s in range(j + 1, t + 1):
                piece = decay[s] * (piece - beta[s] * torch.outer(k[s], k[s] @ piece))
            S += piece
        want.append(S.t() @ q[t])
    assert torch.allclose(plain.delta_recurrence(q, k, v, decay, beta), torch.stack(want), atol=1e-12)
    # a bonus for the current token: o_t = sum_(j < t) (r_t * prod_(j < s < t) w_s) . k_j v_j + (r_t * u) . k_t v_t
    w, u = torch.rand(T, N, generator=g).double(), torch.randn(N, generator=g).double()
    want = torch.stack([sum(((q[t] * w[j + 1 : t].prod(0)) @ k[j]) * v[j] for j in range(t)) + ((q[t] * u) @ k[t]) * v[t] for t in range(T)])
    assert torch.allclose(plain.wkv_recurrence(q, k, v, w, u), want, atol=1e-12)


def test_a_window_of_n_sees_itself_and_the_n_minus_one_before():
    g = torch.Generator().manual_seed(4)
    q, k, v = (torch.randn(9, 5, generator=g).double() for _ in range(3))
    got = plain.windowed_softmax_attention(q, k, v, 0.4, 3)
    for t in range(9):
        lo = max(0, t - 2)
        want = torch.softmax((k[lo : t + 1] @ q[t]) * 0.4, 0) @ v[lo : t + 1]
        assert torch.allclose(got[t], want)
