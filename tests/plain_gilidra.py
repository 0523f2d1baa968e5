"""Gilidra, plainly: one function per mechanism, whole sequences, float64, no cache.

Written from the design's equations only; nothing here is shared with the engine.  ``config`` is
the config.json as a dict, ``w`` maps tensor names to float64 tensors, tokens are a list of ints.

    D(x; n)  = tanh(n.alpha x) * n + n.b                  (no mean, no variance)
    x_p      = D(embed[t_p]; embed.norm)
    layer:     h = D(x; norm1);   x += mixer(h) + experts(h)          (experts may be absent)
    logits   = logit_scale * head D(x; final.norm)
"""

import torch

F64 = torch.float64


def sigmoid(x):
    return 1.0 / (1.0 + torch.exp(-x))


def silu(x):
    return x * sigmoid(x)


def dynamic_tanh(x, w, name):
    return torch.tanh(w[name + ".alpha"] * x) * w[name] + w[name + ".b"]


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def unit_length(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def causal_conv(u, taps_w):
    """``y_t = sum_j w[:, j] u_(t - taps + 1 + j)``, zeros before the start.  ``u`` ``[T, C]``."""
    T, taps = u.shape[0], taps_w.shape[1]
    y = torch.zeros_like(u)
    for j in range(taps):
        back = taps - 1 - j
        if back < T:
            y[back:] += taps_w[:, j] * u[: T - back]
    return y


def delta_recurrence(q, k, v, g, beta):
    """One head: ``q``, ``k`` ``[T, N]``, ``v`` ``[T, P]``, ``g``, ``beta`` ``[T]``.
    The state decays, then takes the step towards ``v`` at ``k``, then answers ``q``."""
    S = torch.zeros(q.shape[1], v.shape[1], dtype=q.dtype)
    out = []
    for t in range(q.shape[0]):
        S = g[t] * S
        S = S + torch.outer(k[t], beta[t] * (v[t] - S.t() @ k[t]))
        out.append(S.t() @ q[t])
    return torch.stack(out)


def delta_mixer(h, w, p, m, eps):
    T, H, N, P = h.shape[0], m["heads"], m["dim"], m["vdim"]
    G = m.get("kv_heads", H)
    q, k, v = (silu(causal_conv(h @ w[p + n].t(), w[p + n + ".conv"])) for n in ("q", "k", "v"))
    q, k, v = unit_length(q.view(T, G, N)) * N ** -0.5, unit_length(k.view(T, G, N)), v.view(T, H, P)
    beta = sigmoid(h @ w[p + "b"].t())
    step = torch.log1p(torch.exp(h @ w[p + "a"].t() + w[p + "dt_bias"]))
    g = torch.exp(-torch.exp(w[p + "A_log"]) * step)
    o = torch.stack([delta_recurrence(q[:, i // (H // G)], k[:, i // (H // G)], v[:, i], g[:, i], beta[:, i])
                     for i in range(H)], 1)
    o = unit_rms(o, eps) * w[p + "norm"] * silu(h @ w[p + "g"].t()).view(T, H, P)
    return o.reshape(T, H * P) @ w[p + "o"].t()


def wkv_recurrence(r, k, v, decay, u):
    """One head: ``r``, ``k``, ``decay`` ``[T, N]``, ``v`` ``[T, N]``, ``u`` ``[N]``.
    The state as it was and the bonus answer ``r``; then the state decays and takes ``k v^T``."""
    S = torch.zeros(r.shape[1], v.shape[1], dtype=r.dtype)
    out = []
    for t in range(r.shape[0]):
        kv = torch.outer(k[t], v[t])
        out.append((S + u[:, None] * kv).t() @ r[t])
        S = decay[t][:, None] * S + kv
    return torch.stack(out)


def wkv_mixer(h, w, p, m, eps):
    T, H, N = h.shape[0], m["heads"], m["dim"]
    before = torch.cat([torch.zeros_like(h[:1]), h[:-1]])
    mix = {n: h + (before - h) * w[p + "mu." + n] for n in ("r", "k", "v", "g", "w")}
    r, k, v = ((mix[n] @ w[p + n].t()).view(T, H, N) for n in ("r", "k", "v"))
    decay = torch.exp(-torch.exp(torch.tanh(mix["w"] @ w[p + "w1"].t()) @ w[p + "w2"].t() + w[p + "w0"])).view(T, H, N)
    u = w[p + "u"].view(H, N)
    o = torch.stack([wkv_recurrence(r[:, i], k[:, i], v[:, i], decay[:, i], u[i]) for i in range(H)], 1)
    o = unit_rms(o, eps).reshape(T, H * N) * w[p + "norm"] * silu(mix["g"] @ w[p + "g"].t())
    return o @ w[p + "o"].t()


def rotate_halves(x, positions, dims, base):
    """``x`` ``[T, ..., n]``: columns ``i`` and ``i + dims / 2`` turn by ``position * base^(-2i / dims)``."""
    half = dims // 2
    f = torch.tensor([base ** (-2.0 * i / dims) for i in range(half)], dtype=x.dtype)
    angle = (positions.to(x.dtype)[:, None] * f).view(x.shape[0], *[1] * (x.dim() - 2), half)
    a, b, rest = x[..., :half], x[..., half:dims], x[..., dims:]
    return torch.cat([a * torch.cos(angle) - b * torch.sin(angle), b * torch.cos(angle) + a * torch.sin(angle), rest], -1)


def windowed_softmax_attention(q, k, v, scale, window):
    """One head; query ``i`` sees ``j`` with ``0 <= i - j < window`` (every earlier key without a window)."""
    T = q.shape[0]
    gap = torch.arange(T)[:, None] - torch.arange(T)[None]
    seen = (gap >= 0) & (gap < window) if window else gap >= 0
    return torch.softmax(((q @ k.t()) * scale).masked_fill(~seen, float("-inf")), -1) @ v


def latents(h, w, p, m, eps):
    """The latent ``c`` ``[T, kv_rank]`` and the turned key part ``[T, rot_dim]`` of a layer with a down-projection."""
    r, rows = m["kv_rank"], h @ w[p + "dkv"].t()
    c = unit_rms(rows[:, :r], eps) * w[p + "dkv.norm"]
    return c, rotate_halves(rows[:, r:], torch.arange(h.shape[0]), m["rot_dim"], float(m["rot"]["base"]))


def latent_mixer(h, w, p, m, eps, kept):
    """``kept``: the pair that the layer named by ``kv_from`` made, or ``None``; returns the output and the pair used."""
    T, H, d, dr, dv = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    cq = unit_rms(h @ w[p + "dq"].t(), eps) * w[p + "dq.norm"]
    q = (cq @ w[p + "uq"].t()).view(T, H, d + dr)
    turned = rotate_halves(q[..., d:], torch.arange(T), dr, float(m["rot"]["base"]))
    c, kr = kept if kept is not None else latents(h, w, p, m, eps)
    k, v = (c @ w[p + "uk"].t()).view(T, H, d), (c @ w[p + "uv"].t()).view(T, H, dv)
    window = (m.get("mask") or {}).get("size", 0)
    o = [windowed_softmax_attention(torch.cat([q[:, i, :d], turned[:, i]], -1), torch.cat([k[:, i], kr], -1), v[:, i],
                                    m["scale"], window) for i in range(H)]
    return torch.cat(o, -1) @ w[p + "o"].t(), (c, kr)


def expert(h, w, p, limit):
    g = torch.clamp(h @ w[p + "gate"].t(), max=limit)
    u = torch.clamp(h @ w[p + "up"].t(), -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ w[p + "down"].t()


def experts(h, w, p, mlp):
    """Every token's ``top`` largest router outputs, weighed by the softmax over those alone."""
    z = h @ w[p + "router"].t()
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        chosen = torch.topk(z[t], mlp["router"]["top"]).indices
        weights = torch.softmax(z[t][chosen], 0)
        for e, s in zip(chosen.tolist(), weights):
            out[t] += s * expert(h[t], w, f"{p}e{e}.", float(mlp["expert"]["limit"]))
    return out


def forward(config, w, tokens, return_layers=False):
    """Logits ``[T, vocab]`` (and the stream after every layer)."""
    eps = float(config["norm"]["eps"])
    x = dynamic_tanh(w["embed"][torch.tensor(tokens)], w, "embed.norm")
    kept, streams = {}, []
    for i, layer in enumerate(config["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        h = dynamic_tanh(x, w, p + "norm1")
        if layer["type"] == "delta":
            y = delta_mixer(h, w, p + "mix.", m, eps)
        elif layer["type"] == "wkv":
            y = wkv_mixer(h, w, p + "mix.", m, eps)
        elif layer["type"] == "latent_attention":
            y, kept[i] = latent_mixer(h, w, p + "mix.", m, eps, kept[m["kv_from"]] if "kv_from" in m else None)
        else:
            raise ValueError(layer["type"])
        if layer.get("mlp") is not None:
            y = y + experts(h, w, p + "mlp.", layer["mlp"])
        x = x + y
        streams.append(x)
    logits = (dynamic_tanh(x, w, "final.norm") @ w["head"].t()) * float(config["logit_scale"])
    return (logits, torch.stack(streams)) if return_layers else logits


def random_weights(config, seed, sharp=1.0, decay_rank=6):
    """Float32 tensors under the checkpoint's names, every one drawn.  ``sharp`` widens the attention
    scores, so that a key which is dropped, doubled or taken from a wrong page shows in the logits."""
    g = torch.Generator().manual_seed(seed)
    D = config["width"]

    def rnd(*shape, std=1.0, mean=0.0):
        return torch.randn(*shape, generator=g) * std + mean

    def norm(name, alpha):
        w[name], w[name + ".b"], w[name + ".alpha"] = rnd(D, std=0.2, mean=1.0), rnd(D, std=0.2), torch.tensor(alpha + 0.1 * torch.rand(1, generator=g).item())

    w = {"embed": rnd(config["vocab"], D), "head": rnd(config["vocab"], D, std=D ** -0.5)}
    norm("embed.norm", 0.9)
    for i, layer in enumerate(config["layers"]):
        p, m = f"l{i}.mix.", layer["mixer"]
        norm(f"l{i}.norm1", 0.5)
        if layer["type"] == "delta":
            H, G, N, P = m["heads"], m.get("kv_heads", m["heads"]), m["dim"], m["vdim"]
            for name, n in (("q", G * N), ("k", G * N), ("v", H * P)):
                w[p + name], w[p + name + ".conv"] = rnd(n, D, std=D ** -0.5), rnd(n, m["conv"], std=0.6)
            w[p + "b"], w[p + "a"] = rnd(H, D, std=D ** -0.5), rnd(H, D, std=D ** -0.5)
            w[p + "A_log"], w[p + "dt_bias"] = rnd(H, std=0.7, mean=-1.0), rnd(H, std=0.7, mean=-1.5)
            w[p + "norm"], w[p + "g"] = rnd(P, std=0.2, mean=1.0), rnd(H * P, D, std=D ** -0.5)
            w[p + "o"] = rnd(D, H * P, std=(H * P) ** -0.5)
        elif layer["type"] == "wkv":
            H, N = m["heads"], m["dim"]
            for name in ("r", "k", "v", "g", "w"):
                w[p + "mu." + name] = torch.rand(D, generator=g)
            for name in ("r", "k", "v", "g"):
                w[p + name] = rnd(H * N, D, std=D ** -0.5)
            w[p + "w1"], w[p + "w2"] = rnd(decay_rank, D, std=D ** -0.5), rnd(H * N, decay_rank, std=decay_rank ** -0.5)
            w[p + "w0"], w[p + "u"], w[p + "norm"] = rnd(H * N, std=1.5, mean=-3.0), rnd(H, N, std=0.7), rnd(H * N, std=0.2, mean=1.0)
            w[p + "o"] = rnd(D, H * N, std=(H * N) ** -0.5)
        else:
            H, d, dr, dv, Q, R = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["q_rank"], m["kv_rank"]
            w[p + "dq"], w[p + "dq.norm"] = rnd(Q, D, std=D ** -0.5), rnd(Q, std=0.2, mean=1.0)
            w[p + "uq"] = rnd(H * (d + dr), Q, std=Q ** -0.5) * sharp
            if "kv_from" not in m:
                w[p + "dkv"], w[p + "dkv.norm"] = rnd(R + dr, D, std=D ** -0.5), rnd(R, std=0.2, mean=1.0)
            w[p + "uk"], w[p + "uv"] = rnd(H * d, R, std=R ** -0.5), rnd(H * dv, R, std=R ** -0.5)
            w[p + "o"] = rnd(D, H * dv, std=(H * dv) ** -0.5)
        mlp = layer.get("mlp")
        if mlp is not None:
            p, F = f"l{i}.mlp.", mlp["expert"]["ff"]
            w[p + "router"] = rnd(mlp["router"]["experts"], D, std=2.0 * D ** -0.5)
            for e in range(mlp["router"]["experts"]):
                q = f"{p}e{e}."
                w[q + "gate"], w[q + "up"] = rnd(F, D, std=D ** -0.5), rnd(F, D, std=D ** -0.5)
                w[q + "down"] = rnd(D, F, std=F ** -0.5)
    norm("final.norm", 0.4)
    return w


def model(weights, config, tokens):
    """Logits ``[T, vocab]`` in float64 from float32 (or rounded) weights."""
    return forward(config, {k: v.double() for k, v in weights.items()}, tokens)


def greedy(weights, config, prompt, n):
    tokens, out = list(prompt), []
    for _ in range(n):
        out.append(int(model(weights, config, tokens)[-1].argmax()))
        tokens.append(out[-1])
    return out
