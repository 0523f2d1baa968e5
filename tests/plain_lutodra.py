"""Lutodra, plainly: one function per mechanism, whole sequences, float64, no cache.

Written from the design's equations only; nothing here is shared with the engine.  ``config`` is
the config.json as a dict, ``w`` maps tensor names to float64 tensors, tokens are a list of ints.

    L(x; n)   = (x - mean) / sqrt(var + eps) * n + n.b
    x_s       = embed[t]                                        for each of the streams s
    sublayer:   u = sum_s in[s] x_s;   y = f(L(u));   x_t <- sum_s mix[s, t] x_s + out[t] y
    layer:      the mixer as the first sublayer, the feed-forward (may be absent) as the second
    loop:       layers start .. stop - 1 run ``times`` times in a row
    logits    = logit_scale * head L(sum_s x_s; final.norm)
"""

import math

import torch

F64 = torch.float64


def sigmoid(x):
    return 1.0 / (1.0 + torch.exp(-x))


def silu(x):
    return x * sigmoid(x)


def softplus(x):
    return torch.clamp(x, min=0.0) + torch.log1p(torch.exp(-torch.abs(x)))


def gelu_tanh(x):
    return 0.5 * x * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (x + 0.044715 * x ** 3)))


def layer_norm(x, w, name, eps):
    mean = x.mean(-1, keepdim=True)
    var = ((x - mean) ** 2).mean(-1, keepdim=True)
    return (x - mean) / torch.sqrt(var + eps) * w[name] + w[name + ".b"]


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def unit_length(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def hyper_read(xs, w, p):
    """``xs`` ``[S, T, D]``: what the sublayer reads."""
    return sum(w[p + "in"][s] * xs[s] for s in range(xs.shape[0]))


def hyper_write(xs, y, w, p):
    S = xs.shape[0]
    return torch.stack([sum(w[p + "mix"][s, t] * xs[s] for s in range(S)) + w[p + "out"][t] * y for t in range(S)])


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
    """One head: ``q``, ``k``, ``g`` ``[T, N]``, ``v`` ``[T, P]``, ``beta`` ``[T]``.
    The state's rows decay, then it takes the step towards ``v`` at ``k``, then answers ``q``."""
    S = torch.zeros(q.shape[1], v.shape[1], dtype=q.dtype)
    out = []
    for t in range(q.shape[0]):
        S = g[t][:, None] * S
        S = S + torch.outer(k[t], beta[t] * (v[t] - S.t() @ k[t]))
        out.append(S.t() @ q[t])
    return torch.stack(out)


def channel_delta_mixer(h, w, p, m, eps):
    T, H, N, P = h.shape[0], m["heads"], m["dim"], m["vdim"]
    G = m["kv_heads"]
    q, k, v = (silu(causal_conv(h @ w[p + n].t(), w[p + n + ".conv"])) for n in ("q", "k", "v"))
    q, k, v = unit_length(q.view(T, G, N)) * N ** -0.5, unit_length(k.view(T, G, N)), v.view(T, H, P)
    beta = sigmoid(h @ w[p + "b"].t())
    step = softplus((h @ w[p + "a1"].t()) @ w[p + "a2"].t() + w[p + "dt_bias"]).view(T, H, N)
    g = torch.exp(-torch.exp(w[p + "A_log"])[:, None] * step)
    o = torch.stack([delta_recurrence(q[:, i // (H // G)], k[:, i // (H // G)], v[:, i], g[:, i], beta[:, i])
                     for i in range(H)], 1)
    gate = sigmoid((h @ w[p + "g1"].t()) @ w[p + "g2"].t()).view(T, H, P)
    o = unit_rms(o, eps) * w[p + "norm"] * gate
    return o.reshape(T, H * P) @ w[p + "o"].t()


def lru_recurrence(u, r, i, lam):
    """``u``, ``r``, ``i`` ``[T, width]``: a gated average per channel whose weights' squares sum to one."""
    a = torch.exp(-8.0 * r * softplus(lam))
    S, out = torch.zeros_like(u[0]), []
    for t in range(u.shape[0]):
        S = a[t] * S + torch.sqrt(1.0 - a[t] ** 2) * i[t] * u[t]
        out.append(S)
    return torch.stack(out)


def rglru_mixer(h, w, p, m):
    T, B = h.shape[0], m["blocks"]
    y = gelu_tanh(h @ w[p + "y"].t() + w[p + "y.b"])
    u = causal_conv(h @ w[p + "x"].t() + w[p + "x.b"], w[p + "conv"]) + w[p + "conv.b"]
    parts = u.view(T, B, -1)
    r, i = (sigmoid(torch.stack([parts[:, b] @ w[p + n][b].t() + w[p + n + ".b"][b] for b in range(B)], 1)).reshape(T, -1)
            for n in ("ra", "ri"))
    return (lru_recurrence(u, r, i, w[p + "lam"]) * y) @ w[p + "o"].t()


def rotary_frequencies(rot):
    """``base^(-2i / dims)``, slow pairs slowed further by ``scaling`` (Llama 3.1)."""
    f = [float(rot["base"]) ** (-2.0 * i / rot["dims"]) for i in range(rot["dims"] // 2)]
    s = rot.get("scaling")
    if not s:
        return f
    out = []
    for fi in f:
        wave = 2.0 * math.pi / fi
        if wave < s["original"] / s["high"]:
            out.append(fi)
        elif wave > s["original"] / s["low"]:
            out.append(fi / s["factor"])
        else:
            keep = (s["original"] / wave - s["low"]) / (s["high"] - s["low"])
            out.append((1.0 - keep) * fi / s["factor"] + keep * fi)
    return out


def rotate_halves(x, positions, rot):
    """``x`` ``[T, ..., n]``: columns ``i`` and ``i + dims / 2`` of the first ``dims`` turn with the position."""
    dims = rot["dims"]
    half = dims // 2
    f = torch.tensor(rotary_frequencies(rot), dtype=x.dtype)
    angle = (positions.to(x.dtype)[:, None] * f).view(x.shape[0], *[1] * (x.dim() - 2), half)
    a, b, rest = x[..., :half], x[..., half:dims], x[..., dims:]
    return torch.cat([a * torch.cos(angle) - b * torch.sin(angle), b * torch.cos(angle) + a * torch.sin(angle), rest], -1)


def sink_attention(q, k, v, scale, sink):
    """One head; the denominator holds ``exp(sink)`` too, which brings no value."""
    T = q.shape[0]
    s = ((q @ k.t()) * scale).masked_fill(torch.arange(T)[:, None] < torch.arange(T)[None], float("-inf"))
    s = torch.cat([s, sink.expand(T, 1)], 1)
    return torch.softmax(s, -1)[:, :T] @ v


def attention_mixer(h, w, p, m, eps):
    T, H, G, d, dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = unit_rms((h @ w[p + "q"].t()).view(T, H, d), eps) * w[p + "q.norm"]
    k = unit_rms((h @ w[p + "k"].t()).view(T, G, d), eps) * w[p + "k.norm"]
    v = (h @ w[p + "v"].t()).view(T, G, dv)
    if m.get("rot"):
        q, k = rotate_halves(q, torch.arange(T), m["rot"]), rotate_halves(k, torch.arange(T), m["rot"])
    gate = sigmoid(h @ w[p + "g"].t())
    o = [sink_attention(q[:, i], k[:, i // (H // G)], v[:, i // (H // G)], m["scale"], w[p + "sink"][i]) * gate[:, i : i + 1]
         for i in range(H)]
    return torch.cat(o, -1) @ w[p + "o"].t()


def gated_mlp(h, w, p):
    return (silu(h @ w[p + "gate"].t()) * (h @ w[p + "up"].t())) @ w[p + "down"].t()


def choose(z, router):
    """One token's experts and their weights from its router outputs."""
    s = sigmoid(z)
    groups = router["groups"]
    size = router["experts"] // groups["count"]
    score = torch.stack([torch.topk(s[g * size : (g + 1) * size], min(2, size)).values.sum() for g in range(groups["count"])])
    allowed = torch.full_like(s, float("-inf"))
    for g in torch.topk(score, groups["keep"]).indices.tolist():
        allowed[g * size : (g + 1) * size] = s[g * size : (g + 1) * size]
    chosen = torch.topk(allowed, router["top"]).indices
    return chosen, s[chosen] / (s[chosen].sum() + 1e-20) * router["scale"]


def experts(h, w, p, mlp):
    z = h @ w[p + "router"].t()
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, s in zip(*(x.tolist() for x in choose(z[t], mlp["router"]))):
            out[t] += s * gated_mlp(h[t], w, f"{p}e{e}.")
    return out


def run_order(config):
    """The layer of every run, in order."""
    n, loop = len(config["layers"]), config.get("loop")
    if not loop:
        return list(range(n))
    a, b = loop["start"], loop["stop"]
    return list(range(a)) + list(range(a, b)) * loop["times"] + list(range(b, n))


def forward(config, w, tokens, return_layers=False):
    """Logits ``[T, vocab]`` (and the sum of the streams after every run of a layer)."""
    eps = float(config["norm"]["eps"])
    xs = w["embed"][torch.tensor(tokens)].expand(config["streams"], -1, -1)
    kept = []
    for i in run_order(config):
        layer, p = config["layers"][i], f"l{i}."
        m = layer["mixer"]
        h = layer_norm(hyper_read(xs, w, p + "hc1."), w, p + "norm1", eps)
        if layer["type"] == "channel_delta":
            y = channel_delta_mixer(h, w, p + "mix.", m, eps)
        elif layer["type"] == "rglru":
            y = rglru_mixer(h, w, p + "mix.", m)
        elif layer["type"] == "attention":
            y = attention_mixer(h, w, p + "mix.", m, eps)
        else:
            raise ValueError(layer["type"])
        xs = hyper_write(xs, y, w, p + "hc1.")
        mlp = layer.get("mlp")
        if mlp is not None:
            h = layer_norm(hyper_read(xs, w, p + "hc2."), w, p + "norm2", eps)
            y = gated_mlp(h, w, p + "mlp.") if mlp["kind"] == "dense" else experts(h, w, p + "mlp.", mlp)
            xs = hyper_write(xs, y, w, p + "hc2.")
        kept.append(xs.sum(0))
    logits = (layer_norm(xs.sum(0), w, "final.norm", eps) @ w["head"].t()) * float(config["logit_scale"])
    return (logits, torch.stack(kept)) if return_layers else logits


def random_weights(config, seed, sharp=1.0, rank=6):
    """Float32 tensors under the checkpoint's names, every one drawn.  ``sharp`` widens the attention
    scores, so that a key which is dropped, doubled or taken from a wrong page shows in the logits;
    ``rank``: the width of the narrow middles of the decay and the gate."""
    g = torch.Generator().manual_seed(seed)
    D, S = config["width"], config["streams"]

    def rnd(*shape, std=1.0, mean=0.0):
        return torch.randn(*shape, generator=g) * std + mean

    def norm(name):
        w[name], w[name + ".b"] = rnd(D, std=0.2, mean=1.0), rnd(D, std=0.2)

    def hyper(p):
        w[p + "in"], w[p + "out"] = rnd(S, std=0.3, mean=1.0 / S), rnd(S, std=0.3, mean=0.7)
        w[p + "mix"] = torch.eye(S) * 0.8 + rnd(S, S, std=0.15)

    def gated(p, F):
        w[p + "gate"], w[p + "up"], w[p + "down"] = rnd(F, D, std=D ** -0.5), rnd(F, D, std=D ** -0.5), rnd(D, F, std=F ** -0.5)

    w = {"embed": rnd(config["vocab"], D), "head": rnd(config["vocab"], D, std=D ** -0.5)}
    for i, layer in enumerate(config["layers"]):
        p, m, mlp = f"l{i}.mix.", layer["mixer"], layer.get("mlp")
        norm(f"l{i}.norm1")
        hyper(f"l{i}.hc1.")
        if layer["type"] == "channel_delta":
            H, G, N, P = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            for name, n in (("q", G * N), ("k", G * N), ("v", H * P)):
                w[p + name], w[p + name + ".conv"] = rnd(n, D, std=D ** -0.5), rnd(n, m["conv"], std=0.6)
            w[p + "b"], w[p + "A_log"] = rnd(H, D, std=D ** -0.5), rnd(H, std=0.7, mean=-1.0)
            w[p + "a1"], w[p + "a2"] = rnd(rank, D, std=D ** -0.5), rnd(H * N, rank, std=rank ** -0.5)
            w[p + "dt_bias"], w[p + "norm"] = rnd(H * N, std=1.2, mean=-2.0), rnd(P, std=0.2, mean=1.0)
            w[p + "g1"], w[p + "g2"] = rnd(rank + 1, D, std=D ** -0.5), rnd(H * P, rank + 1, std=rank ** -0.5)
            w[p + "o"] = rnd(D, H * P, std=(H * P) ** -0.5)
        elif layer["type"] == "rglru":
            W, B = m["width"], m["blocks"]
            for name in ("y", "x"):
                w[p + name], w[p + name + ".b"] = rnd(W, D, std=D ** -0.5), rnd(W, std=0.2)
            w[p + "conv"], w[p + "conv.b"] = rnd(W, m["conv"], std=0.6), rnd(W, std=0.2)
            for name in ("ra", "ri"):
                w[p + name], w[p + name + ".b"] = rnd(B, W // B, W // B, std=(W // B) ** -0.5), rnd(B, W // B, std=0.5)
            w[p + "lam"], w[p + "o"] = rnd(W, std=1.0, mean=-4.0), rnd(D, W, std=W ** -0.5)
        else:
            H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            w[p + "q"], w[p + "k"], w[p + "v"] = rnd(H * d, D, std=D ** -0.5), rnd(G * d, D, std=D ** -0.5), rnd(G * dv, D, std=D ** -0.5)
            w[p + "q.norm"], w[p + "k.norm"] = rnd(d, std=0.2, mean=1.0) * sharp, rnd(d, std=0.2, mean=1.0)
            w[p + "sink"], w[p + "g"] = rnd(H, std=1.0, mean=1.0), rnd(H, D, std=D ** -0.5)
            w[p + "o"] = rnd(D, H * dv, std=(H * dv) ** -0.5)
        if mlp is not None:
            p = f"l{i}.mlp."
            norm(f"l{i}.norm2")
            hyper(f"l{i}.hc2.")
            if mlp["kind"] == "dense":
                gated(p, mlp["ff"])
            else:
                w[p + "router"] = rnd(mlp["router"]["experts"], D, std=2.0 * D ** -0.5)
                for e in range(mlp["router"]["experts"]):
                    gated(f"{p}e{e}.", mlp["expert"]["ff"])
    norm("final.norm")
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
