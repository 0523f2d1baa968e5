"""Gilidra: arguments, plan, tensor names, random weights.

A decoder-only design whose layers run their two sublayers side by side on one norm, ``u = D(x)``, ``x
+= mixer(u) + ff(u)``, where the norm is a dynamic tanh, ``D(x) = tanh(alpha x) * w + b``, which takes no
statistics.  The token embedding passes such a norm too; the model's norm, an untied head and a
constant factor on the logits close it.  Mixers:

* ``delta``: the gated delta rule with grouped key heads, a short convolution and unit-length
  queries and keys (``parts/delta_rule.py``);
* ``wkv``: a token shift, a decay per key channel from a low-rank middle and a bonus for the current
  token (``parts/time_mix.py``);
* ``latent_attention``: attention over a small latent per token in a sliding window; a layer may read
  the latents that an earlier layer cached (``kv_from``), with a window of its own
  (``parts/latent_attention.py``).

The feed-forward is a mixture of clamped gated experts chosen by a softmax over the chosen logits
(``parts/experts.py``); a layer may have none.

config.json names the design under ``architecture`` and gives every size and constant: ``vocab``,
``width``, ``norm.eps`` (of the norms inside the mixers), ``logit_scale`` and ``layers``, a list of
``{"type", "mixer": {...}, "mlp": {"kind": "moe", "expert": {ff, limit}, "router": {experts, top}} |
null}``; ``max_positions`` is optional (the design has no table that bounds it).  Mixer keys:
``delta``: ``heads, kv_heads, dim, vdim, conv`` (taps); ``wkv``: ``heads, dim`` (the width of the decay's
middle is ``decay_rank``, or, as in the design's own files, what the shape of ``w1`` says:
``sizes_from_tensors``); ``latent_attention``: ``heads, dim, rot_dim, vdim, q_rank, kv_rank, scale, rot:
{dims, base}, mask: {size}`` and ``kv_from`` (optional).  Tensors: ``embed``, ``embed.norm``,
``l<i>.norm1``, ``final.norm`` (each with ``.b`` and ``.alpha``), ``l<i>.mix.*``, ``l<i>.mlp.*``,
``head``; linear weights ``[out, in]``.
"""

from dataclasses import dataclass, field
from typing import Any, Dict, List

import torch

from ..config.base import BaseModelArgs
from ..config.plan import LayerSpec, ModelPlan, PartSpec, RunEntry
from ..parts.model import DecoderModel

MIXERS = ("delta", "wkv", "latent_attention")
FEED_FORWARDS = ("moe",)
DEFAULT_POSITIONS = 1 << 15  # nothing in the design bounds a sequence; the cache's tables need a bound
DEFAULT_DECAY_RANK = 16


def _window(mixer):
    return int((mixer.get("mask") or {}).get("size") or 0)


@dataclass
class ModelArgs(BaseModelArgs):
    """Keys of a Gilidra config.json; what the engine cannot run is refused here."""

    architecture: str
    vocab: int
    width: int
    layers: List[Dict[str, Any]]
    norm: Dict[str, Any] = field(default_factory=dict)
    logit_scale: float = 1.0
    max_positions: int = DEFAULT_POSITIONS

    def __post_init__(self):
        for key in ("vocab", "width", "max_positions"):
            if not isinstance(getattr(self, key), int) or getattr(self, key) <= 0:
                raise ValueError(f"{key} must be a positive integer, got {getattr(self, key)!r}")
        if not self.layers:
            raise ValueError("a model needs at least one layer")
        if "eps" not in self.norm:
            raise ValueError("norm.eps is missing")
        for i, entry in enumerate(self.layers):
            if entry.get("type") not in MIXERS:
                raise ValueError(f"layer {i}: mixer type {entry.get('type')!r} is not implemented (known: {MIXERS})")
            mlp = entry.get("mlp")
            if mlp is not None and mlp.get("kind") not in FEED_FORWARDS:
                raise ValueError(f"layer {i}: feed-forward kind {mlp.get('kind')!r} is not implemented (known: {FEED_FORWARDS})")
            if entry["type"] == "latent_attention":
                self._check_latent(i, entry.get("mixer") or {})

    def _check_latent(self, i, m):
        rot = m.get("rot") or {}
        if int(rot.get("dims", m.get("rot_dim", 0))) != int(m.get("rot_dim", 0)):
            raise ValueError(f"layer {i}: the rotated key part has rot_dim columns, all of which turn")
        if "mask" in m and _window(m) <= 0:
            raise ValueError(f"layer {i}: mask.size must be positive, got {m['mask']!r}")
        if m.get("kv_from") is None:
            return
        j = m["kv_from"]
        src = self.layers[j] if isinstance(j, int) and 0 <= j < i else None
        if src is None or src.get("type") != "latent_attention" or src["mixer"].get("kv_from") is not None:
            raise ValueError(f"layer {i}: kv_from {j!r} must name an earlier latent-attention layer with latents of its own")
        for key in ("kv_rank", "rot_dim", "rot"):
            if src["mixer"].get(key) != m.get(key):
                raise ValueError(f"layer {i}: its {key} differs from layer {j}'s, whose latents it reads")

    @property
    def eps(self):
        return float(self.norm["eps"])

    def cache_windows(self):
        """``{layer with latents of its own: the longest window among the layers that read them}`` (0: one
        of them sees every earlier token), which is what the layer's pages have to keep."""
        out = {}
        for i, entry in enumerate(self.layers):
            if entry["type"] == "latent_attention":
                m = entry["mixer"]
                src, w = i if m.get("kv_from") is None else m["kv_from"], _window(m)
                out[src] = 0 if w == 0 or out.get(src) == 0 else max(w, out.get(src, 0))
        return out

    @staticmethod
    def sizes_from_tensors(config, shapes):
        """``config`` with the sizes that only a checkpoint's tensor shapes give: the width of a ``wkv``
        layer's decay middle (rows of ``w1``) and, where ``conv`` is not given, the taps of a ``delta``
        layer's convolution (columns of ``q.conv``)."""
        import copy

        config = copy.deepcopy(config)
        for i, entry in enumerate(config.get("layers") or []):
            m = entry.get("mixer")
            if not isinstance(m, dict):
                continue
            w1, conv = shapes.get(f"l{i}.mix.w1"), shapes.get(f"l{i}.mix.q.conv")
            if entry.get("type") == "wkv" and "decay_rank" not in m and w1 is not None:
                m["decay_rank"] = int(w1[0])
            if entry.get("type") == "delta" and "conv" not in m and conv is not None:
                m["conv"] = int(conv[1])
        return config


class Model:
    """The Gilidra model: a ``DecoderModel`` built from the plan below."""

    def __init__(self, args: ModelArgs):
        self.args = args
        self.model_type = "gilidra"
        self.decoder = DecoderModel(self.plan(args))

    @property
    def layers(self):
        return self.decoder.layers

    @staticmethod
    def mixer_spec(args, entry, p, cache_window):
        D, eps, m = args.width, args.eps, entry["mixer"]
        if entry["type"] == "delta":
            return PartSpec("delta_rule", {
                "width": D, "n_heads": m["heads"], "n_key_heads": m.get("kv_heads", m["heads"]), "key_dim": m["dim"],
                "value_dim": m.get("vdim", m["dim"]), "taps": int(m.get("conv") or 1), "eps": eps}, p)
        if entry["type"] == "wkv":
            return PartSpec("time_mix", {"width": D, "n_heads": m["heads"], "head_dim": m["dim"],
                                         "decay_rank": int(m.get("decay_rank", DEFAULT_DECAY_RANK)), "eps": eps}, p)
        return PartSpec("latent_attention", {
            "width": D, "n_heads": m["heads"], "key_dim": m["dim"], "rot_dim": m["rot_dim"], "value_dim": m.get("vdim", m["dim"]),
            "q_rank": m["q_rank"], "kv_rank": m["kv_rank"], "scale": m.get("scale", (m["dim"] + m["rot_dim"]) ** -0.5),
            "eps": eps, "rot_base": float((m.get("rot") or {}).get("base", 10000.0)), "own_latent": m.get("kv_from") is None,
            "window": _window(m), "cache_window": cache_window, "gate": False, "interleaved": False}, p)

    @staticmethod
    def plan(args: ModelArgs) -> ModelPlan:
        D = args.width

        def norm(name, scale=1.0):
            return PartSpec("dynamic_tanh", {"width": D, "weight_name": name, "scale": scale})

        layers, schedule, slot, slot_of, windows = [], [], 0, {}, args.cache_windows()
        for i, entry in enumerate(args.layers):
            p, m, mlp = f"l{i}.", entry["mixer"], entry.get("mlp")
            source = i if m.get("kv_from") is None else m["kv_from"]
            parts = dict(norm=norm(p + "norm1"), mixer=Model.mixer_spec(args, entry, p + "mix.", windows.get(source)))
            if mlp is not None:
                parts["ffn"] = PartSpec("gated_experts", {
                    "width": D, "n_experts": mlp["router"]["experts"], "inner": mlp["expert"]["ff"], "top": mlp["router"]["top"],
                    "correction": False, "renormalize": True, "activation": "clamped", "limit": float(mlp["expert"]["limit"])}, p + "mlp.")
            # (the layer behind starts with its norm, unless a token shift makes that itself)
            follows = i + 1 < len(args.layers) and args.layers[i + 1]["type"] != "wkv" and mlp is not None
            layers.append(LayerSpec("shared_norm", parts, {"next_norm": norm(f"l{i + 1}.norm1")} if follows else {}))
            if source != i:
                schedule.append(RunEntry(layer=i, cache=slot_of[source], writes_cache=False))
                continue
            slot_of[i] = slot
            schedule.append(RunEntry(layer=i, cache=slot))
            slot += 1
        return ModelPlan(
            width=D, vocab_size=args.vocab, max_positions=args.max_positions,
            embedding=PartSpec("normed_token", {"vocab_size": args.vocab, "width": D, "weight_name": "embed", "norm": norm("embed.norm")}),
            # (the logits' factor rides on the last norm's weight and shift)
            embedding_positions=None, layers=layers, schedule=schedule, final_norm=norm("final.norm", float(args.logit_scale)),
            head=PartSpec("linear", {"vocab_size": args.vocab, "width": D, "weight_name": "head"}))

    def sanitize(self, weights):
        # (one number may be stored as a vector of one)
        return {k: v.reshape(()) if k.endswith(".alpha") and v.numel() == 1 else v for k, v in weights.items()}

    @staticmethod
    def random_weights(args: ModelArgs, seed, scheme="a"):
        """Seeded tensors under the checkpoint's names.  Scheme ``a``: norm weights 1, shifts 0, alphas
        0.5.  Scheme ``b``: all of them drawn."""
        if scheme not in ("a", "b"):
            raise ValueError(f"unknown random-weight scheme '{scheme}'")
        g = torch.Generator().manual_seed(int(seed))
        D = args.width

        def normal(shape, std, mean=0.0):
            return torch.randn(shape, generator=g, dtype=torch.float32) * std + mean

        def vector(n, mean, std):
            return normal((n,), std, mean) if scheme == "b" else torch.full((n,), float(mean))

        def add_norm(name):
            t[name], t[name + ".b"] = vector(D, 1.0, 0.1), vector(D, 0.0, 0.1)
            t[name + ".alpha"] = vector(1, 0.5, 0.05).reshape(())

        t = {"embed": normal((args.vocab, D), 1.0)}
        add_norm("embed.norm")
        for i, entry in enumerate(args.layers):
            p, m, q = f"l{i}.", entry["mixer"], f"l{i}.mix."
            add_norm(p + "norm1")
            if entry["type"] == "delta":
                H, G, N, P = m["heads"], m.get("kv_heads", m["heads"]), m["dim"], m.get("vdim", m["dim"])
                taps = int(m.get("conv") or 1)
                for name, n in (("q", G * N), ("k", G * N), ("v", H * P)):
                    t[q + name], t[q + name + ".conv"] = normal((n, D), D ** -0.5), normal((n, taps), taps ** -0.5)
                t[q + "b"], t[q + "a"], t[q + "g"] = normal((H, D), D ** -0.5), normal((H, D), D ** -0.5), normal((H * P, D), D ** -0.5)
                t[q + "A_log"], t[q + "dt_bias"] = vector(H, 0.0, 0.5), vector(H, -3.0, 0.5)
                t[q + "norm"], t[q + "o"] = vector(P, 1.0, 0.1), normal((D, H * P), (H * P) ** -0.5)
            elif entry["type"] == "wkv":
                H, N, R = m["heads"], m["dim"], int(m.get("decay_rank", DEFAULT_DECAY_RANK))
                for name in ("r", "k", "v", "g", "w"):
                    t[q + "mu." + name] = torch.rand((D,), generator=g) if scheme == "b" else torch.full((D,), 0.5)
                for name in ("r", "k", "v", "g"):
                    t[q + name] = normal((H * N, D), D ** -0.5)
                t[q + "w1"], t[q + "w2"], t[q + "w0"] = normal((R, D), D ** -0.5), normal((H * N, R), R ** -0.5), vector(H * N, -4.0, 1.5)
                t[q + "u"], t[q + "norm"], t[q + "o"] = normal((H, N), 0.5), vector(H * N, 1.0, 0.1), normal((D, H * N), (H * N) ** -0.5)
            else:
                H, d, dr, dv, Q, R = m["heads"], m["dim"], m["rot_dim"], m.get("vdim", m["dim"]), m["q_rank"], m["kv_rank"]
                t[q + "dq"], t[q + "dq.norm"] = normal((Q, D), D ** -0.5), vector(Q, 1.0, 0.1)
                t[q + "uq"] = normal((H * (d + dr), Q), Q ** -0.5)
                if m.get("kv_from") is None:
                    t[q + "dkv"], t[q + "dkv.norm"] = normal((R + dr, D), D ** -0.5), vector(R, 1.0, 0.1)
                t[q + "uk"], t[q + "uv"] = normal((H * d, R), R ** -0.5), normal((H * dv, R), R ** -0.5)
                t[q + "o"] = normal((D, H * dv), (H * dv) ** -0.5)
            mlp = entry.get("mlp")
            if mlp is not None:
                q, F = p + "mlp.", mlp["expert"]["ff"]
                t[q + "router"] = normal((mlp["router"]["experts"], D), D ** -0.5)
                for e in range(mlp["router"]["experts"]):
                    t[f"{q}e{e}.gate"], t[f"{q}e{e}.up"] = normal((F, D), D ** -0.5), normal((F, D), D ** -0.5)
                    t[f"{q}e{e}.down"] = normal((D, F), F ** -0.5)
        add_norm("final.norm")
        t["head"] = normal((args.vocab, D), D ** -0.5)
        return t
