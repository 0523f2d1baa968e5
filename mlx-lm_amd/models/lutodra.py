"""Lutodra: arguments, plan, tensor names, random weights.

A decoder-only design whose residual stream is kept as several streams with hyper-connected sublayers
(``parts/block.py:HyperBlock``): a sublayer reads a weighted sum of the streams through a LayerNorm, and
its output enters all of them while a small matrix mixes them.  A run of layers may be passed several
times with the same weights (``loop``), every pass with a cache and state of its own.  Mixers:

* ``channel_delta``: the gated delta rule with a decay per key channel and an output gate through narrow
  middles (``parts/delta_rule.py:ChannelDeltaRule``);
* ``rglru``: the recurrent block with a real-gated linear recurrent unit (``parts/recurrent_unit.py``);
* ``attention``: grouped softmax attention with normed and rotated queries and keys, a sink in the
  denominator and one output gate a head (``parts/scored_attention.py``).

The feed-forward is dense and gated or a mixture of gated experts chosen by their sigmoid out of the best
groups of neighbours (``parts/experts.py``); a layer may have none.

config.json names the design under ``architecture`` and gives every size and constant: ``vocab``,
``width``, ``streams``, ``norm.eps``, ``logit_scale``, ``loop: {start, stop, times}`` (optional) and ``layers``,
a list of ``{"type", "mixer": {...}, "mlp": {"kind": "dense", "ff"} | {"kind": "moe", "expert": {ff}, "router":
{experts, top, scale, groups: {count, keep}}} | null}``; ``max_positions`` is optional (the design has no table
that bounds it).  Mixer keys: ``channel_delta``: ``heads, kv_heads, dim, vdim, conv`` (taps; the widths of the
middles are ``decay_rank`` and ``gate_rank``, or, as in the design's own files, what the shapes of ``a1`` and ``g1``
say: ``sizes_from_tensors``); ``rglru``: ``width, blocks, conv``; ``attention``: ``heads, kv_heads, dim, vdim, scale,
rot: {dims, base, scaling: {factor, low, high, original}}``.  Tensors: ``embed``, ``l<i>.norm1``, ``l<i>.norm2``,
``final.norm`` (each with ``.b``), ``l<i>.hc1.{in,out,mix}``, ``l<i>.hc2.*``, ``l<i>.mix.*``, ``l<i>.mlp.*``, ``head``;
linear weights ``[out, in]``.
"""

from dataclasses import dataclass, field
from typing import Any, Dict, List, Optional

import torch

from ..config.base import BaseModelArgs
from ..config.plan import LayerSpec, ModelPlan, PartSpec, RunEntry
from ..parts.model import DecoderModel

MIXERS = ("channel_delta", "rglru", "attention")
FEED_FORWARDS = ("dense", "moe")
DEFAULT_POSITIONS = 1 << 15  # nothing in the design bounds a sequence; the cache's tables need a bound
DEFAULT_RANK = 16


@dataclass
class ModelArgs(BaseModelArgs):
    """Keys of a Lutodra config.json; what the engine cannot run is refused here."""

    architecture: str
    vocab: int
    width: int
    layers: List[Dict[str, Any]]
    streams: int = 1
    norm: Dict[str, Any] = field(default_factory=dict)
    loop: Optional[Dict[str, Any]] = None
    logit_scale: float = 1.0
    max_positions: int = DEFAULT_POSITIONS

    def __post_init__(self):
        for key in ("vocab", "width", "streams", "max_positions"):
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
        if self.loop:
            a, b, n = (self.loop.get(k) for k in ("start", "stop", "times"))
            if not all(isinstance(v, int) for v in (a, b, n)) or not 0 <= a < b <= len(self.layers) or n < 1:
                raise ValueError(f"loop {self.loop!r}: layers start .. stop - 1 of {len(self.layers)}, at least once")

    @property
    def eps(self):
        return float(self.norm["eps"])

    def run_order(self):
        """The layer of every run: those of the loop come ``times`` times in a row."""
        n = len(self.layers)
        if not self.loop:
            return list(range(n))
        a, b, times = self.loop["start"], self.loop["stop"], self.loop["times"]
        return list(range(a)) + list(range(a, b)) * times + list(range(b, n))

    @staticmethod
    def sizes_from_tensors(config, shapes):
        """``config`` with the sizes that only a checkpoint's tensor shapes give: the widths of a
        ``channel_delta`` layer's middles (rows of ``a1`` and ``g1``) and, where ``conv`` is not given, the taps
        of a convolution (columns of its weights)."""
        import copy

        config = copy.deepcopy(config)
        for i, entry in enumerate(config.get("layers") or []):
            m, p = entry.get("mixer"), f"l{i}.mix."
            if not isinstance(m, dict):
                continue
            if entry.get("type") == "channel_delta":
                for key, name in (("decay_rank", "a1"), ("gate_rank", "g1")):
                    if key not in m and p + name in shapes:
                        m[key] = int(shapes[p + name][0])
            conv = {"channel_delta": "q.conv", "rglru": "conv"}.get(entry.get("type"))
            if conv and "conv" not in m and p + conv in shapes:
                m["conv"] = int(shapes[p + conv][1])
        return config


class Model:
    """The Lutodra model: a ``DecoderModel`` built from the plan below."""

    def __init__(self, args: ModelArgs):
        self.args = args
        self.model_type = "lutodra"
        self.decoder = DecoderModel(self.plan(args))

    @property
    def layers(self):
        return self.decoder.layers

    @staticmethod
    def mixer_spec(args, entry, p):
        D, eps, m = args.width, args.eps, entry["mixer"]
        if entry["type"] == "channel_delta":
            return PartSpec("channel_delta_rule", {
                "width": D, "n_heads": m["heads"], "n_key_heads": m.get("kv_heads", m["heads"]), "key_dim": m["dim"],
                "value_dim": m.get("vdim", m["dim"]), "taps": int(m.get("conv") or 1), "eps": eps,
                "decay_rank": int(m.get("decay_rank", DEFAULT_RANK)), "gate_rank": int(m.get("gate_rank", DEFAULT_RANK))}, p)
        if entry["type"] == "rglru":
            return PartSpec("recurrent_unit", {"width": D, "inner": m["width"], "blocks": m.get("blocks", 1),
                                               "taps": int(m.get("conv") or 1)}, p)
        rot = m.get("rot") or {}
        return PartSpec("scored_attention", {
            "width": D, "n_heads": m["heads"], "n_kv_heads": m.get("kv_heads", m["heads"]), "key_dim": m["dim"],
            "value_dim": m.get("vdim", m["dim"]), "scale": m.get("scale", m["dim"] ** -0.5), "eps": eps, "head_norm": True,
            "rot_dims": int(rot.get("dims", 0)), "rot_base": float(rot.get("base", 10000.0)), "rot_scaling": rot.get("scaling"),
            "sink": True, "head_gate": True}, p)

    @staticmethod
    def ffn_spec(args, mlp, p):
        if mlp["kind"] == "dense":
            return PartSpec("gated_mlp", {"width": args.width, "inner": mlp["ff"]}, p)
        router = mlp["router"]
        groups = router.get("groups") or {}
        return PartSpec("gated_experts", {
            "width": args.width, "n_experts": router["experts"], "inner": mlp["expert"]["ff"], "top": router["top"], "correction": False,
            "renormalize": True, "weight_scale": float(router.get("scale", 1.0)), "scores": "sigmoid",
            "groups": (groups["count"], groups["keep"]) if groups else None}, p)

    @staticmethod
    def plan(args: ModelArgs) -> ModelPlan:
        D = args.width

        def norm(name, scale=1.0):
            return PartSpec("layernorm", {"width": D, "eps": args.eps, "weight_name": name, "bias_name": name + ".b", "scale": scale})

        order = args.run_order()
        layers = []
        for i, entry in enumerate(args.layers):
            p, mlp = f"l{i}.", entry.get("mlp")
            parts = dict(mixer_norm=norm(p + "norm1"), mixer=Model.mixer_spec(args, entry, p + "mix."))
            if mlp is not None:
                parts["ffn_norm"], parts["ffn"] = norm(p + "norm2"), Model.ffn_spec(args, mlp, p + "mlp.")
            layers.append(LayerSpec("hyper", parts, {"streams": args.streams, "n_runs": len(order), "prefix": p}))
        return ModelPlan(
            width=D, vocab_size=args.vocab, max_positions=args.max_positions,
            embedding=PartSpec("token", {"vocab_size": args.vocab, "width": D, "weight_name": "embed"}),
            # every run has a cache or state of its own; the logits' factor rides on the last norm's weight and bias
            embedding_positions=None, layers=layers, schedule=[RunEntry(layer=i, cache=slot) for slot, i in enumerate(order)],
            final_norm=norm("final.norm", float(args.logit_scale)),
            head=PartSpec("linear", {"vocab_size": args.vocab, "width": D, "weight_name": "head"}))

    def sanitize(self, weights):
        # (a layer without a feed-forward may come with that sublayer's norm and connections: nothing reads them)
        unread = tuple(f"l{i}.{x}" for i, entry in enumerate(self.args.layers) if entry.get("mlp") is None for x in ("norm2", "hc2."))
        return {k: v for k, v in weights.items() if not (unread and k.startswith(unread))}

    @staticmethod
    def random_weights(args: ModelArgs, seed, scheme="a"):
        """Seeded tensors under the checkpoint's names.  Scheme ``a``: norm weights 1, shifts 0, connections
        that read the streams' mean, keep them apart and write to all alike.  Scheme ``b``: all of them drawn."""
        if scheme not in ("a", "b"):
            raise ValueError(f"unknown random-weight scheme '{scheme}'")
        g = torch.Generator().manual_seed(int(seed))
        D, S = args.width, args.streams

        def normal(shape, std, mean=0.0):
            return torch.randn(shape, generator=g, dtype=torch.float32) * std + mean

        def vector(n, mean, std):
            return normal((n,), std, mean) if scheme == "b" else torch.full((n,), float(mean))

        def add_norm(name):
            t[name], t[name + ".b"] = vector(D, 1.0, 0.1), vector(D, 0.0, 0.1)

        def add_connections(p):
            t[p + "in"], t[p + "out"] = vector(S, 1.0 / S, 0.2), vector(S, 1.0, 0.2)
            t[p + "mix"] = torch.eye(S) + (normal((S, S), 0.1) if scheme == "b" else 0.0)

        def add_gated(p, F):
            t[p + "gate"], t[p + "up"], t[p + "down"] = normal((F, D), D ** -0.5), normal((F, D), D ** -0.5), normal((D, F), F ** -0.5)

        t = {"embed": normal((args.vocab, D), 1.0)}
        for i, entry in enumerate(args.layers):
            p, m, q, mlp = f"l{i}.", entry["mixer"], f"l{i}.mix.", entry.get("mlp")
            add_norm(p + "norm1")
            add_connections(p + "hc1.")
            if entry["type"] == "channel_delta":
                H, G, N, P = m["heads"], m.get("kv_heads", m["heads"]), m["dim"], m.get("vdim", m["dim"])
                taps, ra, rg = int(m.get("conv") or 1), int(m.get("decay_rank", DEFAULT_RANK)), int(m.get("gate_rank", DEFAULT_RANK))
                for name, n in (("q", G * N), ("k", G * N), ("v", H * P)):
                    t[q + name], t[q + name + ".conv"] = normal((n, D), D ** -0.5), normal((n, taps), taps ** -0.5)
                t[q + "b"], t[q + "A_log"], t[q + "dt_bias"] = normal((H, D), D ** -0.5), vector(H, 0.0, 0.5), vector(H * N, -3.0, 0.5)
                t[q + "a1"], t[q + "a2"] = normal((ra, D), D ** -0.5), normal((H * N, ra), ra ** -0.5)
                t[q + "g1"], t[q + "g2"] = normal((rg, D), D ** -0.5), normal((H * P, rg), rg ** -0.5)
                t[q + "norm"], t[q + "o"] = vector(P, 1.0, 0.1), normal((D, H * P), (H * P) ** -0.5)
            elif entry["type"] == "rglru":
                C, B, taps = m["width"], m.get("blocks", 1), int(m.get("conv") or 1)
                for name in ("y", "x"):
                    t[q + name], t[q + name + ".b"] = normal((C, D), D ** -0.5), vector(C, 0.0, 0.1)
                t[q + "conv"], t[q + "conv.b"] = normal((C, taps), taps ** -0.5), vector(C, 0.0, 0.1)
                for name in ("ra", "ri"):
                    t[q + name] = normal((B, C // B, C // B), (C // B) ** -0.5)
                    t[q + name + ".b"] = vector(C, 0.0, 0.5).view(B, C // B)
                t[q + "lam"], t[q + "o"] = vector(C, -4.0, 1.0), normal((D, C), C ** -0.5)
            else:
                H, G, d, dv = m["heads"], m.get("kv_heads", m["heads"]), m["dim"], m.get("vdim", m["dim"])
                t[q + "q"], t[q + "k"], t[q + "v"] = normal((H * d, D), D ** -0.5), normal((G * d, D), D ** -0.5), normal((G * dv, D), D ** -0.5)
                t[q + "q.norm"], t[q + "k.norm"], t[q + "sink"] = vector(d, 1.0, 0.1), vector(d, 1.0, 0.1), vector(H, 0.0, 1.0)
                t[q + "g"], t[q + "o"] = normal((H, D), D ** -0.5), normal((D, H * dv), (H * dv) ** -0.5)
            if mlp is not None:
                add_norm(p + "norm2")
                add_connections(p + "hc2.")
                if mlp["kind"] == "dense":
                    add_gated(p + "mlp.", mlp["ff"])
                else:
                    t[p + "mlp.router"] = normal((mlp["router"]["experts"], D), D ** -0.5)
                    for e in range(mlp["router"]["experts"]):
                        add_gated(f"{p}mlp.e{e}.", mlp["expert"]["ff"])
        add_norm("final.norm")
        t["head"] = normal((args.vocab, D), D ** -0.5)
        return t
