"""Typed configuration of the Zevivik design: a decoder of parallel layers whose config.json lists its layers one by one and
may run a stretch of them several times in a row,

    {"architecture": "Zevivik", "vocab": V, "width": W, "norm": {"eps": e}, "embedding": {"scale": s},
     "loop": {"start": a, "stop": b, "times": n},            layers a .. b-1 run n times, a cache per pass
     "layers": [{"type": "attention", "mixer": {"heads", "kv_heads", "dim", "vdim", "scale", "rot": {"dims", "base"},
                                                "mask": {"size": C}}, "mlp": MLP},
                {"type": "latent_attention", "mixer": {"heads", "dim", "vdim", "kv_rank", "scale"}, "mlp": MLP}]}
     MLP: null | {"kind": "dense", "ff": F} | {"kind": "moe", "expert": {"ff", "limit"}, "router": {"experts", "top"},
                                               "shared": {"ff", "limit"} (optional)}

Every size and constant is read from there, layer by layer.  What the design fixes: mixer and feed-forward of a layer side
by side, each behind an RMS norm of its own; attention within chunks of C positions (without `mask`: over all), its first
`dims` numbers per head rotated by halves; latent attention without positions, a normalised latent and one sigmoid gate per
head; dense feed-forwards with gelu's tanh form; experts of the clamped form g sigmoid(1.702 g) (u + 1) whose router has a
bias and weighs the chosen by a softmax over their logits alone; before each pass of the loop a learned vector, and before
every pass but the first the embedding's result, joins the stream.  Tensor names: `embed`, `head`, `final.norm`,
`loop.step`, and per layer `l<i>.` + `norm1`, `norm2`, `mix.*`, `mlp.*`.
"""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Any, Dict, List, Optional

from .pelalix import _number
from .registry import ConfigError, register_architecture
from .spec import LayerSpec, ModelSpec, PartSpec, ScheduleEntry, linear_head, token_embedding

ARCHITECTURE = "Zevivik"
MIXER_TYPES = ("attention", "latent_attention")
MLP_KINDS = ("dense", "moe")


def _mixer(kind: str, m: Any, where: str) -> Dict[str, Any]:
    if not isinstance(m, dict):
        raise ConfigError(f"config.json: {where} must be an object")
    out = {k: _number(m, k, where, int) for k in ("heads", "dim", "vdim")}
    out["scale"] = _number(m, "scale", where, float)
    if kind == "latent_attention":
        out["kv_rank"] = _number(m, "kv_rank", where, int)
        return out
    out["kv_heads"] = _number(m, "kv_heads", where, int, m.get("heads"), required=False)
    mask, rot = m.get("mask"), m.get("rot")
    out["chunk"] = 0 if mask is None else _number(mask, "size", where + ".mask", int)
    out["rot"] = None if rot is None else {"dims": _number(rot, "dims", where + ".rot", int),
                                           "base": _number(rot, "base", where + ".rot", float)}
    return out


def _mlp(raw: Any, where: str) -> Optional[Dict[str, Any]]:
    if raw is None:
        return None
    kind = _number(raw, "kind", where, str)
    if kind not in MLP_KINDS:
        raise ConfigError(f"config.json: {where}.kind {kind!r} is not known (known: " + ", ".join(MLP_KINDS) + ")")
    if kind == "dense":
        return {"kind": kind, "ff": _number(raw, "ff", where, int)}
    sized = lambda key: {"ff": _number(raw.get(key), "ff", f"{where}.{key}", int),
                         "limit": _number(raw.get(key), "limit", f"{where}.{key}", float)}
    router = raw.get("router")
    return {"kind": kind, "expert": sized("expert"), "shared": None if raw.get("shared") is None else sized("shared"),
            "router": {k: _number(router, k, where + ".router", int) for k in ("experts", "top")}}


@dataclass
class ZevivikLayer:
    type: str
    mixer: Dict[str, Any]
    mlp: Optional[Dict[str, Any]] = None


@dataclass
class ZevivikConfig:
    vocab: int
    width: int
    layers: List[ZevivikLayer]
    norm_eps: float = 1e-6
    embedding_scale: float = 1.0
    loop: Optional[Dict[str, int]] = None
    eos_token_ids: List[int] = field(default_factory=list)
    initializer_range: float = 0.02

    architecture = ARCHITECTURE

    @classmethod
    def from_dict(cls, raw: Dict[str, Any]) -> "ZevivikConfig":
        layers_raw = raw.get("layers")
        if not isinstance(layers_raw, list) or not layers_raw:
            raise ConfigError("config.json: 'layers' must be a list with at least one layer")
        layers = []
        for i, lr in enumerate(layers_raw):
            where = f"layers[{i}]"
            kind = _number(lr, "type", where, str)
            if kind not in MIXER_TYPES:
                raise ConfigError(f"config.json: {where}.type {kind!r} is not a mixer of this design (known: "
                                  + ", ".join(MIXER_TYPES) + ")")
            layers.append(ZevivikLayer(kind, _mixer(kind, lr.get("mixer"), where + ".mixer"),
                                       _mlp(lr.get("mlp"), where + ".mlp")))
        eos = raw.get("eos_token_id")
        eos = [] if eos is None else (eos if isinstance(eos, list) else [eos])
        if any(isinstance(x, bool) or not isinstance(x, int) for x in eos):
            raise ConfigError("config.json: eos_token_id must be an integer or a list of integers")
        top, loop = "the configuration", raw.get("loop")
        return cls(vocab=_number(raw, "vocab", top, int), width=_number(raw, "width", top, int), layers=layers,
                   norm_eps=_number(raw.get("norm") or {}, "eps", "norm", float, 1e-6, required=False),
                   embedding_scale=_number(raw.get("embedding") or {}, "scale", "embedding", float, 1.0, required=False),
                   loop=None if loop is None else {k: _number(loop, k, "loop", int) for k in ("start", "stop", "times")},
                   eos_token_ids=list(eos),
                   initializer_range=_number(raw, "initializer_range", top, float, 0.02, required=False))

    def to_dict(self) -> Dict[str, Any]:
        layers = []
        for l in self.layers:
            mixer = {k: v for k, v in l.mixer.items() if k not in ("chunk", "rot")}
            if l.mixer.get("chunk"):
                mixer["mask"] = {"size": l.mixer["chunk"]}
            if l.mixer.get("rot"):
                mixer["rot"] = dict(l.mixer["rot"])
            mlp = None
            if l.mlp is not None:
                mlp = {k: dict(v) if isinstance(v, dict) else v for k, v in l.mlp.items() if v is not None}
            layers.append({"type": l.type, "mixer": mixer, "mlp": mlp})
        d = {"architecture": ARCHITECTURE, "vocab": self.vocab, "width": self.width, "layers": layers,
             "norm": {"eps": self.norm_eps}, "embedding": {"scale": self.embedding_scale},
             "initializer_range": self.initializer_range}
        if self.loop is not None:
            d["loop"] = dict(self.loop)
        if self.eos_token_ids:
            d["eos_token_id"] = self.eos_token_ids[0] if len(self.eos_token_ids) == 1 else self.eos_token_ids
        return d

    def validate(self) -> None:
        def need(ok, msg):
            if not ok:
                raise ConfigError("config.json: " + msg)

        need(self.vocab > 0 and self.width > 0, "vocab and width must be positive")
        need(self.norm_eps > 0, "norm.eps must be positive")
        need(self.initializer_range > 0, "initializer_range must be positive")
        need(all(0 <= t < self.vocab for t in self.eos_token_ids), "eos_token_id names a token outside the vocabulary")
        if self.loop is not None:
            need(0 <= self.loop["start"] < self.loop["stop"] <= len(self.layers),
                 "loop.start .. loop.stop must name layers, at least one")
            need(self.loop["times"] >= 1, "loop.times must be at least 1")
        for i, l in enumerate(self.layers):
            m, w = l.mixer, f"layers[{i}].mixer"
            need(l.type in MIXER_TYPES, f"layers[{i}].type {l.type!r} is not a mixer of this design")
            need(min(m["heads"], m["dim"], m["vdim"]) > 0, f"{w}: heads, dim and vdim must be positive")
            if l.type == "latent_attention":
                need(0 < m["kv_rank"] <= 1024, f"{w}.kv_rank must be between 1 and 1024")
            else:
                need(m["dim"] <= 256 and m["vdim"] <= 256, f"{w}: dim and vdim are at most 256")
                need(m["kv_heads"] > 0 and m["heads"] % m["kv_heads"] == 0, f"{w}.heads must be a multiple of kv_heads")
                need(m["chunk"] >= 0, f"{w}.mask.size must not be negative")
                if m["rot"] is not None:
                    need(m["rot"]["base"] > 0, f"{w}.rot.base must be positive")
                    need(0 < m["rot"]["dims"] <= m["dim"] and m["rot"]["dims"] % 2 == 0,
                         f"{w}.rot.dims must be even, positive and at most dim")
            f, w = l.mlp, f"layers[{i}].mlp"
            if f is None:
                continue
            need(f["kind"] in MLP_KINDS, f"{w}.kind {f['kind']!r} is not known (known: " + ", ".join(MLP_KINDS) + ")")
            if f["kind"] == "dense":
                need(f["ff"] > 0, f"{w}.ff must be positive")
                continue
            for key in ("expert", "shared"):
                if f[key] is not None:
                    need(f[key]["ff"] > 0 and f[key]["limit"] > 0, f"{w}.{key}: ff and limit must be positive")
            need(1 <= f["router"]["top"] <= min(32, f["router"]["experts"]) and f["router"]["experts"] <= 1024,
                 f"{w}.router: top must be between 1 and experts (at most 32 of at most 1024)")

    def schedule(self) -> List[ScheduleEntry]:
        """The layers as they run; the first layer of every pass of the loop says what enters the stream before it."""
        n, loop = len(self.layers), self.loop
        if loop is None:
            return [ScheduleEntry(i) for i in range(n)]
        enter = lambda t: PartSpec("loop", {"width": self.width, "times": loop["times"], "index": t, "embedding": t > 0,
                                            "init_std": self.initializer_range}, rename={"steps": "loop.step"})
        out = [ScheduleEntry(i) for i in range(loop["start"])]
        for t in range(loop["times"]):
            out += [ScheduleEntry(i, enter=enter(t) if i == loop["start"] else None) for i in range(loop["start"], loop["stop"])]
        return out + [ScheduleEntry(i) for i in range(loop["stop"], n)]

    def model_spec(self) -> ModelSpec:
        W, std, eps = self.width, self.initializer_range, self.norm_eps
        norm = lambda name: PartSpec("rmsnorm", {"width": W, "eps": eps}, rename={"weight": name})
        layers = []
        for i, l in enumerate(self.layers):
            p, m, f = f"l{i}.", l.mixer, l.mlp
            sizes = {"hidden_size": W, "num_heads": m["heads"], "head_dim": m["dim"], "value_dim": m["vdim"],
                     "scale": m["scale"], "init_std": std}
            parts = {"mixer_norm": norm(p + "norm1")}
            if l.type == "attention":
                position = None if m["rot"] is None else PartSpec(
                    "rope", {"theta": m["rot"]["base"], "rotary_dim": m["rot"]["dims"]})
                parts["mixer"] = PartSpec(
                    "attention", {**sizes, "num_kv_heads": m["kv_heads"], "qkv_bias": False, "chunk": m["chunk"],
                                  "position": position, "pad": True},
                    prefix=p + "mix.", rename={f"{n}_proj.weight": n for n in "qkvo"})
            else:
                parts["mixer"] = PartSpec(
                    "latent_attention", {**sizes, "rot_dim": 0, "kv_rank": m["kv_rank"], "norm_eps": eps, "head_gate": True},
                    prefix=p + "mix.", rename={**{f"{n}.weight": n for n in ("q", "dkv", "uk", "uv", "g", "o")},
                                               "dkv_norm.weight": "dkv.norm"})
            if f is not None:
                parts["feed_forward_norm"] = norm(p + "norm2")
            if f is not None and f["kind"] == "dense":
                parts["feed_forward"] = PartSpec(
                    "dense_mlp", {"hidden_size": W, "width": f["ff"], "activation": "gelu_tanh", "init_std": std},
                    prefix=p + "mlp.", rename={f"{n}_proj.weight": n for n in ("gate", "up", "down")})
            elif f is not None:
                e, shared = f["expert"], f["shared"]
                names = [(f"experts.{j}", f"e{j}") for j in range(f["router"]["experts"])] + [("shared_expert", "shared")]
                parts["feed_forward"] = PartSpec(
                    "moe", {"hidden_size": W, "num_experts": f["router"]["experts"], "top_k": f["router"]["top"],
                            "expert_width": e["ff"], "activation": "clamped_glu", "limit": e["limit"],
                            "shared_width": 0 if shared is None else shared["ff"],
                            "shared_limit": None if shared is None else shared["limit"], "shared_gated": False,
                            "router_bias": True, "renormalize": True, "init_std": std},
                    prefix=p + "mlp.", rename={"gate.weight": "router", "gate.bias": "router.b",
                                               **{f"{a}.{n}_proj.weight": f"{b}.{n}" for a, b in names
                                                  for n in ("gate", "up", "down")}})
            layers.append(LayerSpec("parallel_norms", parts))
        spec = ModelSpec(
            architecture=ARCHITECTURE, hidden_size=W, vocab_size=self.vocab, max_positions=0, layers=layers,
            schedule=self.schedule(), embedding=token_embedding("embed", self.vocab, W, std, scale=self.embedding_scale),
            final_norm=norm("final.norm"), head=linear_head("head", self.vocab, W, std), init_std=std)
        spec.validate()
        return spec


register_architecture(ARCHITECTURE, ZevivikConfig)
