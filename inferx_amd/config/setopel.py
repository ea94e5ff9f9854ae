"""Typed configuration of the Setopel design: a pre-norm decoder whose residual stream is kept in several copies
(hyper-connections) and whose config.json lists its layers one by one,

    {"architecture": "Setopel", "vocab": V, "width": W, "norm": {"eps": e}, "residual_mult": m, "streams": s,
     "layers": [{"type": "attention", "mixer": {"heads", "kv_heads", "dim", "vdim", "scale", "softcap", "conv",
                                                "q_temp": {"coef", "every"}, "kv_from": j}, "mlp": MLP},
                {"type": "retention", "mixer": {"heads", "dim", "vdim", "decay": [per head],
                                                "rot": {"dims", "base"}}, "mlp": MLP},
                {"type": "latent_attention", "mixer": {"heads", "dim", "vdim", "kv_rank", "scale"}, "mlp": MLP}]}
     MLP: null | {"kind": "dense", "ff": F}

Every size and constant is read from there, layer by layer.  What the design fixes: a norm on the embedding; norm
weights stored around zero; in attention biases on q, k and v, a softmax with one added to its denominator and a sigmoid
gate, and keys and values that a later layer (`kv_from`) may read; in retention keys scaled by dim^(-1/2), a norm per
head without a weight and a silu gate; latents normalised with a plain weight, nothing rotated beside them; feed-forwards
with silu gates.  Without `streams` the stream is one, h + m * branch.  Tensor names: `embed`, `embed.norm`, `head`,
`final.norm`, and per layer `l<i>.` + `norm1`, `norm2`, `hc1.*`, `hc2.*`, `mix.*`, `mlp.*`.
"""
from __future__ import annotations

import copy
from dataclasses import dataclass, field
from typing import Any, Dict, List, Optional

from .pelalix import _number
from .registry import ConfigError, register_architecture
from .spec import LayerSpec, ModelSpec, PartSpec, ScheduleEntry, linear_head

ARCHITECTURE = "Setopel"
MIXER_TYPES = ("attention", "retention", "latent_attention")
MAX_STREAMS = 32


def _mixer(kind: str, m: Any, where: str) -> Dict[str, Any]:
    if not isinstance(m, dict):
        raise ConfigError(f"config.json: {where} must be an object")
    n = lambda key, typ=int, at=m, w=where: _number(at, key, w, typ)
    maybe = lambda key, typ, default: _number(m, key, where, typ, default, required=False)
    if kind == "latent_attention":
        return {"heads": n("heads"), "dim": n("dim"), "vdim": n("vdim"), "kv_rank": n("kv_rank"), "scale": n("scale", float)}
    if kind == "retention":
        decay = m.get("decay")
        if not isinstance(decay, list) or any(isinstance(d, bool) or not isinstance(d, (int, float)) for d in decay):
            raise ConfigError(f"config.json: {where}.decay must be a list of numbers")
        rot = m.get("rot")
        return {"heads": n("heads"), "dim": n("dim"), "vdim": n("vdim"), "decay": [float(d) for d in decay],
                "rot": None if rot is None else {"dims": n("dims", int, rot, where + ".rot"),
                                                 "base": n("base", float, rot, where + ".rot")}}
    temp = m.get("q_temp")
    return {"heads": n("heads"), "kv_heads": maybe("kv_heads", int, m.get("heads")), "dim": n("dim"), "vdim": n("vdim"),
            "scale": n("scale", float), "softcap": maybe("softcap", float, 0.0), "conv": maybe("conv", int, 0),
            "q_temp": None if temp is None else {"coef": n("coef", float, temp, where + ".q_temp"),
                                                 "every": n("every", float, temp, where + ".q_temp")},
            "kv_from": maybe("kv_from", int, None)}


def _mlp(raw: Any, where: str) -> Optional[Dict[str, Any]]:
    if raw is None:
        return None
    kind = _number(raw, "kind", where, str)
    if kind != "dense":
        raise ConfigError(f"config.json: {where}.kind {kind!r} is not known (known: dense)")
    return {"kind": kind, "ff": _number(raw, "ff", where, int)}


@dataclass
class SetopelLayer:
    type: str
    mixer: Dict[str, Any]
    mlp: Optional[Dict[str, Any]] = None


@dataclass
class SetopelConfig:
    vocab: int
    width: int
    layers: List[SetopelLayer]
    norm_eps: float = 1e-6
    residual_mult: float = 1.0
    streams: Optional[int] = None
    eos_token_ids: List[int] = field(default_factory=list)
    initializer_range: float = 0.02

    architecture = ARCHITECTURE

    @classmethod
    def from_dict(cls, raw: Dict[str, Any]) -> "SetopelConfig":
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
            layers.append(SetopelLayer(kind, _mixer(kind, lr.get("mixer"), where + ".mixer"),
                                       _mlp(lr.get("mlp"), where + ".mlp")))
        eos = raw.get("eos_token_id")
        eos = [] if eos is None else (eos if isinstance(eos, list) else [eos])
        if any(isinstance(x, bool) or not isinstance(x, int) for x in eos):
            raise ConfigError("config.json: eos_token_id must be an integer or a list of integers")
        top = "the configuration"
        return cls(vocab=_number(raw, "vocab", top, int), width=_number(raw, "width", top, int), layers=layers,
                   norm_eps=_number(raw.get("norm") or {}, "eps", "norm", float, 1e-6, required=False),
                   residual_mult=_number(raw, "residual_mult", top, float, 1.0, required=False),
                   streams=_number(raw, "streams", top, int, None, required=False), eos_token_ids=list(eos),
                   initializer_range=_number(raw, "initializer_range", top, float, 0.02, required=False))

    def to_dict(self) -> Dict[str, Any]:
        layers = []
        for l in self.layers:
            mixer = {k: copy.deepcopy(v) for k, v in l.mixer.items() if v is not None}
            if l.type == "attention":
                for key in ("softcap", "conv"):
                    if not mixer[key]:
                        del mixer[key]
            layers.append({"type": l.type, "mixer": mixer, "mlp": None if l.mlp is None else dict(l.mlp)})
        d = {"architecture": ARCHITECTURE, "vocab": self.vocab, "width": self.width, "layers": layers,
             "norm": {"eps": self.norm_eps}, "residual_mult": self.residual_mult,
             "initializer_range": self.initializer_range}
        if self.streams is not None:
            d["streams"] = self.streams
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
        need(self.streams is None or 1 <= self.streams <= MAX_STREAMS, f"streams must be between 1 and {MAX_STREAMS}")
        need(all(0 <= t < self.vocab for t in self.eos_token_ids), "eos_token_id names a token outside the vocabulary")
        for i, l in enumerate(self.layers):
            m, w = l.mixer, f"layers[{i}].mixer"
            need(l.type in MIXER_TYPES, f"layers[{i}].type {l.type!r} is not a mixer of this design")
            if l.type == "latent_attention":
                need(min(m["heads"], m["dim"], m["vdim"]) > 0 and 0 < m["kv_rank"] <= 1024,
                     f"{w}: heads, dim, vdim and kv_rank (at most 1024) must be positive")
                need(m["scale"] > 0, f"{w}.scale must be positive")
            elif l.type == "retention":
                need(min(m["heads"], m["vdim"]) > 0 and 0 < m["dim"] <= 256,
                     f"{w}: heads, vdim and dim (at most 256) must be positive")
                need(len(m["decay"]) == m["heads"] and all(0 <= d <= 1 for d in m["decay"]),
                     f"{w}.decay must hold a number from 0 to 1 per head")
                r = m["rot"]
                if r is not None:
                    need(r["base"] > 0, f"{w}.rot.base must be positive")
                    need(0 < r["dims"] <= m["dim"] and r["dims"] % 2 == 0,
                         f"{w}.rot.dims must be even, positive and at most {m['dim']}")
            else:
                need(min(m["heads"], m["kv_heads"]) > 0 and 0 < m["dim"] <= 256 and 0 < m["vdim"] <= 256,
                     f"{w}: heads, kv_heads, dim and vdim (at most 256) must be positive")
                need(m["heads"] % m["kv_heads"] == 0, f"{w}.heads must be a multiple of kv_heads")
                need(m["scale"] > 0 and m["softcap"] >= 0, f"{w}: scale must be positive, softcap not negative")
                need(0 <= m["conv"] <= 64, f"{w}.conv must be at most 64 taps")
                need(m["q_temp"] is None or m["q_temp"]["every"] > 0, f"{w}.q_temp.every must be positive")
                j = m["kv_from"]
                if j is not None:
                    need(0 <= j < i and self.layers[j].type == "attention" and self.layers[j].mixer["kv_from"] is None,
                         f"{w}.kv_from must name an earlier attention layer with keys of its own")
                    need(all(m[k] == self.layers[j].mixer[k] for k in ("kv_heads", "dim", "vdim")),
                         f"{w}.kv_from: kv_heads, dim and vdim must be those of layer {j}")
            if l.mlp is not None:
                need(l.mlp["kind"] == "dense" and l.mlp["ff"] > 0, f"layers[{i}].mlp: a known kind and a positive ff")

    def model_spec(self) -> ModelSpec:
        W, std, eps, s = self.width, self.initializer_range, self.norm_eps, self.streams
        norm = lambda name: PartSpec("rmsnorm", {"width": W, "eps": eps, "offset": 1.0}, rename={"weight": name})
        layers = []
        for i, l in enumerate(self.layers):
            p, m = f"l{i}.", l.mixer
            parts = {"mixer_norm": norm(p + "norm1")}
            names = {f"{n}.weight": n for n in ("q", "k", "v", "g", "o", "dkv", "uk", "uv")}
            common = {"hidden_size": W, "num_heads": m["heads"], "head_dim": m["dim"], "value_dim": m["vdim"], "init_std": std}
            if l.type == "attention":
                temp = m["q_temp"]
                parts["mixer"] = PartSpec(
                    "conv_attention",
                    {**common, "num_kv_heads": m["kv_heads"], "scale": m["scale"], "conv_taps": m["conv"],
                     "own_keys": m["kv_from"] is None, "softcap": m["softcap"],
                     "temperature": None if temp is None else (temp["coef"], temp["every"])},
                    prefix=p + "mix.", rename={**names, **{f"{n}.bias": f"{n}.b" for n in "qkv"}})
            elif l.type == "retention":
                r = m["rot"]
                parts["mixer"] = PartSpec(
                    "retention",
                    {**common, "decay": list(m["decay"]), "norm_eps": eps,
                     "position": None if r is None else PartSpec("rope", {"theta": r["base"], "rotary_dim": r["dims"]})},
                    prefix=p + "mix.", rename=names)
            else:
                parts["mixer"] = PartSpec(
                    "latent_attention", {**common, "rot_dim": 0, "kv_rank": m["kv_rank"], "scale": m["scale"], "norm_eps": eps},
                    prefix=p + "mix.", rename={**names, "dkv_norm.weight": "dkv.norm"})
            if l.mlp is not None:
                parts["feed_forward_norm"] = norm(p + "norm2")
                parts["feed_forward"] = PartSpec("dense_mlp", {"hidden_size": W, "width": l.mlp["ff"], "init_std": std},
                                                 prefix=p + "mlp.",
                                                 rename={f"{n}_proj.weight": n for n in ("gate", "up", "down")})
            sublayers = [("mixer", 1)] + ([("feed_forward", 2)] if l.mlp is not None else [])
            for name, q in sublayers:
                if s is not None:
                    parts[f"{name}_streams"] = PartSpec("hyper_connection", {"streams": s, "factor": self.residual_mult},
                                                        prefix=f"{p}hc{q}.")
                elif self.residual_mult != 1.0:
                    parts[f"{name}_gain"] = PartSpec("constant_gain", {"factor": self.residual_mult})
            layers.append(LayerSpec("hyper_prenorm" if s is not None else "prenorm_gained", parts))
        spec = ModelSpec(
            architecture=ARCHITECTURE, hidden_size=W, vocab_size=self.vocab, max_positions=0, layers=layers,
            schedule=[ScheduleEntry(i, l.mixer.get("kv_from")) for i, l in enumerate(self.layers)],
            embedding=PartSpec("token_embedding", {"vocab_size": self.vocab, "hidden_size": W, "init_std": std,
                                                   "norm_eps": eps, "norm_offset": 1.0, "streams": s},
                               rename={"weight": "embed", "norm.weight": "embed.norm"}),
            final_norm=norm("final.norm"), head=linear_head("head", self.vocab, W, std), init_std=std)
        spec.validate()
        return spec

    def copy(self) -> "SetopelConfig":
        return copy.deepcopy(self)


register_architecture(ARCHITECTURE, SetopelConfig)
