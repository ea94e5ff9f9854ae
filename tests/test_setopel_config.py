"""The Setopel design's configuration, tensor names and cache plan, and the plain implementation's mechanisms by hand
(no GPU needed)."""
import copy
import json
import math

import pytest
import torch

import plain_setopel as ps
import tiny_setopel as ts
from inferx_amd.config import ConfigError, config_from_dict
from inferx_amd.parts import build_model

F = torch.float64


def load(raw):
    return config_from_dict(json.loads(json.dumps(raw)))


@pytest.mark.parametrize("name", sorted(ts.CONFIGS))
def test_round_trip_and_tensor_names(name):
    raw = ts.CONFIGS[name]
    cfg = load(raw)
    assert config_from_dict(cfg.to_dict()).to_dict() == cfg.to_dict()
    tensors = {n: tuple(p.shape) for n, p in build_model(cfg.model_spec()).expected_tensors().items()}
    W, s = raw["width"], raw.get("streams")
    want = {"embed": (raw["vocab"], W), "embed.norm": (W,), "final.norm": (W,), "head": (raw["vocab"], W)}
    for i, l in enumerate(raw["layers"]):
        m, p = l["mixer"], f"l{i}."
        H, d, vd = m["heads"], m["dim"], m["vdim"]
        rows = {"q": H * d, "o": None}
        if l["type"] == "attention":
            rows["g"] = H * vd
            own = ["q"] + ([] if "kv_from" in m else ["k", "v"])
            rows.update({} if "kv_from" in m else {"k": m["kv_heads"] * d, "v": m["kv_heads"] * vd})
            for n in own:
                want[f"{p}mix.{n}.b"] = (rows[n],)
                if m.get("conv"):
                    want[f"{p}mix.{n}.conv"] = (rows[n], m["conv"])
        elif l["type"] == "retention":
            rows.update({"k": H * d, "v": H * vd, "g": H * vd})
        else:
            rows["dkv"] = m["kv_rank"]
            want.update({f"{p}mix.dkv.norm": (m["kv_rank"],), f"{p}mix.uk": (H * d, m["kv_rank"]),
                         f"{p}mix.uv": (H * vd, m["kv_rank"])})
        for n, r in rows.items():
            want[f"{p}mix.{n}"] = (W, H * vd) if n == "o" else (r, W)
        want[p + "norm1"] = (W,)
        if l["mlp"]:
            want.update({p + "norm2": (W,), p + "mlp.gate": (l["mlp"]["ff"], W), p + "mlp.up": (l["mlp"]["ff"], W),
                         p + "mlp.down": (W, l["mlp"]["ff"])})
        for q in (1, 2) if l["mlp"] else (1,):
            if s is not None:
                want.update({f"{p}hc{q}.in": (s,), f"{p}hc{q}.out": (s,), f"{p}hc{q}.mix": (s, s)})
    assert tensors == want


def test_cache_plan():
    """Layers that read another one's keys own no pages; the convolutions' and the retention layers' state is per request."""
    model = build_model(load(ts.A).model_spec())
    plan = model.cache_plan()
    assert [source for _, source in plan] == [None, None, None, 0, None]
    (need, state), = [k["mixer"] for k, _ in plan[:1]]
    assert need.window == 0 and [a.width for a in need.arrays] == [20, 28] and state.shape == (3 * (6 * 20 + 2 * 20 + 2 * 28),)
    need3, state3 = plan[3][0]["mixer"]
    assert need3 == need and state3.shape == (1 * 4 * 20,)  # one earlier input of the queries alone
    assert plan[1][0]["mixer"] == (None, plan[1][0]["mixer"][1]) and plan[1][0]["mixer"][1].shape == (3 * 12 * 20,)
    latent, none = plan[2][0]["mixer"]
    assert none is None and [(a.heads, a.width) for a in latent.arrays] == [(1, 40)]


@pytest.mark.parametrize("path,value,word", [
    (("layers", 0, "type"), "window", "not a mixer"), (("layers", 0, "mixer", "dim"), 300, "at most 256"),
    (("layers", 0, "mixer", "heads"), 5, "multiple of kv_heads"), (("layers", 0, "mixer", "softcap"), -1.0, "softcap"),
    (("layers", 0, "mixer", "conv"), 65, "64 taps"), (("layers", 0, "mixer", "q_temp"), {"coef": 0.1, "every": 0}, "every"),
    (("layers", 0, "mixer", "q_temp"), {"every": 4}, "coef"), (("layers", 3, "mixer", "kv_from"), 1, "kv_from"),
    (("layers", 3, "mixer", "kv_from"), 4, "kv_from"), (("layers", 3, "mixer", "vdim"), 24, "those of layer 0"),
    (("layers", 1, "mixer", "decay"), [0.9, 0.9], "per head"), (("layers", 1, "mixer", "decay"), [0.9, 0.9, 1.5], "from 0 to 1"),
    (("layers", 1, "mixer", "decay"), "slow", "list of numbers"), (("layers", 1, "mixer", "rot", "dims"), 14, "rot.dims"),
    (("layers", 2, "mixer", "kv_rank"), 2000, "kv_rank"), (("layers", 2, "mlp", "kind"), "moe", "not known"),
    (("streams",), 33, "streams"), (("streams",), 0, "streams"), (("vocab",), "many", "vocab"), (("norm", "eps"), 0.0, "eps"),
    (("layers",), [], "at least one layer"), (("eos_token_id",), 320, "outside the vocabulary"),
])
def test_impossible_values_are_named(path, value, word):
    raw = copy.deepcopy(ts.A)
    at = raw
    for key in path[:-1]:
        at = at[key]
    at[path[-1]] = value
    with pytest.raises(ConfigError, match=word):
        load(raw)


# ---- the plain implementation by hand ------------------------------------------------------------------------------------
def test_temperature_steps_up_when_the_count_of_tokens_reaches_a_multiple():
    pos = torch.tensor([0, 2, 3, 6, 7, 11])
    got = ps.temperature(pos, 0.5, 4)   # (p + 1) // 4 = 0, 0, 1, 1, 2, 3
    want = [1 + 0.5 * math.log(k) for k in (1, 1, 2, 2, 3, 4)]
    assert torch.allclose(got, torch.tensor(want, dtype=F), atol=1e-12)
    assert torch.allclose(ps.temperature(torch.arange(3), 1.0, 1), 1 + torch.log(torch.arange(2, 5).double()))


def test_softmax_with_one_in_the_denominator():
    s = torch.tensor([[math.log(2.0), -math.inf, math.log(5.0)], [-200.0, -201.0, -math.inf], [500.0, 499.0, -math.inf]], dtype=F)
    p = ps.softmax_one(s)
    assert torch.allclose(p[0], torch.tensor([2 / 8, 0, 5 / 8], dtype=F))
    assert float(p[1].sum()) < 1e-80 and abs(float(p[2].sum()) - 1.0) < 1e-12
    assert torch.allclose(ps.capped(torch.tensor([1e3, -1e3, 0.1], dtype=F), 2.0),
                          torch.tensor([2.0, -2.0, 2 * math.tanh(0.05)], dtype=F))


def test_streams_by_hand():
    xs = torch.tensor([[[1.0, 2.0], [10.0, 20.0]]], dtype=F)
    assert torch.equal(ps.enter_streams(xs, torch.tensor([2.0, 0.5], dtype=F)), torch.tensor([[7.0, 14.0]], dtype=F))
    M = torch.tensor([[1.0, 3.0], [0.0, 2.0]], dtype=F)  # [from, to]
    got = ps.leave_streams(xs, torch.tensor([[100.0, 200.0]], dtype=F), torch.tensor([1.0, -1.0], dtype=F), M, 0.1)
    assert torch.allclose(got, torch.tensor([[[11.0, 22.0], [13.0, 26.0]]], dtype=F))


def test_convolution_and_retention_by_hand():
    u = torch.tensor([[1.0], [2.0], [4.0]], dtype=F)
    assert torch.equal(ps.short_conv(u, torch.tensor([[10.0, 1.0]], dtype=F)), torch.tensor([[1.0], [12.0], [24.0]], dtype=F))
    # one head of one number: the state is a decayed sum of k v, the result its sign (a head's own norm), gated
    w = {n: torch.tensor([[float(x)]], dtype=F) for n, x in (("q", 1), ("k", 2), ("v", 3), ("g", 1), ("o", 1))}
    m = {"heads": 1, "dim": 1, "vdim": 1, "decay": [0.5]}
    y = ps.retention(torch.tensor([[1.0], [-1.0]], dtype=F), w, m, 0.0, torch.arange(2))
    silu = lambda z: z / (1 + math.exp(-z))
    # token 0: S = 6, o = 6 -> 1; token 1: S = 9, o = -9 -> -1
    assert torch.allclose(y, torch.tensor([[silu(1.0)], [-silu(-1.0)]], dtype=F))


def test_norm_weights_are_stored_around_zero():
    x = torch.tensor([[3.0, 4.0]], dtype=F)
    assert torch.allclose(ps.norm0(x, torch.tensor([0.0, 1.0], dtype=F), 0.0), torch.tensor([[3.0, 8.0]], dtype=F) / math.sqrt(12.5))


def test_a_planted_mistake_shows(tmp_path):
    """The tiny models' random weights let every mechanism show in the logits: leaving one out of the plain
    implementation changes them by far more than rounding."""
    _, w = ts.read_folder(ts.make_folder(ts.A, 3, str(tmp_path), "float32"))
    toks = ts.random_tokens(40, ts.A["vocab"], 5)
    right = ps.forward(ts.A, w, toks)
    scale = float(right.abs().max())

    def changed(edit):
        raw, ww = copy.deepcopy(ts.A), dict(w)
        edit(raw, ww)
        return float((ps.forward(raw, ww, toks) - right).abs().max()) / scale

    for edit in (lambda r, ww: r["layers"][0]["mixer"].pop("q_temp"), lambda r, ww: r["layers"][0]["mixer"].pop("softcap"),
                 lambda r, ww: r["layers"][3]["mixer"]["q_temp"].update(every=6), lambda r, ww: r.update(residual_mult=0.61),
                 lambda r, ww: r["layers"][1]["mixer"].pop("rot"), lambda r, ww: r["layers"][1]["mixer"]["rot"].update(dims=6),
                 lambda r, ww: ww.update({"l2.hc1.mix": w["l2.hc1.mix"].T}),
                 lambda r, ww: ww.update({"l0.hc2.in": w["l0.hc2.in"].flip(0)}),
                 lambda r, ww: ww.update({"embed.norm": w["embed.norm"] * 0}),
                 lambda r, ww: ww.update({"l0.mix.k.conv": w["l0.mix.k.conv"].flip(1)})):
        assert changed(edit) > 1e-3
