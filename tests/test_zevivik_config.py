"""The Zevivik design's configuration, tensor names and cache plan, what enters the stream when, how a bfloat16 run
arranges heads, and the plain implementation's mechanisms by hand (no GPU needed)."""
import copy
import json
import math

import pytest
import torch

import plain_zevivik as pz
import tiny_zevivik as tz
from inferx_amd.config import ConfigError, config_from_dict
from inferx_amd.parts import build_model, build_part

F = torch.float64


def load(raw):
    return config_from_dict(json.loads(json.dumps(raw)))


@pytest.mark.parametrize("name", sorted(tz.CONFIGS))
def test_round_trip_and_tensor_names(name):
    raw = tz.CONFIGS[name]
    cfg = load(raw)
    assert config_from_dict(cfg.to_dict()).to_dict() == cfg.to_dict()
    assert cfg.to_dict()["layers"] == raw["layers"] and cfg.to_dict().get("loop") == raw.get("loop")
    tensors = {n: tuple(p.shape) for n, p in build_model(cfg.model_spec()).expected_tensors().items()}
    W = raw["width"]
    want = {"embed": (raw["vocab"], W), "final.norm": (W,), "head": (raw["vocab"], W)}
    if "loop" in raw:
        want["loop.step"] = (raw["loop"]["times"], W)
    for i, l in enumerate(raw["layers"]):
        m, p, f = l["mixer"], f"l{i}.", l["mlp"]
        H, d, vd = m["heads"], m["dim"], m["vdim"]
        want.update({p + "norm1": (W,), p + "mix.q": (H * d, W), p + "mix.o": (W, H * vd)})
        if l["type"] == "attention":
            want.update({p + "mix.k": (m["kv_heads"] * d, W), p + "mix.v": (m["kv_heads"] * vd, W)})
        else:
            R = m["kv_rank"]
            want.update({p + "mix.dkv": (R, W), p + "mix.dkv.norm": (R,), p + "mix.uk": (H * d, R), p + "mix.uv": (H * vd, R),
                         p + "mix.g": (H, W)})
        if f is None:
            continue
        want[p + "norm2"] = (W,)
        sets = {"": f["ff"]} if f["kind"] == "dense" else {f"e{j}.": f["expert"]["ff"] for j in range(f["router"]["experts"])}
        if f["kind"] == "moe":
            want.update({p + "mlp.router": (f["router"]["experts"], W), p + "mlp.router.b": (f["router"]["experts"],)})
            if "shared" in f:
                sets["shared."] = f["shared"]["ff"]
        for at, ff in sets.items():
            want.update({f"{p}mlp.{at}gate": (ff, W), f"{p}mlp.{at}up": (ff, W), f"{p}mlp.{at}down": (W, ff)})
    assert tensors == want


def test_schedule_and_cache_plan():
    """Every pass of the loop has pages of its own; attention in chunks keeps a chunk, latent attention every token; the
    first pass enters with its vector alone, the others with the embedding's result too."""
    spec = load(tz.A).model_spec()
    assert [e.layer for e in spec.schedule] == [0, 1, 2, 1, 2, 1, 2, 3]
    entered = {i: (e.enter.params["index"], e.enter.params["embedding"]) for i, e in enumerate(spec.schedule) if e.enter}
    assert entered == {1: (0, False), 3: (1, True), 5: (2, True)}
    model = build_model(spec)
    assert model.shared_tensor_names() == ["loop.step"]
    plan = model.cache_plan()
    assert all(source is None for _, source in plan)
    needs = [keeps["mixer"][0] for keeps, _ in plan]
    assert [(n.window, n.chunk) for n in needs] == [(0, 16), (0, 0), (0, 7), (0, 0), (0, 7), (0, 0), (0, 7), (0, 0)]
    assert [(a.heads, a.width) for a in needs[1].arrays] == [(1, 40)] and [a.width for a in needs[0].arrays] == [20, 28]
    assert model.graph_safe()
    none = load(tz.C).model_spec()
    assert [e.layer for e in none.schedule] == [0, 1, 2] and all(e.enter is None for e in none.schedule)


@pytest.mark.parametrize("path,value,word", [
    (("layers", 0, "type"), "window", "not a mixer"), (("layers", 0, "mixer", "dim"), 300, "at most 256"),
    (("layers", 0, "mixer", "heads"), 5, "multiple of kv_heads"), (("layers", 0, "mixer", "mask"), {}, "size"),
    (("layers", 0, "mixer", "mask", "size"), -1, "mask.size"), (("layers", 0, "mixer", "rot", "dims"), 22, "rot.dims"),
    (("layers", 0, "mixer", "rot", "dims"), 5, "rot.dims"), (("layers", 0, "mixer", "rot", "base"), 0.0, "rot.base"),
    (("layers", 0, "mixer", "scale"), None, "scale"), (("layers", 1, "mixer", "kv_rank"), 2000, "kv_rank"),
    (("layers", 1, "mixer", "vdim"), 0, "vdim"), (("layers", 1, "mlp", "kind"), "sparse", "not known"),
    (("layers", 0, "mlp", "router", "top"), 7, "router"), (("layers", 0, "mlp", "expert", "limit"), 0.0, "expert"),
    (("layers", 0, "mlp", "shared"), {"ff": 8}, "limit"), (("loop", "stop"), 5, "loop"), (("loop", "start"), 3, "loop"),
    (("loop", "times"), 0, "times"), (("loop",), {"start": 0, "stop": 1}, "times"), (("vocab",), "many", "vocab"),
    (("norm", "eps"), 0.0, "eps"), (("layers",), [], "at least one layer"), (("eos_token_id",), 320, "outside the vocabulary"),
])
def test_impossible_values_are_named(path, value, word):
    raw = copy.deepcopy(tz.A)
    at = raw
    for key in path[:-1]:
        at = at[key]
    at[path[-1]] = value
    with pytest.raises(ConfigError, match=word):
        load(raw)


# ---- how a bfloat16 run arranges heads ------------------------------------------------------------------------------------
@pytest.mark.parametrize("d,vd,rot,size", [(20, 28, 12, 32), (24, 12, 24, 32), (32, 32, 16, 32), (11, 6, 10, 32), (48, 80, 48, 96),
                                           (64, 64, 64, 64), (13, 13, 0, 32), (200, 160, 100, 224), (8, 8, 2, 32)])
def test_arranged_heads_give_the_same_scores_and_results(d, vd, rot, size):
    """Rows of the projections put into place, then every head rotated whole by the widened table: scores and values are
    those of the plain heads with a part rotated."""
    from inferx_amd.config import PartSpec
    H, G, W, T, base = 4, 2, 10, 5, 30.0
    position = PartSpec("rope", {"theta": base, "rotary_dim": rot}) if rot else None
    part = build_part("mixer", PartSpec("attention", {"hidden_size": W, "num_heads": H, "num_kv_heads": G, "head_dim": d,
                                                      "value_dim": vd, "qkv_bias": False, "position": position, "pad": True}))
    g = torch.Generator().manual_seed(3)
    shapes = {"q": (H * d, W), "k": (G * d, W), "v": (G * vd, W), "o": (W, H * vd)}
    w = {f"{n}_proj.weight": torch.randn(s, generator=g, dtype=F) for n, s in shapes.items()}
    put = part._arrange_heads(w)
    assert part.head_dim == part.value_dim == size and part.rotated == ((0, size) if rot else (0, d)) and not part.general
    x, pos = torch.randn(T, W, generator=g, dtype=F), torch.arange(T) + 7
    turn = (lambda t: pz.rotate_first(t, pos, rot, base)) if rot else (lambda t: t)
    want_q, want_k = (turn((x @ w[f"{n}_proj.weight"].T).view(T, -1, d)) for n in "qk")
    if rot:
        f = part.position.frequencies().double()
        assert f.shape == (size // 2,) and int((f != 0).sum()) == rot // 2

    def whole(t):
        if not rot:
            return t
        a, u, v = (pos.double()[:, None] * f[None, :])[:, None], t[..., :size // 2], t[..., size // 2:]
        return torch.cat([u * a.cos() - v * a.sin(), v * a.cos() + u * a.sin()], dim=-1)
    got_q, got_k = (whole((x @ put[f"{n}_proj.weight"].T).view(T, -1, size)) for n in "qk")
    for h in range(H):
        a, b = want_q[:, h] @ want_k[:, h // 2].T, got_q[:, h] @ got_k[:, h // 2].T
        assert torch.allclose(a, b, atol=1e-5 * float(a.abs().max()))
    v = (x @ put["v_proj.weight"].T).view(T, G, size).repeat_interleave(2, dim=1).reshape(T, -1)
    plain_v = (x @ w["v_proj.weight"].T).view(T, G, vd).repeat_interleave(2, dim=1).reshape(T, -1)
    assert torch.allclose(v @ put["o_proj.weight"].T, plain_v @ w["o_proj.weight"].T)


# ---- the plain implementation by hand ---------------------------------------------------------------------------------------
def test_chunks_are_counted_from_the_start():
    seen = pz.visible(torch.arange(8), 3)
    assert [torch.nonzero(r).flatten().tolist() for r in seen] == [[0], [0, 1], [0, 1, 2], [3], [3, 4], [3, 4, 5], [6], [6, 7]]
    assert torch.equal(pz.visible(torch.arange(4), 1), torch.eye(4, dtype=torch.bool))
    assert torch.equal(pz.visible(torch.arange(4)), torch.ones(4, 4, dtype=torch.bool).tril())


def test_activations_and_router_by_hand():
    z = torch.tensor([-3.0, -0.5, 0.0, 0.7, 4.0], dtype=F)
    assert torch.allclose(pz.gelu_tanh(z), torch.nn.functional.gelu(z, approximate="tanh"))
    w = {"gate": torch.tensor([[1.0]], dtype=F), "up": torch.tensor([[2.0]], dtype=F), "down": torch.tensor([[1.0]], dtype=F)}
    sig = lambda t: 1 / (1 + math.exp(-1.702 * t))
    got = pz.expert(torch.tensor([[0.4], [3.0], [-3.0]], dtype=F), w, 1.5).flatten().tolist()
    want = [0.4 * sig(0.4) * 1.8, 1.5 * sig(1.5) * 2.5, -3.0 * sig(-3.0) * (-1.5 + 1.0)]
    assert all(abs(a - b) < 1e-12 for a, b in zip(got, want))
    wr = {"router": torch.tensor([[1.0], [0.0], [-1.0]], dtype=F), "router.b": torch.tensor([0.0, 2.0, 1.5], dtype=F)}
    idx, p = pz.route(torch.tensor([[0.2], [-4.0]], dtype=F), wr, {"router": {"experts": 3, "top": 2}})
    assert idx.tolist() == [[1, 2], [2, 1]]  # logits (0.2, 2, 1.3) and (-4, 2, 5.5)
    assert torch.allclose(p[:, 0], 1 / (1 + torch.exp(torch.tensor([-0.7, -3.5], dtype=F))))


def test_run_order_and_what_enters():
    assert pz.run_order(tz.A) == [(0, None), (1, 0), (2, 0), (1, 1), (2, 1), (1, 2), (2, 2), (3, None)]
    # a model whose layers leave the stream alone: what is left is the embedding three times and every pass's vector
    raw = {"vocab": 2, "width": 2, "norm": {"eps": 1e-6}, "embedding": {"scale": 2.0}, "loop": {"start": 0, "stop": 1, "times": 3},
           "layers": [{"type": "latent_attention", "mixer": {"heads": 1, "dim": 1, "vdim": 1, "kv_rank": 1, "scale": 1.0}}]}
    w = {"embed": torch.tensor([[1.0, 2.0], [3.0, 5.0]]), "loop.step": torch.tensor([[10.0, 0.0], [0.0, 100.0], [1.0, 1.0]]),
         "head": torch.eye(2), "final.norm": torch.ones(2), "l0.norm1": torch.ones(2)}
    w.update({f"l0.mix.{n}": torch.zeros(s) for n, s in (("q", (1, 2)), ("dkv", (1, 2)), ("dkv.norm", (1,)), ("uk", (1, 1)),
                                                         ("uv", (1, 1)), ("g", (1, 2)), ("o", (2, 1)))})
    trace = []
    pz.forward(raw, w, [1], trace=trace)
    assert [t[0].tolist() for t in trace] == [[16.0, 10.0], [22.0, 120.0], [29.0, 131.0]]


def test_a_planted_mistake_shows(tmp_path):
    """The tiny models' random weights let every mechanism show in the logits: getting one wrong in the plain
    implementation changes them by far more than rounding."""
    _, w = tz.read_folder(tz.make_folder(tz.A, 3, str(tmp_path), "float32"))
    toks = tz.random_tokens(40, tz.A["vocab"], 5)
    right = pz.forward(tz.A, w, toks)
    scale = float(right.abs().max())

    def changed(edit):
        raw, ww = copy.deepcopy(tz.A), dict(w)
        edit(raw, ww)
        return float((pz.forward(raw, ww, toks) - right).abs().max()) / scale

    mixer = lambda r, i: r["layers"][i]["mixer"]
    mlp = lambda r, i: r["layers"][i]["mlp"]
    for edit in (lambda r, ww: mixer(r, 0)["mask"].update(size=15), lambda r, ww: mixer(r, 0)["mask"].update(size=17),
                 lambda r, ww: mixer(r, 2).pop("mask"), lambda r, ww: mixer(r, 0)["rot"].update(dims=20),
                 lambda r, ww: mixer(r, 0)["rot"].update(base=120.0), lambda r, ww: mixer(r, 0).pop("rot"),
                 lambda r, ww: r["embedding"].update(scale=1.75), lambda r, ww: r["loop"].update(times=2),
                 lambda r, ww: ww.update({"loop.step": w["loop.step"].flip(0)}),
                 lambda r, ww: ww.update({"l1.mix.g": w["l1.mix.g"] * 0}),
                 lambda r, ww: ww.update({"l1.mix.g": w["l1.mix.g"].flip(0)}),
                 lambda r, ww: ww.update({"l0.norm2": w["l0.norm1"]}), lambda r, ww: mlp(r, 0)["shared"].update(limit=0.7),
                 lambda r, ww: mlp(r, 0)["expert"].update(limit=1.3), lambda r, ww: mlp(r, 0).pop("shared"),
                 lambda r, ww: ww.update({"l0.mlp.router.b": w["l0.mlp.router.b"] * 0})):
        assert changed(edit) > 1e-3
