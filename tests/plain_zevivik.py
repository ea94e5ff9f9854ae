"""A plain, slow implementation of the Zevivik design: float64 on the CPU, one function per mechanism, a whole sequence at
a time.  It shares no code with the engine; the tests compare the two.

    embedding  : x0 = scale * E[id]
    layer      : x <- x + (mixer(norm1(x)) + ff(norm2(x)))       both read the same x;  norm(x) = x / sqrt(mean(x^2) + eps) * w
    loop       : layers [start, stop) run `times` times with the same tensors; before pass t: x <- x + x0 (t > 0), x <- x + step_t
    attention  : q, k rotated (halves, the first `dims` numbers of a head);  s_ij = q_i . k_j scale for j <= i in i's chunk of
                 `size` positions (chunks counted from position 0);  y = Wo concat(softmax(s) v)
    latent     : c = N(Wdkv x) wn;  k_h = Wuk_h c, v_h = Wuv_h c;  p = softmax(q . k scale), j <= i
                 y = Wo concat_h(sigmoid(Wg x)_h sum_j p_j v_j)
    dense      : Wdown (gelu_tanh(Wgate x) * Wup x)
    experts    : z = Wr x + b;  the `top` largest, weights softmax over them;  sum of weight * expert(x), plus shared(x)
    expert     : g = min(Wgate x, L), u = clamp(Wup x, -L, L);  Wdown (g sigmoid(1.702 g) (u + 1))
"""
import math

import torch

F = torch.float64


def exact(x):
    return x


def bfloat16(x):
    """x rounded to bfloat16 (nearest even) and back: what keeping an activation in 16 bits does to it."""
    return x.to(torch.bfloat16).to(F)


def jittered(seed):
    """Another sample of what 16-bit storage does: x moved at random by up to one part in 512, then rounded."""
    g = torch.Generator().manual_seed(seed)

    def store(x):
        return bfloat16(x * (1.0 + (torch.rand(x.shape, generator=g, dtype=F) * 2.0 - 1.0) / 512.0))
    return store


_S = exact  # what keeping an activation between two operations does to it (`forward(store=...)` sets it)


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def rotate_first(x, positions, dims, base):
    """x [T, heads, d]: of the first `dims` numbers of every head, i and i + dims / 2 turned by p base^(-2 i / dims)."""
    half = dims // 2
    ang = positions.to(F)[:, None] * float(base) ** (-2.0 * torch.arange(half, dtype=F) / dims)[None, :]
    cos, sin = torch.cos(ang)[:, None, :], torch.sin(ang)[:, None, :]
    u, v = x[..., :half], x[..., half:dims]
    return torch.cat([u * cos - v * sin, v * cos + u * sin, x[..., dims:]], dim=-1)


def visible(positions, chunk=0):
    """[i, j]: whether the query at position i reads the key at position j."""
    i, j = positions[:, None], positions[None, :]
    seen = j <= i
    if chunk:
        seen = seen & (torch.div(i, chunk, rounding_mode="floor") == torch.div(j, chunk, rounding_mode="floor"))
    return seen


def attend(q, k, v, scale, seen):
    """q, k [T, H, d], v [T, H, vd] -> [T, H, vd]."""
    score = torch.einsum("ihd,jhd->hij", q, k) * scale
    return torch.einsum("hij,jhv->ihv", torch.softmax(score.masked_fill(~seen[None], -math.inf), dim=-1), v)


def attention(x, w, m, positions):
    T, H, G, d, vd = x.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k = _S(x @ w["q"].T).view(T, H, d), _S(x @ w["k"].T).view(T, G, d)
    v = _S(x @ w["v"].T).view(T, G, vd)
    rot = m.get("rot")
    if rot:
        q, k = (_S(rotate_first(t, positions, rot["dims"], rot["base"])) for t in (q, k))
    k, v = (t.repeat_interleave(H // G, dim=1) for t in (k, v))
    o = attend(q, k, v, m["scale"], visible(positions, (m.get("mask") or {}).get("size", 0)))
    return _S(o).reshape(T, H * vd) @ w["o"].T


def latent_attention(x, w, m, eps, positions):
    T, H, d, vd = x.shape[0], m["heads"], m["dim"], m["vdim"]
    q = _S(x @ w["q"].T).view(T, H, d)
    c = _S(rms_norm(_S(x @ w["dkv"].T), w["dkv.norm"], eps))
    k, v = _S(c @ w["uk"].T).view(T, H, d), _S(c @ w["uv"].T).view(T, H, vd)
    o = attend(q, k, v, m["scale"], visible(positions))
    gate = torch.sigmoid(_S(x @ w["g"].T))                                          # [T, H]
    return _S(o * gate[:, :, None]).reshape(T, H * vd) @ w["o"].T


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def dense(x, w):
    return _S(gelu_tanh(_S(x @ w["gate"].T)) * _S(x @ w["up"].T)) @ w["down"].T


def expert(x, w, limit):
    g, u = torch.clamp(_S(x @ w["gate"].T), max=limit), torch.clamp(_S(x @ w["up"].T), -limit, limit)
    return _S(g * torch.sigmoid(1.702 * g) * (u + 1.0)) @ w["down"].T


def router_logits(x, w):
    return x @ w["router"].T + w["router.b"]


def route(x, w, f):
    """(experts [T, top], weights [T, top]) of every token."""
    val, idx = torch.topk(router_logits(x, w), f["router"]["top"], dim=-1)
    return idx, torch.softmax(val, dim=-1)


def experts(x, w, f, chosen=None):
    """`chosen` [T, top]: experts from outside instead of the router's choice."""
    idx, weight = route(x, w, f)
    if chosen is not None:
        idx = chosen
        weight = torch.softmax(torch.gather(router_logits(x, w), 1, idx), dim=-1)
    out = torch.zeros(x.shape[0], w["e0.down"].shape[0], dtype=F)
    for e in range(f["router"]["experts"]):
        t, s = torch.nonzero(idx == e, as_tuple=True)
        if len(t):
            out[t] += weight[t, s][:, None] * _S(expert(x[t], sub(w, f"e{e}."), f["expert"]["limit"]))
    if f.get("shared"):
        out = out + _S(expert(x, sub(w, "shared."), f["shared"]["limit"]))
    return out


def sub(w, prefix):
    return {k[len(prefix):]: v for k, v in w.items() if k.startswith(prefix)}


def run_order(cfg):
    """[(layer, pass)]: the layers as they run; pass is None outside the loop."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    a, b = loop["start"], loop["stop"]
    return [(i, None) for i in range(a)] + [(i, t) for t in range(loop["times"]) for i in range(a, b)] + [(i, None) for i in range(b, n)]


def forward(cfg, weights, tokens, store=exact, trace=None, experts_of=None, chosen=None, scores=None):
    """Logits [T, vocab] of one sequence from its start.  `weights`: name -> tensor (any float type).  `store`: what
    keeping an activation does (`bfloat16` for a 16-bit engine).  `trace`: a list that receives the stream after every
    layer run.  `experts_of`: per (layer run with experts) the experts [T, top] to use instead of the router's choice;
    `chosen` / `scores`: lists that receive the router's own choice and logits per such run."""
    global _S
    _S = store
    try:
        w = {k: v.to(F) for k, v in weights.items()}
        eps = float(cfg["norm"]["eps"])
        positions = torch.arange(len(tokens))
        x0 = w["embed"][torch.as_tensor(tokens)] * float(cfg["embedding"]["scale"])
        x = x0.clone()
        loop, run = cfg.get("loop"), 0
        for i, t in run_order(cfg):
            layer, lw = cfg["layers"][i], sub(w, f"l{i}.")
            if t is not None and i == loop["start"]:
                x = x + (x0 if t > 0 else 0.0) + w["loop.step"][t]
            h = _S(rms_norm(x, lw["norm1"], eps))
            mw, m = sub(lw, "mix."), layer["mixer"]
            total = (_S(attention(h, mw, m, positions)) if layer["type"] == "attention"
                     else _S(latent_attention(h, mw, m, eps, positions)))
            f = layer.get("mlp")
            if f:
                h = _S(rms_norm(x, lw["norm2"], eps))
                fw = sub(lw, "mlp.")
                if f["kind"] == "dense":
                    total = total + _S(dense(h, fw))
                else:
                    if chosen is not None:
                        chosen.append(route(h, fw, f)[0])
                    if scores is not None:
                        scores.append(router_logits(h, fw))
                    total = total + experts(h, fw, f, None if experts_of is None else experts_of[run])
                    run += 1
            x = x + total
            if trace is not None:
                trace.append(x.clone())
        return _S(rms_norm(x, w["final.norm"], eps)) @ w["head"].T
    finally:
        _S = exact
