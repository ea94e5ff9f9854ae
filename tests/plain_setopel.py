"""A plain, slow implementation of the Setopel design: float64 on the CPU, one function per mechanism, a whole sequence
at a time, the recurrence token by token.  It shares no code with the engine; the tests compare the two.

    embedding  : x = norm0(E[id]);  norm0(x) = x / sqrt(mean(x^2) + eps) * (1 + w)
    streams    : x_1 .. x_s = x;  per sublayer f with numbers a [s], b [s], M [s, s]:
                 y = f(norm0(sum_i a_i x_i));   x_j <- sum_i M[i, j] x_i + m b_j y       (all from the old ones)
                 at the end x = sum_j x_j.  Without streams: x <- x + m f(norm0(x))
    attention  : q, k, v = conv(W x + b);  q *= 1 + coef ln(floor((p + 1) / every) + 1)
                 s_j = cap tanh(q . k_j scale / cap), j <= i;  p_j = exp(s_j) / (1 + sum exp(s))
                 y = Wo (concat(p v) * sigmoid(Wg x));  a layer may take another one's k and v
    retention  : q, k rotated (halves, the first `dims` numbers), k * dim^-1/2;  S <- decay_h S + k v^T;  o = S^T q
                 y = Wo (o / rms(o) * silu(Wg x))
    latent     : c = Wdkv x / rms * wn;  k_h = Wuk_h c, v_h = Wuv_h c;  p = softmax(q . k scale);  y = Wo concat(p v)
    dense      : Wdown (silu(Wgate x) * Wup x)
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


def rms_unit(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def norm0(x, w, eps):
    return rms_unit(x, eps) * (1.0 + w)


def silu(x):
    return x * torch.sigmoid(x)


def rotate_first(x, positions, dims, base):
    """x [T, heads, d]: of the first `dims` numbers of every head, i and i + dims / 2 turned by p base^(-2 i / dims)."""
    half = dims // 2
    ang = positions.to(F)[:, None] * float(base) ** (-2.0 * torch.arange(half, dtype=F) / dims)[None, :]
    cos, sin = torch.cos(ang)[:, None, :], torch.sin(ang)[:, None, :]
    u, v = x[..., :half], x[..., half:dims]
    return torch.cat([u * cos - v * sin, v * cos + u * sin, x[..., dims:]], dim=-1)


def short_conv(u, w):
    """u [T, C], w [C, taps]: y[t] = sum_j w[:, j] u[t - taps + 1 + j], zeros before the start."""
    T, taps = u.shape[0], w.shape[1]
    padded = torch.cat([torch.zeros(taps - 1, u.shape[1], dtype=F), u])
    return sum(padded[j:j + T] * w[:, j] for j in range(taps))


def temperature(positions, coef, every):
    return 1.0 + coef * torch.log(torch.floor((positions.to(F) + 1.0) / every) + 1.0)


def project(x, w, name):
    u = _S(x @ w[name].T + w[name + ".b"])
    return short_conv(u, w[name + ".conv"]) if name + ".conv" in w else u


def capped(score, cap):
    return score if not cap else cap * torch.tanh(score / cap)


def softmax_one(score):
    """Over the last dimension, with one added to the denominator (-inf: not visible)."""
    top = torch.clamp(score.max(-1, keepdim=True).values, min=0.0)
    e = torch.exp(score - top)
    return e / (e.sum(-1, keepdim=True) + torch.exp(-top))


def causal(T):
    return torch.ones(T, T, dtype=torch.bool).tril()


def attention(x, w, m, positions, shared=None):
    """(result, (k, v) as a later layer may use them).  `shared`: another layer's (k, v)."""
    T, H, G, d, vd = x.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = project(x, w, "q").view(T, H, d)
    if m.get("q_temp"):
        q = q * temperature(positions, m["q_temp"]["coef"], m["q_temp"]["every"])[:, None, None]
    q = _S(q)
    if shared is None:
        shared = _S(project(x, w, "k")).view(T, G, d), _S(project(x, w, "v")).view(T, G, vd)
    k, v = (t.repeat_interleave(H // G, dim=1) for t in shared)
    score = capped(torch.einsum("ihd,jhd->hij", q, k) * m["scale"], m.get("softcap"))
    p = softmax_one(score.masked_fill(~causal(T)[None], -math.inf))
    o = torch.einsum("hij,jhv->ihv", p, v).reshape(T, H * vd)
    return _S(_S(o) * torch.sigmoid(_S(x @ w["g"].T))) @ w["o"].T, shared


def retention(x, w, m, eps, positions):
    T, H, d, vd = x.shape[0], m["heads"], m["dim"], m["vdim"]
    q, k = _S(x @ w["q"].T).view(T, H, d), _S(x @ w["k"].T).view(T, H, d)
    v = _S(x @ w["v"].T).view(T, H, vd)
    rot = m.get("rot")
    if rot:
        q, k = (rotate_first(t, positions, rot["dims"], rot["base"]) for t in (q, k))
    k = k * d ** -0.5
    decay = torch.tensor(m["decay"], dtype=F)[:, None, None]
    S = torch.zeros(H, d, vd, dtype=F)
    o = torch.zeros(T, H, vd, dtype=F)
    for t in range(T):
        S = decay * S + k[t][:, :, None] * v[t][:, None, :]
        o[t] = torch.einsum("hdv,hd->hv", S, q[t])
    y = _S(rms_unit(o, eps).reshape(T, H * vd) * silu(_S(x @ w["g"].T)))
    return y @ w["o"].T


def latent_attention(x, w, m, eps):
    T, H, d, vd = x.shape[0], m["heads"], m["dim"], m["vdim"]
    q = _S(x @ w["q"].T).view(T, H, d)
    c = _S(rms_unit(_S(x @ w["dkv"].T), eps) * w["dkv.norm"])
    k, v = _S(c @ w["uk"].T).view(T, H, d), _S(c @ w["uv"].T).view(T, H, vd)
    score = torch.einsum("ihd,jhd->hij", q, k) * m["scale"]
    p = torch.softmax(score.masked_fill(~causal(T)[None], -math.inf), dim=-1)
    return _S(torch.einsum("hij,jhv->ihv", p, v).reshape(T, H * vd)) @ w["o"].T


def dense(x, w):
    return _S(silu(_S(x @ w["gate"].T)) * _S(x @ w["up"].T)) @ w["down"].T


def enter_streams(xs, a):
    """xs [T, s, W] -> sum_i a_i x_i."""
    return (xs * a[None, :, None]).sum(1)


def leave_streams(xs, y, b, M, m):
    """x_j <- sum_i M[i, j] x_i + m b_j y."""
    return torch.einsum("tiw,ij->tjw", xs, M) + m * b[None, :, None] * y[:, None, :]


def sub(w, prefix):
    return {k[len(prefix):]: v for k, v in w.items() if k.startswith(prefix)}


def forward(cfg, weights, tokens, store=exact, trace=None):
    """Logits [T, vocab] of one sequence from its start.  `weights`: name -> tensor (any float type).  `store`: what
    keeping an activation does (`bfloat16` for a 16-bit engine).  `trace`: a list that receives the stream (the sum of
    the streams) after every layer."""
    global _S
    _S = store
    try:
        w = {k: v.to(F) for k, v in weights.items()}
        eps, mult, s = float(cfg["norm"]["eps"]), float(cfg.get("residual_mult", 1.0)), cfg.get("streams")
        positions = torch.arange(len(tokens))
        x = norm0(w["embed"][torch.as_tensor(tokens)], w["embed.norm"], eps)
        xs = x[:, None, :].repeat(1, s or 1, 1)

        def sublayer(xs, lw, q, f):
            """One sublayer around f, with the norm before it."""
            if not s:
                return xs + mult * _S(f(_S(norm0(xs[:, 0], lw[f"norm{q}"], eps))))[:, None, :]
            u = enter_streams(xs, lw[f"hc{q}.in"])
            y = _S(f(_S(norm0(u, lw[f"norm{q}"], eps))))
            return leave_streams(xs, y, lw[f"hc{q}.out"], lw[f"hc{q}.mix"], mult)

        kept = {}
        for i, layer in enumerate(cfg["layers"]):
            lw, m = sub(w, f"l{i}."), layer["mixer"]
            mw = sub(lw, "mix.")

            def mixer(h, i=i, m=m, mw=mw, kind=layer["type"]):
                if kind == "retention":
                    return retention(h, mw, m, eps, positions)
                if kind == "latent_attention":
                    return latent_attention(h, mw, m, eps)
                src = m.get("kv_from")
                y, kept[i] = attention(h, mw, m, positions, None if src is None else kept[src])
                return y

            xs = sublayer(xs, lw, 1, mixer)
            if layer.get("mlp"):
                xs = sublayer(xs, lw, 2, lambda h: dense(h, sub(lw, "mlp.")))
            if trace is not None:
                trace.append(xs.sum(1))
        return _S(norm0(xs.sum(1), w["final.norm"], eps)) @ w["head"].T
    finally:
        _S = exact
