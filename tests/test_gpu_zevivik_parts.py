"""Zevivik's mechanisms one by one, each kernel against a slow float64 function written from the equations (here or in
`plain_zevivik.py`): the branches' sum with one or two norms of the stream, the embedding once more and a pass's vector;
attention in chunks (plain, on the matrix cores in tiles of 16, 64 and 128 queries, single tokens, grouped heads, keys in
slices, pages of passed chunks gone; a key that stands out just inside and just outside the chunk, at page borders); a gate
per head in latent attention, latents of sizes that are brought to a multiple of 32; the router's bias; the gated
activations."""
import math

import numpy as np
import pytest
import torch

import plain_zevivik as pz
from test_gpu_gosuvik_parts import DEV, F, PagedKV, rnd

pytestmark = pytest.mark.gpu


# ---- the branches' sum and the norms after it -----------------------------------------------------------------------------
TERMS = [(), ("a",), ("a", "b"), ("a", "experts"), ("a", "b", "bias"), ("experts", "shared", "gate"), ("a", "experts", "shared"),
         ("again",), ("step",), ("a", "experts", "shared", "again", "step"), ("a", "b", "bias", "again", "step")]


@pytest.mark.parametrize("dtype,tol", [(torch.float32, 3e-6), (torch.bfloat16, 1e-2)])
@pytest.mark.parametrize("width,k", [(96, 2), (74, 3), (90, 1), (1000, 9), (2048, 4), (5120, 8), (9000, 2), (16384, 6), (17000, 2)])
def test_branches_sum_with_norms(width, k, dtype, tol):
    """Every set of terms; two norms, one, none, and one of picked rows (the stream then stays)."""
    from inferx_amd import ops
    T, eps = 6, 1e-3
    h, a, b = rnd((T, width), 1, 2.0), rnd((T, width), 2, 1.5, dtype), rnd((T, width), 3, 1.0, dtype)
    y, shared = rnd((T * k + 3, width), 4, 1.0, dtype), rnd((T, width), 5, 1.0, dtype)
    g = torch.Generator().manual_seed(6)
    dest = torch.randperm(T * k + 3, generator=g)[:T * k].to(torch.int32)
    weight, gate = torch.rand(T, k, generator=g), torch.rand(T, generator=g)
    table, ids, scale = rnd((9, width), 7, 1.0, dtype), torch.tensor([3, 8, 0, 3, 5, 1], dtype=torch.int32), 1.7
    bias, step = rnd((width,), 8, 1.0, dtype), rnd((width,), 9, 2.0, dtype)
    w1, w2 = rnd((width,), 10, 0.3, dtype) + 1.0, rnd((width,), 11, 0.5, dtype) - 1.0
    dev = lambda t: t.to(DEV)
    for terms in TERMS:
        has = lambda n: n in terms
        kw = dict(a=dev(a) if has("a") else None, b=dev(b) if has("b") else None, bias=dev(bias) if has("bias") else None,
                  step=dev(step) if has("step") else None, again=(dev(table), dev(ids), scale) if has("again") else None)
        if has("experts"):
            kw["experts"] = (dev(y), dev(dest), dev(weight), dev(shared) if has("shared") else None, dev(gate) if has("gate") else None)
        want = h.double()
        for n, t in (("a", a), ("b", b), ("bias", bias[None]), ("step", step[None])):
            want = want + (t.double() if has(n) else 0.0)
        if has("again"):
            want = want + table[ids.long()].double() * scale
        if has("experts"):
            want = want + (weight.double()[:, :, None] * y.double()[dest.long().view(T, k)]).sum(1)
            want = want + (shared.double() * (gate.double()[:, None] if has("gate") else 1.0) if has("shared") else 0.0)
        unit = want / torch.sqrt((want * want).mean(1, keepdim=True) + eps)
        at = float(want.abs().max())
        for norms in (2, 1, 0):
            hd, outs = dev(h), [torch.empty(T, width, dtype=dtype, device=DEV) for _ in range(norms)]
            ops.branch_norm(hd, norms=list(zip((dev(w1), dev(w2)), outs)), eps=eps, **kw)
            assert float((hd.cpu().double() - want).abs().max()) <= 3e-6 * at, f"{terms}"
            for w, out in zip((w1, w2), outs):
                expected = unit * w.double()
                assert float((out.cpu().double() - expected).abs().max()) <= tol * float(expected.abs().max()), f"{terms} {norms}"
        rows = torch.tensor([5, 0, 5], dtype=torch.int32, device=DEV)
        hd, out = dev(h), torch.empty(3, width, dtype=dtype, device=DEV)
        ops.branch_norm(hd, norms=[(dev(w2), out)], eps=eps, rows=rows, **kw)
        assert torch.equal(hd.cpu(), h), "with picked rows the stream stays as it was"
        expected = (unit * w2.double())[[5, 0, 5]]
        assert float((out.cpu().double() - expected).abs().max()) <= tol * float(expected.abs().max()), f"{terms} picked"


def test_sums_that_meet_before_a_norm():
    """`BranchSum`: sums of sums, a branch that is not formed yet, one of another type, a tensor for the embedding; formed
    for a norm, for two, and on its own."""
    from inferx_amd.engine.runtime import Runtime
    from inferx_amd.parts import LazyDelta
    from inferx_amd.parts.branch_sum import BranchSum
    from inferx_amd.parts.dense_mlp import BiasedDelta
    from inferx_amd.parts.norm import RMSNorm

    class Later(LazyDelta):
        def __init__(self, t):
            self.t = t

        def materialize(self, ctx):
            return self.t

    class Ctx:
        rt = Runtime("bfloat16")
    T, W = 5, 64
    a, b, c = (rnd((T, W), i, 1.0, torch.bfloat16).to(DEV) for i in (1, 2, 3))
    f32, bias, again, step = rnd((T, W), 4).to(DEV), rnd((W,), 5).to(DEV), rnd((T, W), 6).to(DEV), rnd((W,), 7).to(DEV)
    sums = [(BranchSum(a, b), a.float() + b.float()), (BranchSum(a, BiasedDelta(b, bias)), a.float() + b.float() + bias),
            (BranchSum(BranchSum(a, b), Later(c)), a.float() + b.float() + c.float()), (BranchSum(a, Later(f32)), a.float() + f32),
            (BranchSum(None).entered(again, step), again + step), (BranchSum(a).entered(None, step), a.float() + step),
            (BranchSum(a, b).entered(again, step), a.float() + b.float() + again + step),
            (BranchSum(Later(f32)).entered(None, step), f32 + step)]
    n1, n2 = RMSNorm(W, 1e-5), RMSNorm(W, 1e-5)
    n1.bind({"weight": rnd((W,), 8).to(DEV)}, Ctx.rt)
    n2.bind({"weight": rnd((W,), 9).to(DEV)}, Ctx.rt)
    for i, (total, want) in enumerate(sums):
        assert float((total.materialize(Ctx) - want).abs().max()) <= 1e-5, f"sum {i}"
        h = rnd((T, W), 10).to(DEV)
        left = h + want
        x, z = n1.forward_pair(Ctx, h, total, n2)
        assert float((h - left).abs().max()) <= 1e-5, f"sum {i}"
        for out, n in ((x, n1), (z, n2)):
            expected = left / torch.sqrt((left * left).mean(1, keepdim=True) + 1e-5) * n.weight
            assert float((out.float() - expected).abs().max()) <= 1e-2 * float(expected.abs().max()), f"sum {i}"
    with pytest.raises(ValueError, match="biases"):
        BranchSum(BiasedDelta(a, bias), BiasedDelta(b, bias))
    other = RMSNorm(W, 1e-3)  # another eps: the two norms one after the other
    other.bind({"weight": n2.weight}, Ctx.rt)
    h = rnd((T, W), 10).to(DEV)
    left = h + a.float() + b.float()
    x, z = n1.forward_pair(Ctx, h, BranchSum(a, b), other)
    for out, w, eps in ((x, n1.weight, 1e-5), (z, n2.weight, 1e-3)):
        expected = left / torch.sqrt((left * left).mean(1, keepdim=True) + eps) * w
        assert float((out.float() - expected).abs().max()) <= 1e-2 * float(expected.abs().max())


# ---- attention in chunks ------------------------------------------------------------------------------------------------------
def run_chunked(paged, lengths, contexts, H, scale, chunk, dtype, how, standout=None, splits=1, push=14.0):
    """The last lengths[i] positions of request i as one step's rows; `how`: plain, tiles (16 queries), tiles64, wide (128),
    single (a token per tile), grouped.  standout = (request, key): its queries are made to match that key."""
    from inferx_amd import ops
    G, d, vd = paged.keys[0].shape[1], paged.keys[0].shape[2], paged.values[0].shape[2]
    T = sum(lengths)
    seq = np.repeat(np.arange(len(lengths)), lengths).astype(np.int32)
    pos = np.concatenate([np.arange(c - n, c) for c, n in zip(contexts, lengths)]).astype(np.int32)
    q = rnd((T, H, d), 91, 1.0, dtype)
    if standout is not None:
        i, key = standout
        for t in np.nonzero(seq == i)[0]:
            for h in range(H):
                direction = paged.keys[i][key, h // (H // G)].float()
                q[t, h] += (push / scale * direction / direction.norm() ** 2).to(dtype)
    keys, values = paged.keys, paged.values
    for i, (c, n) in enumerate(zip(contexts, lengths)):  # what the step's first position no longer reads is gone
        paged.give_back(i, (c - n) - (c - n) % chunk)
    span = ops.key_span(0, chunk)
    out = torch.full((T, H, vd), float("nan"), dtype=dtype, device=DEV)
    dev = lambda a: torch.from_numpy(a).to(DEV)
    qd, k, v, table = q.to(DEV), paged.k.to(DEV), paged.v.to(DEV), paged.table.to(DEV)
    if how == "plain":
        ops.attention_plain(qd, k, v, table, dev(seq), dev(pos), out, scale, span)
    else:
        size = {"tiles": 16, "single": 1, "grouped": 1, "tiles64": 64, "wide": 128}[how]
        tiles, at = [], 0
        for i, n in enumerate(lengths):
            tiles += [(i, at + first, min(size, n - first)) for first in range(0, n, size)]
            at += n
        tiles = torch.tensor(tiles, dtype=torch.int32).t().contiguous().to(DEV)
        work = torch.empty(T * H * splits * (d + 2), dtype=torch.float32, device=DEV) if splits > 1 else None
        if how in ("wide", "tiles64"):
            ops.attention_prefill(qd, k, v, table, tiles, dev(pos), out, scale, span, size, None, splits, work)
        else:
            ops.attention_mfma(qd, k, v, table, tiles, dev(pos), out, splits, work, scale, span, 16, prefetch=splits > 1,
                               grouped=how == "grouped")
    want = torch.zeros(T, H, vd, dtype=F)
    for t in range(T):
        i, p = int(seq[t]), int(pos[t])
        lo = p - p % chunk
        for h in range(H):
            s = keys[i][lo:p + 1, h // (H // G)].double() @ q[t, h].double() * scale
            want[t, h] = torch.softmax(s, dim=0) @ values[i][lo:p + 1, h // (H // G)].double()
    return out.cpu().double(), want


CONTEXTS = [170, 33, 1, 350, 48]
PORTIONS = [150, 20, 1, 9, 16]
FEW = [2, 3, 1, 130, 2]
ONES = [1, 1, 1, 1, 1]


@pytest.mark.parametrize("dtype,tol", [(torch.float32, 2e-5), (torch.bfloat16, 2e-2)])
@pytest.mark.parametrize("chunk", [1, 2, 7, 16, 40, 100, 400])
@pytest.mark.parametrize("H,G,d,vd,page", [(4, 2, 16, 24, 16), (3, 3, 11, 6, 8), (2, 1, 33, 48, 48)])
def test_chunked_attention_plain(H, G, d, vd, page, chunk, dtype, tol):
    for lengths in (PORTIONS, ONES):
        got, want = run_chunked(PagedKV(CONTEXTS, G, d, vd, page, dtype, seed=3), lengths, CONTEXTS, H, d ** -0.5, chunk, dtype, "plain")
        assert float((got - want).abs().max()) <= tol * float(want.abs().max()), f"{lengths}"


@pytest.mark.parametrize("chunk", [1, 2, 7, 16, 40, 64, 100, 400])
@pytest.mark.parametrize("H,G,d,page", [(4, 2, 32, 16), (8, 2, 64, 16), (16, 1, 128, 32), (3, 3, 96, 16), (2, 1, 48, 48), (2, 1, 256, 16),
                                        (4, 4, 48, 16)])
def test_chunked_attention_on_the_matrix_cores(H, G, d, page, chunk):
    ways = [("tiles", PORTIONS, 1), ("tiles", FEW, 1), ("tiles", PORTIONS, 4), ("single", ONES, 1), ("single", ONES, 4)]
    if H // G > 1:
        ways += [("grouped", ONES, 1), ("grouped", ONES, 8)]
    if d <= 128 and page & (page - 1) == 0:
        ways += [("tiles64", PORTIONS, 1), ("tiles64", FEW, 2)]
        if d % 32 == 0:
            ways += [("wide", PORTIONS, 1), ("wide", PORTIONS, 2), ("wide", FEW, 4)]
    for how, lengths, splits in ways:
        got, want = run_chunked(PagedKV(CONTEXTS, G, d, d, page, torch.bfloat16, seed=4), lengths, CONTEXTS, H, d ** -0.5, chunk,
                                torch.bfloat16, how, splits=splits)
        assert torch.isfinite(got).all(), f"{how} {lengths} {splits}"
        assert float((got - want).abs().max()) <= 2e-2 * float(want.abs().max()), f"{how} {lengths} {splits}"


@pytest.mark.parametrize("how,splits", [("plain", 1), ("tiles", 1), ("tiles", 4), ("tiles64", 1), ("wide", 1), ("wide", 2), ("single", 4),
                                        ("grouped", 2)])
def test_a_key_that_stands_out_at_the_chunks_edge(how, splits):
    """Chunks of 75 of 300 positions: a key that takes nearly all the weight where it is seen, at the chunk's first and
    second place and the last place of the chunk before, at page borders inside, at the query's own place; portions that
    end just after and well after an edge."""
    H, G, d, page, chunk = 4, 2, 64, 16, 75
    dtype = torch.float32 if how == "plain" else torch.bfloat16
    for n in (226, 227, 260, 300):  # the last query is at the chunk's first, second, a middle and the last place
        start = (n - 1) - (n - 1) % chunk
        for length in ((1,) if how in ("single", "grouped") else (2, 40)):
            for key in {start - chunk, start - 1, start, min(start + 1, n - 1), min(240, n - 1), n - 1}:
                paged = PagedKV([n], G, d, d, page, dtype, seed=6)
                got, want = run_chunked(paged, [length], [n], H, d ** -0.5, chunk, dtype, how, standout=(0, key), splits=splits)
                tol = 1e-4 if how == "plain" else 2e-2
                assert float((got - want).abs().max()) <= tol * float(want.abs().max()), f"n {n} key {key} length {length}"
                value = paged.values[0][key].double().repeat_interleave(H // G, dim=0)
                if start <= key:
                    assert float((want[-1] - value).abs().max()) < 0.2 * float(value.abs().max()), "the test's key does not stand out"
                else:
                    assert float((want[-1] - value).abs().max()) > 0.3 * float(value.abs().max())


@pytest.mark.parametrize("seq_lens,q_lens,chunk", [([5000, 300, 2100], [900, 1, 1], 1500), ([4096, 33], [2048, 1], 700),
                                                   ([3000], [40], 2999), ([700, 700, 9], [1, 1, 1], 256)])
def test_attend_plans_steps_in_chunks(seq_lens, q_lens, chunk):
    """`PagedAttention.attend` on steps of realistic sizes: which kernel serves which request, in how many slices, is its own
    plan; the result is that of float64 attention over each query's chunk."""
    from inferx_amd.engine.runtime import CacheBinding, Runtime, StepContext
    from inferx_amd.parts.attention import PagedAttention
    import attention_util as au
    H, G, d, page = 8, 2, 64, 16
    p = au.paged_on_device(seq_lens, q_lens, H, G, d, page, seed=5)
    part = PagedAttention(64, H, G, d, qkv_bias=False, chunk=chunk)
    rt = Runtime("bfloat16")
    T = sum(q_lens)

    class Host:
        q_start = np.concatenate([[0], np.cumsum(q_lens)]).astype(np.int32)
    Host.seq_lens = np.array(seq_lens, dtype=np.int32)
    i32 = lambda a: torch.tensor(a, dtype=torch.int32, device=DEV)
    ctx = StepContext(rt=rt, num_tokens=T, num_requests=len(q_lens), token_ids=i32([0] * T), positions=p["positions"],
                      seq_of_token=p["seq_of_token"], q_start=i32(Host.q_start), seq_lens=i32(seq_lens), state_slots=i32([0] * len(q_lens)),
                      logits_rows=i32([]), slots=[i32([0] * T)], block_tables=[p["table"]], host=Host,
                      one_token_each=all(n == 1 for n in q_lens))
    out = torch.empty(T, H, d, dtype=torch.bfloat16, device=DEV)
    part.attend(ctx, p["q"], CacheBinding(group=0, arrays={"k": p["k_cache"], "v": p["v_cache"]}), out)
    row = 0
    for (k, v), q, L, n in zip(p["dense"], p["qs"], seq_lens, q_lens):
        pos = torch.arange(L - n, L)
        for c in sorted({int(x) // chunk for x in pos}):
            mine = torch.nonzero(pos // chunk == c).flatten()
            a, b = c * chunk, int(pos[mine[-1]]) + 1
            want = au.reference_attention(q[mine], k[a:b], v[a:b], pos[mine] - a, d ** -0.5)
            assert au.rel_err(out[row + mine], want) <= 2e-2, f"context {L}, chunk {c}"
        row += n


# ---- a gate per head in latent attention --------------------------------------------------------------------------------------
@pytest.mark.parametrize("mfma", [False, True])
@pytest.mark.parametrize("H,rank,rot,page", [(3, 64, 32, 16), (16, 96, 0, 16), (6, 32, 0, 48), (20, 512, 64, 16), (5, 256, 0, 8)])
def test_latent_attention_with_a_gate_per_head(H, rank, rot, page, mfma):
    from inferx_amd import ops
    from test_gpu_bibevik_parts import Paged, plain_latent_scores
    contexts, scale = [70, 33, 1, 150, 48], 0.2
    dtype = torch.bfloat16 if mfma else torch.float32
    paged = Paged(contexts, rank + rot, page, dtype, seed=7)
    for lengths in ([70, 20, 1, 9, 16], [1, 1, 1, 1, 1], [2, 1, 1, 40, 3]):
        T, one = sum(lengths), all(n == 1 for n in lengths)
        q_lat, q_rot = rnd((T, H, rank), 1, 0.5, dtype), rnd((T, H, rot), 2, 0.5, dtype)
        wide = rnd((T, H + 5), 3, 2.0, dtype)  # the gate's numbers are a view into a wider product
        seq = np.repeat(np.arange(len(lengths)), lengths).astype(np.int32)
        pos = np.concatenate([np.arange(c - n, c) for c, n in zip(contexts, lengths)]).astype(np.int32)
        dev = lambda a: torch.from_numpy(a).to(DEV)
        ql, qr, gates = q_lat.to(DEV), q_rot.to(DEV), wide.to(DEV)[:, 5:]
        qr = qr if rot else ql
        out = torch.full((T, H, rank), float("nan"), dtype=dtype, device=DEV)
        args = (ql, qr, paged.cache.to(DEV), paged.table.to(DEV), dev(seq), dev(pos), out, rank, rot, scale)
        if mfma:
            splits, work = 1, None
            if one:
                splits = ops.latent_mfma_splits(T, H)
                work = (torch.empty(T * H * splits, rank, device=DEV), torch.empty(T * H * splits, 2, device=DEV))
            ops.latent_attention_mfma(*args, one, splits, work, 0, gates)
            if one:  # the keys whole as well
                whole = torch.empty_like(out)
                ops.latent_attention_mfma(*args[:6], whole, *args[7:], one, 1, None, 0, gates)
                assert float((whole.double() - out.double()).abs().max()) <= 2e-2 * float(out.double().abs().max())
        else:
            ops.latent_attention_plain(*args, 0, gates)
        want = torch.zeros(T, H, rank, dtype=F)
        for i in range(len(lengths)):
            rows = np.nonzero(seq == i)[0]
            want[rows] = plain_latent_scores(q_lat[rows].double(), q_rot[rows].double(), paged.rows[i].double(),
                                             [int(p) for p in pos[rows]], scale)
        want = want * torch.sigmoid(wide[:, 5:].double())[:, :, None]
        assert float((out.cpu().double() - want).abs().max()) <= (2e-2 if mfma else 1e-5) * float(want.abs().max()), f"{lengths}"


# ---- the router's bias ----------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("T,W,E,k", [(1, 96, 6, 2), (7, 74, 5, 1), (16, 256, 70, 6), (40, 90, 9, 9), (128, 64, 12, 3), (129, 96, 6, 2),
                                     (300, 200, 130, 8), (3, 64, 300, 4)])
def test_router_with_a_bias(T, W, E, k, dtype):
    """The chosen are the largest biased logits, their weights a softmax over those alone; the one-launch form for few
    tokens, the two-launch form, and the product on the matrix cores give the same."""
    from inferx_amd import ops
    x, w, bias = rnd((T, W), 1, 1.0, dtype), rnd((E, W), 2, W ** -0.5, dtype), rnd((E,), 3, 1.0)
    z = pz.router_logits(x.double(), {"router": w.double(), "router.b": bias.double()})
    val, idx = torch.topk(z, k, dim=1)
    weight = torch.softmax(val, dim=1)
    close = (val[:, -1] - torch.sort(z, dim=1, descending=True).values[:, min(k, E - 1)]).abs() < 1e-4 if k < E else torch.zeros(T, dtype=torch.bool)
    out = []
    tw, te = torch.empty(T, k, device=DEV), torch.empty(T, k, dtype=torch.int32, device=DEV)
    ops.moe_route(x.to(DEV), w.to(DEV), None, tw, te, None, True, 1.0, bias=bias.to(DEV))
    out.append((tw, te))
    if ops.route_one_launch_fits(T, W, E):
        tw, te = torch.empty(T, k, device=DEV), torch.empty(T, k, dtype=torch.int32, device=DEV)
        i32 = lambda n: torch.empty(n, dtype=torch.int32, device=DEV)
        ops.moe_route_dispatch(x.to(DEV), w.to(DEV), None, tw, te, None, True, 1.0, i32(E + 1), i32(T * k), i32(T * k), bias=bias.to(DEV))
        out.append((tw, te))
    for tw, te in out:
        for t in range(T):
            if not bool(close[t]):
                got = dict(zip(te[t].tolist(), tw[t].tolist()))
                want = dict(zip(idx[t].tolist(), weight[t].tolist()))
                assert got.keys() == want.keys() and all(abs(got[e] - want[e]) < 1e-4 for e in want), f"token {t}"
    always = 2  # pieces of a shared expert behind the chosen ones keep their weight of one
    tw, te = torch.empty(T, k + always, device=DEV), torch.empty(T, k + always, dtype=torch.int32, device=DEV)
    ops.moe_route(x.to(DEV), w.to(DEV), None, tw, te, None, True, 1.0, always, bias=bias.to(DEV))
    assert torch.equal(tw[:, :k], out[0][0]) and (tw[:, k:] == 1).all() and te[:, k:].tolist() == [[E, E + 1]] * T


# ---- the gated activations --------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype,tol", [(torch.float32, 2e-6), (torch.bfloat16, 1e-2)])
@pytest.mark.parametrize("width", [24, 50, 333, 1408])
def test_gated_activations(width, dtype, tol):
    from inferx_amd import ops
    from inferx_amd.engine.runtime import Runtime
    gu, bias = rnd((9, 2 * width), 1, 3.0, dtype), rnd((2 * width,), 2, 1.0, dtype)
    gu[0, :4] = torch.tensor([-40.0, 40.0, -9.0, 0.0]).to(dtype)

    def glu(t, limit):
        g, u = t[:, :width], t[:, width:]
        if limit < 0:
            return pz.gelu_tanh(g) * u
        if limit == 0:
            return g * torch.sigmoid(g) * u
        g, u = torch.clamp(g, max=limit), torch.clamp(u, -limit, limit)
        return g * torch.sigmoid(1.702 * g) * (u + 1.0)
    for limit in (0.0, 1.3, ops.GLU_GELU_TANH):
        for b in (None, bias):
            out = torch.empty(9, width, dtype=dtype, device=DEV)
            ops.glu_bias(gu.to(DEV), None if b is None else b.to(DEV), out, limit)
            want = glu(gu.double() + (0.0 if b is None else b.double()), limit)
            assert float((out.cpu().double() - want).abs().max()) <= tol * float(want.abs().max()), f"limit {limit}"
        rt = Runtime("float32" if dtype == torch.float32 else "bfloat16")
        for T in (3, 20, 70):  # few rows: the activation in the product's kernel
            x, w = rnd((T, 64), 3, 1.0, dtype), rnd((2 * width, 64), 4, 0.2, dtype)
            got = rt.gated_linear(x.to(DEV), w.to(DEV), limit).cpu().double()
            want = glu(x.double() @ w.double().T, limit)
            assert float((got - want).abs().max()) <= 2 * tol * float(want.abs().max()), f"limit {limit}, {T} rows"
