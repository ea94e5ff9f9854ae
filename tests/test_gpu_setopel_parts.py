"""Setopel's mechanisms one by one, each kernel against a slow float64 function written from the equations (here or in
`plain_setopel.py`): the norm over a stream of several copies and the embedding that starts it; the convolution with a
query temperature; attention with capped scores, a zero sink and a gate (plain, on the matrix cores in tiles of 16 and of
128 queries, single tokens, keys in slices; one key made to stand out far back, at page borders, at the first token and
the query's own); heads that are widened; retention row by row and in chunks, carried over steps, portions around the
chunk's length."""
import math

import numpy as np
import pytest
import torch

import plain_setopel as ps
from test_gpu_gosuvik_parts import DEV, F, PagedKV, rnd, step_rows

pytestmark = pytest.mark.gpu


# ---- a stream of several copies --------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype,tol", [(torch.float32, 2e-6), (torch.bfloat16, 1e-2)])
@pytest.mark.parametrize("streams,width", [(1, 40), (2, 74), (3, 96), (4, 2048), (5, 90), (7, 1000), (8, 256), (9, 48), (4, 5120),
                                           (2, 9000), (32, 20), (6, 4)])
def test_norm_over_streams(streams, width, dtype, tol):
    from inferx_amd import ops
    T = 7
    xs, y = rnd((T, streams, width), 1, 2.0), rnd((T, width), 2, 1.5, dtype)
    mix, gain, enter = rnd((streams, streams), 3), rnd((streams,), 4), rnd((streams,), 5)
    weight = rnd((width,), 6, 0.3) + 1.0
    w0, eps = weight.double() - 1.0, 1e-3
    left = ps.leave_streams(xs.double(), y.double(), gain.double(), mix.double(), 1.0)
    for come_back, named in ((True, True), (True, False), (False, True)):
        h, out = xs.to(DEV), torch.empty(T, width, dtype=dtype, device=DEV)
        ops.stream_norm(h, y.to(DEV) if come_back else None, mix.to(DEV), gain.to(DEV), enter.to(DEV) if named else None,
                        weight.to(DEV), out, eps)
        state = left if come_back else xs.double()
        u = ps.enter_streams(state, enter.double()) if named else state.sum(1)
        want = ps.norm0(u, w0, eps)
        assert float((h.cpu().double() - state).abs().max()) <= 2e-6 * float(state.abs().max())
        assert float((out.cpu().double() - want).abs().max()) <= tol * float(want.abs().max())
    rows = torch.tensor([5, 0, 5], dtype=torch.int32, device=DEV)
    h, out = xs.to(DEV), torch.empty(3, width, dtype=dtype, device=DEV)
    ops.stream_norm(h, y.to(DEV), mix.to(DEV), gain.to(DEV), None, weight.to(DEV), out, eps, rows)
    assert torch.equal(h.cpu(), xs), "with picked rows the copies stay as they were"
    want = ps.norm0(left.sum(1), w0, eps)[[5, 0, 5]]
    assert float((out.cpu().double() - want).abs().max()) <= tol * float(want.abs().max())


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("streams,width", [(1, 40), (4, 256), (3, 2050)])
def test_embedding_with_a_norm_starts_every_copy(streams, width, dtype):
    from inferx_amd import ops
    table, weight = rnd((11, width), 1, 0.2, dtype), rnd((width,), 2, 0.3) + 1.0
    ids = torch.tensor([3, 0, 10, 3], dtype=torch.int32, device=DEV)
    h = torch.empty(4, streams, width, dtype=torch.float32, device=DEV)
    ops.embed_norm(h, table.to(DEV), ids, weight.to(DEV), 1e-4, 0.7)
    want = ps.norm0(table[[3, 0, 10, 3]].double() * 0.7, weight.double() - 1.0, 1e-4)
    for j in range(streams):
        assert float((h[:, j].cpu().double() - want).abs().max()) <= 2e-6 * float(want.abs().max())
    ops.embed_norm(h, table.to(DEV), ids, None, 0.0)
    assert torch.equal(h.cpu(), table[[3, 0, 10, 3]].float()[:, None, :].repeat(1, streams, 1))


# ---- the convolution with a temperature ------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype,tol", [(torch.float32, 2e-6), (torch.bfloat16, 1e-2)])
@pytest.mark.parametrize("H,G,d,vd,taps,temp,keys", [(4, 2, 16, 24, 3, (0.4, 8), True), (3, 3, 10, 6, 4, (1.0, 1), True),
                                                     (2, 1, 32, 32, 1, (0.3, 5), True), (8, 2, 64, 64, 4, None, True),
                                                     (4, 2, 16, 16, 3, (0.5, 7), False), (2, 2, 7, 7, 5, (0.2, 3), False)])
def test_convolution_with_a_query_temperature(H, G, d, vd, taps, temp, keys, dtype, tol):
    """Requests in portions of changing size (down to two tokens and one, up to several tiles of rows), slots out of order, the state carried;
    the first token whose count reaches a multiple of the step, and the one before; queries alone (no keys of its own)."""
    from inferx_amd.parts.short_conv import ShortConv
    names = ("q", "k", "v") if keys else ("q",)
    cq, ck, cv = H * d, (G * d if keys else 0), (G * vd if keys else 0)
    C = cq + ck + cv
    w, bias = rnd((C, taps), 3, 0.5, dtype), rnd((C,), 4, 0.7, dtype)
    conv = ShortConv(cq, ck, cv, d, vd, taps)
    at = {"q": slice(0, cq), "k": slice(cq, cq + ck), "v": slice(cq + ck, C)}
    conv.bind({f"{n}.conv": w[at[n]].to(DEV) for n in names}, names=names, bias=bias.to(DEV))
    lengths = [110, 40, 60]
    x = [rnd((n, C + 8), 10 + i, 1.0, dtype) for i, n in enumerate(lengths)]  # rows longer than the channels: a gate behind
    state = torch.full((4, max(1, (taps - 1) * C)), float("nan"), device=DEV)
    slots = [2, 0, 3]
    state[slots] = 0
    page = 16
    kc, vc = torch.zeros(16, G, page, d, dtype=dtype, device=DEV), torch.zeros(16, G, vd, page, dtype=dtype, device=DEV)
    first_slot = [0, 112, 160]
    done, got = [0, 0, 0], [[], [], []]
    for portions in ((7, 31, 1), (1, 0, 1), (8, 0, 2), (94, 9, 56)):
        rows = step_rows(portions, slots)
        pos = np.concatenate([np.arange(a, a + n) for a, n in zip(done, portions)]).astype(np.int32)
        cache_slots = np.concatenate([f + np.arange(a, a + n) for f, a, n in zip(first_slot, done, portions)]).astype(np.int32)
        T = len(pos)

        class Ctx:
            seq_of_token, q_start, state_slots = rows.seq_of_token, rows.q_start, rows.state_slots
        xin = torch.cat([t[a:a + n] for t, a, n in zip(x, done, portions)]).to(DEV)
        q = torch.empty(T, H, d, dtype=dtype, device=DEV)
        temperature = None if temp is None else (torch.from_numpy(pos).to(DEV),) + temp
        if keys:
            conv.apply(Ctx, xin, state, q, kc, vc, slots=torch.from_numpy(cache_slots).to(DEV), temperature=temperature)
        else:
            conv.apply(Ctx, xin, state, q, q, q, temperature=temperature)
        row = 0
        for i, n in enumerate(portions):
            got[i].append(q[row:row + n].cpu())
            row += n
            done[i] += n
    assert done == lengths
    for i, n in enumerate(lengths):
        u = x[i][:, :C].double() + bias.double()
        y = ps.short_conv(u, w.double())
        want = y[:, at["q"]].view(n, H, d)
        if temp is not None:
            want = want * ps.temperature(torch.arange(n), *temp)[:, None, None]
        assert float((torch.cat(got[i]).double() - want).abs().max()) <= tol * float(want.abs().max())
        if keys:
            s = first_slot[i] + torch.arange(n)
            k = kc.cpu().double()[s // page, :, s % page]
            v = vc.cpu().double()[s // page, :, :, s % page]
            assert float((k - y[:, at["k"]].view(n, G, d)).abs().max()) <= tol * float(y.abs().max())
            assert float((v - y[:, at["v"]].view(n, G, vd)).abs().max()) <= tol * float(y.abs().max())


# ---- attention with capped scores, a zero sink and a gate -------------------------------------------------------------------
def plain_capped(q, keys, values, pos, scale, cap, sink, gate):
    """q [H, d] at position pos over keys [n, G, d], values [n, G, vd]; gate [H, vd] or None."""
    H, G = q.shape[0], keys.shape[1]
    out = torch.zeros(H, values.shape[2], dtype=F)
    for h in range(H):
        s = ps.capped(keys[:pos + 1, h // (H // G)] @ q[h] * scale, cap)
        p = ps.softmax_one(s) if sink else torch.softmax(s, dim=-1)
        out[h] = p @ values[:pos + 1, h // (H // G)]
    return out if gate is None else out * torch.sigmoid(gate)


def run_capped(paged, lengths, contexts, H, scale, cap, dtype, how, sink=True, use_gate=True, standout=None, splits=1,
               push=14.0, noise=1.0):
    """The last lengths[i] positions of request i as one step's rows; `how`: plain, tiles (16 queries), single (a token
    per tile), grouped, wide (tiles of 128 queries).  standout = (request, key): its queries are made to match that key
    with a raw score of `push`."""
    from inferx_amd import ops
    G, d, vd = paged.keys[0].shape[1], paged.keys[0].shape[2], paged.values[0].shape[2]
    T = sum(lengths)
    seq = np.repeat(np.arange(len(lengths)), lengths).astype(np.int32)
    pos = np.concatenate([np.arange(c - n, c) for c, n in zip(contexts, lengths)]).astype(np.int32)
    q = rnd((T, H, d), 91, noise, dtype)
    if standout is not None:
        i, key = standout
        for t in np.nonzero(seq == i)[0]:
            for h in range(H):
                direction = paged.keys[i][key, h // (H // G)].float()
                q[t, h] += (push / scale * direction / direction.norm() ** 2).to(dtype)
    wide = rnd((T, H * vd + 8), 92, 1.5, dtype).to(DEV)  # the gate's rows are a view into a wider product
    gate = wide[:, 8:] if use_gate else None
    zero = torch.zeros(H, device=DEV) if sink else None
    out = torch.full((T, H, vd), float("nan"), dtype=dtype, device=DEV)
    dev = lambda a: torch.from_numpy(a).to(DEV)
    qd, k, v, table = q.to(DEV), paged.k.to(DEV), paged.v.to(DEV), paged.table.to(DEV)
    if how == "plain":
        ops.attention_plain(qd, k, v, table, dev(seq), dev(pos), out, scale, 0, zero, None, cap)
        if use_gate:
            ops.sigmoid_gate(out.view(T, -1), gate)
    else:
        size = {"tiles": 16, "single": 1, "grouped": 1, "wide": 128}[how]
        tiles, at = [], 0
        for i, n in enumerate(lengths):
            tiles += [(i, at + first, min(size, n - first)) for first in range(0, n, size)]
            at += n
        tiles = torch.tensor(tiles, dtype=torch.int32).t().contiguous().to(DEV)
        work = torch.empty(T * H * splits * (d + 2), dtype=torch.float32, device=DEV) if splits > 1 else None
        if how == "wide":
            ops.attention_prefill(qd, k, v, table, tiles, dev(pos), out, scale, 0, 128, None, splits, work, sink=zero,
                                  softcap=cap, gate=gate)
        else:
            ops.attention_mfma(qd, k, v, table, tiles, dev(pos), out, splits, work, scale, 0, 16, prefetch=splits > 1,
                               grouped=how == "grouped", sink=zero, softcap=cap, gate=gate)
    gates = None if gate is None else gate.cpu().double().reshape(T, H, vd)
    want = torch.stack([plain_capped(q[t].double(), paged.keys[seq[t]].double(), paged.values[seq[t]].double(), int(pos[t]),
                                     scale, cap, sink, None if gates is None else gates[t]) for t in range(T)])
    return out.cpu().double(), want


CONTEXTS = [70, 33, 1, 150, 48]
PORTIONS = [70, 20, 1, 9, 16]
ONES = [1, 1, 1, 1, 1]


@pytest.mark.parametrize("dtype,tol", [(torch.float32, 2e-5), (torch.bfloat16, 2e-2)])
@pytest.mark.parametrize("H,G,d,vd,page,cap", [(4, 2, 16, 24, 16, 3.0), (3, 3, 10, 6, 8, 0.0), (6, 1, 64, 64, 16, 50.0),
                                               (2, 1, 33, 48, 48, 1.0), (1, 1, 8, 8, 16, 20.0)])
def test_capped_attention_plain(H, G, d, vd, page, cap, dtype, tol):
    for lengths in (PORTIONS, ONES):
        for sink, gate in ((True, True), (False, False)):
            got, want = run_capped(PagedKV(CONTEXTS, G, d, vd, page, dtype, seed=3), lengths, CONTEXTS, H, d ** -0.5, cap, dtype,
                                   "plain", sink, gate)
            assert float((got - want).abs().max()) <= tol * float(want.abs().max()), f"{lengths} sink {sink}"


@pytest.mark.parametrize("H,G,d,page,cap", [(4, 2, 32, 16, 3.0), (8, 2, 64, 16, 50.0), (16, 1, 128, 32, 10.0), (3, 3, 96, 16, 0.0),
                                            (2, 1, 48, 48, 1.5), (4, 4, 16, 16, 5.0), (2, 1, 256, 16, 8.0)])
def test_capped_attention_on_the_matrix_cores(H, G, d, page, cap):
    ways = [("tiles", PORTIONS, 1), ("tiles", [3, 1, 1, 2, 1], 1), ("tiles", PORTIONS, 4), ("single", ONES, 4)]
    if H // G > 1:
        ways += [("grouped", ONES, 1), ("grouped", ONES, 8)]
    if d % 32 == 0 and d <= 128 and page & (page - 1) == 0:
        ways += [("wide", PORTIONS, 1), ("wide", PORTIONS, 2), ("wide", [2, 33, 1, 150, 3], 4)]
    for how, lengths, splits in ways:
        for sink, gate in ((True, True), (False, True), (True, False)):
            got, want = run_capped(PagedKV(CONTEXTS, G, d, d, page, torch.bfloat16, seed=4), lengths, CONTEXTS, H, d ** -0.5,
                                   cap, torch.bfloat16, how, sink, gate, splits=splits)
            assert torch.isfinite(got).all(), f"{how} {splits}"
            assert float((got - want).abs().max()) <= 2e-2 * float(want.abs().max()), f"{how} {lengths} {splits} sink {sink}"


@pytest.mark.parametrize("how,splits", [("plain", 1), ("tiles", 1), ("tiles", 4), ("wide", 1), ("wide", 2), ("single", 4),
                                        ("grouped", 2)])
def test_one_key_that_stands_out(how, splits):
    """A key whose score is far above the others', at every kind of place: the first tokens, both sides of a page border,
    the far past, the last keys.  The capped score still outweighs hundreds of others; with a cap below what it would
    take, the weight is spread as the cap says."""
    H, G, d, page = 4, 2, 64, 16
    n = 300
    for length in ((1,) if how in ("single", "grouped") else (2, 40)):
        for key in (0, 1, 15, 16, 47, 48, 255, 256, n - length - 1, n - length):
            for cap, push in ((30.0, 18.0), (2.0, 18.0)):
                dtype = torch.float32 if how == "plain" else torch.bfloat16
                got, want = run_capped(PagedKV([n], G, d, d, page, dtype, seed=6), [length], [n], H, d ** -0.5, cap, dtype, how,
                                       standout=(0, key), splits=splits, push=push)
                tol = 1e-4 if how == "plain" else 2e-2
                assert float((got - want).abs().max()) <= tol * float(want.abs().max()), f"key {key} cap {cap} length {length}"


def test_the_zero_sink_takes_what_low_scores_leave():
    """All scores far below zero: nearly everything goes to the sink, and the result nearly vanishes; far above: the sink
    takes nothing.  (One key per request, so the weights are known.)"""
    for push in (-8.0, -2.0, 0.0, 9.0):
        for how in ("plain", "tiles", "wide", "single"):
            dtype = torch.float32 if how == "plain" else torch.bfloat16
            paged = PagedKV([1, 1], 1, 32, 32, 16, dtype, seed=8)
            got, want = run_capped(paged, [1, 1], [1, 1], 2, 1.0, 12.0, dtype, how, standout=(0, 0), push=push, use_gate=False,
                                   noise=0.0)
            assert float((got[0] - want[0]).abs().max()) <= 2e-2 * float(want[0].abs().max()) + 1e-6
            expected = 1.0 / (1.0 + math.exp(-12 * math.tanh(push / 12.0)))
            share = float((want[0, 0] @ paged.values[0][0, 0].double()) / (paged.values[0][0, 0].double() ** 2).sum())
            assert abs(share - expected) < 0.05 * expected  # (the query is rounded)


def test_heads_are_widened_with_zeros():
    from inferx_amd.parts.attention_conv import pad_heads, padded_head
    assert [padded_head(*s) for s in ((16,), (10, 6), (17, 3), (20, 28), (64, 64))] == [16, 16, 32, 32, 64]
    t = rnd((6, 5), 1)
    wide = pad_heads(t, 3, 2, 4)
    assert wide.shape == (12, 5) and torch.equal(wide.view(3, 4, 5)[:, :2].reshape(6, 5), t) and not wide.view(3, 4, 5)[:, 2:].any()
    wide = pad_heads(t.t().contiguous(), 3, 2, 3, dim=1)
    assert wide.shape == (5, 9) and torch.equal(wide.view(5, 3, 3)[..., :2].reshape(5, 6), t.t())


# ---- retention ----------------------------------------------------------------------------------------------------------------
def plain_decayed(q, k, v, decay, S, silu=False):
    """Row by row in float64: q, k [n, H, d], v [n, H, vd], S [H, d, vd]; (o, the new S)."""
    if silu:
        q, k, v = ps.silu(q), ps.silu(k), ps.silu(v)
    o = torch.zeros(q.shape[0], q.shape[1], v.shape[2], dtype=F)
    for t in range(q.shape[0]):
        S = decay[:, None, None] * S + k[t][:, :, None] * v[t][:, None, :]
        o[t] = torch.einsum("hdv,hd->hv", S, q[t])
    return o, S


class StepCtx:
    """What `decayed_state` reads of a step."""

    def __init__(self, lengths, slots):
        from inferx_amd.engine.runtime import Runtime
        rows = step_rows(lengths, slots)
        self.rt, self.memo = Runtime("float32"), {}
        self.seq_of_token, self.q_start, self.state_slots = rows.seq_of_token, rows.q_start, rows.state_slots
        self.one_token_each = all(n == 1 for n in lengths)

        class host:
            q_start = np.concatenate([[0], np.cumsum(lengths)]).astype(np.int32)
        self.host = host


SIZES = [(2, 16, 16, 16), (3, 12, 20, 8), (2, 64, 40, 64), (1, 128, 136, 32), (2, 96, 12, 48), (2, 32, 33, 0), (1, 10, 7, 6),
         (2, 30, 16, 30), (4, 128, 128, 128), (1, 160, 24, 160), (2, 36, 260, 12), (1, 4, 4, 2)]


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,d,vd,rot", SIZES)
def test_retention_carried_over_steps(H, d, vd, rot, dtype):
    """Three requests in slots out of order, in steps of portions around the chunks' length, single tokens and none, so that
    portions worked in chunks stand beside rows worked one by one and follow each other; a decay of one, of zero, and
    strong ones."""
    from inferx_amd import ops
    from inferx_amd.parts.linear_state import decayed_state
    decay = [1.0, 0.99, 0.5, 0.0][:H] if H > 1 else [0.9]
    lengths = [16 + 65 + 1 + 3, 1 + 64 + 2 + 130, 15 + 17 + 0 + 63]
    steps = list(zip((16, 65, 1, 3), (1, 64, 2, 130), (15, 17, 0, 63)))
    slots = [3, 0, 2]
    q, k = ([rnd((n, H * d), s + i, 1.0, dtype) for i, n in enumerate(lengths)] for s in (10, 20))
    v = [rnd((n, H * vd), 30 + i, 1.0, dtype) for i, n in enumerate(lengths)]
    state = rnd((5, H * d * vd + 4), 40).to(DEV)
    view = state[:, :H * d * vd]
    view[slots] = 0
    kept = state.clone()
    freq = 100.0 ** (-2.0 * torch.arange(rot // 2, dtype=F) / rot) if rot else None
    done, got = [0, 0, 0], [[], [], []]
    for lens in steps:
        part = lambda x: torch.cat([t[a:a + n] for t, a, n in zip(x, done, lens)]).to(DEV)
        pos = np.concatenate([np.arange(a, a + n) for a, n in zip(done, lens)])
        table = None
        if rot:
            ang = torch.from_numpy(pos).double()[:, None] * freq[None, :]
            table = torch.stack([torch.cos(ang), torch.sin(ang)], dim=-1).float().contiguous().to(DEV)
        proj = torch.cat([part(q), part(k), part(v)], dim=1)  # rows of one product, as the mixer has them
        out = torch.full((len(pos), H, vd), float("nan"), device=DEV)
        decayed_state(StepCtx(lens, slots), proj[:, :H * d], proj[:, H * d:2 * H * d], proj[:, 2 * H * d:], view, out, H, d, vd,
                      torch.tensor(decay, device=DEV), cos_sin=table, k_scale=d ** -0.5)
        row = 0
        for i, n in enumerate(lens):
            got[i].append(out[row:row + n].cpu().double())
            row += n
            done[i] += n
    assert done == lengths
    for i, n in enumerate(lengths):
        p = torch.arange(n)
        rotated = [ps.rotate_first(t[i].double().view(n, H, d), p, rot, 100.0) if rot else t[i].double().view(n, H, d) for t in (q, k)]
        want, S = plain_decayed(rotated[0], rotated[1] * d ** -0.5, v[i].double().view(n, H, vd), torch.tensor(decay, dtype=F),
                                torch.zeros(H, d, vd, dtype=F))
        g = torch.cat(got[i])
        assert float((g - want).abs().max()) <= 2e-5 * float(want.abs().max()), f"request {i}"
        held = view[slots[i]].cpu().double().view(H, vd, d).transpose(1, 2)
        assert float((held - S).abs().max()) <= 2e-5 * float(S.abs().max()), f"request {i}: state"
    for slot in (1, 4):
        assert torch.equal(state[slot], kept[slot]), "a slot that no request holds was touched"
    assert torch.equal(state[:, H * d * vd:], kept[:, H * d * vd:])


@pytest.mark.parametrize("n", [1, 2, 15, 16, 31, 32, 33, 63, 64, 65, 127, 128, 129, 193])
def test_retention_portions_of_every_length(n):
    """One portion that begins from a state, in chunks against row by row; one row of keys that stands out at the chunk's
    first and last rows."""
    from inferx_amd import ops
    H, d, vd = 2, 32, 48
    q, k, v = rnd((n, H * d), 1), rnd((n, H * d), 2), rnd((n, H * vd), 3)
    for row in (0, 31, 32, 63, 64, n - 1):
        if row < n:
            k[row] *= 20.0
    decay = torch.tensor([0.97, 1.0])
    S0 = rnd((H, d, vd), 4)
    state = S0.transpose(1, 2).reshape(1, -1).contiguous().to(DEV)
    count = -(-n // 64)
    chunks = torch.tensor([[64 * i for i in range(count)], [min(64, n - 64 * i) for i in range(count)]], dtype=torch.int32, device=DEV)
    seqs = torch.tensor([[0], [0], [count]], dtype=torch.int32, device=DEV)
    out = torch.empty(n, H, vd, device=DEV)
    ops.linear_chunks(q.to(DEV), k.to(DEV), v.to(DEV), state, torch.zeros(1, dtype=torch.int32, device=DEV), chunks, seqs, out, H, d,
                      vd, decay.to(DEV))
    want, S = plain_decayed(q.double().view(n, H, d), k.double().view(n, H, d), v.double().view(n, H, vd), decay.double(), S0.double())
    assert float((out.cpu().double() - want).abs().max()) <= 2e-5 * float(want.abs().max())
    assert float((state.cpu().double().view(H, vd, d).transpose(1, 2) - S).abs().max()) <= 2e-5 * float(S.abs().max())


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_decayed_attention_through_silu_in_chunks(dtype):
    """The other user of the chunks: queries, keys and values through silu, nothing rotated."""
    from inferx_amd.parts.linear_state import decayed_state
    H, d, vd, lens = 3, 64, 64, (100, 5, 1, 64)
    T = sum(lens)
    proj = rnd((T, H * (2 * d + vd)), 5, 1.0, dtype)
    decay = torch.tensor([0.9, 0.99, 0.999])
    state = torch.zeros(4, H * d * vd, device=DEV)
    out = torch.full((T, H, vd), float("nan"), device=DEV)
    pd = proj.to(DEV)
    decayed_state(StepCtx(lens, [1, 3, 0, 2]), pd[:, :H * d], pd[:, H * d:2 * H * d], pd[:, 2 * H * d:], state, out, H, d, vd,
                  decay.to(DEV), silu=True)
    row = 0
    for n in lens:
        x = proj[row:row + n].double()
        want, _ = plain_decayed(x[:, :H * d].view(n, H, d), x[:, H * d:2 * H * d].view(n, H, d), x[:, 2 * H * d:].view(n, H, vd),
                                decay.double(), torch.zeros(H, d, vd, dtype=F), silu=True)
        assert float((out[row:row + n].cpu().double() - want).abs().max()) <= 2e-5 * float(want.abs().max())
        row += n
