"""The Nuzivik decoder on the GPU against the plain implementation (tests/plain/nuzivik.py): every
new kernel alone (the pass between two sublayers, the scaled embedding, keys as values beside
per-head norms, the squashed router, every form of the attention kernels with kept first
positions), the attention part and the mixture of experts over portions and single tokens, keys
made to stand out just inside and just outside every edge (window, kept tokens, pages), a sink
that decides, whole models of five tiny configurations under the four schedule families in
float32 and bfloat16 with pools so small that pages and slots are used again, long decoding, a
batch against its requests alone, the residual stream after every layer, and greedy generation
through the engine and its scheduler."""
import math

import numpy as np
import pytest
import torch

import schedules
from plain import nuzivik as P
from replay_common import collect, make_requests
from tiny_nuzivik import TINY, assert_matches_plain, read_model_dir, telling, write_tiny

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
F32, BF16, F64, I32 = torch.float32, torch.bfloat16, torch.float64, torch.int32

LENGTHS = {"A": [70, 45, 100, 37], "B": [66, 35, 90], "C": [50, 81, 36], "D": [40, 75, 130],
           "E": [61, 30, 45]}
MIXED_LENGTHS = {"A": [70, 45, 100, 37, 83, 64, 29, 58], "B": [66, 35, 90, 41, 23, 77, 50, 62, 88],
                 "C": [50, 81, 36, 67, 44, 72, 90, 33, 58], "D": [40, 75, 52, 33, 61, 28, 97],
                 "E": [61, 30, 45, 38, 52, 27, 66]}


def gen(seed):
    return torch.Generator().manual_seed(seed)


def rel(got, want):
    got = got.detach().to("cpu", F64)
    return float((got - want).abs().max() / want.abs().max().clamp_min(1e-30))


def bind_random(part, seed, dtype, std=0.2, change=None):
    from kappai_amd.weights import random_tensors, stored_to_runtime
    t = telling(random_tensors(part.tensor_specs(), seed, std=std, norm_jitter=0.2), seed)
    if change:
        change(t)
    part.bind({k: stored_to_runtime(v, dtype).to(DEV) for k, v in t.items()})
    return t


def step_through(part, cm, x, portions, view):
    """One request through a mixer in ``portions``; returns the outputs in order."""
    from test_parts_gpu import one_segment_batch
    rc, outs, done = None, [], 0
    for n in portions:
        rc, b = one_segment_batch(cm, n, rc=rc)
        y = part.forward(x[done:done + n].to(DEV), b, view)
        outs.append(y if y.dim() == 2 else y.sum(0))
        cm.commit(rc, n)
        cm.check()
        done += n
    assert done == x.shape[0]
    return torch.cat(outs).float(), rc


PORTIONS_150 = [37, 3] + [1] * 50 + [2, 33] + [1] * 25


# ---------------------------------------------------------------------------------------------
# kernels alone
# ---------------------------------------------------------------------------------------------
@pytest.mark.parametrize("W", [72, 64, 328, 2048, 100, 67, 30, 4096])
def test_one_pass_between_two_sublayers(W):
    """Norm of the update, sum and norm of the new stream in one kernel, against their formulas in
    float64: the update as float32 rows, bfloat16 rows, float32 partial sums and a mixture's
    experts' results; with and without the norm on it; the read alone; the sum alone; some rows
    only."""
    from kappai_amd.kernels import ops
    T, E, top = 19, 5, 3
    g = gen(W)
    x = torch.randn(T, W, generator=g) * 3

    def weights(alpha):
        return alpha, 1 + 0.3 * torch.randn(W, generator=g), 0.5 * torch.randn(W, generator=g)

    def on_gpu(n):
        return ops.TanhNormWeights(n[0], n[1].to(DEV), n[2].to(DEV))

    def n_of(n, v):
        return torch.tanh(n[0] * v) * n[1].double() + n[2].double()

    post, pre = weights(0.7), weights(0.3)
    for kind in ("f32", "bf16", "parts", "terms", "read"):
        y = torch.randn(T, W, generator=g)
        given = y.to(DEV)
        summed = y.double()
        if kind == "bf16":
            given = y.to(BF16).to(DEV)
            summed = y.to(BF16).double()
        elif kind == "parts":
            y = torch.randn(5, T, W, generator=g)
            given, summed = y.to(DEV), y.double().sum(0)
        elif kind == "terms":
            chosen = torch.stack([torch.randperm(E, generator=g)[:top] for _ in range(T)])
            plan = ops.moe_plan(chosen.to(I32).to(DEV), E)
            wts = torch.rand(T, top, generator=g)
            slots = torch.full((plan.n_tiles * plan.tile_rows, W), float("nan"))
            each = torch.randn(T, top, W, generator=g)
            slots[plan.slot_of_pair.cpu().long()] = each.reshape(T * top, W)
            given = ops.ExpertTerms(slots.to(DEV), wts.to(DEV), plan)
            summed = (each.double() * wts.double()[:, :, None]).sum(1)
            assert rel(given.combined(), summed) < 1e-6
        elif kind == "read":
            given, summed = None, torch.zeros(T, W, dtype=F64)
        for post_n in ((None,) if kind == "read" else (post, None)):
            upd = summed if post_n is None else n_of(post_n, summed)
            new = x.double() + upd
            resid = x.clone().to(DEV)
            rows = ops.tanh_norm_step(resid, given, post=post_n and on_gpu(post_n),
                                      pre=on_gpu(pre), rows_dtype=F32)
            assert rel(resid, new) < 1e-6 and rel(rows, n_of(pre, new)) < 1e-6, kind
            rows = ops.tanh_norm_step(x.clone().to(DEV), given, post=post_n and on_gpu(post_n),
                                      pre=on_gpu(pre), rows_dtype=BF16)
            assert rows.dtype == BF16 and rel(rows.float(), n_of(pre, new)) < 5e-3
            resid = x.clone().to(DEV)
            assert ops.tanh_norm_step(resid, given, post=post_n and on_gpu(post_n)) is None
            assert rel(resid, new) < 1e-6
            pick = torch.tensor([17, 0, 5, 17], dtype=I32)
            resid = x.clone().to(DEV)
            rows = ops.tanh_norm_step(resid, given, post=post_n and on_gpu(post_n),
                                      pre=on_gpu(pre), rows=pick.to(DEV), rows_dtype=F32)
            assert torch.equal(resid.cpu(), x)
            assert rel(rows, n_of(pre, new)[pick.long()]) < 1e-6
    with pytest.raises(ValueError, match="tanh_norm_step: y"):
        ops.tanh_norm_step(torch.zeros(4, W, device=DEV), torch.zeros(5, W, device=DEV))


def test_the_norms_own_interface():
    from kappai_amd.parts import TanhNorm
    T, W = 9, 88
    norm = TanhNorm("n", W, BF16)
    t = bind_random(norm, 3, BF16)
    x, d = torch.randn(T, W, generator=gen(1)) * 4, torch.randn(3, T, W, generator=gen(2))
    resid = x.clone().to(DEV)
    rows = norm.norm_output(resid, d.to(DEV), rows_dtype=BF16)
    want = x.double() + P.saturating_norm(d.double().sum(0), t, "n")
    assert rel(resid, want) < 1e-6 and torch.equal(rows, resid.to(BF16))
    got = norm.add_norm(resid, d[0].to(DEV))
    assert rel(resid, want + d[0].double()) < 1e-6
    assert rel(got.float(), P.saturating_norm(want + d[0].double(), t, "n")) < 5e-3


def test_embedded_rows_times_a_constant():
    from kappai_amd.kernels import ops
    table = torch.randn(96, 64, generator=gen(1))
    ids = torch.tensor([3, 95, 0, 41, 3], dtype=I32, device=DEV)
    for t in (table.to(DEV), table.to(BF16).to(DEV), ops.InFragments.of(table.to(BF16).to(DEV))):
        want = (table if t.dtype == F32 else table.to(BF16)).float()[ids.cpu().long()] * 8.25
        assert torch.equal(ops.embed_rows(ids, t, scale=8.25).cpu(), want)
        assert torch.equal(ops.embed_rows(ids, t).cpu() * 8.25, want)


@pytest.mark.parametrize("dtype,tol", [(F32, 2e-6), (BF16, 8e-3)])
@pytest.mark.parametrize("H,G,d,rot", [(6, 2, 16, 0), (3, 3, 24, 0), (4, 1, 64, 32), (2, 2, 10, 4),
                                       (8, 2, 128, 0), (1, 1, 48, 0), (2, 1, 256, 0)])
def test_keys_as_values_beside_per_head_norms(dtype, tol, H, G, d, rot):
    """Queries and keys normed head by head (and rotated), the value of a token the key as it was
    projected, before either."""
    from kappai_amd.kernels import ops
    T, ps, D = 21, 16, 16 * ((d + 15) // 16)
    g = gen(H * 100 + d)
    proj = (torch.randn(T, (H + G) * d, generator=g) * 2).to(dtype)
    pos = torch.arange(T) + 5
    bt = torch.tensor([[3, 1]], dtype=I32)
    cos = sin = None
    if rot:
        ang = torch.randn(64, rot // 2, generator=g)
        cos, sin = torch.cos(ang), torch.sin(ang)
    w = torch.ones(d)
    k_pool = torch.full((4, G, ps, D), float("nan"), dtype=dtype, device=DEV)
    v_pool = torch.full((4, G, D, ps), float("nan"), dtype=dtype, device=DEV)
    q = ops.head_norm_rotate_store(
        proj.to(DEV), H, G, d, d, D, w.to(DEV), w.to(DEV), 1e-5, None if cos is None else cos.to(DEV),
        None if sin is None else sin.to(DEV), rot, ops.ROT_HALF if rot else ops.ROT_NONE, k_pool,
        v_pool, pos.to(I32).to(DEV), torch.zeros(T, dtype=I32, device=DEV), bt.to(DEV), ps,
        values_are_keys=True)

    def turned(x):
        x = P.unit_rms(x, 1e-5)
        if rot:
            c, s = cos[pos].double()[:, None], sin[pos].double()[:, None]
            a, b = x[..., :rot // 2], x[..., rot // 2:rot]
            x = torch.cat([a * c - b * s, a * s + b * c, x[..., rot:]], dim=-1)
        return x

    pd = proj.double()
    want_q = torch.zeros(T, H, D, dtype=F64)
    want_q[..., :d] = turned(pd[:, :H * d].reshape(T, H, d))
    k = pd[:, H * d:].reshape(T, G, d)
    assert rel(q.float(), want_q.reshape(T, H * D)) < tol
    for t in range(T):
        page, slot = int(bt[0, pos[t] // ps]), int(pos[t] % ps)
        key, val = k_pool[page, :, slot].float().cpu(), v_pool[page, :, :, slot].float().cpu()
        assert torch.equal(val[:, :d].double(), k[t]) and bool((val[:, d:] == 0).all())
        assert rel(key[:, :d], turned(k)[t]) < tol and bool((key[:, d:] == 0).all())


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("W,E,top,groups,keep,scale,T", [
    (72, 6, 2, 3, 2, 1.7, 37), (64, 8, 3, 1, 1, 0.5, 150), (48, 3, 3, 1, 1, 1.0, 5),
    (100, 12, 4, 2, 1, 2.5, 64), (67, 64, 8, 8, 3, 1.3, 90), (320, 160, 6, 16, 4, 16.0, 33),
    (96, 130, 16, 13, 13, 1.0, 21), (54, 5, 2, 5, 3, 1.2, 1), (64, 256, 8, 128, 70, 1.0, 9)])
def test_squashed_router(dtype, W, E, top, groups, keep, scale, T):
    """The chosen experts and their weights against the plain choice, with corrections so far below
    zero that an expert of a dropped group at zero would be chosen."""
    from kappai_amd.kernels import ops
    g = gen(E * 31 + top)
    x = torch.randn(T, W, generator=g).to(dtype)
    router = (torch.randn(E, W, generator=g) * 2 / math.sqrt(W)).to(BF16).float()
    corr = -3.0 + 0.8 * torch.randn(E, generator=g)
    cfg = {"experts": E, "top": top, "groups": {"count": groups, "keep": keep}}
    s = torch.sigmoid(x.double() @ router.double().T)
    for c in (corr, None):
        chosen, wts = ops.moe_route_scored(x.to(DEV), router.to(DEV), top, scale,
                                             correction=None if c is None else c.to(DEV),
                                             groups=groups, keep_groups=keep)
        chosen, wts = chosen.cpu(), wts.cpu().double()
        clear = 0
        for i in range(T):
            order, gap = P.choose(s[i], torch.zeros(E) if c is None else c.double(), cfg)
            if gap < 1e-5:
                continue
            clear += 1
            got = dict(zip(chosen[i].tolist(), wts[i].tolist()))
            assert sorted(got) == sorted(order), i
            assert all(abs(got[e] - float(s[i, e]) * scale) < 1e-5 * scale for e in order)
        assert clear >= 0.9 * T
    bias = torch.randn(E, generator=g)
    chosen, wts = ops.moe_route_scored(x.to(DEV), router.to(DEV), top, bias=bias.to(DEV))
    want = torch.sigmoid(x.double() @ router.double().T + bias.double())
    assert rel(wts, want.gather(1, chosen.cpu().long())) < 1e-5
    with pytest.raises(ValueError, match="groups"):
        ops.moe_route_scored(x.to(DEV), router.to(DEV), top, groups=E + 1)


def dense_attention(q, k, v, pos, window, chunk, keep, scale, table, sink, cap=0.0):
    """Float64 reference for rows at positions ``pos``: q [T, H, d], k and v [N, G, d] of all
    positions, table [H, n] by distance (the last column for all beyond), sink [H]."""
    T, H, _ = q.shape
    k, v = (x.repeat_interleave(H // x.shape[1], dim=1) for x in (k, v))
    j = torch.arange(k.shape[0])
    out = torch.zeros(T, H, v.shape[2], dtype=F64)
    for t in range(T):
        p = int(pos[t])
        ok = j <= p
        if window:
            ok &= (p - j < window) | (j < keep)
        if chunk:
            ok &= (j >= p - p % chunk) | (j < keep)
        sc = torch.einsum("hd,jhd->hj", q[t], k[ok]) * scale
        if cap:
            sc = cap * torch.tanh(sc / cap)
        if table is not None:
            sc = sc + table[:, (p - j[ok]).clamp(max=table.shape[1] - 1)]
        if sink is not None:
            w = torch.softmax(torch.cat([sc, sink[:, None]], 1), dim=1)[:, :-1]
        else:
            w = torch.softmax(sc, dim=1)
        out[t] = torch.einsum("hj,jhd->hd", w, v[ok])
    return out.reshape(T, -1)


def paged(x, blocks, ps, transposed):
    """[N, G, d] into NaN-poisoned pages by ``blocks`` (-1: that page is not held)."""
    N, G, d = x.shape
    n_pages = max(blocks) + 2
    pool = torch.full((n_pages, G, d, ps) if transposed else (n_pages, G, ps, d), float("nan"),
                      dtype=x.dtype)
    for p in range(N):
        b = blocks[p // ps]
        if b >= 0:
            if transposed:
                pool[b, :, :, p % ps] = x[p]
            else:
                pool[b, :, p % ps] = x[p]
    return pool.to(DEV)


ATTENTION_CASES = [
    # (H, G, d, window, chunk, keep, table columns, cap, page size)
    (6, 2, 16, 24, 0, 3, 52, 0.0, 16), (4, 1, 48, 17, 0, 20, 9, 0.0, 16),
    (8, 8, 64, 16, 0, 16, 40, 0.0, 16), (8, 2, 64, 33, 0, 40, 300, 0.0, 32),
    (4, 4, 32, 1, 0, 5, 3, 0.0, 16), (4, 2, 128, 96, 0, 1, 242, 30.0, 16),
    (2, 1, 96, 31, 0, 33, None, 0.0, 64), (3, 1, 80, 50, 0, 49, 2, 0.0, 16),
    (16, 1, 16, 20, 0, 64, 130, 0.0, 16), (2, 2, 256, 40, 0, 7, 60, 0.0, 16),
    (4, 2, 32, 0, 48, 10, 70, 0.0, 16), (2, 1, 64, 100, 0, 90, 5000, 0.0, 16),
    (4, 1, 192, 64, 0, 32, 100, 5.0, 16)]


@pytest.mark.parametrize("form", ["rows-f32", "rows", "prefill", "decode-block", "decode-split",
                                  "lone"])
@pytest.mark.parametrize("case", range(len(ATTENTION_CASES)))
def test_attention_kernels_with_kept_first_positions(form, case):
    """Rows of one request at many positions: before the window has passed anything, when the
    window's edge meets the kept tokens, at page borders, far behind.  Pages that the window has
    passed are not held (block table -1) and everything unwritten is NaN."""
    from kappai_amd.kernels import ops
    H, G, d, window, chunk, keep, cols, cap, ps = ATTENTION_CASES[case]
    dtype = F32 if form == "rows-f32" else BF16
    g = gen(1000 * case + 7)
    N, scale = 420, 1.5 / math.sqrt(d)
    q, k, v = (torch.randn(N, n, d, generator=g).to(dtype) for n in (H, G, G))
    table = None if cols is None else torch.randn(H, cols, generator=g) * 1.5
    sink = torch.randn(H, generator=g) + 1
    mods = ops.ScoreMods(cap, None if table is None else table.to(DEV), sink.to(DEV), keep)
    size = window or chunk
    edges = sorted({p for p in (0, 1, 15, 16, 17, 31, 32, 33, keep - 1, keep, keep + 1, size - 1, size,
                                size + 1, size + keep - 1, size + keep, size + keep + 1, 127, 128,
                                200, 255, 256, 300, 383, N - 1) if 0 <= p < N})

    def table_row(first, length):
        """The block table of a request with ``length`` tokens whose oldest row wants ``first``
        (the first position of that row's window)."""
        order = torch.randperm(N // ps + 2, generator=g).tolist()
        return [order[b] if b * ps < length and (b < (keep + ps - 1) // ps or (b + 1) * ps > first)
                else -1 for b in range(N // ps + 1)]

    def first_seen(p):
        if window:
            return max(0, p + 1 - window)
        return p - p % chunk

    tab = None if table is None else table.double()
    dense = lambda rows, pos: dense_attention(q[rows].double(), k.double(), v.double(), pos, window,
                                              chunk, keep, scale, tab, sink.double(), cap)
    tol = 1e-5 if dtype == F32 else 2e-2
    common = dict(window=window, chunk=chunk, mods=mods)
    if form in ("rows-f32", "rows", "decode-block", "decode-split"):
        # every row a request of its own: its own pages and block table
        rows = edges
        if form.startswith("decode") and H // G > 16:
            pytest.skip("at most 16 query heads a kv head")
        blocks, pools_k, pools_v, at = [], [], [], 0
        for p in rows:
            b = table_row(first_seen(p), p + 1)
            kp, vp = paged(k[:p + 1], b, ps, False), paged(v[:p + 1], b, ps, True)
            blocks.append([x + at if x >= 0 else -1 for x in b])
            at += kp.shape[0]
            pools_k.append(kp)
            pools_v.append(vp)
        pos = torch.tensor(rows, dtype=I32)
        got = ops.paged_attention(
            q[rows].reshape(len(rows), H * d).to(DEV), H, G, d, torch.cat(pools_k), torch.cat(pools_v),
            pos.to(DEV), torch.arange(len(rows), dtype=I32, device=DEV),
            torch.tensor(blocks, dtype=I32, device=DEV), ps, scale, single_rows=True,
            max_position=max(rows), kernel=form.replace("-f32", ""), **common)
        want = dense(rows, pos)
        assert rel(got.float(), want) < tol
        return
    # portions of one request, cut at odd places; "lone": a single row beside each portion
    for start, n in ((0, 70), (keep, 1 + size), (97, 33), (max(0, size + keep - 20), 45), (300, 120)):
        n = min(n, N - start)
        rows = list(range(start, start + n))
        lone_pos = N - 1
        if form == "lone":
            rows.append(lone_pos)
        b0 = table_row(first_seen(start), start + n)
        kp, vp = paged(k[:start + n], b0, ps, False), paged(v[:start + n], b0, ps, True)
        blocks = [b0]
        if form == "lone":
            b1 = table_row(first_seen(lone_pos), N)
            blocks.append([x + kp.shape[0] if x >= 0 else -1 for x in b1])
            kp = torch.cat([kp, paged(k, b1, ps, False)])
            vp = torch.cat([vp, paged(v, b1, ps, True)])
        n_tiles = (n + 31) // 32
        tiles = [[0, 32 * i, min(32, n - 32 * i), i | (n_tiles << 16)] for i in range(n_tiles)]
        pos = torch.tensor(rows, dtype=I32)
        more = dict(lone_rows=torch.tensor([n], dtype=I32, device=DEV),
                    max_lone_position=lone_pos) if form == "lone" else {}
        got = ops.paged_attention(
            q[rows].reshape(len(rows), H * d).to(DEV), H, G, d, kp, vp, pos.to(DEV),
            torch.tensor([0] * n + ([1] if form == "lone" else []), dtype=I32, device=DEV),
            torch.tensor(blocks, dtype=I32, device=DEV), ps, scale,
            q_tiles=torch.tensor(tiles, dtype=I32, device=DEV), max_position=max(rows),
            kernel="prefill", **common, **more)
        assert rel(got.float(), dense(rows, pos)) < tol, (start, n)


# ---------------------------------------------------------------------------------------------
# parts
# ---------------------------------------------------------------------------------------------
def attention_dict(H, G, d, scale, far, size, keep):
    m = {"heads": H, "kv_heads": G, "dim": d, "vdim": d, "scale": scale, "bias_max": far}
    if size is not None:
        m["mask"] = {"size": size, "keep_first": keep}
    return m


def make_attention(W, m, buckets, dtype):
    from kappai_amd.parts import ScoredAttention
    mask = m.get("mask") or {}
    return ScoredAttention("a.", W, m["heads"], m["kv_heads"], m["dim"], m["dim"], m["scale"], dtype,
                           norm_eps=1e-5, head_qk_norm=True, head_norm_weight=False,
                           values_from_keys=True, bias_buckets=buckets, bias_far=m["bias_max"],
                           sink=True, window=mask.get("size"), keep_first=mask.get("keep_first", 0),
                           weight_suffix="")


@pytest.mark.parametrize("dtype,tol", [(F32, 2e-5), (BF16, 3e-2)])
@pytest.mark.parametrize("H,G,d,scale,far,buckets,size,keep", [
    (6, 2, 16, 0.3, 50, 10, 24, 3), (3, 3, 24, 0.25, 300, 7, 40, 0), (4, 1, 40, 0.2, 33, 16, 17, 20),
    (8, 8, 8, 0.6, 64, 8, 16, 16), (1, 1, 96, 0.1, 1000, 32, None, 0), (2, 1, 90, 0.15, 20, 2, 1, 5),
    (20, 1, 16, 0.4, 90, 12, 64, 33), (2, 2, 272, 0.05, 40, 6, 30, 18)])
def test_attention_part(dtype, tol, H, G, d, scale, far, buckets, size, keep):
    """Per-head norms, values that are the keys, distance biases, the window beside the first
    tokens and the sinks, over portions down to one token; also more query heads a kv head and
    wider heads than the matrix-core kernels take."""
    from kappai_amd.cache import CacheManager
    m = attention_dict(H, G, d, scale, far, size, keep)
    part = make_attention(72, m, buckets, dtype)
    t = bind_random(part, 4, dtype)
    pages = 10 if size is None else (size + keep + 37) // 16 + 4
    cm = CacheManager([part.cache_spec()], 16, pages, 1)
    cm.allocate_storage(dtype, DEV, poison=True)
    x = torch.randn(150, 72, generator=gen(14)).to(BF16)
    got, _ = step_through(part, cm, x.to(dtype), PORTIONS_150, cm.view(0))
    assert rel(got, P.attention(x.double(), t, "a.", m, 1e-5)) < tol


def needle_case(H, d, size, keep, buckets, far, dtype, scale=0.7):
    """A part whose queries read the first half of the input and whose keys read the second, one
    for one; biases and sinks small."""
    half = H * d
    m = attention_dict(H, H, d, scale, far, size, keep)
    part = make_attention(2 * half, m, buckets, dtype)

    def change(t):
        eye, zero = torch.eye(half), torch.zeros(half, half)
        t["a.q"] = torch.cat([eye, zero], 1).to(BF16)
        t["a.k"] = torch.cat([zero, eye], 1).to(BF16)
        t["a.rel"] = (t["a.rel"].float() * 0.2).to(BF16)
    return part, bind_random(part, 4, dtype, std=0.3, change=change), m, half


def needle_rows(T, needle, half, seed):
    """[T, 2 half]: every query points along ``u``; the needle's key does too, every other key lies
    at right angles to it but for a little noise."""
    u = torch.ones(half) / math.sqrt(half)
    r = u * torch.tensor([1.0, -1.0]).repeat(half // 2)
    x = torch.randn(T, 2 * half, generator=gen(seed)) * 0.02
    x[:, half:] += r
    x[needle, half:] = 3.0 * u
    x[:, :half] += 1.5 * u
    return x.to(BF16)


@pytest.mark.parametrize("dtype,tol", [(F32, 1e-4), (BF16, 5e-2)])
@pytest.mark.parametrize("size,keep", [(40, 6), (48, 16), (33, 17), (100, 0), (64, 70)])
def test_a_key_that_stands_out_at_every_edge(dtype, tol, size, keep):
    """One key takes nearly all the weight of every query that sees it.  It is put at the first
    position, at the last kept one and the next, at page borders and far from both; a query sees it
    while it lies in the window (and not one token longer) or for good when it is kept, in prompts,
    in portions cut right at the edge, and token by token over the edge."""
    from kappai_amd.cache import CacheManager
    part, t, m, half = needle_case(2, 16, size, keep, 8, 60, dtype)
    out_of = lambda x: P.attention(x.double(), t, "a.", m, 1e-5)
    for needle in sorted({0, max(0, keep - 1), keep, 15, 16, 31, 32, 63, 90}):
        T = needle + size + 40
        x = needle_rows(T, needle, half, needle)
        want = out_of(x)
        # the rows on both sides of the edge differ by far more than the tolerance
        inside, outside = needle + size - 1, needle + size
        jump = float((want[inside] - want[outside]).abs().max() / want.abs().max())
        assert (jump < 0.2) if needle < keep else (jump > 0.3), (needle, jump)
        for portions in ([T], [needle + size, T - needle - size], [needle + size - 1, 2, 39],
                         [needle + 1] + [size - 3] + [1] * 42, [3, needle + size + 7] + [2] * 15):
            assert sum(portions) == T
            held = (size + max(portions) + 30) // 16 + (keep + 15) // 16 + 2
            cm = CacheManager([part.cache_spec()], 16, min(held, T // 16 + 1), 1)
            cm.allocate_storage(dtype, DEV, poison=True)
            got, _ = step_through(part, cm, x.to(dtype), portions, cm.view(0))
            err = (got.cpu().double() - want).abs().max(dim=1).values / want.abs().max()
            assert float(err.max()) < tol, (needle, portions[:4], int(err.argmax()), float(err.max()))


@pytest.mark.parametrize("dtype,tol", [(F32, 1e-4), (BF16, 5e-2)])
def test_far_kept_keys_with_their_true_distance(dtype, tol):
    """A kept key hundreds of tokens back wins or loses by the bias of its true distance: the table
    favours the last row by far, then the first ones."""
    from kappai_amd.cache import CacheManager
    from kappai_amd.weights import stored_to_runtime
    for far_bias, near_bias in ((6.0, -3.0), (-6.0, 3.0)):
        part, t, m, half = needle_case(2, 16, 50, 20, 8, 200, dtype, scale=0.2)
        table = torch.full((8, 2), near_bias)
        table[6:] = far_bias
        t["a.rel"] = table.to(BF16)
        part.bind({k: stored_to_runtime(v, dtype).to(DEV) for k, v in t.items()})
        x = needle_rows(480, 9, half, 5)
        want = P.attention(x.double(), t, "a.", m, 1e-5)
        other = dict(t)
        other["a.rel"] = torch.full((8, 2), near_bias).to(BF16)
        shift = P.attention(x.double(), other, "a.", m, 1e-5)
        assert float((want[-1] - shift[-1]).abs().max()) > 0.15 * float(want.abs().max())
        for portions in ([480], [300, 2] + [1] * 178):
            cm = CacheManager([part.cache_spec()], 16, 31, 1)
            cm.allocate_storage(dtype, DEV, poison=True)
            got, _ = step_through(part, cm, x.to(dtype), portions, cm.view(0))
            assert rel(got, want) < tol


@pytest.mark.parametrize("dtype", [F32, BF16])
def test_the_sink_takes_the_weight(dtype):
    """Every key points away from the queries: all scores lie far below the sinks, and the result
    is near nothing, where a softmax without the sink would return a mean of the values."""
    from kappai_amd.cache import CacheManager
    part, t, m, half = needle_case(2, 16, 30, 4, 8, 60, dtype)
    T = 90
    u = torch.ones(half) / math.sqrt(half)
    x = torch.randn(T, 2 * half, generator=gen(7)) * 0.02
    x[:, :half] += 1.5 * u
    x[:, half:] -= u
    x = x.to(BF16)
    want = P.attention(x.double(), t, "a.", m, 1e-5)
    full = float((x.double() @ t["a.k"].double().T @ t["a.o"].double().T).abs().max())
    assert float(want.abs().max()) < 2e-2 * full
    cm = CacheManager([part.cache_spec()], 16, 8, 1)
    cm.allocate_storage(dtype, DEV, poison=True)
    got, _ = step_through(part, cm, x.to(dtype), [40, 2] + [1] * 48, cm.view(0))
    assert float((got.cpu().double() - want).abs().max()) < 1e-3 * full


@pytest.mark.parametrize("dtype,tol", [(F32, 2e-5), (BF16, 3e-2)])
@pytest.mark.parametrize("W,F,E,top,groups,scale,T", [
    (72, 24, 6, 2, (3, 2), 1.7, 37), (64, 32, 8, 3, None, 0.5, 150), (48, 8, 3, 3, None, 1.0, 5),
    (96, 48, 12, 4, (2, 1), 2.5, 300), (100, 40, 10, 4, (5, 3), 1.3, 1), (54, 10, 5, 2, (5, 3), 1.2, 20),
    (64, 64, 16, 2, (4, 2), 1.0, 700)])
def test_experts_with_a_squashed_router(dtype, tol, W, F, E, top, groups, scale, T):
    """The whole feed-forward: with the sum over the experts made here and left to the caller, for
    rows whose choice is no close call."""
    from kappai_amd.parts import MixtureOfExperts
    n, keep = groups or (1, 1)
    part = MixtureOfExperts("f.", W, F, E, top, dtype, weight_suffix="", scoring="sigmoid",
                            correction=True, groups=n, keep_groups=keep, weight_scale=scale)
    t = bind_random(part, 8, dtype)
    x = torch.randn(T, W, generator=gen(18)).to(BF16)
    router = {"experts": E, "top": top, "scale": scale}
    if groups:
        router["groups"] = {"count": n, "keep": keep}
    margins = []
    want = P.moe_ff(x.double(), t, "f.", {"router": router}, margins=margins)
    clear = margins[0] > 1e-4
    assert clear.sum() >= 0.9 * T
    for got in (part.forward(x.to(dtype).to(DEV), None),
                part.forward(x.to(dtype).to(DEV), None, terms=True).combined()):
        got = got.float().cpu().double()
        assert float((got[clear] - want[clear]).abs().max() / want.abs().max()) < tol


@pytest.mark.parametrize("E,P_", [(3, 5), (16, 32), (16, 8192), (64, 4096), (160, 777), (1, 130),
                                  (4096, 200), (5, 64), (8, 1)])
def test_plan_sorts_pairs_by_expert(E, P_):
    """Every pair has a slot in a tile of its expert, in the order of the pairs; other slots are
    empty."""
    from kappai_amd.kernels import ops
    top = 1 if P_ % 2 else 2
    idx = torch.randint(0, E, (P_ // top, top), generator=gen(E + P_), dtype=I32)
    idx[: P_ // top // 3] = E - 1                       # one expert with a long run
    plan = ops.moe_plan(idx.to(DEV), E)
    slot = plan.slot_of_pair.cpu().long()
    back = plan.pair_of_slot.cpu().long()
    tile_expert = plan.tile_expert.cpu().long()
    flat = idx.flatten().long()
    assert slot.unique().numel() == P_ and torch.equal(back[slot], torch.arange(P_))
    assert int((back >= 0).sum()) == P_
    assert torch.equal(tile_expert[slot // plan.tile_rows], flat)
    for e in flat.unique().tolist():
        mine = slot[flat == e]
        assert torch.equal(mine, int(mine[0]) + torch.arange(mine.numel()))
        assert int(mine[0]) % plan.tile_rows == 0


# ---------------------------------------------------------------------------------------------
# whole models
# ---------------------------------------------------------------------------------------------
@pytest.fixture(scope="module")
def model_dirs(tmp_path_factory):
    base = tmp_path_factory.mktemp("nuzivik")
    return {name: write_tiny(name, base / name) for name in TINY}


_models = {}


def gpu_model(model_dir, dtype):
    from kappai_amd.models import load_model
    key = (str(model_dir), dtype)
    if key not in _models:
        _models[key] = load_model(model_dir, dtype, DEV)
    return _models[key]


def replay(model_dir, dtype, steps, index, max_tokens, out_dir, slots=4, graphs=True):
    from kappai_amd.engine.replay import TraceReplayer, make_replay_cache
    from kappai_amd.engine.step import StepRunner
    model = gpu_model(model_dir, dtype)
    cache = make_replay_cache(model, max_tokens, 16, num_slots=slots)
    cache.allocate_storage(model.dtype, DEV, poison=True)
    runner = StepRunner(model, cache, DEV, decode_graphs=graphs)
    rep = TraceReplayer(runner, out_dir)
    outputs = {}
    for obj in steps:
        res = rep.run_step(obj)
        if res is not None:
            outputs[obj["step"]] = res
    cache.check()
    assert not cache.live_requests()
    return collect(index, outputs, model.vocab_size), runner


# a request with less than this share of its rows before a close call says little in bfloat16
MIN_STRICT = {"A": 0.3, "B": 1.0, "C": 0.2, "D": 0.03, "E": 0.1}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["A", "B", "C", "D", "E"])
@pytest.mark.parametrize("family", ["whole", "prefill_then_decode", "changing_portions", "mixed"])
def test_schedules(tmp_path, model_dirs, name, family, dtype):
    """Every logit of every request.  The mixed family runs in a pool smaller than its requests
    together with four state slots, so pages and slots are taken again."""
    requests = make_requests(TINY[name][0]["vocab"],
                             MIXED_LENGTHS[name] if family == "mixed" else LENGTHS[name], seed=21)
    steps, index, peak = getattr(schedules, family)(requests)
    if family == "mixed":
        assert sum(len(t) for t in requests.values()) > peak
    got, runner = replay(model_dirs[name], dtype, steps, index, peak, tmp_path / "out")
    assert len(got) == sum(len(t) for t in requests.values())
    assert_matches_plain(got, model_dirs[name], requests, dtype, (name, family, dtype),
                         min_strict=MIN_STRICT[name])
    if family == "prefill_then_decode":
        assert runner.graph_replays > 0        # single tokens ran from captured graphs


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding(tmp_path, model_dirs, dtype):
    """A short prompt and 330 tokens one by one (windows pass over decoded tokens, pages go back
    and are taken again, the block tables of a graph grow), two requests side by side."""
    for name in ("A", "B", "D"):
        requests = make_requests(TINY[name][0]["vocab"], [350, 290], seed=22)
        plans = {"r0": (0, [20] + [1] * 330), "r1": (5, [3] + [1] * 287)}
        steps, index, peak = schedules.build(requests, plans)
        got, runner = replay(model_dirs[name], dtype, steps, index, peak, tmp_path / name)
        assert_matches_plain(got, model_dirs[name], requests, dtype, (name, dtype),
                             min_strict=1.0 if name == "B" else 0.0)
        assert runner.graph_replays > 250


def test_a_batch_gives_what_its_requests_give_alone(tmp_path, model_dirs):
    """Unequal requests in one step (a long portion, a short one, single tokens) against each
    request stepped alone: the same logits up to rounding, with and without graphs."""
    requests = make_requests(TINY["A"][0]["vocab"], [120, 9, 40], seed=23)
    alone, _ = replay(model_dirs["A"], "float32", *schedules.changing_portions(requests),
                      tmp_path / "alone", graphs=False)
    plans = {"r0": (0, [100] + [1] * 20), "r1": (1, [2, 2] + [1] * 5), "r2": (0, [1, 30, 2, 7])}
    together, _ = replay(model_dirs["A"], "float32", *schedules.build(requests, plans),
                         tmp_path / "together")
    assert alone.keys() == together.keys()
    scale = max(float(np.abs(v).max()) for v in alone.values())
    worst = max(float(np.abs(alone[k] - together[k]).max()) / scale for k in alone)
    assert worst < 1e-5


@pytest.mark.parametrize("name", ["A", "C"])
def test_the_residual_stream_layer_by_layer(model_dirs, name):
    """The stream after every layer of a whole prompt, in float32, against the plain
    implementation's (a layer leaves its last update pending; it is applied here)."""
    from kappai_amd.cache import CacheManager
    from kappai_amd.engine import StepEntry, StepRunner
    model = gpu_model(model_dirs[name], "float32")
    cfg, t = read_model_dir(model_dirs[name])
    tokens = [int(x) for x in np.random.default_rng(3).integers(0, cfg["vocab"], size=61)]
    streams = []
    P.forward(cfg, t, tokens, layers_out=streams)
    cm = CacheManager(model.cache_specs(), 16, 8, 1)
    cm.allocate_storage(model.dtype, DEV, poison=True)
    runner = StepRunner(model, cm, DEV, decode_graphs=False)
    seen = []
    for layer in model.layers:
        inner = layer.forward

        def spy(h, batch, cache, shared_cache=False, inner=inner):
            out = inner(h, batch, cache, shared_cache=shared_cache)
            x = out.resid.clone()
            out.delta.norm.norm_output(x, out.delta.y)
            seen.append(x)
            return out
        layer.forward = spy
    try:
        runner.step([StepEntry(cm.open("a"), tokens, [len(tokens) - 1])])
    finally:
        for layer in model.layers:
            del layer.forward
    assert len(seen) == len(streams)
    for i, (got, want) in enumerate(zip(seen, streams)):
        assert rel(got, want) < 2e-5, i


def test_greedy_generation_through_the_engine(model_dirs):
    """Prompts of unequal length through ``Engine.generate`` (its scheduler cuts the prompts into
    portions of 16 beside decoding) against the plain implementation's greedy choice."""
    from kappai_amd.engine import Engine
    from kappai_amd.sampling import SamplingParams
    for name in ("A", "C"):
        rng = np.random.default_rng(5)
        prompts = [[int(t) for t in rng.integers(0, TINY[name][0]["vocab"], size=n)]
                   for n in (45, 7, 23)]
        cfg, t = read_model_dir(model_dirs[name])
        want = []
        for p in prompts:
            toks = list(p)
            for _ in range(10):
                toks.append(int(P.forward(cfg, t, toks)[-1].argmax()))
            want.append(toks[len(p):])
        eng = Engine(str(model_dirs[name]), dtype="float32", num_pages=24, max_batch=3, chunk=16,
                     token_budget=24)
        got = eng.generate(prompts, SamplingParams.greedy(n_predict=10))
        assert got == want
        assert eng.cache.num_free_slots == 3
        assert all(g.allocator.num_used == 0 for g in eng.cache.paged_groups)
        eng.shutdown()


def test_command_line(model_dirs, tmp_path):
    """The command line on a model folder and in random-weights mode (a named shape), with the
    sampling options of any other model."""
    import subprocess
    import sys
    from pathlib import Path
    root = Path(__file__).resolve().parent.parent
    prompt = [5, 17, 3, 88, 41, 7, 120]
    cfg, t = read_model_dir(model_dirs["A"])
    toks = list(prompt)
    for _ in range(6):
        toks.append(int(P.forward(cfg, t, toks)[-1].argmax()))
    out = subprocess.run(
        [sys.executable, "-m", "kappai_amd", "-m", str(model_dirs["A"]), "--dtype", "float32",
         "-p", ",".join(map(str, prompt)), "-n", "6", "-t", "0", "--num-pages", "16", "--time"],
        cwd=str(root), capture_output=True, text=True, timeout=300)
    assert out.returncode == 0, out.stderr
    assert [int(x) for x in out.stdout.split()] == toks[len(prompt):]
    assert "router" in out.stderr and "attn" in out.stderr
    made = tmp_path / "made"
    out = subprocess.run(
        [sys.executable, str(root / "bin" / "kappai-cli"), "--random-weights", "nuzivik-tiny",
         "--model", str(made), "--weight-seed", "2", "--weight-std", "0.1", "-n", "5", "-t", "0.8",
         "-k", "20", "-s", "3", "--num-pages", "16", "7 8 9 10"],
        cwd=str(tmp_path), capture_output=True, text=True, timeout=300)
    assert out.returncode == 0, out.stderr
    assert len(out.stdout.split()) == 5 and (made / "config.json").is_file()
