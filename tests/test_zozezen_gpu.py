"""The Zozezen decoder on the GPU against the plain implementation (tests/plain/zozezen.py): every
new kernel alone (RMS norms on both sides of a sublayer in one pass, the convolution in whole pieces
and for single rows, the state-space walk and its chunks on the matrix cores, the gate before a
grouped norm, the softmax router with groups, experts without tensors and a gate row, clamped
experts), the attention with keys of its own and on another layer's, the state-space mixer and the
mixture of experts over portions and single tokens, keys made to stand out far back and at page
borders, a token that only the state remembers, a sink that decides, whole models of five tiny
configurations under the four schedule families in float32 and bfloat16 with pools so small that
pages and slots are used again, long decoding, a batch against its requests alone, the residual
stream after every layer, and greedy generation through the engine and its scheduler."""
import math

import numpy as np
import pytest
import torch

import schedules
from plain import zozezen as P
from replay_common import collect, make_requests
from tiny_zozezen import TINY, assert_matches_plain, read_model_dir, telling, write_tiny

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
F32, BF16, F64, I32 = torch.float32, torch.bfloat16, torch.float64, torch.int32

LENGTHS = {"A": [70, 45, 100, 37], "B": [66, 35, 90], "C": [50, 300, 129], "D": [40, 75, 130],
           "E": [61, 30, 45]}
MIXED_LENGTHS = {"A": [70, 45, 100, 37, 83, 64, 29, 58], "B": [66, 35, 90, 41, 23, 77, 50, 62, 88],
                 "C": [50, 181, 36, 67, 144, 72, 90, 33, 58], "D": [40, 75, 52, 33, 61, 28, 97],
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


def one_segment_batch(cm, n, rc=None):
    """A RowBatch for ``n`` more tokens of one request, with the tables the parts ask for (tiles of
    query rows, chunks of rows for the scan)."""
    from kappai_amd.engine import StepEntry, StepRunner
    from kappai_amd.kernels import ops
    from kappai_amd.parts.attention import AttentionTiles
    from kappai_amd.parts.mingru import ScanChunks
    rc = rc or cm.open("r")
    cm.extend(rc, n)
    runner = StepRunner.__new__(StepRunner)
    runner.model = type("M", (), {"vocab_size": 10 ** 9})()
    runner.step_tables = [AttentionTiles(ops.ATTENTION_TILE_ROWS),
                          ScanChunks(ops.STATE_SPACE_CHUNK_ROWS)]
    runner.cache, runner.device, runner._staging, runner._staged = cm, torch.device(DEV), None, None
    return rc, runner.make_batch([StepEntry(rc, [0] * n, [])])


def summed(y):
    return y if y.dim() == 2 else y.sum(0)


def step_through(part, cm, x, portions, view, reader=None):
    """One request through a mixer in ``portions``; returns the outputs in order.  ``reader``: another
    mixer that reads what this one keeps; its outputs come second."""
    rc, outs, more, done = None, [], [], 0
    for n in portions:
        rc, b = one_segment_batch(cm, n, rc=rc)
        rows = x[done:done + n].to(DEV)
        outs.append(summed(part.forward(rows, b, view)))
        if reader is not None:
            more.append(summed(reader.forward(rows, b, view, shared_cache=True)))
        cm.commit(rc, n)
        cm.check()
        done += n
    assert done == x.shape[0]
    if reader is not None:
        return torch.cat(outs).float(), torch.cat(more).float()
    return torch.cat(outs).float(), rc


PORTIONS_150 = [37, 3] + [1] * 50 + [2, 33] + [1] * 25


def tables(segments):
    """The row tables for segments [(first position, rows, slot), ...]."""
    pos, seg, start = [], [], [0]
    for s, (p0, n, _) in enumerate(segments):
        pos += range(p0, p0 + n)
        seg += [s] * n
        start.append(start[-1] + n)
    i32 = lambda v: torch.tensor(v, dtype=I32, device=DEV)
    return {"row_pos": i32(pos), "row_seg": i32(seg), "seg_start": i32(start),
            "seg_pos0": i32([p for p, _, _ in segments]),
            "seg_slot": i32([s for _, _, s in segments])}


def chunk_tables(segments, rows):
    chunks, first, row = [], [0], 0
    for s, (_, n, _) in enumerate(segments):
        for at in range(0, n, rows):
            chunks.append([s, row + at, min(rows, n - at)])
        row += n
        first.append(len(chunks))
    return (torch.tensor(chunks, dtype=I32, device=DEV), torch.tensor(first, dtype=I32, device=DEV))


# ---------------------------------------------------------------------------------------------
# kernels alone
# ---------------------------------------------------------------------------------------------
@pytest.mark.parametrize("W", [72, 64, 328, 2048, 100, 67, 30, 4096, 4100, 1100, 8192, 5001])
def test_rms_norms_on_both_sides_in_one_pass(W):
    """Norm of the update, sum and norm of the new stream in one kernel, against their formulas in
    float64: the update as float32 rows, bfloat16 rows, float32 partial sums and a mixture's
    experts' results (alone; with a shared expert's rows or partial sums behind a gate and experts
    that hand their input on); with and without the norm on it; the read alone; some rows only."""
    from kappai_amd.kernels import ops
    T, E, top = 11, 5, 3
    g = gen(W)
    x = torch.randn(T, W, generator=g) * 3
    post = (1 + 0.3 * torch.randn(W, generator=g), 1e-5)
    pre = (1 + 0.3 * torch.randn(W, generator=g), 1e-2)

    def on_gpu(n):
        return n[0].to(DEV), n[1]

    def n_of(n, v):
        return v / torch.sqrt((v * v).mean(-1, keepdim=True) + n[1]) * n[0].double()

    for kind in ("f32", "bf16", "parts", "terms", "more-f32", "more-bf16", "read"):
        y = torch.randn(T, W, generator=g)
        given, summed_ = y.to(DEV), y.double()
        if kind == "bf16":
            given = y.to(BF16).to(DEV)
            summed_ = y.to(BF16).double()
        elif kind == "parts":
            y = torch.randn(5, T, W, generator=g)
            given, summed_ = y.to(DEV), y.double().sum(0)
        elif kind == "read":
            given, summed_ = None, torch.zeros(T, W, dtype=F64)
        elif kind != "f32":
            more = kind != "terms"
            n_real = E - 2 if more else E
            chosen = torch.stack([torch.randperm(E, generator=g)[:top] for _ in range(T)])
            plan = ops.moe_plan(chosen.to(I32).to(DEV), n_real)
            slot = plan.slot_of_pair.cpu().long()
            real = (chosen < n_real).flatten()
            assert torch.equal(slot >= 0, real)
            wts = torch.rand(T, top, generator=g)
            slots = torch.full((plan.n_tiles * plan.tile_rows, W), float("nan"))
            each = torch.randn(T, top, W, generator=g)
            slots[slot[real]] = each.reshape(T * top, W)[real]
            dt = BF16 if kind == "more-bf16" else F32
            rows_in = torch.randn(T, W, generator=g).to(dt)
            also = (torch.randn(T, W, generator=g).to(BF16) if kind == "more-bf16" else
                    torch.randn(3, T, W, generator=g)) if more else None
            gate = torch.rand(T, generator=g)
            each = torch.where((chosen < n_real)[:, :, None], each, rows_in.float()[:, None, :])
            summed_ = (each.double() * wts.double()[:, :, None]).sum(1)
            given = ops.ExpertTerms(slots.to(DEV), wts.to(DEV), plan)
            if more:
                a = also.double() if also.dim() == 2 else also.double().sum(0)
                summed_ = summed_ + a * gate.double()[:, None]
                given.also, given.also_gate, given.rows = also.to(DEV), gate.to(DEV), rows_in.to(DEV)
            assert rel(given.combined(), summed_) < 1e-6
        for post_n in ((None,) if kind == "read" else (post, None)):
            new = x.double() + (summed_ if post_n is None else n_of(post_n, summed_))
            resid = x.clone().to(DEV)
            rows = ops.rms_norm_step(resid, given, post=post_n and on_gpu(post_n), pre=on_gpu(pre),
                                     rows_dtype=F32)
            assert rel(resid, new) < 2e-6 and rel(rows, n_of(pre, new)) < 2e-6, kind
            rows = ops.rms_norm_step(x.clone().to(DEV), given, post=post_n and on_gpu(post_n),
                                     pre=on_gpu(pre), rows_dtype=BF16)
            assert rows.dtype == BF16 and rel(rows.float(), n_of(pre, new)) < 5e-3
            resid = x.clone().to(DEV)
            assert ops.rms_norm_step(resid, given, post=post_n and on_gpu(post_n)) is None
            assert rel(resid, new) < 2e-6
            pick = torch.tensor([8, 0, 5, 8], dtype=I32)
            resid = x.clone().to(DEV)
            rows = ops.rms_norm_step(resid, given, post=post_n and on_gpu(post_n), pre=on_gpu(pre),
                                     rows=pick.to(DEV), rows_dtype=F32)
            assert torch.equal(resid.cpu(), x)
            assert rel(rows, n_of(pre, new)[pick.long()]) < 2e-6
    with pytest.raises(ValueError, match="rms_norm_step: y"):
        ops.rms_norm_step(torch.zeros(4, W, device=DEV), torch.zeros(5, W, device=DEV))


def test_rms_norm_steps_of_one_value_wider_than_the_kernel_takes():
    from kappai_amd.kernels import ops
    from kappai_amd.parts import RMSNorm
    from kappai_amd.parts.base import NormedUpdate
    W = ops.RMS_STEP_MAX_WIDTH + 8
    with pytest.raises(ValueError, match="resid"):
        ops.rms_norm_step(torch.zeros(2, W, device=DEV))
    a, b = (RMSNorm(n, W, 1e-5, F32, suffix="", weight_offset=1.0) for n in "ab")
    ta, tb = bind_random(a, 1, F32), bind_random(b, 2, F32)
    x, y = torch.randn(3, W, generator=gen(3)), torch.randn(3, W, generator=gen(4))
    resid = x.clone().to(DEV)
    rows = b.add_norm(resid, NormedUpdate(y.to(DEV), a))
    new = x.double() + P.one_plus_norm(y.double(), ta["a"], 1e-5)
    assert rel(resid, new) < 2e-6 and rel(rows, P.one_plus_norm(new, tb["b"], 1e-5)) < 2e-6


@pytest.mark.parametrize("taps", [1, 2, 3, 4, 5, 8])
@pytest.mark.parametrize("dtype,C", [(F32, 40), (BF16, 40), (BF16, 2056), (BF16, 37)])
def test_convolution_with_bias_over_portions_and_slots(taps, dtype, C):
    """Three requests side by side in slots of states that hold NaN, in portions down to one row (and
    steps of nothing but single rows), against the whole sequences at once."""
    from kappai_amd.kernels import ops
    w, bias = torch.randn(C, taps, generator=gen(6)) * 0.5, torch.randn(C, generator=gen(5))
    lens = [7, 1, 1, 2, 9, 1, 1, 12, 3]
    xs = [torch.randn(sum(lens) + 6, C + 8, generator=gen(7 + i)).to(BF16) for i in range(3)]
    state = torch.full((6, taps - 1, C), float("nan"), device=DEV)
    outs, done = [[], [], []], [0, 0, 0]
    for k, n in enumerate(lens):
        ns = [n, n, 1 if n == 1 else n + (1 if k % 3 == 0 else 0)]
        segs = [(done[i], ns[i], slot) for i, slot in enumerate((3, 1, 4))]
        tb = tables(segs)
        x = torch.cat([xs[i][done[i]:done[i] + ns[i]] for i in range(3)]).to(dtype).to(DEV)
        for act in (False, True):                  # the last one brings the histories up to date
            st = state if act else state.clone()
            y = ops.conv_silu(x, w.to(DEV), st, tb["row_pos"], tb["row_seg"], tb["seg_start"],
                              tb["seg_pos0"], tb["seg_slot"], bias=bias.to(DEV), activation=act)
        for i, part in enumerate(y.split(ns)):
            outs[i].append(part)
            done[i] += ns[i]
    for i in range(3):
        want = P.short_conv(xs[i][:done[i], :C].double(), w, bias)
        assert rel(torch.cat(outs[i]).float(), want) < (1e-5 if dtype == F32 else 1e-2)


STATE_SPACE_CASES = [
    # (H, G, N, dv): sizes for the chunks and for the walk only
    (4, 2, 32, 16), (8, 1, 64, 64), (6, 3, 128, 72), (2, 2, 16, 8), (3, 1, 256, 40), (4, 4, 40, 136),
    (2, 1, 8, 200), (4, 1, 136, 64),
    (3, 1, 7, 10), (5, 5, 33, 9), (2, 1, 1, 1), (2, 1, 300, 24), (1, 1, 600, 6), (6, 2, 20, 12)]


def state_space_case(H, G, N, dv, lengths, dtype, seed=0, z_shift=0.0):
    g = gen(100 * H + N + seed)
    cols = H * dv + 2 * G * N
    rows = [torch.randn(n, cols, generator=g).to(BF16) for n in lengths]
    zs = [(torch.randn(n, H, generator=g) + z_shift).to(BF16) for n in lengths]
    vec = {"z_bias": torch.randn(H, generator=g) - 1,
           "rate": torch.exp(-1.5 + 1.5 * torch.randn(H, generator=g)),
           "skip": 1 + 0.5 * torch.randn(H, generator=g)}
    want = []
    for x, z in zip(rows, zs):
        xx, B, C = x.double().split([H * dv, G * N, G * N], dim=1)
        n = x.shape[0]
        dt = torch.nn.functional.softplus(z.double() + vec["z_bias"].double())
        want.append(P.state_space(xx.reshape(n, H, dv), B.reshape(n, G, N), C.reshape(n, G, N), dt,
                                  vec["rate"].double(), vec["skip"].double()).reshape(n, H * dv))
    return rows, zs, {k: v.to(DEV) for k, v in vec.items()}, want


@pytest.mark.parametrize("form,case", [
    (form, i) for i, (_, _, N, dv) in enumerate(STATE_SPACE_CASES)
    for form in ("walk-f32", "walk", "chunks-128", "chunks-50", "chunks-16")
    if form.startswith("walk") or (N % 8 == 0 and dv % 8 == 0 and N <= 256)])
def test_state_space_recurrence(form, case):
    """Three requests side by side, in portions of several chunks, a few rows and one row, in states
    that hold NaN before, against the recurrence in float64 token by token; every form carries on
    from what the others would have left.  Chunks keep float32's accuracy although they run on the
    matrix cores."""
    from kappai_amd.kernels import ops
    H, G, N, dv = STATE_SPACE_CASES[case]
    dtype = F32 if form == "walk-f32" else BF16
    lengths = [345, 150, 61] if form.startswith("chunks") else [75, 40, 21]
    plan = ([[200, 3, 1], [1, 130, 2], [129, 1, 57], [15, 16, 1]] if form.startswith("chunks") else
            [[40, 3, 1], [1, 30, 2], [33, 1, 17], [1, 6, 1]])
    rows, zs, vec, want = state_space_case(H, G, N, dv, lengths, dtype)
    state = torch.full((5, H, dv, N), float("nan"), device=DEV)
    done, outs = [0, 0, 0], [[], [], []]
    for ns in plan:
        segs = [(done[i], ns[i], slot) for i, slot in enumerate((4, 0, 2))]
        tb = tables(segs)
        x = torch.cat([rows[i][done[i]:done[i] + ns[i]] for i in range(3)]).to(dtype).to(DEV)
        z = torch.cat([zs[i][done[i]:done[i] + ns[i]] for i in range(3)]).to(dtype)
        z = torch.cat([z, torch.full((z.shape[0], 3), float("nan"), dtype=dtype)], 1).to(DEV)
        kw = {}
        if form.startswith("chunks"):
            n = int(form.split("-")[1])
            ch, first = chunk_tables(segs, n)
            kw = dict(chunks=ch, seg_chunk0=first, chunk_rows=n)
        y = ops.state_space(x, z, H, G, N, dv, state=state, seg_start=tb["seg_start"],
                            seg_pos0=tb["seg_pos0"], seg_slot=tb["seg_slot"], **vec, **kw)
        for i, part in enumerate(y.split(ns)):
            outs[i].append(part)
            done[i] += ns[i]
    for i in range(3):
        assert done[i] == lengths[i]
        assert rel(torch.cat(outs[i]), want[i]) < 1e-5, i
    assert bool(state[[1, 3]].isnan().all())


@pytest.mark.parametrize("z_shift", [-12.0, 4.0, 30.0])
def test_state_space_with_extreme_steps(z_shift):
    """Decays within 1e-5 of one over hundreds of tokens, and decays that leave nothing: the chunks
    against the float64 recurrence."""
    from kappai_amd.kernels import ops
    H, G, N, dv, T = 4, 2, 64, 32, 300
    rows, zs, vec, want = state_space_case(H, G, N, dv, [T], BF16, seed=3, z_shift=z_shift)
    seg = [(0, T, 0)]
    tb, (ch, first) = tables(seg), chunk_tables(seg, 128)
    for kw in (dict(chunks=ch, seg_chunk0=first, chunk_rows=128), {}):
        state = torch.full((1, H, dv, N), float("nan"), device=DEV)
        y = ops.state_space(rows[0].to(DEV), zs[0].to(DEV), H, G, N, dv, state=state,
                            seg_start=tb["seg_start"], seg_pos0=tb["seg_pos0"],
                            seg_slot=tb["seg_slot"], **vec, **kw)
        assert rel(y, want[0]) < 2e-5


@pytest.mark.parametrize("dtype,tol", [(F32, 2e-6), (BF16, 6e-3)])
@pytest.mark.parametrize("parts,n", [(1, 72), (4, 16), (2, 512), (8, 512), (1, 4096), (3, 1000), (1, 8192),
                                     (5, 6), (2, 700), (1, 9000)])
@pytest.mark.parametrize("kind", [0, 1])
def test_a_gate_before_and_behind_a_grouped_norm(dtype, tol, parts, n, kind):
    from kappai_amd.kernels import ops
    T, g = 7, gen(parts * n)
    o = torch.randn(T, parts * n, generator=g) * 2
    gate = torch.randn(T, parts * n + 8, generator=g).to(BF16)
    w = 1 + 0.2 * torch.randn(parts, n, generator=g)
    gd = gate[:, :parts * n].double()
    s = (gd if kind == ops.GATE_SILU else 1.0) * torch.sigmoid(gd)
    for first in (True, False):
        x = o.double() * (s if first else 1.0)
        want = P.unit_rms(x.reshape(T, parts, n), 1e-5) * w.double()
        want = want.reshape(T, -1) * (1.0 if first else s)
        got = ops.head_norm_gate(o.to(DEV), w.to(DEV), 1e-5, gate.to(dtype).to(DEV), kind, parts, n,
                                 dtype, gate_first=first)
        assert rel(got.float(), want) < tol


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("W,E,top,groups,keep,T", [
    (72, 9, 2, 3, 2, 37), (64, 8, 3, 1, 1, 150), (48, 4, 4, 1, 1, 5), (100, 12, 4, 2, 1, 64),
    (67, 64, 8, 8, 3, 90), (320, 160, 6, 16, 4, 33), (96, 130, 16, 13, 13, 21), (54, 5, 2, 5, 3, 1),
    (64, 256, 8, 128, 70, 9), (2048, 20, 4, 4, 2, 70), (128, 15, 3, 3, 1, 40), (128, 31, 3, 1, 1, 40)])
def test_router_with_a_softmax_over_all_experts(dtype, W, E, top, groups, keep, T):
    """The chosen experts and their weights against the plain choice, with corrections below zero (an
    expert of a dropped group at zero would be chosen); the gate row beside them."""
    from kappai_amd.kernels import ops
    g = gen(E * 31 + top)
    x = torch.randn(T, W, generator=g).to(dtype)
    router = (torch.randn(E + 1, W, generator=g) * 2 / math.sqrt(W)).to(BF16).float()
    corr = -1.0 + 0.2 * torch.randn(E, generator=g)
    cfg = {"top": top, "groups": {"count": groups, "keep": keep}}
    s = torch.softmax(x.double() @ router[:E].double().T, dim=-1)
    want_gate = torch.sigmoid(x.double() @ router[E].double())
    for c, gate in ((corr, True), (None, True), (corr, False)):
        out = ops.moe_route_scored(x.to(DEV), router.to(DEV) if gate else router[:E].to(DEV), top, 1.5,
                                   correction=None if c is None else c.to(DEV), groups=groups,
                                   keep_groups=keep, score="softmax", group_best=1, gate=gate)
        if gate:
            assert rel(out[2], want_gate) < 1e-5
        chosen, wts = out[0].cpu(), out[1].cpu().double()
        clear = 0
        for i in range(T):
            order, gap = P.choose(s[i], torch.zeros(E) if c is None else c.double(), cfg)
            if gap < 1e-6:
                continue
            clear += 1
            got = dict(zip(chosen[i].tolist(), wts[i].tolist()))
            assert sorted(got) == sorted(order), i
            assert all(abs(got[e] - 1.5 * float(s[i, e])) < 1e-5 for e in order)
        assert clear >= 0.9 * T
    with pytest.raises(ValueError, match="score"):
        ops.moe_route_scored(x.to(DEV), router.to(DEV), top, score="tanh")


@pytest.mark.parametrize("E,identity,P_", [(3, 2, 5), (16, 4, 32), (16, 4, 8192), (64, 64, 4096),
                                           (1, 3, 130), (5, 1, 64), (8, 8, 1)])
def test_plan_leaves_out_experts_without_tensors(E, identity, P_):
    from kappai_amd.kernels import ops
    idx = torch.randint(0, E + identity, (P_, 1), generator=gen(E + P_), dtype=I32)
    idx[: P_ // 3] = E                                      # a long run that has no place
    plan = ops.moe_plan(idx.to(DEV), E)
    slot, back = plan.slot_of_pair.cpu().long(), plan.pair_of_slot.cpu().long()
    flat = idx.flatten().long()
    real = flat < E
    assert torch.equal(slot >= 0, real) and bool((slot[~real] == -1).all())
    assert torch.equal(back[slot[real]], torch.arange(P_)[real])
    assert int((back >= 0).sum()) == int(real.sum())
    assert torch.equal(plan.tile_expert.cpu().long()[slot[real] // plan.tile_rows], flat[real])


@pytest.mark.parametrize("dtype,tol", [(F32, 1e-5), (BF16, 1e-2)])
@pytest.mark.parametrize("F", [24, 7, 64])
def test_clamped_gate_of_a_dense_product(dtype, tol, F):
    from kappai_amd.kernels import ops
    x = (torch.randn(9, 2 * F, generator=gen(F)) * 3).to(dtype)
    g, u = x[:, :F].double().clamp(max=1.3), x[:, F:].double().clamp(-1.3, 1.3)
    want = g * torch.sigmoid(1.5 * g) * (u + 0.5)
    assert rel(ops.glu(x.to(DEV), ops.GLU_CLAMPED, ops.ClampedGate(1.3, 1.5, 0.5)).float(),
               want) < tol
    with pytest.raises(ValueError, match="constants"):
        ops.glu(x.to(DEV), ops.GLU_CLAMPED)


@pytest.mark.parametrize("M", [1, 8, 16, 20, 33, 64, 100, 300, 2100])
@pytest.mark.parametrize("F,K", [(64, 64), (48, 72), (512, 256)])
def test_clamped_gate_in_the_epilogue_of_a_product(M, F, K):
    """Every form of the gated product kernels, at row counts that select each, against its formula;
    inputs wide enough for the limit to bite on both sides."""
    from kappai_amd.kernels import ops
    g = gen(M + F)
    x = torch.randn(M, K, generator=g).to(BF16)
    wg, wu = ((torch.randn(F, K, generator=g) * 2 / math.sqrt(K)).to(BF16) for _ in range(2))
    w = ops.interleave_gate_up(wg, wu).to(DEV)
    a, b = x.double() @ wg.double().T, x.double() @ wu.double().T
    a, b = a.clamp(max=1.3), b.clamp(-1.3, 1.3)
    want = a * torch.sigmoid(1.6 * a) * (b + 0.75)
    clamp = ops.ClampedGate(1.3, 1.6, 0.75)
    forms = [w] + ([ops.InFragments.of(w)] if ops.InFragments.of(w) is not None else [])
    for m in forms:
        got = ops.linear_swiglu(x.to(DEV), m, activation=ops.GLU_CLAMPED, clamp=clamp)
        assert rel(got.float(), want) < 1e-2
    with pytest.raises(ValueError, match="constants"):
        ops.linear_swiglu(x.to(DEV), w, activation=ops.GLU_CLAMPED)


# ---------------------------------------------------------------------------------------------
# parts
# ---------------------------------------------------------------------------------------------
def make_attention(W, m, dtype, own=True, prefix="a."):
    from kappai_amd.parts import RotaryEncoding, ScoredAttention
    rot = m.get("rot")
    return ScoredAttention(prefix, W, m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["scale"], dtype,
                           norm_eps=1e-5, head_qk_norm=True, sink_value=0.0, head_gate=True,
                           position=RotaryEncoding(m["dim"], rot["base"], rot["dims"]) if rot else None,
                           own_keys=own, weight_suffix="")


def attention_dict(H, G, d, dv, scale, rot):
    m = {"heads": H, "kv_heads": G, "dim": d, "vdim": dv, "scale": scale}
    if rot:
        m["rot"] = {"base": rot[0], "dims": rot[1]}
    return m


@pytest.mark.parametrize("dtype,tol", [(F32, 2e-5), (BF16, 3e-2)])
@pytest.mark.parametrize("H,G,d,dv,scale,rot", [
    (6, 2, 16, 24, 0.3, (1e4, 8)), (4, 1, 64, 32, 0.15, (1e6, 64)), (8, 8, 8, 16, 0.6, None),
    (3, 1, 10, 14, 0.4, (700.0, 6)), (20, 1, 16, 8, 0.4, (1e4, 16)), (6, 3, 64, 96, 0.12, (1e4, 32)),
    (2, 2, 272, 16, 0.05, (1e5, 16)), (1, 1, 128, 128, 0.1, (1e4, 128))])
def test_attention_with_keys_of_its_own_and_on_another_layers(dtype, tol, H, G, d, dv, scale, rot):
    """Per-head norms, rotation, the one in the denominator and the gates over portions down to one
    token; a second mixer with queries, gates and a scale of its own on the same keys and values."""
    from kappai_amd.cache import CacheManager
    m = attention_dict(H, G, d, dv, scale, rot)
    m2 = dict(m, scale=scale * 1.7)
    part, reader = make_attention(72, m, dtype), make_attention(72, m2, dtype, own=False, prefix="b.")
    t, t2 = bind_random(part, 4, dtype), bind_random(reader, 5, dtype)
    cm = CacheManager([part.cache_spec()], 16, 10, 1)
    cm.allocate_storage(dtype, DEV, poison=True)
    x = torch.randn(150, 72, generator=gen(14)).to(BF16)
    got, read = step_through(part, cm, x.to(dtype), PORTIONS_150, cm.view(0), reader=reader)
    made = []
    want = P.attention(x.double(), t, "a.", m, 1e-5, made=made)
    assert rel(got, want) < tol
    want2 = P.attention(x.double(), t2, "b.", m2, 1e-5, kv=made[0])
    assert rel(read, want2) < tol
    assert float((want - want2).abs().max()) > 0.2 * float(want.abs().max())


@pytest.mark.parametrize("variant", [1, 2])
@pytest.mark.parametrize("H,G,d", [(8, 2, 64), (4, 1, 64), (8, 1, 128), (16, 4, 128)])
def test_a_sink_in_both_forms_of_the_prompt_kernel(variant, H, G, d):
    """The tiled kernel whose blocks share key tiles among four heads, and the one of a block a head,
    with a sink a head from negligible to overwhelming; portions that start at a page's border and
    in the middle of one."""
    from kappai_amd.kernels import ops
    N, ps, scale = 300, 16, 1.0 / math.sqrt(d)
    g = gen(H + d)
    q, k, v = (torch.randn(N, n, d, generator=g).to(BF16) for n in (H, G, G))
    sink = torch.linspace(-60.0, 9.0, H)
    sink[1] = 0.0
    n_pages = (N + ps - 1) // ps
    order = torch.randperm(n_pages, generator=g)
    kp = torch.full((n_pages, G, ps, d), float("nan"), dtype=BF16)
    vp = torch.full((n_pages, G, d, ps), float("nan"), dtype=BF16)
    for p in range(N):
        kp[order[p // ps], :, p % ps] = k[p]
        vp[order[p // ps], :, :, p % ps] = v[p]
    kk, vv = (x.double().repeat_interleave(H // G, dim=1) for x in (k, v))
    sc = torch.einsum("ihd,jhd->hij", q.double(), kk) * scale
    sc = sc.masked_fill(torch.arange(N)[None, :] > torch.arange(N)[:, None], -math.inf)
    w = torch.softmax(torch.cat([sc, sink.double()[:, None, None].expand(-1, N, 1)], 2), 2)[..., :-1]
    want = torch.einsum("hij,jhd->ihd", w, vv).reshape(N, -1)
    for start, n in ((0, N), (32, 200), (77, 33), (N - 2, 2)):
        nt = (n + 31) // 32
        tiles = [[0, 32 * i, min(32, n - 32 * i), i | (nt << 16)] for i in range(nt)]
        i32 = lambda x: torch.tensor(x, dtype=I32, device=DEV)
        got = ops.paged_attention(
            q[start:start + n].reshape(n, H * d).to(DEV), H, G, d, kp.to(DEV), vp.to(DEV),
            i32(list(range(start, start + n))), i32([0] * n), order.to(I32)[None].to(DEV), ps, scale,
            q_tiles=i32(tiles), max_position=start + n - 1, kernel="prefill",
            prefill_variant=variant, mods=ops.ScoreMods(0.0, None, sink.to(DEV)))
        assert rel(got.float(), want[start:start + n]) < 2e-2, (start, n)


def needle_case(H, d, dtype, scale):
    """A part whose queries read the first half of the input and whose keys and values read the second,
    one for one; norm weights of one and open gates."""
    half = H * d
    m = attention_dict(H, H, d, d, scale, None)
    part = make_attention(2 * half, m, dtype)

    def change(t):
        eye, zero = torch.eye(half), torch.zeros(half, half)
        t["a.q"] = torch.cat([eye, zero], 1).to(BF16)
        t["a.k"] = t["a.v"] = torch.cat([zero, eye], 1).to(BF16)
        t["a.q.norm"] = t["a.k.norm"] = torch.ones(d).to(BF16)
        t["a.g"] = torch.zeros_like(t["a.g"])
    return part, bind_random(part, 4, dtype, std=0.3, change=change), m, half


@pytest.mark.parametrize("dtype,tol", [(F32, 1e-4), (BF16, 5e-2)])
@pytest.mark.parametrize("needle", [0, 1, 15, 16, 31, 127, 128, 300])
def test_a_key_far_back_that_takes_the_weight(dtype, tol, needle):
    """One key among hundreds at right angles to every query takes most of the weight, from the first
    position, page borders and the middle; in prompts, in portions cut right behind it, and token by
    token hundreds of tokens later.  Without that key the rows would be something else entirely."""
    from kappai_amd.cache import CacheManager
    part, t, m, half = needle_case(2, 16, dtype, 0.7)
    T = needle + 260
    u = torch.ones(half) / math.sqrt(half)
    r = u * torch.tensor([1.0, -1.0]).repeat(half // 2)
    x = torch.randn(T, 2 * half, generator=gen(needle)) * 0.02
    x[:, half:] += r
    x[needle, half:] = 3.0 * u
    x[:, :half] += 1.5 * u
    x = x.to(BF16)
    want = P.attention(x.double(), t, "a.", m, 1e-5)
    without = x.clone()
    without[needle, half:] = r.to(BF16)
    gone = P.attention(without.double(), t, "a.", m, 1e-5)
    assert float((want[-1] - gone[-1]).abs().max()) > 0.5 * float(want.abs().max())
    for portions in ([T], [needle + 1, 2, T - needle - 3], [needle + 3, 200] + [1] * 57,
                     [max(1, needle), T - max(1, needle) - 2, 1, 1]):
        assert sum(portions) == T
        cm = CacheManager([part.cache_spec()], 16, T // 16 + 1, 1)
        cm.allocate_storage(dtype, DEV, poison=True)
        got, _ = step_through(part, cm, x.to(dtype), portions, cm.view(0))
        err = (got.cpu().double() - want).abs().max(dim=1).values / want.abs().max()
        assert float(err.max()) < tol, (portions[:4], int(err.argmax()), float(err.max()))


@pytest.mark.parametrize("dtype", [F32, BF16])
def test_the_one_in_the_denominator_takes_the_weight(dtype):
    """Every key points away from the queries: all scores lie far below zero, and the result is near
    nothing, where a softmax without the sink would return a mean of the values."""
    from kappai_amd.cache import CacheManager
    part, t, m, half = needle_case(2, 16, dtype, 0.7)
    T = 90
    u = torch.ones(half) / math.sqrt(half)
    x = torch.randn(T, 2 * half, generator=gen(7)) * 0.02
    x[:, :half] += 1.5 * u
    x[:, half:] -= u
    x = x.to(BF16)
    want = P.attention(x.double(), t, "a.", m, 1e-5)
    full = float((x.double() @ t["a.v"].double().T @ t["a.o"].double().T).abs().max())
    assert float(want.abs().max()) < 2e-2 * full
    cm = CacheManager([part.cache_spec()], 16, 8, 1)
    cm.allocate_storage(dtype, DEV, poison=True)
    got, _ = step_through(part, cm, x.to(dtype), [40, 2] + [1] * 48, cm.view(0))
    assert float((got.cpu().double() - want).abs().max()) < 1e-3 * full


def make_state_space(W, m, dtype):
    from kappai_amd.parts import StateSpaceDual
    return StateSpaceDual("m.", W, m["heads"], m["vdim"], m["state"], m["groups"], m["conv"],
                          m["norm_groups"], 1e-5, dtype, weight_suffix="", bias_suffix=".b")


def state_space_dict(H, dv, N, G, conv, norm_groups):
    return {"heads": H, "vdim": dv, "state": N, "groups": G, "conv": conv, "norm_groups": norm_groups}


@pytest.mark.parametrize("dtype,tol", [(F32, 2e-5), (BF16, 3e-2)])
@pytest.mark.parametrize("H,dv,N,G,conv,norm_groups", [
    (6, 12, 20, 3, 3, 2), (8, 16, 32, 2, 4, 4), (2, 24, 16, 1, 1, 1), (4, 72, 40, 1, 4, 1),
    (3, 104, 136, 3, 4, 6), (5, 9, 33, 5, 2, 3), (16, 64, 128, 2, 4, 2), (1, 8, 8, 1, 7, 1)])
def test_state_space_part(dtype, tol, H, dv, N, G, conv, norm_groups):
    """Projection, convolution, recurrence and gated norm over portions: long ones in chunks, short
    ones and single tokens in the walk, cut across chunk borders, one after the other."""
    from kappai_amd.cache import CacheManager
    m = state_space_dict(H, dv, N, G, conv, norm_groups)
    part = make_state_space(72, m, dtype)
    t = bind_random(part, 6, dtype)
    T = 420
    x = torch.randn(T, 72, generator=gen(15)).to(BF16)
    want = P.mamba2(x.double(), t, "m.", m, 1e-5)
    for portions in ([T], [128, 1, 127, 2, 17, 16, 129], [2] * 20 + [1] * 60 + [320]):
        assert sum(portions) == T
        cm = CacheManager([part.cache_spec()], 16, 4, 2)
        cm.allocate_storage(dtype, DEV, poison=True)
        got, rc = step_through(part, cm, x.to(dtype), portions, cm.view(0))
        assert rel(got, want) < tol, portions[:3]


@pytest.mark.parametrize("dtype,tol", [(F32, 1e-3), (BF16, 5e-2)])
@pytest.mark.parametrize("needle", [0, 2, 63, 126, 127, 128, 200])
def test_a_token_that_only_the_state_remembers(dtype, tol, needle):
    """One token is written with a large step, every other token steps so little that it neither writes
    nor lets the state fade: rows hundreds of tokens later read that token, over chunk borders,
    portions and single steps.  Without it they would read next to nothing."""
    from kappai_amd.cache import CacheManager
    m = state_space_dict(2, 16, 16, 1, 4, 1)
    part = make_state_space(96, m, dtype)

    def change(t):
        w = torch.zeros_like(t["m.in"]).float()
        w[:96] = torch.randn(96, 96, generator=gen(1)) * 0.2         # z, x, B, C
        w[96:] = 0
        w[96:, 95] = 1.0                                             # the steps: the last input
        w[:96, 95] = 0
        t["m.in"] = w.to(BF16)
        t["m.dt_bias"], t["m.A_log"] = torch.zeros(2).to(BF16), torch.full((2,), -3.0).to(BF16)
        t["m.D"] = torch.zeros(2).to(BF16)
    t = bind_random(part, 6, dtype, change=change)
    T = needle + 330
    x = torch.randn(T, 96, generator=gen(16)).to(BF16)
    x[:, 95] = -14.0
    x[needle, 95] = 6.0
    want = P.mamba2(x.double(), t, "m.", m, 1e-5)
    without = x.clone()
    without[needle, 95] = -14.0
    gone = P.mamba2(without.double(), t, "m.", m, 1e-5)
    assert float((want[-1] - gone[-1]).abs().max()) > 0.3 * float(want.abs().max())
    # (a row whose read-out nearly cancels is a matter of rounding once the norm has blown it up)
    own = P.mamba2(x.double(), t, "m.", m, 1e-5, BF16) - want
    steady = own[needle:].abs().amax(1) < 0.02 * want.abs().max()
    assert float(steady.double().mean()) > 0.98
    for portions in ([T], [needle + 1, 128, 1, T - needle - 130], [needle + 2, 30] + [1] * 298):
        assert sum(portions) == T
        cm = CacheManager([part.cache_spec()], 16, 4, 1)
        cm.allocate_storage(dtype, DEV, poison=True)
        got, _ = step_through(part, cm, x.to(dtype), portions, cm.view(0))
        err = (got.cpu().double() - want)[needle:].abs().amax(1) / want[needle:].abs().max()
        assert bool((err < tol)[steady].all()), (portions[:3], float(err[steady].max()))


@pytest.mark.parametrize("dtype,tol", [(F32, 2e-5), (BF16, 3e-2)])
@pytest.mark.parametrize("W,F,E,top,identity,groups,shared,T", [
    (72, 24, 7, 2, 2, (3, 2), 40, 37), (64, 32, 8, 3, 0, None, 64, 150), (48, 8, 3, 4, 1, None, None, 5),
    (96, 48, 12, 4, 3, (5, 3), 24, 300), (100, 40, 6, 3, 6, (2, 1), 10, 1), (54, 10, 4, 2, 1, (5, 3), 14, 20),
    (64, 64, 16, 2, 4, (4, 2), 128, 700), (64, 32, 2, 5, 6, None, 32, 90)])
def test_experts_with_clamped_gates(dtype, tol, W, F, E, top, identity, groups, shared, T):
    """The whole feed-forward: with the sum over the experts made here and left to the caller, for
    rows whose choice is no close call; limits that bite, another one for the shared expert."""
    from kappai_amd.kernels import ops
    from kappai_amd.parts import MixtureOfExperts
    n, keep = groups or (1, 1)
    part = MixtureOfExperts("f.", W, F, E, top, dtype, weight_suffix="", activation="clamped",
                            clamp=ops.ClampedGate(0.7), scoring="softmax_all", correction=True,
                            groups=n, keep_groups=keep, group_best=1, identity=identity,
                            shared_hidden=shared, shared_gate=shared is not None,
                            shared_clamp=ops.ClampedGate(1.1) if shared else None)
    t = bind_random(part, 8, dtype)
    x = torch.randn(T, W, generator=gen(18)).to(BF16)
    mlp = {"expert": {"ff": F, "limit": 0.7}, "router": {"experts": E, "top": top,
                                                         "identity": identity}}
    if groups:
        mlp["router"]["groups"] = {"count": n, "keep": keep}
    if shared:
        mlp["shared"] = {"ff": shared, "limit": 1.1}
    margins = []
    want = P.moe_ff(x.double(), t, "f.", mlp, margins=margins)
    clear = margins[0] > 1e-4
    assert clear.sum() >= 0.9 * T
    up = x.double() @ t["f.e0.up"].double().T
    assert float((up.abs() > 0.7).double().mean()) > 0.1                # (the limit does bite)
    for got in (part.forward(x.to(dtype).to(DEV), None),
                part.forward(x.to(dtype).to(DEV), None, terms=True).combined()):
        got = got.float().cpu().double()
        assert float((got[clear] - want[clear]).abs().max() / want.abs().max()) < tol


# ---------------------------------------------------------------------------------------------
# whole models
# ---------------------------------------------------------------------------------------------
@pytest.fixture(scope="module")
def model_dirs(tmp_path_factory):
    base = tmp_path_factory.mktemp("zozezen")
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
MIN_STRICT = {"A": 0.05, "B": 1.0, "C": 1.0, "D": 0.02, "E": 0.02}


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
    """A short prompt and 330 tokens one by one (states carried on hundreds of times, the block
    tables of a graph grow), two requests side by side."""
    for name in ("A", "B", "C"):
        requests = make_requests(TINY[name][0]["vocab"], [350, 290], seed=22)
        plans = {"r0": (0, [20] + [1] * 330), "r1": (5, [3] + [1] * 287)}
        steps, index, peak = schedules.build(requests, plans)
        got, runner = replay(model_dirs[name], dtype, steps, index, peak, tmp_path / name)
        assert_matches_plain(got, model_dirs[name], requests, dtype, (name, dtype),
                             min_strict=0.0 if name == "A" else 1.0)
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
    assert "router" in out.stderr and "scan" in out.stderr
    made = tmp_path / "made"
    out = subprocess.run(
        [sys.executable, str(root / "bin" / "kappai-cli"), "--random-weights", "zozezen-tiny",
         "--model", str(made), "--weight-seed", "2", "--weight-std", "0.1", "-n", "5", "-t", "0.8",
         "-k", "20", "-s", "3", "--num-pages", "16", "7 8 9 10"],
        cwd=str(tmp_path), capture_output=True, text=True, timeout=300)
    assert out.returncode == 0, out.stderr
    assert len(out.stdout.split()) == 5 and (made / "config.json").is_file()
