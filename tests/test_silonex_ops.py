"""The mechanisms of the Silonex design, each alone, against plain float64 formulas written here
or in tests/_ref_silonex.py (no code shared with ``lumen``).  CPU tensors take the ops' torch
path; marked ``gpu``, the same cases run the HIP kernels in fp32 and bf16.

Where random inputs would hide a fault the inputs are made so that it shows: connection matrices
that move one copy onto another, one key whose score towers over the rest placed just inside and
just outside a window, states and tails left in a slot by another sequence, decays of 0 and 1,
a write that must survive hundreds of tokens, a key that is written twice."""
import math

import pytest
import torch

import _ref_silonex as ref
from test_dalavik_ops import CASES, F64, close, paged, rnd, segments

from lumen.ops.attention import head_norm_rotary_write, row_attention
from lumen.ops.conv import short_conv
from lumen.ops.norm import gated_rms_norm, hyper_mix, hyper_start, weight_layer_norm
from lumen.ops.recurrent import head_scan
from lumen.ops.rope import stretched_inv_freq
from lumen.ops.segments import TILE_ROWS, SegBatch, tile_list


def f64(t):
    return t.detach().cpu().to(F64)


# ---- norms -------------------------------------------------------------------------------------------
@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("W", [96, 37, 1028])
def test_layer_norm_with_shift(device, dtype, W):
    x = rnd(5, W, seed=1, device=device, scale=3.0) + 40.0          # a mean far from zero
    w, b = rnd(W, seed=2, device=device) + 1.0, rnd(W, seed=3, device=device)
    close(weight_layer_norm(x, w, 1e-5, dtype, b), ref.layer_norm(f64(x), f64(w), f64(b), 1e-5),
          dtype, scale=8.0)
    close(weight_layer_norm(x, w, 1e-5, dtype), ref.layer_norm(f64(x), f64(w), 0.0, 1e-5), dtype,
          scale=8.0)


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("W,groups,shared", [(96, 3, False), (80, 5, True), (64, 1, False),
                                             (2048, 16, True), (30, 2, False), (63, 9, True),
                                             (4096, 8, False), (24, 1, True)])
@pytest.mark.parametrize("gate,first", [("silu", True), ("silu", False), ("sigmoid", False)])
def test_gated_rms_norm(device, dtype, W, groups, shared, gate, first):
    T = 6
    x = rnd(T, W, seed=1, device=device, scale=0.02)                # eps counts at this size
    g = rnd(T, W + 24, seed=2, dtype=dtype, device=device, scale=2.0)[:, 8:8 + W]
    w = rnd(W // groups if shared else W, seed=3, device=device) + 1.0
    a = torch.sigmoid(f64(g)) * (f64(g) if gate == "silu" else 1.0)
    wf = f64(w).repeat(groups) if shared else f64(w)
    want = (ref.grouped_rms(f64(x) * a, groups, 1e-4) * wf if first
            else ref.grouped_rms(f64(x), groups, 1e-4) * wf * a)
    got = gated_rms_norm(x, g, w, groups, 1e-4, gate, first)
    assert got.dtype == dtype
    close(got, want, dtype)


# ---- hyper-connections -------------------------------------------------------------------------------
@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("S,W", [(1, 96), (2, 1028), (3, 37), (4, 256), (8, 64), (5, 40)])
def test_hyper_start_and_mix(device, dtype, S, W):
    T, V = 7, 33
    table = rnd(V, W, seed=1, dtype=dtype, device=device)
    toks = torch.tensor([0, 32, 5, 5, 17, 1, 9], device=device)
    w_in, w2 = rnd(S, seed=2, device=device), rnd(S, seed=3, device=device)
    norm = (rnd(W, seed=4, device=device) + 1.0, rnd(W, seed=5, device=device))
    x, h = hyper_start(toks, table, S, w_in, norm, 1e-5, dtype)
    assert x.dtype == torch.float32 and tuple(x.shape) == (T, S, W) and h.dtype == dtype
    xs = f64(table)[toks.cpu()].unsqueeze(0).repeat(S, 1, 1)
    assert torch.equal(f64(x).transpose(0, 1), xs)
    ln = lambda u: ref.layer_norm(u, f64(norm[0]), f64(norm[1]), 1e-5)  # noqa: E731
    close(h, ln(ref.hyper_in(xs, f64(w_in))), dtype)
    # every copy different from here on: one output, then two normed outputs, then the last sum
    x += rnd(T, S, W, seed=6, device=device)
    for k, pair in ((0, False), (1, True), (2, False)):
        xs = f64(x).transpose(0, 1)
        ys = [rnd(T, W, seed=10 + 3 * k + j, dtype=dtype, device=device, scale=1.5)
              for j in range(2 if pair else 1)]
        mix, out = rnd(S, S, seed=20 + k, device=device), rnd(S, seed=30 + k, device=device)
        pw = (rnd(W, seed=40, device=device), rnd(W, seed=41, device=device), 1e-3)
        y = f64(ys[0])
        if pair:
            y = (ref.rms_unit(y, 1e-3) * f64(pw[0]) + ref.rms_unit(f64(ys[1]), 1e-3) * f64(pw[1]))
        new = ref.hyper_out(xs, f64(mix), f64(out), y)
        before = x.clone()
        last = k == 2
        got = hyper_mix(x, ys, pw if pair else None, mix, out, w2, None if last else norm, 1e-5,
                        dtype, keep=not last)
        u = ref.hyper_in(new, f64(w2))
        if last:
            assert got.dtype == torch.float32
            close(got, u, torch.float32)
            if device == "cuda":
                assert torch.equal(x, before)                    # nothing stored
        else:
            close(got, ln(u), dtype)
            close(x.transpose(0, 1), new, torch.float32)


@pytest.mark.parametrize("device,dtype", CASES)
def test_hyper_mix_matrix_is_from_to(device, dtype):
    """mix with a single one at [from 0, to 2]: copy 2 becomes the old copy 0, all others only take
    their share of the output."""
    S, W = 3, 16
    x = rnd(4, S, W, seed=1, device=device)
    old = f64(x)
    y = rnd(4, W, seed=2, dtype=dtype, device=device)
    mix = torch.zeros(S, S, device=device)
    mix[0, 2] = 1.0
    out = torch.tensor([0.5, 0.0, 2.0], device=device)
    got = hyper_mix(x, [y], None, mix, out, torch.tensor([0.0, 0.0, 1.0], device=device), None, 1e-5,
                    dtype)
    close(x[:, 0], 0.5 * f64(y), torch.float32)
    assert bool((x[:, 1] == 0).all())
    close(x[:, 2], old[:, 0] + 2.0 * f64(y), torch.float32)
    close(got, old[:, 0] + 2.0 * f64(y), torch.float32)


# ---- rotary with stretched frequencies, per-head norms, caches ------------------------------------------
@pytest.mark.parametrize("scaling", [None, {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 64},
                                     {"factor": 3.0, "low": 2.0, "high": 2.5, "original": 500}])
@pytest.mark.parametrize("dims,base", [(16, 10000.0), (64, 500000.0), (2, 100.0), (20, 40.0)])
def test_stretched_frequencies(dims, base, scaling):
    rot = {"dims": dims, "base": base, "scaling": scaling}
    got = stretched_inv_freq(dims, base, scaling, "cpu")
    want = ref.frequencies(rot)
    assert float(((f64(got) - want) / want).abs().max()) <= 1e-7
    if scaling and base >= 10000:                    # all three regimes occur, or the test says little
        plain = ref.frequencies({"dims": dims, "base": base})
        ratio = want / plain
        assert float(ratio.max()) == 1.0 and float(ratio.min()) == pytest.approx(1 / scaling["factor"])


def turn(x, pos, rot):
    """x [T, n, D] in float64 at arbitrary positions."""
    half = rot["dims"] // 2
    a = pos.to(F64).view(-1, 1, 1) * ref.frequencies(rot).view(1, 1, -1)
    u, v = x[..., :half], x[..., half:2 * half]
    return torch.cat([u * torch.cos(a) - v * torch.sin(a), v * torch.cos(a) + u * torch.sin(a),
                      x[..., 2 * half:]], -1)


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("H,G,D,Dv,dims", [(6, 2, 24, 16, 16), (3, 3, 10, 14, 6), (8, 1, 64, 128, 64),
                                           (1, 1, 128, 128, 32), (4, 2, 40, 24, 0), (5, 5, 256, 8, 256),
                                           (2, 1, 48, 72, 48), (3, 1, 300, 20, 8), (2, 2, 16, 16, 4)])
@pytest.mark.parametrize("vnorm", [True, False])
def test_head_norm_rotary_write(device, dtype, H, G, D, Dv, dims, vnorm):
    T = 5
    width = (H + G) * D + G * Dv
    z = rnd(T, width + 8, seed=9, dtype=dtype, device=device, scale=1.5)
    before = f64(z)
    pos = torch.tensor([0, 1, 97, 31, 400], dtype=torch.int32, device=device)
    slots = torch.tensor([3, -1, 30, 0, 31], device=device)
    wq, wk = rnd(D, seed=1, device=device) + 1.0, rnd(D, seed=2, device=device) + 1.0
    sc = {"factor": 4.0, "low": 1.0, "high": 4.0, "original": 100}
    rot = {"dims": dims, "base": 5000.0, "scaling": sc}
    kc = torch.full((2, 16, G, D), 7.0, dtype=dtype, device=device)
    vc = torch.full((2, 16, G, Dv), 7.0, dtype=dtype, device=device)
    head_norm_rotary_write(z, wq, wk, pos, slots, kc, vc, H, G, D, Dv, dims,
                           stretched_inv_freq(dims, 5000.0, sc, device), 1e-3, vnorm)
    q = ref.rms_unit(before[:, :H * D].view(T, H, D), 1e-3) * f64(wq)
    k = ref.rms_unit(before[:, H * D:(H + G) * D].view(T, G, D), 1e-3) * f64(wk)
    v = before[:, (H + G) * D:width].view(T, G, Dv)
    v = ref.rms_unit(v, 1e-3) if vnorm else v
    q, k = turn(q, pos.cpu(), rot), turn(k, pos.cpu(), rot)
    close(z[:, :H * D].view(T, H, D), q, dtype, scale=16.0)     # fp32 angles: 400 rad carry 2e-5
    assert torch.equal(f64(z)[:, H * D:], before[:, H * D:])    # keys and values stay in the row
    for t, s in enumerate(slots.tolist()):
        if s >= 0:
            close(kc.view(32, G, D)[s], k[t], dtype, scale=16.0)
            close(vc.view(32, G, Dv)[s], v[t], dtype)
    assert bool((kc.view(32, -1)[1] == 7.0).all()) and bool((vc.view(32, -1)[5] == 7.0).all())


# ---- segments of a step: prompt portions first, decoded rows after them ---------------------------------
def step_of(spans, slots, n_pre, device):
    """spans: [(first position, rows)]; the first ``n_pre`` are prompt portions."""
    cu, row_seg = [0], []
    for i, (_, n) in enumerate(spans):
        cu.append(cu[-1] + n)
        row_seg += [i] * n
    i32 = dict(dtype=torch.int32, device=device)
    seg = SegBatch(torch.tensor(cu, **i32), torch.tensor(slots, **i32),
                   torch.tensor([p for p, _ in spans], **i32), torch.tensor(row_seg, **i32),
                   torch.zeros(cu[-1], **i32))
    if n_pre is not None:
        seg.q_tiles = torch.tensor(tile_list(cu, n_pre, TILE_ROWS), **i32).view(-1, 2)
        seg.tile_rows, seg.tile_size = cu[n_pre], TILE_ROWS
    return seg, cu


SPANS = [(0, 70), (40, 33), (0, 2), (7, 1), (64, 32), (0, 1), (99, 1), (3, 1)]
SLOTS = [2, 0, 5, 7, 1, 4, 3, 6]                            # slot 8 belongs to nobody


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("C,taps", [(40, 4), (37, 3), (64, 1), (24, 2), (12, 7), (1000, 4), (9, 16)])
@pytest.mark.parametrize("n_pre", [5, None])
def test_short_conv(device, dtype, C, taps, n_pre):
    """Portions longer than a strip and shorter than the taps, decoded rows, sequences that start
    (stale tails must read as zeros) and that go on; with and without a bias."""
    seg, cu = step_of(SPANS, SLOTS, n_pre, device)
    x = rnd(cu[-1], C + 12, seed=1, dtype=dtype, device=device)[:, 4:4 + C]
    w = rnd(C, taps, seed=2, device=device)
    for bias in (None, rnd(C, seed=3, device=device)):
        tail = rnd(9, taps - 1, C, seed=4, dtype=dtype, device=device, scale=5.0)
        t0 = f64(tail)
        got = short_conv(x, w, bias, tail, seg)
        assert got.dtype == dtype
        for i, (p0, n) in enumerate(SPANS):
            hist = t0[SLOTS[i]].clone()
            hist[:max(0, taps - 1 - p0)] = 0                 # positions below 0
            ext = torch.cat([hist, f64(x)[cu[i]:cu[i + 1]]])
            want = ref.silu(ref.short_conv(ext, f64(w), None if bias is None else f64(bias)))
            close(got[cu[i]:cu[i + 1]], want[taps - 1:], dtype, scale=max(4.0, float(want.abs().max())))
            if taps > 1:
                assert torch.equal(f64(tail)[SLOTS[i]], ext[-(taps - 1):])   # inputs as they are
        assert torch.equal(f64(tail)[8], t0[8])


# ---- matrix-state scans -----------------------------------------------------------------------------
def run_scan(kind, seg, cu, spans, slots, H, G, Dk, Dv, device, dtype, scale=1.0, silu_in=False,
             decay=None, a_shift=0.0, tol_scale=None):
    """The op against the token loop of the oracle for every segment; returns the op's output."""
    T = cu[-1]
    q = rnd(T, G * Dk + 4, seed=1, dtype=dtype, device=device, scale=scale)[:, :G * Dk]
    k = rnd(T, G * Dk + 8, seed=2, dtype=dtype, device=device, scale=scale)[:, 8:]
    v = rnd(T, H * Dv, seed=3, dtype=dtype, device=device)
    lg = rnd(T, 2 * H + 2, seed=4, dtype=dtype, device=device, scale=1.5)
    a, b = lg[:, :H] + a_shift, lg[:, H:2 * H]
    A_log, dt_bias = rnd(H, seed=5, device=device), rnd(H, seed=6, device=device) - 1.0
    skip = rnd(H, seed=7, device=device) if kind == "ssd" else None
    state = rnd(9, H, Dk, Dv, seed=8, device=device)
    s0 = f64(state)
    if kind == "const":
        dec = torch.tensor(decay, dtype=F64)
        dk = torch.log(dec).clamp(min=-1e4).float().to(device)
    else:
        dk = (a, A_log, dt_bias)
    delta = kind == "delta"
    got = head_scan(q, k, v, state, seg, H, Dk, Dv, dk, beta=b if delta else None, skip=skip,
                    rep=H // G, silu_in=silu_in, key_eps=1e-6 if delta else 0.0,
                    q_scale=Dk ** -0.5 if delta else 1.0)
    assert got.dtype == torch.float32
    act = ref.silu if silu_in else (lambda t: t)
    hg = torch.arange(H) // (H // G)
    stored = lambda t: act(t).to(dtype).to(F64)  # noqa: E731
    qd, kd = stored(f64(q).reshape(T, G, Dk)), stored(f64(k).reshape(T, G, Dk))
    vd = act(f64(v).reshape(T, H, Dv))
    if delta:
        qd, kd = ref.unit_vector(qd) * Dk ** -0.5, ref.unit_vector(kd)
    qd, kd = qd[:, hg], kd[:, hg]
    if kind == "const":
        g, vin = dec.view(1, H).expand(T, H), vd
    else:
        dt = ref.softplus(f64(a) + f64(dt_bias))
        g = torch.exp(-torch.exp(f64(A_log)) * dt)
        vin = vd if delta else dt.unsqueeze(-1) * vd
    for i, (p0, n) in enumerate(spans):
        r = slice(cu[i], cu[i + 1])
        S = s0[slots[i]] if p0 > 0 else None                 # a sequence's start: zeros
        if delta:
            o, S = ref.delta_recurrence(qd[r], kd[r], vd[r], torch.sigmoid(f64(b))[r], g[r], S)
        else:
            o, S = ref.decayed_recurrence(qd[r], kd[r], vin[r], g[r], S)
        if skip is not None:
            o = o + f64(skip).view(1, H, 1) * vd[r]
        o = o.reshape(n, H * Dv)
        # fp32-level arithmetic in every dtype: inputs are exact, only sums round (bf16: operands are
        # kept to 16 bits; a silu that rounds the other way is one bf16 unit of one element)
        f = 2.0 if dtype == torch.float32 else 8.0
        f *= 20.0 if silu_in and dtype != torch.float32 else 1.0
        close(got[r], o, torch.float32, scale=f * max(1.0, float(o.abs().max())))
        close(state[slots[i]], S, torch.float32, scale=f * max(1.0, float(S.abs().max())))
    assert torch.equal(f64(state)[8], s0[8])                 # nobody's slot is untouched
    return got


SIZES = [(4, 2, 16, 24), (3, 3, 64, 64), (2, 1, 33, 10), (6, 1, 128, 128), (1, 1, 100, 5),
         (2, 2, 256, 160), (4, 4, 8, 32)]


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("H,G,Dk,Dv", SIZES)
@pytest.mark.parametrize("kind", ["ssd", "delta"])
def test_head_scan(device, dtype, H, G, Dk, Dv, kind):
    seg, cu = step_of(SPANS, SLOTS, 5, device)
    run_scan(kind, seg, cu, SPANS, SLOTS, H, G, Dk, Dv, device, dtype, scale=0.5)


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("H,Dk,Dv", [(4, 16, 24), (3, 64, 40), (2, 36, 6), (4, 128, 128)])
def test_head_scan_constant_decay(device, dtype, H, Dk, Dv):
    """Constant decays, also exactly 0 (only the current token is left) and 1 (nothing fades);
    silu on q, k and v."""
    seg, cu = step_of(SPANS, SLOTS, 5, device)
    run_scan("const", seg, cu, SPANS, SLOTS, H, H, Dk, Dv, device, dtype, silu_in=True,
             decay=[0.0, 1.0, 0.5, 0.999][:H])


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("kind", ["ssd", "delta"])
@pytest.mark.parametrize("n_pre,spans", [(1, [(0, 300)]), (1, [(5, 257)]), (0, [(0, 1), (9, 1)]),
                                         (None, [(0, 3), (4, 65)]), (2, [(0, 31), (31, 32)])])
def test_head_scan_portions(device, dtype, kind, n_pre, spans):
    slots = [3, 1][:len(spans)]
    seg, cu = step_of(spans, slots, n_pre, device)
    run_scan(kind, seg, cu, spans, slots, 4, 2, 32, 48, device, dtype, scale=0.5)


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("kind", ["ssd", "delta"])
@pytest.mark.parametrize("shift", [30.0, -12.0])
def test_head_scan_extreme_steps(device, dtype, kind, shift):
    """Step sizes of ~30 (log decays of tens to hundreds per token: sums over a chunk reach the
    thousands, neighbours' weights must still be right) and of ~1e-6 (no decay at all)."""
    seg, cu = step_of(SPANS, SLOTS, 5, device)
    run_scan(kind, seg, cu, SPANS, SLOTS, 4, 2, 32, 40, device, dtype, scale=0.3, a_shift=shift)


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("split", [[280], [33, 2, 200, 45], [1] * 280, [250] + [1] * 30])
def test_a_far_write_survives(device, dtype, split):
    """One token writes value 3 along a key of its own; the last token, 279 later, asks for it: a
    delta-rule state with no decay returns exactly that value, however the tokens were cut."""
    T, Dk, Dv = 280, 16, 8
    k = torch.zeros(T, Dk)
    k[:, 0] = 1.0
    k[0] = 0.0
    k[0, 5] = 2.0                                    # unit vector e_5
    q = k.clone()
    q[-1] = 0.0
    q[-1, 5] = 0.5
    v = rnd(T, Dv, seed=1)
    v[0] = 3.0
    state = torch.full((2, 1, Dk, Dv), 9.0, device=device)
    a = torch.full((T, 1), -40.0)                    # softplus ~ 0: decay 1
    b = torch.full((T, 1), 40.0)                     # beta 1
    cast = lambda t: t.to(dtype).to(device)  # noqa: E731
    zero = torch.zeros(1, device=device)
    at, outs = 0, []
    for n in split:
        r = slice(at, at + n)
        seg, _ = step_of([(at, n)], [1], 0 if n == 1 and at > 0 else 1, device)
        outs.append(head_scan(cast(q[r]), cast(k[r]), cast(v[r]), state, seg, 1, Dk, Dv,
                              (cast(a[r]), zero, zero), beta=cast(b[r]), key_eps=1e-6, q_scale=1.0))
        at += n
    out = torch.cat(outs).cpu()
    assert at == T and float((out[-1] - 3.0).abs().max()) < 1e-4
    # writing e_0 again and again with beta 1 REPLACES: token t reads its own value, not a sum
    close(out[1:-1], cast(v)[1:-1].cpu().to(F64), torch.float32, scale=4.0)


# ---- window attention with a soft cap ----------------------------------------------------------------
@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("D,Dv,H,G", [(32, 32, 4, 2), (24, 40, 3, 1), (64, 64, 4, 1)])
@pytest.mark.parametrize("window", [1, 31, 32, 33, 100])
def test_window_edge_with_soft_cap(device, dtype, D, Dv, H, G, window):
    """Key j's score towers over all others.  Rows j .. j + window - 1 must return its value, rows
    before and after must not see it at all -- as a prompt's portion and as decoded rows, at block
    and tile borders."""
    n, bs = 210, 8
    cap = 20.0
    for j in (0, 7, 8, 63, 64, 101):
        k = 0.05 * rnd(n, G, D, seed=j)
        k[:, :, 0] = 0.0
        k[j, :, 0] = 40.0
        v = rnd(n, G, Dv, seed=j + 1)
        v[j] = 50.0
        kc, tb = paged([k.reshape(n, -1)], bs, 40, G * D, dtype, device, 3)
        vc, _ = paged([v.reshape(n, -1)], bs, 40, G * Dv, dtype, device, 3)
        kc, vc = kc.view(-1, bs, G, D), vc.view(-1, bs, G, Dv)
        q = 0.05 * rnd(n, H, D, seed=j + 2)
        q[:, :, 0] = 4.0
        q = q.to(dtype).to(device)
        hg = torch.arange(H) // (H // G)
        s = torch.einsum("thd,nhd->htn", f64(q), k.to(dtype).to(F64)[:, hg])
        s = torch.where(ref.window_mask(n, window), cap * torch.tanh(s / cap),
                        torch.tensor(-math.inf, dtype=F64))
        want = torch.einsum("htn,nhd->thd", torch.softmax(s, -1), v.to(dtype).to(F64)[:, hg])
        assert float(want[j].min()) > 49 and float(want[min(n - 1, j + window - 1)].min()) > 49
        if j + window < n:
            assert float(want[j + window].max()) < 10
        probe = [t for t in (j - 1, j, j + window - 1, j + window) if 0 <= t < n]
        for spans, pre in (([(0, 0, n)], 1), ([(0, t, 1) for t in probe], 0)):
            seg = segments(spans, tb, device)
            rows = [t for _, p0, c in spans for t in range(p0, p0 + c)]
            if pre:
                i32 = dict(dtype=torch.int32, device=device)
                seg.q_tiles = torch.tensor(tile_list([0, n], 1, TILE_ROWS), **i32).view(-1, 2)
                seg.tile_rows, seg.tile_size = n, TILE_ROWS
            o = torch.empty(len(rows), H, Dv, dtype=dtype, device=device)
            row_attention(q[rows].contiguous(), None, kc, vc, Dv, o, seg, H, G, 1.0, cap,
                          window=window)
            close(o, want[rows], dtype, scale=50.0)
