"""The mechanisms of the Tazulix design, each alone, against plain float64 formulas written here
or in tests/_ref_tazulix.py (no code shared with ``lumen``).  CPU tensors take the ops' torch
path; marked ``gpu``, the same cases run the HIP kernels in fp32 and bf16.

Where random inputs would hide a fault the inputs are made so that it shows: one head a hundred times
larger than the others (a norm per head would hide it), gates and up values beyond their limits, one
key whose score towers over the rest, a write that must survive hundreds of tokens."""
import math

import pytest
import torch

import _ref_tazulix as ref
from test_dalavik_ops import CASES, F64, close, paged, rnd, segments
from test_silonex_ops import f64, step_of

from lumen.ops.attention import row_attention, row_norm_rotary_write
from lumen.ops.moe import (ClampedGate, gated_act, grouped_mm_ok, moe, moe_dense, moe_grouped,
                           moe_grouped_mm, route_groups, scaled_act)
from lumen.ops.norm import SPLIT, embed_rms, parts_rms, residual_rms
from lumen.ops.recurrent import head_scan
from lumen.ops.rope import interleaved_inv_freq, yarn_inv_freq
from lumen.ops.segments import TILE_ROWS, tile_list

GATE = ClampedGate(0.9, 1.6, ref.GATE_SLOPE, 1.0)


# ---- YaRN --------------------------------------------------------------------------------------------
SCALINGS = [{"factor": 8.0, "original": 128, "fast": 16.0, "slow": 1.0},
            {"factor": 2.5, "original": 4096, "fast": 32.0, "slow": 1.0},
            {"factor": 40.0, "original": 64, "fast": 8.0, "slow": 2.0},
            {"factor": 1.0, "original": 1000, "fast": 32.0, "slow": 1.0},
            {"factor": 3.0, "original": 20, "fast": 500.0, "slow": 400.0},     # both borders below 0
            {"factor": 3.0, "original": 10 ** 9, "fast": 2.0, "slow": 1.9}]    # and beyond the end


@pytest.mark.parametrize("scaling", [None] + SCALINGS)
@pytest.mark.parametrize("dims,base", [(24, 5000.0), (64, 500000.0), (2, 100.0), (20, 40.0),
                                       (128, 10000.0)])
def test_yarn_frequencies(dims, base, scaling):
    got, amp = yarn_inv_freq(dims, base, scaling, "cpu")
    want, want_amp = ref.frequencies({"dims": dims, "base": base, "scaling": scaling})
    assert float(((f64(got) - want) / want).abs().max()) <= 1e-7
    assert amp == pytest.approx(want_amp, rel=1e-12)
    if not scaling:
        assert amp == 1.0 and torch.equal(got, interleaved_inv_freq(dims, base, "cpu"))


def test_yarn_regimes():
    """Fast dimensions keep their frequency, slow ones are divided by the factor, the ramp lies
    between and is linear in the dimension's index."""
    f, amp = yarn_inv_freq(64, 10000.0, {"factor": 4.0, "original": 2048, "fast": 32.0, "slow": 1.0},
                           "cpu")
    plain = torch.tensor([10000.0 ** (-2.0 * i / 64) for i in range(32)], dtype=F64)
    kept = f64(f) / plain
    # borders: 64 ln(2048 / (2 pi 32)) / (2 ln 10000) = 8.06 -> 8, 64 ln(2048 / 2 pi) / .. = 20.1 -> 21
    ramp = torch.clamp((torch.arange(32).to(F64) - 8) / 13, 0.0, 1.0)
    assert float((kept - (1.0 - 0.75 * ramp)).abs().max()) < 1e-6
    assert amp == pytest.approx(1.0 + 0.1 * math.log(4.0))


# ---- whole-projection norm, rotation, caches ---------------------------------------------------------
@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("H,G,D,Dv,dims", [(6, 2, 24, 16, 16), (3, 3, 10, 14, 6), (8, 1, 64, 128, 64),
                                           (1, 1, 128, 128, 32), (4, 2, 40, 24, 0), (5, 5, 256, 8, 256),
                                           (2, 1, 48, 72, 48), (3, 1, 300, 20, 8), (2, 2, 16, 16, 4),
                                           (7, 7, 12, 12, 8), (16, 4, 128, 128, 128), (2, 1, 512, 64, 512)])
@pytest.mark.parametrize("amp", [1.0, 1.3])
def test_row_norm_rotary_write(device, dtype, H, G, D, Dv, dims, amp):
    T = 5
    width = (H + G) * D + G * Dv
    z = rnd(T, width + 8, seed=9, dtype=dtype, device=device, scale=0.05)   # eps counts at this size
    z[:, :D] *= 100.0                                   # the first query head dwarfs the others
    z[:, H * D:H * D + D] *= 10.0
    before = f64(z)
    pos = torch.tensor([0, 1, 97, 31, 400], dtype=torch.int32, device=device)
    slots = torch.tensor([3, -1, 30, 0, 31], device=device)
    wq, wk = rnd(H * D, seed=1, device=device) + 1.0, rnd(G * D, seed=2, device=device) + 1.0
    rot = {"dims": dims, "base": 5000.0}
    kc = torch.full((2, 16, G, D), 7.0, dtype=dtype, device=device)
    vc = torch.full((2, 16, G, Dv), 7.0, dtype=dtype, device=device)
    row_norm_rotary_write(z, wq, wk, pos, slots, kc, vc, H, G, D, Dv, dims,
                          interleaved_inv_freq(dims, 5000.0, device), amp, 1e-3)
    q = ref.rms_unit(before[:, :H * D], 1e-3) * f64(wq)
    k = ref.rms_unit(before[:, H * D:(H + G) * D], 1e-3) * f64(wk)
    per_head = ref.rms_unit(before[:, :H * D].view(T, H, D), 1e-3).reshape(T, H * D) * f64(wq)
    if H > 1:
        assert float((per_head - q).abs().max()) > 0.5

    def turn(x):
        x = ref.rotate(x, pos.cpu(), rot) if dims else x
        return torch.cat([x[..., :dims] * amp, x[..., dims:]], -1)   # what passes is not scaled

    q, k = turn(q.view(T, H, D)), turn(k.view(T, G, D))
    scale = lambda w: max(1.0, float(w.abs().max()))  # noqa: E731  (fp32 angles: 400 rad carry 2e-5)
    close(z[:, :H * D].view(T, H, D), q, dtype, scale=3.0 * scale(q))
    assert torch.equal(f64(z)[:, H * D:], before[:, H * D:])    # keys and values stay in the row
    v = before[:, (H + G) * D:width].view(T, G, Dv)
    for t, s in enumerate(slots.tolist()):
        if s >= 0:
            close(kc.view(32, G, D)[s], k[t], dtype, scale=3.0 * scale(k))
            assert torch.equal(f64(vc.view(32, G, Dv)[s]), v[t])
    assert bool((kc.view(32, -1)[1] == 7.0).all()) and bool((vc.view(32, -1)[5] == 7.0).all())


def test_row_norm_rotary_write_rejects_bad_shapes():
    z = torch.zeros(1, 64)
    pos, slots = torch.zeros(1, dtype=torch.int32), torch.zeros(1, dtype=torch.long)
    kc, vc = torch.zeros(1, 16, 2, 8), torch.zeros(1, 16, 2, 8)
    f = interleaved_inv_freq(8, 100.0, "cpu")
    w4, w2 = torch.ones(32), torch.ones(16)
    ok = (z, w4, w2, pos, slots, kc, vc, 4, 2, 8, 8, 8, f, 1.0, 1e-5)
    row_norm_rotary_write(*ok)
    for at, value in ((1, w2), (2, w4), (5, torch.zeros(1, 16, 1, 8)), (11, 7), (11, 10), (7, 6)):
        bad = list(ok)
        bad[at] = value
        with pytest.raises(ValueError):
            row_norm_rotary_write(*bad)


# ---- the residual stream -----------------------------------------------------------------------------
@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("W", [96, 37, 1028, 2048])
def test_stream_start_and_residual(device, dtype, W):
    V = 33
    table = rnd(V, W, seed=1, dtype=dtype, device=device, scale=0.1)
    toks = torch.tensor([0, 32, 5, 5, 17, 1, 9], device=device)
    w = rnd(W, seed=4, device=device) + 1.0
    x, h, e = embed_rms(toks, table, 8.5, w, 1e-2)
    assert e is None
    xd = f64(table)[toks.cpu()] * 8.5
    assert x.dtype == torch.float32 and h.dtype == dtype
    close(x, xd, torch.float32)
    close(h, ref.rms_unit(xd, 1e-2) * f64(w), dtype)
    y = rnd(7, W, seed=5, dtype=dtype, device=device)
    xd = f64(x) + f64(y)
    ptr = x.data_ptr()
    h = residual_rms(x, y, w, 1e-2)
    assert x.data_ptr() == ptr and h.dtype == dtype
    close(x, xd, torch.float32)
    close(h, ref.rms_unit(xd, 1e-2) * f64(w), dtype)
    xd = f64(x) + f64(y)
    assert residual_rms(x, y, None, 1e-2) is None              # nothing reads the stream normed
    close(x, xd, torch.float32)


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("W", [96, 37, 1028])
def test_stream_through_its_own_projection(device, dtype, W):
    """x <- A x + scale * (B e): the stream enters the GEMM in two parts, so that what comes out
    keeps far more of it than one 16-bit rounding would leave."""
    T = 7
    table = rnd(33, W, seed=1, dtype=dtype, device=device, scale=0.3)
    toks = torch.tensor([0, 32, 5, 5, 17, 1, 9], device=device)
    A, B = (rnd(W, W, seed=s, dtype=dtype, device=device, scale=W ** -0.5) for s in (2, 3))
    w = rnd(W, seed=4, device=device) + 1.0
    mm = lambda a, b: (a.double() @ b.double().t()).float()  # noqa: E731
    base = mm(table[toks], B)
    for start in (True, False):
        if start:
            x, parts, e = embed_rms(toks, table, 3.0, SPLIT, 1e-5, rows=True)
            assert torch.equal(e, table[toks])
        else:
            parts = residual_rms(x, rnd(T, W, seed=6, dtype=dtype, device=device), SPLIT, 1e-5)
        xd = f64(x)
        if dtype == torch.float32:
            assert parts is x
        else:
            assert tuple(parts.shape) == (2 * T, W) and parts.dtype == dtype
            hi, lo = f64(parts[:T]), f64(parts[T:])
            assert torch.equal(hi, f64(x.to(dtype)))
            assert float((hi + lo - xd).abs().max()) <= 2.0 ** -16 * float(xd.abs().max())
        x2, h = parts_rms(mm(parts, A), base, 3.0, w, 1e-5, dtype)
        want = xd @ f64(A).T + 3.0 * f64(base)
        assert x2.dtype == torch.float32 and h.dtype == dtype and x2.data_ptr() != x.data_ptr()
        err = float((f64(x2) - want).abs().max()) / float(want.abs().max())
        assert err <= (2e-6 if dtype == torch.float32 else 5e-5)      # one bf16 rounding: ~2e-3
        close(h, ref.rms_unit(want, 1e-5) * f64(w), dtype)


# ---- experts -----------------------------------------------------------------------------------------
@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("E,ff,ffs", [(3, 40, 0), (4, 37, 11), (0, 0, 48), (2, 16, 24)])
@pytest.mark.parametrize("weigh", ["input", "output"])
def test_clamped_gate(device, dtype, E, ff, ffs, weigh):
    """Gates and up values on both sides of the limits (a gate has no lower one), another limit for
    the shared block, an expert nobody chose, the weight before or after the clamps."""
    T = 11
    gu = rnd(T, 2 * (E * ff + ffs), seed=60, dtype=dtype, device=device, scale=3.0)
    wts = None
    if E:
        wts = torch.rand(T, E, generator=torch.Generator().manual_seed(61)).to(device)
        wts[:, 0] = 0.0

    def pair(g, u, limit):
        g, u = torch.clamp(g, max=limit), torch.clamp(u, min=-limit, max=limit)
        return g * torch.sigmoid(ref.GATE_SLOPE * g) * (u + 1.0)

    want, z = [], f64(gu)
    for e in range(E):
        g, u = z[:, 2 * e * ff:(2 * e + 1) * ff], z[:, (2 * e + 1) * ff:(2 * e + 2) * ff]
        s = f64(wts)[:, e, None]
        want.append(pair(s * g, s * u, 0.9) if weigh == "input" else s * pair(g, u, 0.9))
    if ffs:
        want.append(pair(z[:, 2 * E * ff:2 * E * ff + ffs], z[:, 2 * E * ff + ffs:], 1.6))
    want = torch.cat(want, 1)
    close(gated_act(gu, wts, E, ff, ffs, GATE, weigh), want, dtype)
    if E:                                  # the two places differ, and so do the limits
        other = gated_act(gu, wts, E, ff, ffs, GATE, "output" if weigh == "input" else "input")
        assert float((f64(other) - want).abs().max()) > 0.1
    if ffs:
        same = gated_act(gu, wts, E, ff, ffs, ClampedGate(0.9, 0.9, ref.GATE_SLOPE, 1.0), weigh)
        assert float((f64(same) - want).abs().max()) > 0.1


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("act", ["silu", "relu", "gelu_tanh"])
def test_weighted_input_of_plain_gates(device, dtype, act):
    """weigh="input" with the older activations: act(w g) * (w u)."""
    gu = rnd(5, 2 * 3 * 16, seed=62, dtype=dtype, device=device, scale=2.0)
    wts = torch.rand(5, 3, generator=torch.Generator().manual_seed(63)).to(device)
    z = f64(gu).view(5, 3, 2, 16) * f64(wts).view(5, 3, 1, 1)
    fn = {"silu": ref.silu, "relu": torch.relu,
          "gelu_tanh": lambda t: torch.nn.functional.gelu(t, approximate="tanh")}[act]
    close(gated_act(gu, wts, 3, 16, 0, act, "input"), (fn(z[:, :, 0]) * z[:, :, 1]).reshape(5, 48),
          dtype)
    with pytest.raises(ValueError):
        gated_act(gu, wts, 3, 16, 0, act, "both")


@pytest.mark.parametrize("device", ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)])
@pytest.mark.parametrize("E,top", [(1, 1), (5, 5), (6, 2), (16, 1), (64, 6), (130, 4)])
def test_sigmoid_router_keeps_the_scores(device, E, top):
    z = rnd(37, E, seed=50, device=device, scale=2.0)
    got = route_groups(z, None, top, 1, 1, normalize=False)
    close(got, ref.route(f64(z), top), torch.float32, scale=1.0)
    assert bool(((got > 0).sum(-1) == top).all())


def _experts(E, ff, ffs, W, dtype, device):
    w = {"m.router": rnd(E, W, seed=63, dtype=dtype, scale=0.5)}
    names = [f"m.e{e}." for e in range(E)] + (["m.shared."] if ffs else [])
    for i, n in enumerate(names):
        f = ffs if n == "m.shared." else ff
        w[n + "gate"] = rnd(f, W, seed=100 + i, dtype=dtype, scale=2.0 * W ** -0.5)
        w[n + "up"] = rnd(f, W, seed=200 + i, dtype=dtype, scale=2.0 * W ** -0.5)
        w[n + "down"] = rnd(W, f, seed=300 + i, dtype=dtype, scale=f ** -0.5)
    gu = torch.cat([w[n + s] for n in names for s in ("gate", "up")], 0).to(device)
    down = torch.cat([w[n + "down"] for n in names], 1).contiguous().to(device)
    return w, gu, down


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("E,top,ff,ffs", [(6, 2, 24, 40), (5, 1, 20, 12), (3, 3, 17, 0), (1, 1, 16, 8)])
def test_experts_of_weighted_inputs_match_oracle(device, dtype, E, top, ff, ffs):
    """Every way to run the experts against the oracle's loop, which feeds an expert w * h."""
    T, W = 60, 32
    h = rnd(T, W, seed=62, dtype=dtype, device=device)
    w, gu, down = _experts(E, ff, ffs, W, dtype, device)
    f = {"expert": {"ff": ff, "limit": 0.9}, "router": {"experts": E, "top": top}}
    if ffs:
        f["shared"] = {"ff": ffs, "limit": 1.6}
    wd = {k: v.to(F64) for k, v in w.items()}
    want = ref.moe_ff(f64(h), wd, "m.", f)
    r = route_groups(h.float() @ w["m.router"].float().to(device).t(), None, top, 1, 1,
                     normalize=False)
    for fn in (moe_dense, moe_grouped):
        got = fn(h, r, gu, down, E, ff, ffs, GATE, weigh="input")
        assert got.dtype == dtype
        close(got, want, dtype)
    close(moe(h, r, gu, down, E, top, ff, ffs, GATE, weigh="input"), want, dtype)
    if grouped_mm_ok(h, ff):
        close(moe_grouped_mm(h, r, gu, down, E, top, ff, ffs, GATE, weigh="input"), want, dtype)
    off = moe_dense(h, r, gu, down, E, ff, ffs, GATE, weigh="output")
    assert float((f64(off) - want).abs().max()) > 0.1


def test_grouped_form_is_chosen_by_what_it_saves():
    from lumen.ops.moe import grouped_pays

    big = 2 * 2816 * 4096
    assert grouped_pays(2048, 16, 3, big) and not grouped_pays(8, 16, 3, big)
    assert not grouped_pays(1 << 20, 16, 6, big)               # 3 top > E: nothing to save
    assert not grouped_pays(4096, 16, 3, 2 * 704 * 1024)       # narrow layers: sorting costs more


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("E,top,ff,ffs,T", [(40, 2, 16, 24, 1000), (33, 1, 24, 0, 1100)])
def test_grouped_experts_of_weighted_inputs(dtype, E, top, ff, ffs, T, monkeypatch):
    """``moe`` leaving the dense form: the grouped GEMM in 16 bits, per-expert GEMMs in fp32."""
    import lumen.ops.moe as moe_ops

    monkeypatch.setattr(moe_ops, "GROUPED_MIN_SAVING", 1)
    W = 64
    h = rnd(T, W, seed=62, dtype=dtype, device="cuda")
    w, gu, down = _experts(E, ff, ffs, W, dtype, "cuda")
    f = {"expert": {"ff": ff, "limit": 0.9}, "router": {"experts": E, "top": top}}
    if ffs:
        f["shared"] = {"ff": ffs, "limit": 1.6}
    want = ref.moe_ff(f64(h), {k: v.to(F64) for k, v in w.items()}, "m.", f)
    r = route_groups(h.float() @ w["m.router"].float().cuda().t(), None, top, 1, 1, normalize=False)
    assert moe_ops.grouped_pays(T, E, top, 2 * ff * W)
    close(moe(h, r, gu, down, E, top, ff, ffs, GATE, weigh="input"), want, dtype)


@pytest.mark.parametrize("device,dtype", CASES)
def test_squared_relu_dense(device, dtype):
    u = rnd(9, 52, seed=64, dtype=dtype, device=device, scale=2.0)
    close(scaled_act(u, None, 0, 0, 52, "relu2"), torch.clamp(f64(u), min=0.0) ** 2, dtype)


# ---- causal attention over pages ---------------------------------------------------------------------
@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("D,Dv,H,G", [(32, 32, 4, 2), (24, 40, 3, 1), (64, 128, 4, 4), (128, 128, 4, 1)])
def test_far_keys_at_page_borders(device, dtype, D, Dv, H, G):
    """Key j's score towers over all others: every row from j on must return its value, the rows
    before it must not see it -- as a prompt's portion and as decoded rows, j and the rows at block
    and tile borders, hundreds of keys apart."""
    n, bs = 420, 8
    for j in (63, 0, 7, 8, 64, 127, 128, 300):
        k = 0.05 * rnd(n, G, D, seed=j)
        k[:, :, 0] = 0.0
        k[j, :, 0] = 40.0
        v = rnd(n, G, Dv, seed=j + 1)
        v[j] = 50.0
        kc, tb = paged([k.reshape(n, -1)], bs, 60, G * D, dtype, device, 3)
        vc, _ = paged([v.reshape(n, -1)], bs, 60, G * Dv, dtype, device, 3)
        kc, vc = kc.view(-1, bs, G, D), vc.view(-1, bs, G, Dv)
        q = 0.05 * rnd(n, H, D, seed=j + 2)
        q[:, :, 0] = 1.0
        q = q.to(dtype).to(device)
        want = ref.causal_attention(f64(q), k.to(dtype).to(F64), v.to(dtype).to(F64), 0.5)
        assert float(want[j:].min()) > 49 and (j == 0 or float(want[:j].max()) < 10)
        probe = sorted({t for t in (j - 1, j, j + 1, 63, 64, 255, 256, n - 1) if 0 <= t < n})
        for spans, pre in (([(0, 0, n)], 1), ([(0, t, 1) for t in probe], 0)):
            seg = segments(spans, tb, device)
            rows = [t for _, p0, c in spans for t in range(p0, p0 + c)]
            if pre:
                i32 = dict(dtype=torch.int32, device=device)
                seg.q_tiles = torch.tensor(tile_list([0, n], 1, TILE_ROWS), **i32).view(-1, 2)
                seg.tile_rows, seg.tile_size = n, TILE_ROWS
            o = torch.empty(len(rows), H, Dv, dtype=dtype, device=device)
            row_attention(q[rows].contiguous(), None, kc, vc, Dv, o, seg, H, G, 0.5)
            close(o, want[rows], dtype, scale=50.0)
        if device == "cpu":
            break                                        # the torch path is slow: one place is enough


# ---- lightning attention -----------------------------------------------------------------------------
@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("split", [[280], [33, 2, 200, 45], [1] * 280, [250] + [1] * 30])
def test_a_far_write_fades_by_its_decay(device, dtype, split):
    """Token 0 writes value 3 along a key of its own; the last token, 279 later, asks for it: it finds
    decay^279 of it, per head, however the tokens were cut -- in a slot full of another sequence's
    state."""
    T, H, Dk, Dv = 280, 4, 16, 8
    decay = [1.0, 0.999, 0.97, 0.0]
    k, q = torch.zeros(T, H, Dk), torch.zeros(T, H, Dk)
    k[:, :, 0] = 1.0
    k[0] = 0.0
    k[0, :, 5] = 1.0
    q[:, :, 0] = 1.0
    q[-1] = 0.0
    q[-1, :, 5] = 1.0
    v = rnd(T, H, Dv, seed=1)
    v[0] = 3.0
    state = torch.full((2, H, Dk, Dv), 9.0, device=device)
    log_decay = torch.log(torch.tensor(decay)).clamp(min=-1e4).to(device)
    cast = lambda t: t.reshape(T, -1).to(dtype).to(device)  # noqa: E731
    at, outs = 0, []
    for n in split:
        r = slice(at, at + n)
        seg, _ = step_of([(at, n)], [1], 0 if n == 1 and at > 0 else 1, device)
        outs.append(head_scan(cast(q)[r], cast(k)[r], cast(v)[r], state, seg, H, Dk, Dv, log_decay))
        at += n
    out = torch.cat(outs).cpu().view(T, H, Dv)
    for h, d in enumerate(decay):
        assert float((out[-1, h] - 3.0 * d ** 279).abs().max()) < 1e-4 * 3.0
    o, _ = ref.decayed_recurrence(q.to(F64), k.to(F64), v.to(dtype).to(F64),
                                  torch.tensor(decay, dtype=F64))
    close(out, o, torch.float32, scale=2.0 * float(o.abs().max()))
