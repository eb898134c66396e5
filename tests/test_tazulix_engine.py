"""Tazulix through the serving engine (model registry, loader, block manager, state slots,
scheduler, hybrid runner, trace replay) against the float64 whole-sequence oracle of
tests/_ref_tazulix.py.

Every test runs on the CPU (the ops' torch path) and, marked ``gpu``, on the HIP kernels.  The
configurations are small and unlike each other: head sizes that are and are not multiples of the
vector and matrix-core widths, values wider and narrower than keys, grouped, multi-query and full
heads, rotary on a part of the head and on all of it, with and without YaRN, loops at the start, in
the middle and over the whole stack, one expert and many, one chosen and all, layers without a
feed-forward, stacks that begin with either kind of layer."""
import copy
import os

import pytest
import torch

import _ref_tazulix as ref
from test_foderax_engine import engine, replay_alone, tokens
from test_silonex_engine import check_conditioned

from lumen.models import build_model
from lumen.models.config import ModelConfig, get_config, tazulix_to_dict
from lumen.models.tazulix import TazulixForCausalLM, layer_runs, pass_starts
from lumen.serve.hybrid_runner import key_bytes_per_token, state_bytes_per_slot
from lumen.serve.sequence import SamplingParams
from lumen.serve.trace import TraceReplay

DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]


def _cfg(name, vocab, width, scale, loop, eps, layers):
    return ModelConfig(arch="tazulix", vocab_size=vocab, hidden_size=width, embedding_scale=scale,
                       loop=loop, num_hidden_layers=len(layers), rms_norm_eps=eps,
                       intermediate_size=0, num_attention_heads=0, num_key_value_heads=0,
                       max_position_embeddings=1 << 20, eos_token_id=-1, name=name,
                       layer_specs=layers)


def _ff(n):
    return {"kind": "dense", "ff": n} if n else None


def _moe(E, top, ff, ffs=0, limit=0.8, limit_s=1.5):
    f = {"kind": "moe", "router": {"experts": E, "top": top}, "expert": {"ff": ff, "limit": limit}}
    if ffs:
        f["shared"] = {"ff": ffs, "limit": limit_s}
    return f


def _att(H, G, D, Dv, dims, mlp, base=3000.0, scale=0.3, scaling="default"):
    r = {"base": base, "dims": dims}
    if scaling == "default":
        r["scaling"] = {"factor": 6.0, "original": 128, "fast": 12.0, "slow": 1.0}
    elif scaling:
        r["scaling"] = scaling
    return {"type": "attention", "mlp": mlp, "mixer": {"heads": H, "kv_heads": G, "dim": D,
                                                       "vdim": Dv, "scale": scale, "rot": r}}


def _lin(H, D, Dv, decay, mlp):
    return {"type": "lightning", "mlp": mlp,
            "mixer": {"heads": H, "dim": D, "vdim": Dv, "decay": decay}}


CONFIGS = {
    "tiny": lambda: copy.deepcopy(get_config("tiny-tazulix")),
    # nothing a multiple of 8: scalar paths everywhere; three passes over the first two layers; a
    # layer without a feed-forward; plain frequencies; every expert chosen
    "odd": lambda: _cfg("odd", 131, 60, 3.5, {"start": 0, "stop": 2, "times": 3}, 3e-6, [
        _att(3, 3, 10, 14, 6, _moe(5, 2, 28, 13), scaling=None),
        _lin(3, 11, 7, [0.3, 1.0, 0.97], None),
        _att(6, 2, 14, 6, 14, _moe(3, 3, 9, 0, limit=2.0)),
        _lin(1, 9, 31, [0.995], _ff(33))]),
    # one of everything: one head, one expert, no loop, an embedding factor of 1
    "one": lambda: _cfg("one", 64, 48, 1.0, None, 1e-4, [
        _lin(1, 16, 16, [0.9], _moe(1, 1, 24, 16)),
        _att(1, 1, 16, 16, 16, _ff(40))]),
    # head sizes 64 and 128 (the matrix-core attention's shapes), values twice as wide as keys, wide
    # states, the whole stack looped, one expert of many
    "wide": lambda: _cfg("wide", 200, 128, 11.3, {"start": 0, "stop": 3, "times": 2}, 1e-5, [
        _att(4, 1, 64, 64, 32, _moe(12, 1, 48, 64), base=500000.0, scale=0.13),
        _lin(2, 128, 64, [0.8, 0.995], _moe(8, 4, 32, 32, 3.0, 0.6)),
        _att(2, 2, 64, 128, 64, _ff(96), base=10000.0, scale=0.12)]),
}


def make(name, device, dtype=torch.float32, seed=0):
    m = TazulixForCausalLM(CONFIGS[name](), dtype=dtype, device=device)
    m.init_weights(seed=seed)
    return m


class Oracle:
    def __init__(self, model):
        self.cfg = tazulix_to_dict(model.config)
        self.w = {n: model.tensor(n).detach().cpu() for n in model.tensor_names()}

    def forward(self, toks, cfg=None, w=None, dtype=ref.F64):
        return ref.forward(cfg or self.cfg, w or self.w, toks, dtype=dtype)

    def expect(self, toks):
        """(logits, yardstick) of one sequence."""
        want = self.forward(toks)
        return want, yardstick(self, toks, want)


def yardstick(orc, toks, want):
    """[T] how far rounding alone moves each position's logits: the oracle's own arithmetic in fp32
    against float64, and float64 with the embeddings moved by 3e-7 of themselves.  A norm over a
    read-out that is nearly zero, or a router's close call, magnifies rounding at that position in any
    implementation."""
    g = torch.Generator().manual_seed(99)
    e = orc.w["embed"].to(ref.F64)
    moved = dict(orc.w, embed=e * (1.0 + 3e-7 * torch.randn(e.shape, generator=g, dtype=ref.F64)))
    runs = (orc.forward(toks, dtype=torch.float32).to(ref.F64), orc.forward(toks, w=moved))
    return torch.stack([(r - want).abs().max(-1).values for r in runs]).max(0).values


def close_to_rounding(m, toks, want, *gots):
    """16-bit serving: every result's error (per position, root mean square over the logits) against
    what 16-bit storage alone does, measured on the ops' torch path: typical and unusual positions
    both within a factor of it, and the results as close to each other.  (A router's close call may
    fall either way in 16 bits at single positions: quantiles.)"""
    twin = TazulixForCausalLM(m.config, dtype=m.dtype, device="cpu")
    for n in m.tensor_names():
        twin.tensor(n).data.copy_(m.tensor(n).cpu())
    rms = lambda a, b: (a.to(ref.F64) - b.to(ref.F64)).pow(2).mean(-1).sqrt()  # noqa: E731
    stick = rms(twin(torch.tensor(toks))[0], want)
    for a, b in [(g, want) for g in gots] + [(g, gots[0]) for g in gots[1:]]:
        per = rms(a, b)
        for q in (0.5, 0.9):
            e, s = float(per.quantile(q)), float(stick.quantile(q))
            assert e <= (1.5 if q == 0.5 else 2.5) * s, f"quantile {q}: {e:.3e} against {s:.3e}"


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_whole_prompt_matches_oracle(device, name):
    m = make(name, device)
    toks = tokens(m, 150, 1)
    want, stick = Oracle(m).expect(toks)
    check_conditioned(replay_alone(m, device, toks, [1000]), want, stick)
    # the model's own forward (fresh caches, every row) is the same step function
    check_conditioned(m(torch.tensor(toks, device=device))[0].cpu(), want, stick)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_stream_after_every_pass(device, name):
    """The runner's per-layer hook against the oracle's stream after every pass of a layer: a fault
    shows at its layer."""
    m = make(name, device, seed=13)
    toks = tokens(m, 29, 14)
    layers = []
    o = Oracle(m)
    ref.forward(o.cfg, o.w, toks, layers)
    eng = engine(m, device)
    seen = {}
    eng.runner.observe = lambda i, x: seen.__setitem__(i, x.detach().float().cpu().clone())
    TraceReplay(eng).step([{"id": "a", "tokens": toks, "want": []}], ["a"])
    assert sorted(seen) == list(range(len(layers)))
    for i, want in enumerate(layers):
        err = float((seen[i].to(ref.F64) - want).abs().max())
        assert err <= 1e-4 * max(1.0, float(want.abs().max())), f"pass {i}: {err:.3e}"


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_prefill_then_long_decode(device, name):
    """A short prompt, then token by token across block, tile and chunk borders: states and caches
    carried from step to step."""
    m = make(name, device, seed=1)
    toks = tokens(m, 170, 2)
    want, stick = Oracle(m).expect(toks)
    check_conditioned(replay_alone(m, device, toks, [5] + [1] * 300), want, stick)
    # from the very first token on, one at a time (the first token is a one-row prefill)
    check_conditioned(replay_alone(m, device, toks[:40], [1]), want[:40], stick[:40])


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("pieces", [[2], [3, 1, 2, 17, 2, 1, 1, 30], [16], [15, 1, 17], [64, 2, 63],
                                    [33, 2], [129, 2]])
def test_portions_of_several_sizes(device, pieces):
    m = make("tiny", device, seed=2)
    toks = tokens(m, 137, 3)
    check_conditioned(replay_alone(m, device, toks, pieces, bs=8), *Oracle(m).expect(toks))


@pytest.mark.parametrize("device", DEVICES)
def test_long_portions_carry_state(device):
    """Portions longer than the scans' chunks and the attention's tiles, cut off their grids."""
    m = make("odd", device, seed=12)
    toks = tokens(m, 330, 4)
    want, stick = Oracle(m).expect(toks)
    check_conditioned(replay_alone(m, device, toks, [1000]), want, stick)
    check_conditioned(replay_alone(m, device, toks, [197, 1, 130, 2]), want, stick)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_first_tokens(device, name):
    m = make(name, device, seed=3)
    orc = Oracle(m)
    for n in (1, 2, 3, 6):
        toks = tokens(m, n, 10 + n)
        want, stick = orc.expect(toks)
        check_conditioned(replay_alone(m, device, toks, [1000]), want, stick)
        check_conditioned(replay_alone(m, device, toks, [1]), want, stick)


def _sharpen(m, factor=6.0):
    """Scale the attention layers' query weights up: a few keys, wherever they lie, carry a row's
    weight, so that a wrong key or angle shows."""
    with torch.no_grad():
        for i, L in enumerate(m.config.layer_specs):
            if L["type"] == "attention":
                m.tensor(f"l{i}.mix.q.norm").mul_(factor)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("name", ["tiny", "wide"])
def test_every_constant_counts(device, name):
    """Sharp scores.  The oracle itself says that every constant of the configuration and every branch
    of the design, changed or dropped, would move the logits far beyond the tolerance -- and the
    engine matches the true model whole, in ragged portions and decoded token by token."""
    m = make(name, device, seed=21)
    _sharpen(m)
    toks = tokens(m, 160, 22)
    orc = Oracle(m)
    want = orc.forward(toks)
    scale = max(float(want.std()), 1.0)
    specs = orc.cfg["layers"]
    ia = next(i for i, L in enumerate(specs) if L["type"] == "attention"
              and L["mixer"]["rot"].get("scaling"))
    il = next(i for i, L in enumerate(specs) if L["type"] == "lightning")
    im = next(i for i, L in enumerate(specs) if (L["mlp"] or {}).get("kind") == "moe")
    idn = next(i for i, L in enumerate(specs) if (L["mlp"] or {}).get("kind") == "dense")

    def cfg_with(fn):
        c = copy.deepcopy(orc.cfg)
        fn(c)
        return c, None, {}

    def w_with(name_, fn):
        w = dict(orc.w)
        w[name_] = fn(w[name_].float()).to(w[name_].dtype)
        return None, w, {}

    att = lambda c: c["layers"][ia]["mixer"]  # noqa: E731
    mlp = lambda c: c["layers"][im]["mlp"]  # noqa: E731
    yarn = lambda **kw: cfg_with(lambda c: att(c)["rot"]["scaling"].update(**kw))  # noqa: E731

    def set_(d, k, v):
        d[k] = v

    def no_reinjection(w, W=m.config.hidden_size):
        w = w.clone()
        w[:, W:] = 0
        return w

    def swapped(w, W=m.config.hidden_size):
        return torch.cat([w[:, W:], w[:, :W]], 1)

    def per_head(h, w, p, mm, eps):
        """the attention mixer with q and k normed head by head"""
        T, (H, G, D, Dv) = h.shape[0], (mm[k] for k in ("heads", "kv_heads", "dim", "vdim"))
        proj = lambda n: h @ w[p + n].T + w[p + n + ".b"]  # noqa: E731
        q = ref.rms_unit(proj("q").view(T, H, D), eps) * w[p + "q.norm"].view(H, D)
        k = ref.rms_unit(proj("k").view(T, G, D), eps) * w[p + "k.norm"].view(G, D)
        pos = torch.arange(T)
        o = ref.causal_attention(ref.rotate(q, pos, mm["rot"]), ref.rotate(k, pos, mm["rot"]),
                                 proj("v").view(T, G, Dv), mm["scale"])
        return o.reshape(T, H * Dv) @ w[p + "o"].T

    def weigh_output(h, w, p, f):
        wt = ref.route(h @ w[p + "router"].T, f["router"]["top"])
        y = sum(wt[:, e, None] * ref.expert(h, w, p + f"e{e}.", f["expert"]["limit"])
                for e in range(f["router"]["experts"]))
        return y + ref.expert(h, w, p + "shared.", f["shared"]["limit"])

    def rescore(h, w, p, f):
        """routing weights that sum to one"""
        wt = ref.route(h @ w[p + "router"].T, f["router"]["top"])
        wt = wt / wt.sum(-1, keepdim=True)
        y = sum((wt[:, e, None] > 0) * ref.expert(wt[:, e, None] * h, w, p + f"e{e}.",
                                                  f["expert"]["limit"])
                for e in range(f["router"]["experts"]))
        return y + ref.expert(h, w, p + "shared.", f["shared"]["limit"])

    true_order = ref.layer_order

    def first_pass_only(c):
        out, begun = [], False
        for i, enter in true_order(c):
            out.append((i, enter and not begun))
            begun |= enter
        return out

    A, M = f"l{ia}.mix.", f"l{im}.mlp."
    changes = {
        "yarn off": cfg_with(lambda c: set_(att(c)["rot"], "scaling", None)),
        "yarn factor": yarn(factor=att(orc.cfg)["rot"]["scaling"]["factor"] * 1.5),
        "yarn original": yarn(original=att(orc.cfg)["rot"]["scaling"]["original"] * 8),
        "yarn fast": yarn(fast=att(orc.cfg)["rot"]["scaling"]["fast"] / 6),
        "yarn slow": yarn(slow=4.0),
        "rotary base": cfg_with(lambda c: set_(att(c)["rot"], "base", 2000.0)),
        "rotary dims": cfg_with(lambda c: set_(att(c)["rot"], "dims", att(c)["rot"]["dims"] - 2)),
        "scale": cfg_with(lambda c: set_(att(c), "scale", att(c)["scale"] * 0.9)),
        "q bias": w_with(A + "q.b", lambda t: t * 0.0),
        "k bias": w_with(A + "k.b", lambda t: t * 0.0),
        "v bias": w_with(A + "v.b", lambda t: t * 0.0),
        "q norm weight": w_with(A + "q.norm", lambda t: t * 0.0 + 6.0),
        "k norm weight": w_with(A + "k.norm", lambda t: t * 0.0 + 1.0),
        "norms per head": (None, None, {"MIXERS": dict(ref.MIXERS, attention=per_head)}),
        "decay": cfg_with(lambda c: set_(c["layers"][il]["mixer"], "decay",
                                         [d * 0.95 for d in c["layers"][il]["mixer"]["decay"]])),
        "decay order": cfg_with(lambda c: c["layers"][il]["mixer"]["decay"].reverse()),
        "read-out norm": w_with(f"l{il}.mix.norm", lambda t: t * 0.0 + 1.0),
        "gate": w_with(f"l{il}.mix.g", lambda t: t * 0.0),
        "expert limit": cfg_with(lambda c: set_(mlp(c)["expert"], "limit",
                                                mlp(c)["expert"]["limit"] * 1.2)),
        "shared limit": cfg_with(lambda c: set_(mlp(c)["shared"], "limit",
                                                mlp(c)["expert"]["limit"])),
        "top": cfg_with(lambda c: set_(mlp(c)["router"], "top", mlp(c)["router"]["top"] + 1)),
        "no shared expert": w_with(M + "shared.down", lambda t: t * 0.0),
        "weight on the output": (None, None, {"FEED_FORWARDS": dict(ref.FEED_FORWARDS,
                                                                    moe=weigh_output)}),
        "weights sum to one": (None, None, {"FEED_FORWARDS": dict(ref.FEED_FORWARDS, moe=rescore)}),
        "gate slope": (None, None, {"GATE_SLOPE": 1.0}),
        "dense act": (None, None, {"FEED_FORWARDS": dict(
            ref.FEED_FORWARDS, dense=lambda h, w, p, f: torch.relu(h @ w[p + "up"].T)
            @ w[p + "down"].T)}),
        "dense": w_with(f"l{idn}.mlp.down", lambda t: t * 0.0),
        "loop count": cfg_with(lambda c: set_(c["loop"], "times", c["loop"]["times"] + 1)),
        "loop stop": cfg_with(lambda c: set_(c["loop"], "stop", c["loop"]["stop"] - 1)),
        "no re-injection": w_with("loop.in", no_reinjection),
        "loop halves swapped": w_with("loop.in", swapped),
        "injected at the first pass only": (None, None, {"layer_order": first_pass_only}),
        "embedding scale": cfg_with(lambda c: set_(c["embedding"], "scale", 1.0)),
        "norm2": w_with(f"l{im}.norm2", lambda t: t * 0.0 + 1.0),
        "eps": cfg_with(lambda c: set_(c["norm"], "eps", 1e-1)),
    }
    for what, (c, w, patch) in changes.items():
        with pytest.MonkeyPatch.context() as mp:
            for k, v in patch.items():
                mp.setattr(ref, k, v)
            moved = float((orc.forward(toks, c, w) - want).abs().max())
        assert moved > 20 * 5e-4 * scale, f"{what}: moves the logits by {moved:.2e} only"
    stick = yardstick(orc, toks, want)
    check_conditioned(replay_alone(m, device, toks, [1000]), want, stick, rtol=5e-4)
    check_conditioned(replay_alone(m, device, toks, [37, 2, 50, 1, 64, 3], bs=8), want, stick,
                      rtol=5e-4)
    check_conditioned(replay_alone(m, device, toks, [90] + [1] * 200), want, stick, rtol=5e-4)


@pytest.mark.parametrize("device", DEVICES)
def test_far_token_is_seen(device):
    """Changing the FIRST token of a long prompt changes the last logits, through the states alone (a
    stack of lightning layers) and through the attention; the engine agrees with the oracle on both
    prompts."""
    for name in ("tiny", "states"):
        if name == "states":
            cfg = _cfg("states", 90, 64, 4.0, {"start": 1, "stop": 2, "times": 2}, 1e-5,
                       [_lin(2, 16, 24, [0.9995, 1.0], _ff(64)), _lin(2, 24, 16, [0.999, 1.0], None)])
            m = TazulixForCausalLM(cfg, dtype=torch.float32, device=device)
            m.init_weights(seed=23)
        else:
            m = make(name, device, seed=23)
        orc = Oracle(m)
        a = tokens(m, 260, 24)
        b = list(a)
        b[0] = (a[0] + 1) % m.config.vocab_size
        wa, wb = orc.forward(a)[-1], orc.forward(b)[-1]
        assert float((wa - wb).abs().max()) > 10 * 5e-4 * float(wa.std())
        for toks in (a, b):
            want, stick = orc.expect(toks)
            for pieces in ([230, 7, 1], [200] + [1] * 60):
                check_conditioned(replay_alone(m, device, toks, pieces, bs=8), want, stick)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("name", ["tiny", "odd"])
def test_mixed_batches_reuse_blocks_and_slots(device, name):
    """Seven unequal requests through three sequence slots and a pool of 20 blocks of 8: portions
    of some beside single tokens of others; finished requests hand their blocks and their state
    slot (with states still in it) to new ones.  Every request must come out as if it had run
    alone."""
    m = make(name, device, seed=4)
    orc = Oracle(m)
    lens = [41, 9, 66, 2, 30, 17, 50]
    reqs = {f"r{i}": tokens(m, n, 20 + i) for i, n in enumerate(lens)}
    eng = engine(m, device, blocks=20, bs=8, seqs=3)
    rp = TraceReplay(eng)
    g = torch.Generator().manual_seed(5)
    waiting = list(reqs)
    live, at, got = [], {}, {r: [] for r in reqs}
    sizes = [2, 1, 1, 13, 1, 5, 1, 1, 24, 3]
    k = 0
    seen_blocks, seen_slots = [], []
    while waiting or live:
        while waiting and len(live) < 3:
            need = sum((len(reqs[r]) + 7) // 8 for r in live + [waiting[0]])
            if need > 20:
                break
            r = waiting.pop(0)
            live.append(r)
            at[r] = 0
        entries, end = [], []
        for r in list(live):
            if len(live) > 1 and torch.rand((), generator=g) < 0.3:
                continue                                   # left out of this step
            c = min(sizes[k % len(sizes)], len(reqs[r]) - at[r])
            k += 1
            entries.append({"id": r, "tokens": reqs[r][at[r]:at[r] + c], "want": list(range(c))})
            at[r] += c
            if at[r] == len(reqs[r]):
                end.append(r)
                live.remove(r)
        if not entries:
            continue
        seen_slots += list(eng.states.owner.values())
        out = rp.step(entries, end)
        seen_blocks += [b for t in eng.blocks.tables.values() for b in t]
        o = 0
        for e in entries:
            got[e["id"]].append(out[o:o + len(e["tokens"])])
            o += len(e["tokens"])
    assert eng.blocks.num_free == 20 and len(set(seen_blocks)) <= 20
    assert eng.states.num_free == 3 and set(seen_slots) <= {0, 1, 2}
    for r, toks in reqs.items():
        check_conditioned(torch.cat(got[r], 0), *orc.expect(toks))


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("name", ["tiny", "odd"])
def test_blocks_and_slot_reused_after_finish(device, name):
    """The second request gets the first one's blocks and state slot, full of its keys, values and
    states."""
    m = make(name, device, seed=6)
    orc = Oracle(m)
    eng = engine(m, device, blocks=8, bs=16, seqs=1)
    rp = TraceReplay(eng)
    a, b = tokens(m, 100, 30), tokens(m, 60, 31)
    rp.step([{"id": "a", "tokens": a, "want": []}], ["a"])
    got = torch.cat([rp.step([{"id": "b", "tokens": b[:1], "want": [0]}], []),
                     rp.step([{"id": "b", "tokens": b[1:33], "want": list(range(32))}], []),
                     rp.step([{"id": "b", "tokens": b[33:], "want": list(range(27))}], ["b"])], 0)
    check_conditioned(got, *orc.expect(b))


def test_every_pass_has_caches_of_its_own():
    """A looped layer's passes must not share memory, and the byte counts follow the passes."""
    m = make("tiny", "cpu")
    eng = engine(m, "cpu", blocks=4, bs=8, seqs=2)
    st = eng.runner.state
    assert eng.weights.runs == [0, 1, 2, 1, 2, 1, 2, 3]
    assert eng.weights.starts == [False, True, False, True, False, True, False, False]
    ptrs = [t.data_ptr() for group in (st.k, st.v, st.S) for t in group if t is not None]
    assert len(ptrs) == len(set(ptrs)) == 12
    per_tok = sum(t[0, 0].numel() for g in (st.k, st.v) for t in g if t is not None) * 4
    assert key_bytes_per_token(m.config, 4) == per_tok
    assert state_bytes_per_slot(m.config, 4) == sum(t[0].numel() for t in st.S if t is not None) * 4


def test_loop_plan():
    def plan(n, loop):
        c = _cfg("p", 9, 8, 1.0, loop, 1e-5, [_lin(1, 4, 4, [0.5], None)] * n)
        order = ref.layer_order(tazulix_to_dict(c))
        assert list(zip(layer_runs(c), pass_starts(c))) == order
        return order

    assert plan(2, None) == [(0, False), (1, False)]
    assert plan(3, {"start": 1, "stop": 2, "times": 1}) == [(0, False), (1, True), (2, False)]
    assert plan(2, {"start": 0, "stop": 2, "times": 2}) == [(0, True), (1, False)] * 2
    assert plan(2, {"start": 1, "stop": 1, "times": 3}) == [(0, False), (1, False)]


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("name", ["tiny", "one"])
def test_greedy_generation_through_scheduler(device, name):
    """LLMEngine.generate: chunked prefill under a small token budget, more prompts than
    sequence slots, async scheduling, greedy sampling -- every generated token is the oracle's
    arg-max (up to a tie within the tolerance) given the tokens before it."""
    m = make(name, device, seed=7)
    orc = Oracle(m)
    eng = engine(m, device, blocks=48, bs=8, seqs=3, budget=24)
    prompts = [tokens(m, n, 40 + n) for n in (5, 37, 1, 20, 52)]
    seqs = eng.generate(prompts, SamplingParams(max_tokens=10, temperature=0.0, ignore_eos=True))
    assert eng.blocks.num_free == 48 and eng.states.num_free == 3
    for p, s in zip(prompts, seqs):
        assert len(s.output_ids) == 10
        want = orc.forward(p + s.output_ids[:-1])
        for j, tok in enumerate(s.output_ids):
            row = want[len(p) - 1 + j]
            assert float(row.max() - row[tok]) <= 1e-3 * max(float(row.std()), 1.0)


@pytest.mark.parametrize("device", DEVICES)
def test_preemption_recomputes_caches_and_state(device):
    """A pool too small for all running sequences: the scheduler preempts and later recomputes a
    sequence from its first token in whatever blocks and slot it then gets; outputs stay the
    oracle's."""
    m = make("odd", device, seed=8)
    orc = Oracle(m)
    eng = engine(m, device, blocks=12, bs=4, seqs=3, budget=64, async_scheduling=False)
    prompts = [tokens(m, n, 60 + n) for n in (9, 11, 10)]
    seqs = eng.generate(prompts, SamplingParams(max_tokens=14, temperature=0.0, ignore_eos=True))
    assert eng.scheduler.num_preemptions > 0
    for p, s in zip(prompts, seqs):
        want = orc.forward(p + s.output_ids[:-1])
        for j, tok in enumerate(s.output_ids):
            row = want[len(p) - 1 + j]
            assert float(row.max() - row[tok]) <= 1e-3 * max(float(row.std()), 1.0)


def _random_config(seed):
    """A random stack: 1 - 5 layers in random order with a random loop, sizes that are and are not
    multiples of the vector and matrix-core widths."""
    import random

    rng = random.Random(seed)
    layers = []
    for _ in range(rng.randint(1, 5)):
        kind = rng.choice([None, "dense", "moe", "moe"])
        mlp = None if kind is None else _ff(rng.choice([40, 92, 128]))
        if kind == "moe":
            E = rng.choice([1, 2, 5, 8, 20])
            mlp = _moe(E, rng.randint(1, min(E, 6)), rng.choice([8, 20, 48]),
                       rng.choice([0, 24, 31, 64]), rng.choice([0.5, 1.0, 7.0]),
                       rng.choice([0.7, 1.0, 5.0]))
        H = rng.choice([1, 2, 3, 4, 6, 8])
        D, Dv = rng.choice([8, 12, 20, 32, 64]), rng.choice([8, 12, 24, 32, 64, 72])
        if rng.random() < 0.6:
            G = rng.choice([g for g in (1, 2, 3, 4, H) if H % g == 0])
            layers.append(_att(H, G, D, Dv, rng.choice([2, D // 4 * 2, D]), mlp,
                               base=rng.choice([100.0, 10000.0]), scale=rng.uniform(0.1, 0.6),
                               scaling=rng.choice([None, "default",
                                                   {"factor": 2.0, "original": 1000, "fast": 32.0,
                                                    "slow": 1.0}])))
        else:
            layers.append(_lin(H, D, Dv, [rng.choice([0.4, 0.9, 0.99, 1.0]) for _ in range(H)], mlp))
    a = rng.randint(0, len(layers) - 1)
    loop = {"start": a, "stop": rng.randint(a, len(layers)), "times": rng.randint(1, 3)}
    return _cfg(f"random{seed}", rng.randint(50, 400), rng.choice([64, 96, 100, 192]),
                rng.choice([1.0, 6.0]), rng.choice([None, loop, loop]), rng.choice([1e-6, 1e-5]),
                layers)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("seed", range(10))
def test_random_configurations(device, seed):
    """Whole, in ragged portions, and decoded across a tile border: the oracle's logits (fp32)
    and, on the GPU in 16 bits, the same logits however the prompt was cut."""
    cfg = _random_config(seed)
    m = TazulixForCausalLM(cfg, dtype=torch.float32, device=device)
    m.init_weights(seed=seed)
    toks = tokens(m, 150, seed)
    want, stick = Oracle(m).expect(toks)
    for pieces in ([1000], [37, 2, 1, 50, 1, 1, 1, 3], [120] + [1] * 30):
        check_conditioned(replay_alone(m, device, toks, pieces), want, stick)
    if device == "cuda":
        m16 = TazulixForCausalLM(cfg, dtype=torch.bfloat16, device=device)
        m16.init_weights(seed=seed)
        whole = replay_alone(m16, device, toks, [1000])
        close_to_rounding(m16, toks, Oracle(m16).forward(toks), whole,
                          replay_alone(m16, device, toks, [37, 2, 1, 50, 1, 1, 1, 3]),
                          replay_alone(m16, device, toks, [120] + [1] * 30))


def test_configuration_is_validated():
    def bad(fn, name="odd"):
        c = CONFIGS[name]()
        fn(c)
        with pytest.raises(ValueError):
            TazulixForCausalLM(c, dtype=torch.float32, device="cpu")

    mixer = lambda c, i: c.layer_specs[i]["mixer"]  # noqa: E731
    bad(lambda c: mixer(c, 0).update(kv_heads=2))             # 3 heads on 2 key heads
    bad(lambda c: mixer(c, 0)["rot"].update(dims=7))
    bad(lambda c: mixer(c, 0)["rot"].update(dims=12))         # heads of 10
    bad(lambda c: mixer(c, 0).update(vdim=600))
    bad(lambda c: mixer(c, 2)["rot"]["scaling"].update(factor=0.0))
    bad(lambda c: mixer(c, 1).update(dim=300))                # a state row the scan has no kernel for
    bad(lambda c: mixer(c, 1).update(decay=[0.5]))            # 3 heads
    bad(lambda c: mixer(c, 1).update(decay=[0.5, -0.1, 0.5]))
    bad(lambda c: c.loop.update(stop=9))
    bad(lambda c: c.loop.update(times=0))
    bad(lambda c: c.layer_specs[0].update(type="window"))
    bad(lambda c: c.layer_specs[0]["mlp"].update(kind="routed"))
    bad(lambda c: c.layer_specs[0]["mlp"]["router"].update(top=6))
    bad(lambda c: c.layer_specs[0]["mlp"]["expert"].update(limit=0.0))


def test_checkpoint_roundtrip(tmp_path):
    """save -> config.json + model.safetensors under the design's tensor names -> load by
    directory (the class is picked by config.json); a missing tensor or a wrong shape is an
    error."""
    from safetensors.torch import load_file, save_file

    from lumen.models.loading import save_hf_weights

    for name in ("one", "odd"):
        m = make(name, "cpu", dtype=torch.bfloat16)
        d = str(tmp_path / name)
        save_hf_weights(m, d)
        m2 = build_model(d, dtype=torch.bfloat16, device="cpu")
        assert m2.config.arch == "tazulix" and type(m2) is TazulixForCausalLM
        for f in ("loop", "embedding_scale", "layer_specs", "rms_norm_eps", "vocab_size"):
            assert getattr(m2.config, f) == getattr(m.config, f), f
        for n in m.tensor_names():
            assert torch.equal(m.tensor(n), m2.tensor(n)), n
    f = os.path.join(d, "model.safetensors")
    sd = load_file(f)
    assert "l1.norm2" not in sd and "l2.mlp.shared.up" not in sd and "loop.in" in sd
    short = dict(sd)
    short.pop("l0.mix.k.b")
    save_file(short, f)
    with pytest.raises(KeyError):
        build_model(d, dtype=torch.bfloat16, device="cpu")
    sd["l0.mix.q.norm"] = torch.zeros(10, dtype=torch.bfloat16)
    save_file(sd, f)
    with pytest.raises(ValueError):
        build_model(d, dtype=torch.bfloat16, device="cpu")


def test_trace_run_command_line(tmp_path):
    """bin/trace_run as a user runs it: a checkpoint directory, JSON steps on stdin, one logits
    file per step that wants any, `done <step>` after every step, exit code 0 at end of input."""
    import json
    import subprocess
    import sys

    import numpy as np

    from lumen.models.loading import save_hf_weights

    m = make("odd", "cpu", dtype=torch.bfloat16)
    d = str(tmp_path / "ckpt")
    out = str(tmp_path / "out")
    save_hf_weights(m, d)
    a, b = tokens(m, 21, 70), tokens(m, 12, 71)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:9], "want": [0, 8]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[9:10], "want": []},
                                     {"id": "b", "tokens": b[:11], "want": [10]}], "end": []},
             {"step": 2, "entries": [{"id": "b", "tokens": b[11:], "want": [0]},
                                     {"id": "a", "tokens": a[10:], "want": [10]}],
              "end": ["a", "b"]}]
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    r = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", d,
                        "--dtype", "float32", "--out", out, "--max-tokens", "128", "--device", "cpu"],
                       input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True,
                       text=True, timeout=300)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [ln for ln in r.stdout.splitlines() if ln.startswith("done")] == ["done 0", "done 1", "done 2"]
    orc = Oracle(m)
    (ra, sa), (rb, sb) = orc.expect(a), orc.expect(b)
    V = m.config.vocab_size
    got = {i: torch.from_numpy(np.fromfile(os.path.join(out, f"{i}.f32"), dtype="<f4")).view(-1, V)
           for i in range(3)}
    check_conditioned(got[0], ra[[0, 8]], sa[[0, 8]])
    check_conditioned(got[1], rb[[10]], sb[[10]])
    check_conditioned(got[2], torch.stack([rb[11], ra[20]]), torch.stack([sb[11], sa[20]]))


@pytest.mark.gpu
@pytest.mark.parametrize("name", list(CONFIGS))
def test_bf16_close_to_oracle_and_cut_invariant(name):
    """bf16 serving: within rounding of the float64 oracle, and the same logits (to rounding)
    however the prompt is cut and whether rows decode through the hipGraph path or eagerly."""
    m = make(name, "cuda", dtype=torch.bfloat16, seed=9)
    toks = tokens(m, 170, 50)
    want = Oracle(m).forward(toks)
    whole = replay_alone(m, "cuda", toks, [1000])
    cut = replay_alone(m, "cuda", toks, [7, 1, 2, 1, 1, 16])
    eager = replay_alone(m, "cuda", toks, [30] + [1] * 150, graphs=False)
    close_to_rounding(m, toks, want, whole, cut, eager)


@pytest.mark.gpu
def test_graph_replayed_decode_matches_eager():
    """Decode steps replay a captured hipGraph per batch bucket; several replays, with eager
    prefill steps of other requests between them, give what eager decoding gives."""
    m = make("tiny", "cuda", seed=10)
    a, b = tokens(m, 50, 51), tokens(m, 33, 52)
    orc = Oracle(m)
    (wa, sa), (wb, sb) = orc.expect(a), orc.expect(b)
    rp = TraceReplay(engine(m, "cuda", graphs=True))
    got_a = [rp.step([{"id": "a", "tokens": a[:20], "want": list(range(20))}], [])]
    for i in range(20, 35):                                # graph bucket 1
        got_a.append(rp.step([{"id": "a", "tokens": a[i:i + 1], "want": [0]}], []))
    got_b = [rp.step([{"id": "b", "tokens": b[:10], "want": list(range(10))}], [])]
    for i in range(15):                                    # graph bucket 2, both decoding
        o = rp.step([{"id": "a", "tokens": a[35 + i:36 + i], "want": [0]},
                     {"id": "b", "tokens": b[10 + i:11 + i], "want": [0]}], [])
        got_a.append(o[0:1])
        got_b.append(o[1:2])
    check_conditioned(torch.cat(got_a, 0), wa, sa)
    check_conditioned(torch.cat(got_b, 0), wb[:25], sb[:25])
