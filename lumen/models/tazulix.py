"""Tazulix: a decoder-only pre-norm stack of softmax attention and lightning attention layers with
dense or routed feed-forwards, in which a run of layers can be passed through more than once and
reads the embedding anew at every pass.

The stream starts as x0 = embed[token] * ``embedding_scale`` and is kept in fp32.  Per layer, with
N(z) = z / sqrt(mean(z^2) + eps) * w:

    x <- x + mixer(N_1(x));   x <- x + ff(N_2(x))        (the second one where there is a feed-forward)

``loop`` {start, stop, times}: layers start .. stop - 1 run ``times`` times in a row with the same
weights; every pass has caches and state of its own.  Ahead of the first layer of EVERY pass

    x <- W_in [x; x0]                                     (``loop.in``, [width, 2 width])

Mixers (``layers[i].type``), h being the layer's normed input:

``attention``  grouped-query attention.  q = W_q h + b_q and k = W_k h + b_k are RMS-normed over the
    WHOLE projection (all heads at once) with weights of that size, then turned in the half layout
    on the first ``rot.dims`` entries of each head; v = W_v h + b_v.  With ``rot.scaling`` the
    frequencies are YaRN's (interpolated by ``factor`` where a dimension turns less than ``slow``
    times within ``original`` positions, kept where it turns more than ``fast`` times, a ramp
    between) and cosine and sine carry the factor 0.1 ln(factor) + 1.  score = q.k * scale, ordinary
    softmax over all earlier keys.

``lightning``  q, k, v = silu of their projections; S <- decay_h S + k v^T, o = S^T q; the heads
    RMS-normed together, times sigmoid(W_g h), through W_o.

Feed-forwards (``layers[i].mlp``): ``dense``  W_down relu(W_up h)^2.  ``moe``  the ``top`` experts with
the largest s = sigmoid(W_r h) each take s_e h as their input -- the weight multiplies what goes in,
not what comes out --, plus a shared expert on h itself; an expert is

    g = min(W_gate z, limit),  u = clamp(W_up z, -limit, limit);   W_down (g sigmoid(1.702 g) (u + 1))

Output: N with ``final.norm``, logits through ``head``.

The checkpoint names tensors ``embed`` / ``loop.in`` / ``l<i>.<part>`` / ``final.norm`` / ``head``;
this module keeps exactly those names.  The serving step function is
``lumen.serve.hybrid_runner.TazulixWeights.run_layers``; ``forward`` runs it on fresh caches.
"""
from __future__ import annotations

import math
from typing import Dict, List

import torch

from .config import ModelConfig
from .named import NamedTensorModel
from .silonex import MAX_STATE_KEY, layer_runs

MIXERS = ("attention", "lightning")
# an expert's gate is g * sigmoid(GATE_SLOPE * g), its up projection enters as u + UP_SHIFT: the
# design fixes both
GATE_SLOPE = 1.702
UP_SHIFT = 1.0
MAX_NORM_WIDTH = 16000              # a row of the read-out's norm is held in LDS


def pass_starts(cfg: ModelConfig) -> List[bool]:
    """For every entry of ``layer_runs``: does a pass of the loop begin with it?"""
    n = len(layer_runs(cfg))
    out = [False] * n
    if cfg.loop:
        a, b, t = (int(cfg.loop[k]) for k in ("start", "stop", "times"))
        for p in range(t if b > a else 0):
            out[a + p * (b - a)] = True
    return out


def rotary(m: dict) -> tuple:
    """(rotated entries per head, base, scaling or None) of an attention mixer."""
    r = m.get("rot") or {}
    return int(r.get("dims", 0)), float(r.get("base", 1.0)), r.get("scaling") or None


def tensor_shapes(cfg: ModelConfig) -> Dict[str, tuple]:
    """{checkpoint tensor name: shape} of a configuration."""
    W, V = cfg.hidden_size, cfg.vocab_size
    out: Dict[str, tuple] = {"embed": (V, W)}
    if any(pass_starts(cfg)):
        out["loop.in"] = (W, 2 * W)

    def expert(p, ff):
        out[p + "gate"], out[p + "up"], out[p + "down"] = (ff, W), (ff, W), (W, ff)

    for i, L in enumerate(cfg.layer_specs):
        p, m, f = f"l{i}.", L["mixer"], L.get("mlp")
        x, y = p + "mix.", p + "mlp."
        H, D, Dv = m["heads"], m["dim"], m["vdim"]
        out[p + "norm1"] = (W,)
        if L["type"] == "attention":
            G = m["kv_heads"]
            for n, rows in (("q", H * D), ("k", G * D), ("v", G * Dv)):
                out[x + n], out[x + n + ".b"] = (rows, W), (rows,)
            out[x + "q.norm"], out[x + "k.norm"] = (H * D,), (G * D,)
        else:
            for n, rows in (("q", H * D), ("k", H * D), ("v", H * Dv), ("g", H * Dv)):
                out[x + n] = (rows, W)
            out[x + "norm"] = (H * Dv,)
        out[x + "o"] = (W, H * Dv)
        if f:
            out[p + "norm2"] = (W,)
            if f["kind"] == "dense":
                out[y + "up"], out[y + "down"] = (f["ff"], W), (W, f["ff"])
            else:
                for e in range(f["router"]["experts"]):
                    expert(y + f"e{e}.", f["expert"]["ff"])
                out[y + "router"] = (f["router"]["experts"], W)
                if f.get("shared"):
                    expert(y + "shared.", f["shared"]["ff"])
    out["final.norm"] = (W,)
    out["head"] = (V, W)
    return out


def validate(cfg: ModelConfig) -> None:
    """Reject configurations the step function or its kernels cannot run, with the reason."""
    n = len(cfg.layer_specs)
    if cfg.loop:
        a, b, t = (int(cfg.loop[k]) for k in ("start", "stop", "times"))
        if not 0 <= a <= b <= n or t < 1:
            raise ValueError(f"loop {cfg.loop} does not fit {n} layers")
    for i, L in enumerate(cfg.layer_specs):
        m = L["mixer"]
        if L["type"] == "attention":
            if m["heads"] % m["kv_heads"]:
                raise ValueError(f"layer {i}: heads {m['heads']} not a multiple of kv_heads "
                                 f"{m['kv_heads']}")
            dims, _, sc = rotary(m)
            if dims % 2 or not 0 <= dims <= m["dim"]:
                raise ValueError(f"layer {i}: rot.dims {dims} must be even and at most dim "
                                 f"{m['dim']}")
            if sc and not (float(sc["factor"]) > 0 and float(sc["original"]) > 0
                           and float(sc["fast"]) > 0 and float(sc["slow"]) > 0):
                raise ValueError(f"layer {i}: rot.scaling needs positive values, got {sc}")
            if max(m["dim"], m["vdim"]) > 512:
                raise ValueError(f"layer {i}: head sizes above 512 are not supported")
        elif L["type"] == "lightning":
            if not 1 <= int(m["dim"]) <= MAX_STATE_KEY:
                raise ValueError(f"layer {i}: recurrent key size {m['dim']} must be in "
                                 f"[1, {MAX_STATE_KEY}]")
            if m["heads"] * m["vdim"] > MAX_NORM_WIDTH:
                raise ValueError(f"layer {i}: {m['heads']} heads of {m['vdim']} are wider than "
                                 f"{MAX_NORM_WIDTH}")
            d = m["decay"]
            if len(d) != m["heads"] or not all(0.0 <= float(x) for x in d):
                raise ValueError(f"layer {i}: decay must give one value >= 0 per head")
        else:
            raise ValueError(f"layer {i}: unknown mixer type {L['type']!r}")
        f = L.get("mlp")
        if not f or f.get("kind") == "dense":
            continue
        if f.get("kind") != "moe":
            raise ValueError(f"layer {i}: unknown feed-forward kind {f.get('kind')!r}")
        E, top = int(f["router"]["experts"]), int(f["router"]["top"])
        if not 1 <= top <= E <= 1024:
            raise ValueError(f"layer {i}: top {top} of {E} experts: at least 1, at most all of at "
                             "most 1024")
        for part in ("expert", "shared"):
            if f.get(part) and not float(f[part]["limit"]) > 0:
                raise ValueError(f"layer {i}: mlp.{part}.limit must be positive")


class TazulixForCausalLM(NamedTensorModel):
    supports_packing = False

    def __init__(self, config: ModelConfig, dtype=torch.bfloat16, device=None):
        validate(config)
        super().__init__(config, tensor_shapes(config), dtype, device)

    @torch.no_grad()
    def init_weights(self, std: float = 0.02, seed: int = 0):
        """Random weights for synthetic runs: projections Normal(0, 1 / sqrt(fan_in)), norm
        weights near 1, small biases, embeddings whose scaled rows have unit spread."""
        g = torch.Generator(device="cpu").manual_seed(seed)
        for name in self.tensor_names():
            p = self.tensor(name)
            if name == "embed":
                v = torch.randn(p.shape, generator=g) / self.config.embedding_scale
            elif p.dim() == 2:
                v = torch.randn(p.shape, generator=g) / math.sqrt(p.shape[1])
            elif name.endswith(".b"):
                v = 0.1 * torch.randn(p.shape, generator=g)
            else:                                                  # norm weights
                v = 1.0 + 0.1 * torch.randn(p.shape, generator=g)
            p.copy_(v.to(p.dtype))

    @torch.no_grad()
    def forward(self, input_ids: torch.Tensor) -> torch.Tensor:
        """Logits [B, S, V] of whole sequences starting at position 0: the serving step function
        on a private cache, every row's logits kept."""
        from ..serve.hybrid_runner import forward_fresh

        if input_ids.dim() == 1:
            input_ids = input_ids.view(1, -1)
        return forward_fresh(self, input_ids)
