"""Silonex: a decoder-only stack whose residual stream is kept as several copies, with a run of
layers that is passed through more than once.

The stream starts as S copies x_s = embed[token] and is kept in fp32.  Every sublayer (mixer,
then feed-forward) reads one combination of the copies and writes back through a matrix (the
layer's ``hc1`` / ``hc2`` tensors):

    y    = sublayer(LN(sum_s in[s] x_s))                 LN with weight and shift
    x_t <- sum_s mix[s, t] x_s + out[t] y                 all copies from the old ones

``loop`` {start, stop, times}: layers start .. stop - 1 run ``times`` times in a row with the same
weights; every pass has caches and state of its own (``layer_runs``).

Mixers (``layers[i].type``):

``parallel``  two token mixers on the same input; each output is RMS-normed over the model width
    with its own weight, and the result is half their sum.
    left: grouped-query attention; q and k RMS-normed per head, then rotary in the half layout on
    ``rot.dims`` entries with frequencies stretched by wavelength (``rot.scaling``); values divided
    by their own root mean square; score = softcap * tanh(q.k * scale / softcap); row i sees the
    keys j with 0 <= i - j < ``mask.size``; ordinary softmax.
    right: gated delta rule.  q, k and v pass a short causal convolution and silu; q and k become
    unit vectors, q times dim^-1/2; beta = sigmoid(W_b h), g = exp(-exp(A_log) softplus(W_a h +
    dt_bias)) per head; S <- g S, u = beta (v - S^T k), S <- S + k u^T, o = S^T q; o RMS-normed per
    head with a shared weight, times silu(W_g h).

``lightning``  q, k, v = silu of their projections; S <- decay_h S + k v^T, o = S^T q; the heads
    RMS-normed together, times sigmoid(W_g h).

``mamba2``  one projection [z | x | B | C | dt]; x, B, C pass a short causal convolution (with a
    bias) and silu; dt = softplus(dt + dt_bias); S <- exp(-exp(A_log) dt) S + dt B x^T, y = S^T C
    + D x; y * silu(z) RMS-normed in ``norm_groups`` equal parts.

Feed-forward ``dense``: W_down (silu(W_gate h) * (W_up h)).

Output: the sum of the copies, LN with ``final.norm``, logits = embed (.) * logit_scale.

The checkpoint names tensors ``embed`` / ``l<i>.<part>`` / ``final.norm``; this module keeps
exactly those names.  The serving step function is
``lumen.serve.hybrid_runner.SilonexWeights.run_layers``; ``forward`` runs it on fresh caches.
"""
from __future__ import annotations

import math
from typing import Dict, List

import torch

from .config import ModelConfig
from .named import NamedTensorModel

MIXERS = ("parallel", "lightning", "mamba2")
# the delta rule's q and k become x / sqrt(sum x^2 + UNIT_EPS): the design fixes it
UNIT_EPS = 1e-6
MAX_STREAMS = 8
MAX_STATE_KEY = 256
MAX_TAPS = 16


def layer_runs(cfg: ModelConfig) -> List[int]:
    """The layer each pass of a step runs, in order: the looped layers appear ``times`` times."""
    n = len(cfg.layer_specs)
    lp = cfg.loop
    if not lp:
        return list(range(n))
    a, b, t = int(lp["start"]), int(lp["stop"]), int(lp["times"])
    return list(range(a)) + list(range(a, b)) * t + list(range(b, n))


def window(m: dict) -> int:
    """An attention half's window in tokens (0: everything before a row is seen)."""
    return int((m.get("mask") or {}).get("size") or 0)


def tensor_shapes(cfg: ModelConfig) -> Dict[str, tuple]:
    """{checkpoint tensor name: shape} of a configuration."""
    W, V, S = cfg.hidden_size, cfg.vocab_size, cfg.streams
    out: Dict[str, tuple] = {"embed": (V, W)}

    def norm(name):
        out[name], out[name + ".b"] = (W,), (W,)

    for i, L in enumerate(cfg.layer_specs):
        p, m, f = f"l{i}.", L["mixer"], L.get("mlp")
        x = p + "mix."
        for q in (1, 2) if f else (1,):
            norm(p + f"norm{q}")
            out[p + f"hc{q}.in"], out[p + f"hc{q}.out"] = (S,), (S,)
            out[p + f"hc{q}.mix"] = (S, S)
        if L["type"] == "parallel":
            a = m["left"]
            H, G, D, Dv = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
            y = x + "left."
            out[y + "q"], out[y + "k"], out[y + "v"] = (H * D, W), (G * D, W), (G * Dv, W)
            out[y + "q.norm"], out[y + "k.norm"] = (D,), (D,)
            out[y + "o"], out[y + "out"] = (W, H * Dv), (W,)
            a = m["right"]
            H, G, D, Dv, K = a["heads"], a["kv_heads"], a["dim"], a["vdim"], a["conv"]
            y = x + "right."
            for n, rows in (("q", G * D), ("k", G * D), ("v", H * Dv)):
                out[y + n], out[y + n + ".conv"] = (rows, W), (rows, K)
            for n in ("a", "b"):
                out[y + n] = (H, W)
            out[y + "A_log"], out[y + "dt_bias"] = (H,), (H,)
            out[y + "norm"], out[y + "g"] = (Dv,), (H * Dv, W)
            out[y + "o"], out[y + "out"] = (W, H * Dv), (W,)
        elif L["type"] == "lightning":
            H, D, Dv = m["heads"], m["dim"], m["vdim"]
            out[x + "q"], out[x + "k"] = (H * D, W), (H * D, W)
            out[x + "v"], out[x + "g"] = (H * Dv, W), (H * Dv, W)
            out[x + "norm"], out[x + "o"] = (H * Dv,), (W, H * Dv)
        else:
            H, P, N, G, K = m["heads"], m["vdim"], m["state"], m["groups"], m["conv"]
            C = H * P + 2 * G * N
            out[x + "in"] = (H * P + C + H, W)
            out[x + "conv"], out[x + "conv.b"] = (C, K), (C,)
            for n in ("dt_bias", "A_log", "D"):
                out[x + n] = (H,)
            out[x + "norm"], out[x + "o"] = (H * P,), (W, H * P)
        if f:
            y = p + "mlp."
            out[y + "gate"], out[y + "up"], out[y + "down"] = (f["ff"], W), (f["ff"], W), (W, f["ff"])
    norm("final.norm")
    return out


def validate(cfg: ModelConfig) -> None:
    """Reject configurations the step function or its kernels cannot run, with the reason."""
    n = len(cfg.layer_specs)
    if not 1 <= cfg.streams <= MAX_STREAMS:
        raise ValueError(f"streams must be in [1, {MAX_STREAMS}], got {cfg.streams}")
    if cfg.loop:
        a, b, t = (int(cfg.loop[k]) for k in ("start", "stop", "times"))
        if not 0 <= a <= b <= n or t < 1:
            raise ValueError(f"loop {cfg.loop} does not fit {n} layers")

    def multiple(i, what, a, b):
        if b < 1 or a % b:
            raise ValueError(f"layer {i}: {what}: {a} is not a multiple of {b}")

    def taps(i, k):
        if not 1 <= int(k) <= MAX_TAPS:
            raise ValueError(f"layer {i}: conv taps must be in [1, {MAX_TAPS}], got {k}")

    def state_key(i, d):
        if not 1 <= int(d) <= MAX_STATE_KEY:
            raise ValueError(f"layer {i}: recurrent key size {d} must be in [1, {MAX_STATE_KEY}]")

    for i, L in enumerate(cfg.layer_specs):
        m = L["mixer"]
        if L["type"] == "parallel":
            a, r = m["left"], m["right"]
            multiple(i, "heads over kv_heads (left)", a["heads"], a["kv_heads"])
            dims = a["rot"]["dims"]
            if dims % 2 or not 0 <= dims <= a["dim"]:
                raise ValueError(f"layer {i}: rot.dims {dims} must be even and at most dim "
                                 f"{a['dim']}")
            if max(a["dim"], a["vdim"]) > 512:
                raise ValueError(f"layer {i}: head sizes above 512 are not supported")
            multiple(i, "heads over kv_heads (right)", r["heads"], r["kv_heads"])
            taps(i, r["conv"])
            state_key(i, r["dim"])
        elif L["type"] == "lightning":
            state_key(i, m["dim"])
            d = m["decay"]
            if len(d) != m["heads"] or not all(0.0 <= float(x) for x in d):
                raise ValueError(f"layer {i}: decay must give one value >= 0 per head")
        elif L["type"] == "mamba2":
            multiple(i, "heads over groups", m["heads"], m["groups"])
            multiple(i, "channels over norm_groups", m["heads"] * m["vdim"], m["norm_groups"])
            taps(i, m["conv"])
            state_key(i, m["state"])
        else:
            raise ValueError(f"layer {i}: unknown mixer type {L['type']!r}")
        f = L.get("mlp")
        if f and f.get("kind", "dense") != "dense":
            raise ValueError(f"layer {i}: unknown feed-forward kind {f.get('kind')!r}")


class SilonexForCausalLM(NamedTensorModel):
    supports_packing = False

    def __init__(self, config: ModelConfig, dtype=torch.bfloat16, device=None):
        validate(config)
        super().__init__(config, tensor_shapes(config), dtype, device)

    @torch.no_grad()
    def init_weights(self, std: float = 0.02, seed: int = 0):
        """Random weights for synthetic runs: projections Normal(0, 1 / sqrt(fan_in)), norm
        weights near 1 with small shifts, copies that mostly keep themselves, decays spread from
        slow to fast heads."""
        g = torch.Generator(device="cpu").manual_seed(seed)
        for name in self.tensor_names():
            p = self.tensor(name)
            leaf = name.rsplit(".", 1)[-1]
            if leaf == "mix" and ".hc" in name:
                v = 0.9 * torch.eye(p.shape[0]) + 0.1 * torch.randn(p.shape, generator=g)
            elif leaf in ("in", "out") and ".hc" in name:
                v = 1.0 / p.shape[0] + 0.1 * torch.randn(p.shape, generator=g)
            elif leaf == "conv":
                v = torch.randn(p.shape, generator=g) / math.sqrt(p.shape[1])
            elif p.dim() == 2:
                v = torch.randn(p.shape, generator=g) / math.sqrt(p.shape[1])
            elif leaf == "A_log":
                v = torch.log(torch.linspace(0.5, 8.0, p.numel()))
            elif leaf == "dt_bias":
                v = -2.0 + torch.randn(p.shape, generator=g)
            elif leaf == "b":
                v = 0.1 * torch.randn(p.shape, generator=g)
            else:                                                  # norm weights, D
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
