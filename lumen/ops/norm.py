"""Fused residual-add + RMSNorm (HIP kernel ``kernels/rmsnorm.hip``; torch reference on CPU).

``rms_norm(x, w, eps, residual)`` returns ``(y, s)`` with ``s = x + residual`` (the new residual
stream, ``x`` itself when no residual is given) and ``y = s * rsqrt(mean(s^2) + eps) * w``.
Mirrors transformers' LlamaRMSNorm (used by the model loaded at
reference training/train_baseline.py:122) with the residual add of the decoder layer fused in.
"""
from __future__ import annotations

from typing import Optional, Tuple

import torch

from ._native import native, use_native

def _occupancy_cap(C) -> None:
    """(No-op.)  An occupancy cap through reserved dynamic LDS per workgroup measured no gain;
    the knob stays reachable for scripts/probes/rmsnorm_probe.py via ``C.set_rms_lds``."""


def rms_norm_ref(x, w, eps, residual=None):
    s = x if residual is None else (x.float() + residual.float()).to(x.dtype)
    sf = s.float()
    rstd = torch.rsqrt(sf.pow(2).mean(-1, keepdim=True) + eps)
    wf = (w if w.requires_grad else w.detach()).float()  # never save a ZeRO-3 param object
    y = (sf * rstd * wf).to(x.dtype)
    return y, s


class _FusedAddRMSNorm(torch.autograd.Function):
    @staticmethod
    def forward(ctx, x, residual, w, eps, ext=0):
        C = native()
        _occupancy_cap(C)
        x = x.contiguous()
        if ext and x.dim() == 2:
            # y as the first H columns of a [rows, H + ext] buffer (row-strided kernel output)
            y = torch.empty(x.shape[0], x.shape[1] + ext, dtype=x.dtype,
                            device=x.device)[:, :x.shape[1]]
        else:
            y = torch.empty_like(x)
        rows = x.numel() // x.shape[-1]
        rstd = torch.empty(rows, dtype=torch.float32, device=x.device)
        if residual is not None:
            s = torch.empty_like(x)
            C.rmsnorm_fwd(x, residual.contiguous(), w, y, s, rstd, eps)
        else:
            s = x
            C.rmsnorm_fwd(x, None, w, y, None, rstd, eps)
        ctx.save_for_backward(s, w, rstd)
        ctx.has_res = residual is not None
        ctx.w_grad = w.requires_grad
        if residual is not None:
            return y, s
        # no residual: s is x itself; hand back a view so autograd tracks it as an output
        return y, s.view_as(s)

    @staticmethod
    def backward(ctx, dy, ds):
        C = native()
        _occupancy_cap(C)
        s, w, rstd = ctx.saved_tensors
        dx = torch.empty_like(s)
        dw = torch.zeros(w.shape, dtype=torch.float32, device=w.device) if ctx.w_grad else None
        C.rmsnorm_bwd(dy.contiguous(), s, w, rstd,
                      ds.contiguous() if ds is not None else None, dx, dw)
        dres = dx if ctx.has_res else None
        return dx, dres, (dw.to(w.dtype) if dw is not None else None), None, None


def rms_norm(x: torch.Tensor, w: torch.Tensor, eps: float,
             residual: Optional[torch.Tensor] = None,
             ext: int = 0) -> Tuple[torch.Tensor, torch.Tensor]:
    if use_native(x):
        return _FusedAddRMSNorm.apply(x, residual, w, eps, ext)
    return rms_norm_ref(x, w, eps, residual)


def layer_norm(x, w, b, eps):
    """OPT LayerNorm (torch op); frozen params enter autograd as detached aliases."""
    fz = lambda t: t if (t is None or t.requires_grad) else t.detach()  # noqa: E731
    return torch.nn.functional.layer_norm(x, (x.shape[-1],), fz(w), fz(b), eps)


# ---- Dynamic Tanh (DyT): tanh(alpha * x) * w + b, no mean or variance ------------------------
# A DyT norm is the triple (w [W], b [W], alpha [] ) of fp32 tensors; alpha stays on the device
# (the kernels read it there, so a captured graph never bakes a value in).  Everything is
# computed in fp32; only the result is rounded to ``out_dtype``.
def dyt_ref(x, norm, out_dtype=None):
    w, b, alpha = norm
    y = torch.tanh(alpha.float() * x.float()) * w.float() + b.float()
    return y.to(out_dtype or x.dtype)


def dyt(x: torch.Tensor, norm, out_dtype=None) -> torch.Tensor:
    """DyT of the rows of ``x`` [rows, W] (fp32 or 16-bit) in ``out_dtype``."""
    from ._seqmix import DT, call, use_seqmix

    out_dtype = out_dtype or x.dtype
    if not use_seqmix(x):
        return dyt_ref(x, norm, out_dtype)
    x = x.contiguous()
    out = torch.empty(x.shape, dtype=out_dtype, device=x.device)
    call("sm_dyt", DT[x.dtype], DT[out_dtype], x, norm[0], norm[1], norm[2], out,
         x.numel() // x.shape[-1], x.shape[-1])
    return out


def dyt_residual_ref(x, y, post, pre=None, out_dtype=None):
    x.add_(dyt_ref(y, post, torch.float32))
    return x, (dyt_ref(x, pre, out_dtype or y.dtype) if pre is not None else None)


def dyt_residual(x: torch.Tensor, y: torch.Tensor, post, pre=None, out_dtype=None):
    """The fp32 residual stream ``x`` [T, W] takes a sublayer's output in place,
    x += DyT_post(y), and -- fused -- the next sublayer's input h = DyT_pre(x) is produced in
    ``out_dtype``.  Returns (x, h or None)."""
    from ._seqmix import DT, call, use_seqmix

    out_dtype = out_dtype or y.dtype
    if not use_seqmix(x):
        return dyt_residual_ref(x, y, post, pre, out_dtype)
    assert x.dtype == torch.float32 and x.is_contiguous() and y.is_contiguous()
    h = torch.empty(x.shape, dtype=out_dtype, device=x.device) if pre is not None else None
    p = pre or (None, None, None)
    call("sm_dyt_residual", DT[y.dtype], DT[out_dtype], x, y, post[0], post[1], post[2], h,
         p[0], p[1], p[2], x.shape[0], x.shape[1])
    return x, h


# ---- RMS norm in groups ------------------------------------------------------------------------
# The row is split into ``groups`` equal consecutive parts and each part is divided by its own
# sqrt(mean(part^2) + eps); the whole row is then multiplied by w (groups = 1: the ordinary RMS
# norm with a plain weight).  fp32 throughout; only a stored result is rounded.
# (HIP: ``csrc/seqmix/rms_group.hip``.)
def group_rms_norm_ref(x, w, groups, eps, out_dtype=None):
    shp = x.shape
    g = x.float().reshape(*shp[:-1], groups, shp[-1] // groups)
    y = (g / torch.sqrt((g * g).mean(-1, keepdim=True) + eps)).reshape(shp) * w.float()
    return y.to(out_dtype or x.dtype)


def group_rms_norm(x: torch.Tensor, w: torch.Tensor, groups: int, eps: float,
                   out_dtype=None) -> torch.Tensor:
    """Group RMS norm of the rows of ``x`` [rows, W] (fp32 or 16-bit; the rows may be a column
    slice of a wider buffer) with the fp32 weight ``w`` [W], stored in ``out_dtype``."""
    from ._seqmix import DT, call, use_seqmix

    out_dtype = out_dtype or x.dtype
    if x.shape[-1] % groups:
        raise ValueError(f"width {x.shape[-1]} is not a multiple of {groups} groups")
    if not use_seqmix(x):
        return group_rms_norm_ref(x, w, groups, eps, out_dtype)
    assert x.dim() == 2 and x.stride(1) == 1 and w.dtype == torch.float32
    out = torch.empty(x.shape, dtype=out_dtype, device=x.device)
    call("sm_group_rms", DT[x.dtype], DT[out_dtype], x, x.stride(0), w, None, out, out.stride(0),
         x.shape[0], x.shape[1], groups, eps)
    return out


def group_rms_residual_ref(x, y, w, groups, eps, cast=None):
    x.add_(group_rms_norm_ref(y, w, groups, eps, torch.float32))
    return x, (x.to(cast) if cast is not None and cast != x.dtype else None)


def group_rms_residual(x: torch.Tensor, y: torch.Tensor, w: torch.Tensor, groups: int,
                       eps: float, cast=None):
    """The fp32 residual stream ``x`` [T, W] takes a sublayer's normed output in place,
    x += group_rms_norm(y) * w, and -- fused, when ``cast`` is a 16-bit dtype -- the new stream is
    also returned rounded to ``cast`` (what the next sublayer's GEMMs read).  Returns
    (x, x in ``cast`` or None)."""
    from ._seqmix import DT, call, use_seqmix

    if x.shape[-1] % groups:
        raise ValueError(f"width {x.shape[-1]} is not a multiple of {groups} groups")
    if not use_seqmix(x):
        return group_rms_residual_ref(x, y, w, groups, eps, cast)
    assert x.dtype == torch.float32 and x.is_contiguous() and y.stride(1) == 1
    xb = None
    if cast is not None and cast != torch.float32:
        xb = torch.empty(x.shape, dtype=cast, device=x.device)
    call("sm_group_rms", DT[y.dtype], DT[cast if xb is not None else torch.float32], y,
         y.stride(0), w, x, xb, x.shape[1], x.shape[0], x.shape[1], groups, eps)
    return x, xb


# ---- layer norm with a weight (and optionally a shift), fused with a scaled residual add ----------
# LN(x) = (x - mean) / sqrt(mean((x - mean)^2) + eps) * w (+ b).  The fp32 residual stream takes a
# sublayer's output multiplied by a constant, x += mult * y, and the same pass produces the next
# sublayer's input LN(x) in the model dtype.  fp32 throughout; only a stored result is rounded.
# (HIP: ``csrc/seqmix/layer_norm.hip``.)
def weight_layer_norm_ref(x, w, eps, out_dtype=None, b=None):
    xf = x.float()
    d = xf - xf.mean(-1, keepdim=True)
    y = d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * w.float()
    if b is not None:
        y = y + b.float()
    return y.to(out_dtype or x.dtype)


def scaled_residual_layer_norm_ref(x, y, mult, w, eps, out_dtype=None, b=None):
    if y is not None:
        x.add_(y.float(), alpha=mult)
    return x, (weight_layer_norm_ref(x, w, eps, out_dtype or x.dtype, b) if w is not None
               else None)


def scaled_residual_layer_norm(x: torch.Tensor, y: Optional[torch.Tensor], mult: float,
                               w: Optional[torch.Tensor], eps: float, out_dtype=None,
                               b: Optional[torch.Tensor] = None):
    """The fp32 residual stream ``x`` [T, W] takes ``mult * y`` in place (``y`` None: nothing is
    added) and -- fused, when ``w`` [W] (fp32) is given -- h = LN(x) * w (+ ``b``) is produced in
    ``out_dtype``.  Returns (x, h or None)."""
    from ._seqmix import DT, call, use_seqmix

    if not use_seqmix(x):
        return scaled_residual_layer_norm_ref(x, y, mult, w, eps, out_dtype, b)
    assert x.dtype == torch.float32 and x.is_contiguous()
    assert y is None or (y.is_contiguous() and y.shape == x.shape)
    assert w is None or (w.dtype == torch.float32 and w.is_contiguous())
    assert b is None or (b.dtype == torch.float32 and b.is_contiguous())
    if y is None and w is None:
        return x, None
    out_dtype = out_dtype or (y.dtype if y is not None else x.dtype)
    h = torch.empty(x.shape, dtype=out_dtype, device=x.device) if w is not None else None
    call("sm_layer_norm", DT[y.dtype] if y is not None else 0, DT[out_dtype], x, y, float(mult), w,
         b, h, x.shape[0], x.shape[1], eps)
    return x, h


def weight_layer_norm(x: torch.Tensor, w: torch.Tensor, eps: float, out_dtype=None,
                      b: Optional[torch.Tensor] = None) -> torch.Tensor:
    """LN(x) * w (+ ``b``) of the fp32 rows ``x`` [T, W] in ``out_dtype``."""
    return scaled_residual_layer_norm(x, None, 0.0, w, eps, out_dtype or x.dtype, b)[1]


# ---- pre-norm residual stream with RMS norms ---------------------------------------------------------
# The fp32 stream takes what joins it and the same pass hands on the next sublayer's input,
# h = x / sqrt(mean(x^2) + eps) * w in the compute dtype -- or, where a GEMM reads the stream itself,
# its two 16-bit parts (rounded value, rounded remainder) as [2 T, W]: their products summed in fp32
# keep about 16 bits of the stream's mantissa.  (HIP: ``csrc/seqmix/stream_rms.hip``.)
SPLIT = "split"


def rms_norm_rows_ref(x, w, eps, out_dtype):
    return (x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w.float()).to(out_dtype)


def _stream_rms(x, keep, out, eps, dtype, tokens=None, table=None, scale=1.0, rows=None, y=None,
                f=(), f2=None, coef=0.0):
    """The new stream in ``x`` [T, W]; ``out``: a norm weight, SPLIT or None -> h, parts or None."""
    from ._seqmix import DT, call, use_seqmix

    split = isinstance(out, str)
    w = None if split else out
    if not use_seqmix(x):
        v = x if keep else torch.zeros_like(x)
        if table is not None:
            v = v + table[tokens].float() * scale
            if rows is not None:
                rows.copy_(table[tokens])
        for p in ([y] if y is not None else []) + list(f):
            v = v + p.float()
        if f2 is not None:
            v = v + coef * f2
        x.copy_(v)
        if w is not None:
            return rms_norm_rows_ref(x, w, eps, dtype)
        if not split or dtype == torch.float32:
            return x if split else None
        hi = x.to(dtype)
        return torch.cat([hi, (x - hi.float()).to(dtype)], 0)
    T, W = x.shape
    assert x.dtype == torch.float32 and x.is_contiguous() and len(f) <= 2
    assert y is None or (y.is_contiguous() and y.dtype == dtype and tuple(y.shape) == (T, W))
    for p in tuple(f) + ((f2,) if f2 is not None else ()):
        assert p.dtype == torch.float32 and p.is_contiguous() and tuple(p.shape) == (T, W)
    assert w is None or (w.dtype == torch.float32 and w.is_contiguous() and w.numel() == W)
    vocab = 0
    if table is not None:
        assert table.is_contiguous() and table.dtype == dtype and table.shape[1] == W
        assert tokens.dtype == torch.int64 and tokens.is_contiguous() and tokens.numel() == T
        vocab = table.shape[0]
    parts = split and dtype != torch.float32
    h = None
    if w is not None or parts:
        h = torch.empty(2 * T if parts else T, W, dtype=dtype, device=x.device)
    fp = list(f) + [None] * (2 - len(f))
    call("sm_stream_rms", DT[dtype], x, int(bool(keep)), table, tokens, vocab, float(scale), rows,
         y, fp[0], fp[1], f2, float(coef), w, h, int(parts), T, W, eps)
    return x if split and not parts else h


def embed_rms(tokens: torch.Tensor, table: torch.Tensor, scale: float, out, eps: float,
              rows: bool = False):
    """The start of a stream: x [T, W] fp32 = table[token] * ``scale`` and, in the table's dtype,
    what ``out`` asks for: RMS norm with the fp32 weight ``out`` [W], SPLIT for the two 16-bit
    parts [2 T, W] (fp32 model: x itself), None for nothing.  Returns (x, h, e), e being the table's
    rows as they are when ``rows`` asks for them, else None."""
    shape = (tokens.shape[0], table.shape[1])
    x = torch.empty(shape, dtype=torch.float32, device=table.device)
    e = torch.empty(shape, dtype=table.dtype, device=table.device) if rows else None
    return x, _stream_rms(x, False, out, eps, table.dtype, tokens, table, scale, e), e


def residual_rms(x: torch.Tensor, y: torch.Tensor, out, eps: float):
    """The stream ``x`` [T, W] fp32 takes a sublayer's output ``y`` (compute dtype) in place;
    returns what ``out`` asks for (see ``embed_rms``)."""
    return _stream_rms(x, True, out, eps, y.dtype, y=y)


def parts_rms(parts: torch.Tensor, base: torch.Tensor, coef: float, out, eps: float, dtype):
    """A new stream from a GEMM over the old one's parts: ``parts`` [T, W] or [2 T, W] fp32 (high
    rows, then low rows) summed, plus ``coef`` * ``base`` [T, W] fp32.  Returns (x, h)."""
    T, W = base.shape
    x = torch.empty(T, W, dtype=torch.float32, device=base.device)
    f = (parts,) if parts.shape[0] == T else (parts[:T], parts[T:])
    return x, _stream_rms(x, False, out, eps, dtype, f=f, f2=base, coef=coef)


# ---- a recurrence's read-out: group RMS norm and output gate ---------------------------------------
# The fp32 row x is normed in ``groups`` equal parts (each by its own root mean square), weighted,
# and gated by act(g) with act = SiLU or the sigmoid; the gate multiplies either before the norm or
# after it.  fp32 throughout; only the result is rounded.  (HIP: ``csrc/seqmix/rms_group.hip``.)
GATES = {"silu": 0, "sigmoid": 1}


def gated_rms_norm_ref(x, g, w, groups, eps, gate, gate_first):
    a = torch.sigmoid(g.float())
    a = a * g.float() if gate == "silu" else a
    xf = x.float() * a if gate_first else x.float()
    T, W = x.shape
    p = xf.reshape(T, groups, W // groups)
    p = p / torch.sqrt((p * p).mean(-1, keepdim=True) + eps)
    wf = w.float()
    y = p.reshape(T, W) * (wf if wf.numel() == W else wf.repeat(groups))
    return (y if gate_first else y * a).to(g.dtype)


def gated_rms_norm(x: torch.Tensor, g: torch.Tensor, w: torch.Tensor, groups: int, eps: float,
                   gate: str, gate_first: bool) -> torch.Tensor:
    """``x`` [T, W] fp32 and its gate logits ``g`` [T, W] (a column slice of a fused projection is
    fine) -> [T, W] in g's dtype; ``w`` fp32 [W], or [W / groups] shared by the groups; ``gate``:
    silu | sigmoid; ``gate_first``: norm(x * act(g)) * w instead of norm(x) * w * act(g)."""
    from ._seqmix import DT, call, use_seqmix

    T, W = x.shape
    if W % groups:
        raise ValueError(f"width {W} is not a multiple of {groups} groups")
    if w.numel() not in (W, W // groups):
        raise ValueError(f"{w.numel()} weights for rows of {W} in {groups} groups")
    if not use_seqmix(x):
        return gated_rms_norm_ref(x, g, w, groups, eps, gate, gate_first)
    assert x.dtype == torch.float32 and x.is_contiguous() and w.dtype == torch.float32
    assert g.stride(1) == 1 and tuple(g.shape) == (T, W)
    out = torch.empty(T, W, dtype=g.dtype, device=x.device)
    call("sm_gated_rms", DT[g.dtype], x, g, g.stride(0), w, out, T, W, groups,
         int(w.numel() != W), int(bool(gate_first)), GATES[gate], eps)
    return out


# ---- hyper-connections: a residual stream kept as several copies --------------------------------------
# Between two sublayers, on the copies x_1 .. x_S of a row:
#     x'_t = sum_s mix[s, t] x_s + out[t] y          (y: the sublayer's output)
#     h    = LN(sum_t in[t] x'_t) * w + b            (the next sublayer's input)
# fp32 throughout; only h is rounded.  (HIP: ``csrc/seqmix/hyper.hip``.)
def hyper_start(tokens: torch.Tensor, table: torch.Tensor, S: int, w_in: torch.Tensor,
                norm, eps: float, out_dtype):
    """The start of a step: ``S`` copies of each token's embedding row -> (x [T, S, W] fp32,
    h [T, W] = LN(sum_t w_in[t] x_t) * norm[0] + norm[1] in ``out_dtype``)."""
    from ._seqmix import DT, call, use_seqmix

    T, W = tokens.shape[0], table.shape[1]
    if not use_seqmix(table):
        x = table[tokens].float().view(T, 1, W).repeat(1, S, 1)
        u = (x * w_in.float().view(1, S, 1)).sum(1)
        return x, weight_layer_norm_ref(u, norm[0], eps, out_dtype, norm[1])
    assert table.is_contiguous() and tokens.dtype == torch.int64 and tokens.is_contiguous()
    assert table.dtype == out_dtype
    x = torch.empty(T, S, W, dtype=torch.float32, device=table.device)
    h = torch.empty(T, W, dtype=out_dtype, device=table.device)
    call("sm_hyper_mix", DT[out_dtype], x, table, tokens, table.shape[0], None, None, None, None,
         0.0, None, None, w_in, norm[0], norm[1], eps, h, None, 1, T, S, W)
    return x, h


def hyper_mix_ref(x, ys, pair, mix, out, w_in, norm, eps, out_dtype):
    y = ys[0].float()
    if len(ys) == 2:
        wa, wb, eps_y = pair
        rms = lambda t: t / torch.sqrt((t * t).mean(-1, keepdim=True) + eps_y)  # noqa: E731
        y = rms(y) * wa.float() + rms(ys[1].float()) * wb.float()
    new = torch.einsum("nsw,st->ntw", x, mix.float()) + out.float().view(1, -1, 1) * y[:, None]
    x.copy_(new)
    u = (x * w_in.float().view(1, -1, 1)).sum(1)
    return u if norm is None else weight_layer_norm_ref(u, norm[0], eps, out_dtype, norm[1])


def hyper_mix(x: torch.Tensor, ys, pair, mix: torch.Tensor, out: torch.Tensor,
              w_in: torch.Tensor, norm, eps: float, out_dtype=None, keep: bool = True):
    """``x`` [T, S, W] fp32 takes a sublayer's output through ``mix`` [S, S] (from, to) and ``out``
    [S] in place (``keep`` False: the copies are not needed any more and need not be stored);
    returns LN(sum_t w_in[t] x_t) with ``norm`` = (w, b) in ``out_dtype``, or with ``norm`` None the
    fp32 sum itself.  ``ys``: one output [T, W] in the compute dtype, or two that are RMS-normed over
    the row with the weights of ``pair`` = (w_a, w_b, eps) and added."""
    from ._seqmix import DT, call, use_seqmix

    T, S, W = x.shape
    if len(ys) not in (1, 2) or (len(ys) == 2) != (pair is not None):
        raise ValueError("one sublayer output, or two with their norms' weights")
    out_dtype = out_dtype or ys[0].dtype
    if not use_seqmix(x):
        return hyper_mix_ref(x, ys, pair, mix, out, w_in, norm, eps, out_dtype)
    if S > 8:
        raise ValueError(f"{S} residual copies > 8 are not supported")
    assert x.dtype == torch.float32 and x.is_contiguous()
    for y in ys:
        assert y.is_contiguous() and tuple(y.shape) == (T, W) and y.dtype == out_dtype
    for f in (mix, out, w_in) + tuple(norm or ()) + tuple((pair or ())[:2]):
        assert f.dtype == torch.float32 and f.is_contiguous()
    dst = torch.empty(T, W, dtype=torch.float32 if norm is None else out_dtype, device=x.device)
    wa, wb, eps_y = pair if pair is not None else (None, None, 0.0)
    call("sm_hyper_mix", DT[out_dtype], x, None, None, 0, ys[0], ys[1] if len(ys) == 2 else None,
         wa, wb, eps_y, mix, out, w_in, norm[0] if norm else None, norm[1] if norm else None, eps,
         dst if norm else None, None if norm else dst, int(bool(keep)), T, S, W)
    return dst


# ---- depth-weighted layer inputs: layer scale, history, weighted average, next norm ---------------
# A stack whose layer i reads a weighted average of everything before it keeps every layer's
# result X_0 .. X_L of the step's rows in ``hist`` [L + 1, T, W] (fp32).  One pass per layer:
#     X_n = x + sum_k scale_k * y_k          (the sublayers' outputs with per-channel scales)
#     x  <- sum_{j <= n} mix[j] * X_j         (what the next layer reads)
#     h   = x / sqrt(mean(x^2) + eps) * w     (its norm, in the compute dtype)
# fp32 throughout; only h is rounded.  (HIP: ``csrc/seqmix/depth_mix.hip``.)
def depth_mix_norm_ref(hist, n, x, ys, scales, mix, w, eps, out_dtype):
    new = x.float().clone()
    for y, sc in zip(ys, scales):
        new += y.float() * sc.float()
    hist[n] = new
    xn = (hist[:n + 1] * mix.float().view(n + 1, 1, 1)).sum(0)
    h = None
    if w is not None:
        h = (xn / torch.sqrt((xn * xn).mean(-1, keepdim=True) + eps) * w.float()).to(out_dtype)
    return xn, h


def depth_mix_norm(hist: torch.Tensor, n: int, x: torch.Tensor, ys, scales, mix: torch.Tensor,
                   w: Optional[torch.Tensor], eps: float, out_dtype=None):
    """``hist`` [L + 1, T, W] fp32 holds X_0 .. X_(n-1); ``x`` [T, W] fp32 is the stream layer
    n - 1 read; ``ys`` (up to three [T, W] sublayer outputs in the compute dtype) join it with the
    per-channel fp32 ``scales`` [W] and the sum is stored as X_n; the new stream is
    sum_j ``mix``[j] X_j over j = 0 .. n (``mix`` [n + 1] fp32) and, with ``w`` [W] (fp32, the
    weight the normed row is multiplied by), h = rms_norm(stream) * w in ``out_dtype``.  Returns
    (stream fp32 [T, W], h or None)."""
    from ._seqmix import DT, call, use_seqmix

    if not 1 <= len(ys) <= 3 or len(ys) != len(scales):
        raise ValueError("one to three sublayer outputs, each with its scale")
    if not 1 <= n < hist.shape[0] or mix.numel() != n + 1:
        raise ValueError(f"history of {hist.shape[0]} entries, entry {n}, {mix.numel()} weights")
    out_dtype = out_dtype or ys[0].dtype
    if not use_seqmix(x):
        return depth_mix_norm_ref(hist, n, x, ys, scales, mix, w, eps, out_dtype)
    T, W = x.shape
    assert hist.dtype == torch.float32 and hist.is_contiguous() and tuple(hist.shape[1:]) == (T, W)
    assert x.dtype == torch.float32 and x.is_contiguous() and mix.dtype == torch.float32
    for y, sc in zip(ys, scales):
        assert y.is_contiguous() and y.shape == x.shape and y.dtype == ys[0].dtype
        assert sc.dtype == torch.float32 and sc.is_contiguous() and sc.numel() == W
    assert w is None or (w.dtype == torch.float32 and w.is_contiguous())
    xn = torch.empty_like(x)
    h = torch.empty(T, W, dtype=out_dtype, device=x.device) if w is not None else None
    yp = list(ys) + [None] * (3 - len(ys))
    sp = list(scales) + [None] * (3 - len(ys))
    call("sm_depth_mix", DT[ys[0].dtype], DT[out_dtype], hist, n, x, yp[0], sp[0], yp[1], sp[1],
         yp[2], sp[2], mix, w, xn, h, T, W, eps)
    return xn, h
