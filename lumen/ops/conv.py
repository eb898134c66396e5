"""Causal depthwise convolutions over time with per-sequence tails.

``dyt_canon``, on a layer's normed input (below); ``short_conv``, on columns of a projection:
y_t = silu(sum_j w[:, taps - 1 - j] x_(t - j) (+ bias)).  Its tail holds the last taps - 1 INPUT
rows of every sequence as the projection stored them, [slots, taps - 1, C] in the model dtype.
(HIP: ``csrc/seqmix/head_scan_step.hip``.)

``dyt_canon``: h = DyT(x) on every row, then out_t = h_t + sum_j w[:, j] * h_(t - taps + 1 + j)
with zeros before a sequence's start.  The last ``taps - 1`` normed rows of every sequence live
in ``tail`` [slots, taps - 1, W] (fp32), so a step may begin anywhere in a sequence: rows before
the step's first row come from the tail (positions below 0 read as zero, whatever a reused slot
still holds), and the tail is moved on to the step's last rows afterwards.  (HIP:
``csrc/seqmix/norm_conv.hip``, norm and convolution in one pass over x.)
"""
from __future__ import annotations

from typing import Optional

import torch
import torch.nn.functional as F

from .norm import dyt_ref
from .segments import SegBatch


def dyt_canon_ref(x, norm, conv_w, tail, seg: SegBatch, out_dtype):
    taps = conv_w.shape[1]
    K = taps - 1
    h = dyt_ref(x, norm, torch.float32)
    out = torch.empty_like(h)
    cu, slots, starts = seg.cu.tolist(), seg.slot.tolist(), seg.start.tolist()
    w = conv_w.float()
    for s in range(seg.S):
        a, b, sl, p0 = cu[s], cu[s + 1], slots[s], starts[s]
        if b == a:
            continue
        hist = tail[sl].clone() if K else h.new_zeros(0, h.shape[1])
        for i in range(K):                     # tail row i is position p0 - K + i
            if p0 - K + i < 0:
                hist[i] = 0
        ext = torch.cat([hist, h[a:b]], 0)     # row K + t is the segment's row t
        acc = h[a:b].clone()
        for j in range(taps):
            acc += w[:, j] * ext[j:j + (b - a)]
        out[a:b] = acc
        if K:
            tail[sl] = ext[-K:]
    return out.to(out_dtype)


def dyt_canon(x: torch.Tensor, norm, conv_w: torch.Tensor, tail: torch.Tensor, seg: SegBatch,
              out_dtype) -> torch.Tensor:
    from ._seqmix import DT, call, use_seqmix

    if not use_seqmix(x):
        return dyt_canon_ref(x, norm, conv_w, tail, seg, out_dtype)
    T, W = x.shape
    taps = conv_w.shape[1]
    assert x.dtype == torch.float32 and x.is_contiguous() and conv_w.dtype == torch.float32
    assert tail.dtype == torch.float32 and tail.shape[1:] == (max(taps - 1, 0), W) or taps == 1
    out = torch.empty(T, W, dtype=out_dtype, device=x.device)
    call("sm_dyt_canon", DT[out_dtype], x, norm[0], norm[1], norm[2], conv_w, tail, out, seg.cu,
         seg.slot, seg.start, seg.row_seg, T, W, taps)
    if taps > 1:
        call("sm_canon_tail", x, norm[0], norm[1], norm[2], tail, seg.cu, seg.slot, seg.start,
             seg.S, W, taps)
    return out


def short_conv_ref(x, w, bias, tail, seg: SegBatch):
    taps = w.shape[1]
    K = taps - 1
    out = torch.empty(x.shape, dtype=torch.float32, device=x.device)
    cu, slots, starts = seg.cu.tolist(), seg.slot.tolist(), seg.start.tolist()
    for s in range(seg.S):
        a, b, sl, p0 = cu[s], cu[s + 1], slots[s], starts[s]
        if b == a:
            continue
        hist = tail[sl].float().clone()
        for i in range(K):                     # tail row i is position p0 - K + i
            if p0 - K + i < 0:
                hist[i] = 0
        ext = torch.cat([hist, x[a:b].float()], 0)
        acc = sum(w[:, j].float() * ext[j:j + (b - a)] for j in range(taps))
        out[a:b] = F.silu(acc if bias is None else acc + bias.float())
        if K:
            tail[sl] = ext[-K:].to(tail.dtype)
    return out.to(x.dtype)


def short_conv(x: torch.Tensor, w: torch.Tensor, bias: Optional[torch.Tensor],
               tail: torch.Tensor, seg: SegBatch) -> torch.Tensor:
    """x [T, C] (rows may be a column slice of a fused projection), w [C, taps] fp32, bias [C]
    fp32 or None, tail [slots, taps - 1, C] in x's dtype -> silu(conv(x)) [T, C] in x's dtype; the
    tail moves on.  One launch for decoded rows; prompt portions take one pass over strips of rows
    and one over the segments' tails."""
    from ._seqmix import DT, call, use_seqmix

    T, C = x.shape
    taps = w.shape[1]
    if w.shape[0] != C or tuple(tail.shape[1:]) != (taps - 1, C):
        raise ValueError(f"convolution {tuple(w.shape)} / tail {tuple(tail.shape)} for {C} channels")
    if not use_seqmix(x):
        return short_conv_ref(x, w, bias, tail, seg)
    if taps > 16:
        raise ValueError(f"{taps} convolution taps > 16 are not supported")
    assert x.stride(1) == 1 and w.dtype == torch.float32 and w.is_contiguous()
    assert tail.dtype == x.dtype and tail.is_contiguous()
    assert bias is None or (bias.dtype == torch.float32 and bias.is_contiguous())
    out = torch.empty(T, C, dtype=x.dtype, device=x.device)
    P, Tp = seg.portions()
    if P:
        call("sm_short_conv", DT[x.dtype], x, x.stride(0), w, bias, tail, out, seg.cu, seg.slot,
             seg.start, seg.row_seg, Tp, C, taps)
        call("sm_conv_tail", DT[x.dtype], 0, x, x.stride(0), w, bias, tail, out, seg.cu, seg.slot,
             seg.start, P, C, taps)
    if seg.S > P:
        call("sm_conv_tail", DT[x.dtype], 1, x, x.stride(0), w, bias, tail, out, seg.cu[P:],
             seg.slot[P:], seg.start[P:], seg.S - P, C, taps)
    return out
