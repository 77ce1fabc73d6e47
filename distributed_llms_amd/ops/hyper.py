"""Hyper-connections: the residual state of a token is several float32 streams X [T, S, W] instead of one.

A sublayer reads one weighted sum of the streams and its output goes back to all of them while they are mixed:

    u = sum_s in[s] x_s;   h = u / sqrt(mean(u^2) + eps) * gain       (read: the sublayer's normed input)
    x_t <- sum_s mix[s, t] x_s + out[t] y                             (write: all streams at once, from the old ones)

  :func:`embed_streams`   every stream starts as the scaled token embedding
  :func:`stream_read`     the read alone (the first sublayer; with ``in`` = ones the model's last norm)
  :func:`stream_step`     the write of one sublayer and the read of the next in one launch

``y`` is one output or two that are normed apart before they are summed.  Streams, mixing and norms are float32
whatever the activation type.  CUDA tensors go to the in-tree HIP kernels (csrc/kernels/hyper.hip) and raise if
those are not built; CPU tensors run the plain PyTorch forms.
"""
from __future__ import annotations

from typing import Optional, Tuple

import torch

from .seqmix import _ck, _f32flag, _k, _ptr, _ref_rms, _stream

MAX_STREAMS = 16
MAX_WIDTH = 16384          # the read keeps one row in LDS


def embed_streams(ids: torch.Tensor, table: torch.Tensor, streams: int, scale: float = 1.0) -> torch.Tensor:
    """X [T, streams, W] float32, every stream = table[ids] * scale."""
    t, (v, w) = ids.numel(), table.shape
    if not table.is_cuda:
        return (table.index_select(0, ids.long()).float() * scale)[:, None, :].repeat(1, streams, 1)
    _ck(ids, "ids", torch.int32)
    _ck(table, "table")
    x = torch.empty(t, streams, w, dtype=torch.float32, device=table.device)
    _k().hc_embed(x.data_ptr(), ids.data_ptr(), table.data_ptr(), t, streams, w, v, float(scale), _f32flag(table), _stream())
    return x


def _ref_read(x: torch.Tensor, w_in: torch.Tensor, gain: float, eps: float, act_dtype) -> torch.Tensor:
    u = (x * w_in.float()[None, :, None]).sum(1)
    return (u * torch.rsqrt(u.pow(2).mean(-1, keepdim=True) + eps) * gain).to(act_dtype)


def _check_streams(x: torch.Tensor, *vecs):
    if x.dim() != 3 or x.dtype != torch.float32 or not 1 <= x.shape[1] <= MAX_STREAMS or x.shape[2] > MAX_WIDTH:
        raise ValueError("hyper-connections: X [T, streams, W] float32, at most 16 streams of width 16384")
    for v in vecs:
        if v is not None and (v.dtype != torch.float32 or v.numel() != x.shape[1] or v.device != x.device):
            raise ValueError("hyper-connections: one float32 weight per stream")


def stream_read(x: torch.Tensor, w_in: torch.Tensor, gain: float, eps: float, act_dtype) -> torch.Tensor:
    """h [T, W] in ``act_dtype``: the RMS norm (scalar weight ``gain``) of sum_s w_in[s] X[:, s]."""
    _check_streams(x, w_in)
    if not x.is_cuda:
        return _ref_read(x, w_in, gain, eps, act_dtype)
    _ck(x, "x", torch.float32)
    _ck(w_in, "w_in", torch.float32)
    t, s, w = x.shape
    h = torch.empty(t, w, dtype=act_dtype, device=x.device)
    _k().hc_step(x.data_ptr(), 0, 0, 0, 0, 0, 0, 1.0, w_in.data_ptr(), float(gain), h.data_ptr(), t, s, w, float(eps),
                 _f32flag(h), _stream())
    return h


def stream_step(x: torch.Tensor, mix: torch.Tensor, w_out: torch.Tensor, o: torch.Tensor, eps: float,
                w_o: Optional[torch.Tensor] = None, o2: Optional[torch.Tensor] = None, w_o2: Optional[torch.Tensor] = None,
                coef: float = 1.0, nxt: Optional[Tuple[torch.Tensor, float]] = None):
    """The close of a sublayer, in place on X: x_t <- sum_s mix[s, t] x_s + w_out[t] y with
    y = coef * (f(o, w_o) + f(o2, w_o2)), f(o, w) = rms_norm(o) * w (plain weight) when ``w`` is given and o itself
    otherwise (``o2`` None: one term).  ``nxt`` = (w_in, gain): also returns the next sublayer's input
    (:func:`stream_read` of the new streams) in ``o``'s dtype.  Returns (x, h or None)."""
    t, s, w = x.shape
    _check_streams(x, w_out, None if nxt is None else nxt[0])
    if mix.shape != (s, s) or mix.dtype != torch.float32 or o.shape != (t, w) or (
            o2 is not None and (o2.shape != o.shape or o2.dtype != o.dtype)):
        raise ValueError("stream_step: shape / dtype mismatch")
    if not x.is_cuda:
        f = lambda a, g: a.float() if g is None else _ref_rms(a, g, eps, 0.0)
        y = f(o, w_o)
        if o2 is not None:
            y = y + f(o2, w_o2)
        x.copy_(torch.einsum("tsw,sd->tdw", x, mix) + w_out[None, :, None] * (coef * y)[:, None, :])
        return x, (None if nxt is None else _ref_read(x, nxt[0], nxt[1], eps, o.dtype))
    _ck(x, "x", torch.float32)
    _ck(mix, "mix", torch.float32)
    _ck(w_out, "w_out", torch.float32)
    _ck(o, "o")
    if o2 is not None:
        _ck(o2, "o2")
    for n, g in (("w_o", w_o), ("w_o2", w_o2)):
        if g is not None:
            _ck(g, n, o.dtype)
            if g.numel() != w:
                raise ValueError(f"stream_step: {n} width")
    h, w_in, gain = None, None, 0.0
    if nxt is not None:
        w_in, gain = nxt
        _ck(w_in, "w_in", torch.float32)
        h = torch.empty_like(o)
    _k().hc_step(x.data_ptr(), mix.data_ptr(), w_out.data_ptr(), o.data_ptr(), _ptr(w_o), _ptr(o2), _ptr(w_o2), float(coef),
                 _ptr(w_in), float(gain), _ptr(h), t, s, w, float(eps), _f32flag(o), _stream())
    return x, h
