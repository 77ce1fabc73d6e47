"""Linear attention with a decayed float32 matrix state per head.

Per head, with queries and keys q, k [dim], values v [vdim] and a decay a in (0, 1] per key channel:

    S <- diag(a) S + k v^T;   o = S^T q

so the read-out sees the current token's write.  ``S`` starts at zero and is carried from token to token in
a state slot (float32, whatever the activation type).  Two forms of the decay share the scan:

  * one fixed number per head (``decay`` [heads] float32) -- every key channel of the head, every token;
  * one number per key channel and token from a logit z: a = sigmoid(z + bias)^(1 / tau), evaluated in
    float32 as exp(log_sigmoid(z + bias) / tau).

A third form has exponential gates (:class:`MatrixMemorySpec`, :func:`memory_gates`): per head and token one decay
a, a weight b of the write and a factor c of the read-out, S <- a S + b k v^T, o = c S^T q, from log gates that are
kept in range by a running maximum, with a normaliser vector n beside the matrix.

q, k and v are columns of a fused projection; ``act`` "silu" applies x sigmoid(x) to each as it is read, and
``q_scale`` multiplies q.  The state pool is [slots, heads, vdim, dim]: a value column's key channels are
contiguous, which is how the scan kernel holds them in registers.

  :func:`decay_scan`        the recurrence over a varlen batch, state slots read and written
  :func:`memory_gates`      the gates a, b, c of the exponentially gated form, its maximum and normaliser state
  :func:`memory_scan`       gates and recurrence of the exponentially gated form (prompts in blocks on the matrix cores)
  :func:`memory_mixer`      the same with the output norm and gate (one launch for steps of one token per sequence)
  :func:`gated_norm`        o / rms(o) * w * act(gate) per group of channels (``ops.delta.gated_head_norm``
                            with the gate's activation as a parameter)

Same dispatch as the other ops: CUDA tensors go to the in-tree HIP kernels (csrc/kernels/linattn.hip,
memory.hip) and raise if those are not built; CPU tensors run the plain PyTorch forms.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Optional

import torch
import torch.nn.functional as F

from .seqmix import SeqBatch, _ck, _f32flag, _k, _ptr, _stream

MAX_KEY_DIM = 256        # the scan kernel keeps a state column in registers
MEMORY_STEP_MAX_VDIM = 8192    # the one-token step keeps a head's read-out in LDS
MEMORY_BLOCK_MIN = 16    # longest chunk of a step from which the matrix memory runs in blocks on the matrix cores


@dataclass
class LinAttnSpec:
    """Sizes of one linear-attention mixer."""
    heads: int
    dim: int             # query / key size per head
    vdim: int            # value size per head


@dataclass
class MatrixMemorySpec(LinAttnSpec):
    """Sizes and constants of an exponentially gated matrix memory."""
    cap: float = 15.0            # both gate logits z become cap tanh(z / cap)
    den_eps: float = 1e-6        # added to the read-out's divisor


def memory_gates(proj: torch.Tensor, qcol: int, kcol: int, icol: int, fcol: int, spec: MatrixMemorySpec,
                 i_bias: torch.Tensor, f_bias: torch.Tensor, n_state: torch.Tensor, m_state: torch.Tensor, sb: SeqBatch,
                 q_scale: float = 1.0) -> torch.Tensor:
    """Gates [T, heads, 4] float32 = (a, b, c, m) of every token: with i = cap tanh((zi + i_bias) / cap) and
    f = log_sigmoid(cap tanh((zf + f_bias) / cap)) (zi, zf [heads] at columns ``icol`` / ``fcol`` of ``proj``) the running
    maximum m_t = max(f + m_(t-1), i), which starts at 0; a = exp(f + m_(t-1) - m_t), b = exp(i - m_t); the normaliser
    n <- a n + b k; c = 1 / (max(|n . q|, exp(-m_t)) + den_eps).  ``n_state`` [slots, heads, dim] and ``m_state``
    [slots, heads] float32 carry n and m from chunk to chunk."""
    t = proj.shape[0]
    hh, d = spec.heads, spec.dim
    if n_state.shape[1:] != (hh, d) or m_state.shape[1:] != (hh,) or n_state.dtype != torch.float32 or \
            m_state.dtype != torch.float32 or proj.shape[1] < max(qcol + hh * d, kcol + hh * d, icol + hh, fcol + hh):
        raise ValueError("memory_gates: shape / dtype mismatch")
    if i_bias.numel() != hh or f_bias.numel() != hh or i_bias.dtype != torch.float32 or f_bias.dtype != torch.float32:
        raise ValueError("memory_gates: gate biases [heads] float32")
    if not proj.is_cuda:
        q = proj[:, qcol:qcol + hh * d].float().view(t, hh, d) * q_scale
        k = proj[:, kcol:kcol + hh * d].float().view(t, hh, d)
        ig = spec.cap * torch.tanh((proj[:, icol:icol + hh].float() + i_bias) / spec.cap)
        fg = F.logsigmoid(spec.cap * torch.tanh((proj[:, fcol:fcol + hh].float() + f_bias) / spec.cap))
        g = torch.empty(t, hh, 4, dtype=torch.float32)
        cu, pos, slots = sb.cu.tolist(), sb.positions.tolist(), sb.state_slots.tolist()
        for b in range(sb.num_seqs):
            lo, hi = cu[b], cu[b + 1]
            if hi == lo:
                continue
            n = n_state[slots[b]].clone() if pos[lo] > 0 else torch.zeros(hh, d)
            m = m_state[slots[b]].clone() if pos[lo] > 0 else torch.zeros(hh)
            for j in range(lo, hi):
                mn = torch.maximum(fg[j] + m, ig[j])
                a, w = torch.exp(fg[j] + m - mn), torch.exp(ig[j] - mn)
                m = mn
                n = a[:, None] * n + w[:, None] * k[j]
                den = torch.maximum((n * q[j]).sum(-1).abs(), torch.exp(-m)) + spec.den_eps
                g[j] = torch.stack([a, w, 1.0 / den, m], -1)
            n_state[slots[b]], m_state[slots[b]] = n, m
        return g
    if d > MAX_KEY_DIM:
        raise ValueError(f"memory_gates: key size {d} > {MAX_KEY_DIM}")
    _ck(proj, "proj")
    for nm, x in (("i_bias", i_bias), ("f_bias", f_bias), ("n_state", n_state), ("m_state", m_state)):
        _ck(x, nm, torch.float32)
    g = torch.empty(t, hh, 4, dtype=torch.float32, device=proj.device)
    _k().ml_gates(g.data_ptr(), proj.data_ptr(), proj.shape[1], int(qcol), int(kcol), int(icol), int(fcol), i_bias.data_ptr(),
                  f_bias.data_ptr(), float(spec.cap), float(q_scale), float(spec.den_eps), n_state.data_ptr(),
                  m_state.data_ptr(), sb.cu.data_ptr(), sb.positions.data_ptr(), sb.state_slots.data_ptr(), sb.num_seqs,
                  sb.max_q_len, hh, d, _f32flag(proj), _stream())
    return g


def decay_scan(proj: torch.Tensor, qcol: int, kcol: int, vcol: int, spec: LinAttnSpec, state: torch.Tensor,
               sb: SeqBatch, act: Optional[str] = None, q_scale: float = 1.0, decay: Optional[torch.Tensor] = None,
               z: Optional[torch.Tensor] = None, z_bias: Optional[torch.Tensor] = None, tau: float = 1.0,
               gates: Optional[torch.Tensor] = None) -> torch.Tensor:
    """The recurrence.  ``proj`` [T, *] holds q [heads, dim] from column ``qcol``, k from ``kcol``, v
    [heads, vdim] from ``vcol``.  Decay: ``decay`` [heads] float32, or ``z`` [T, heads dim] (activation
    type) with ``z_bias`` [heads dim] float32 and ``tau``, or ``gates`` [T, heads, 4] of :func:`memory_gates` (decay, weight of
    the write, factor of the read-out).  ``state`` [slots, heads, vdim, dim] float32: a chunk
    that starts at position 0 starts from zero, any other from its slot; the slot holds the state after the
    chunk's last token.  Returns o [T, heads, vdim] float32."""
    t = proj.shape[0]
    hh, d, dv = spec.heads, spec.dim, spec.vdim
    if act not in (None, "silu"):
        raise ValueError(f"decay_scan: activation {act!r} (None, 'silu')")
    if sum(x is not None for x in (decay, z, gates)) != 1:
        raise ValueError("decay_scan: a decay per head, a logit per key channel or gates, one of them")
    if gates is not None and (gates.shape != (t, hh, 4) or gates.dtype != torch.float32):
        raise ValueError("decay_scan: gates [T, heads, 4] float32")
    if state.shape[1:] != (hh, dv, d) or state.dtype != torch.float32 or proj.shape[1] < max(
            qcol + hh * d, kcol + hh * d, vcol + hh * dv):
        raise ValueError("decay_scan: shape / dtype mismatch")
    if decay is not None and (decay.numel() != hh or decay.dtype != torch.float32):
        raise ValueError("decay_scan: decay [heads] float32")
    if z is not None and (z.shape != (t, hh * d) or z_bias is None or z_bias.numel() != hh * d
                          or z_bias.dtype != torch.float32 or z.dtype != proj.dtype):
        raise ValueError("decay_scan: z [T, heads dim] with a float32 bias [heads dim]")
    if not proj.is_cuda:
        f = (lambda x: x * torch.sigmoid(x)) if act == "silu" else (lambda x: x)
        q = f(proj[:, qcol:qcol + hh * d].float()).view(t, hh, d) * q_scale
        k = f(proj[:, kcol:kcol + hh * d].float()).view(t, hh, d)
        v = f(proj[:, vcol:vcol + hh * dv].float()).view(t, hh, dv)
        if decay is not None:
            a = decay.float().view(1, hh, 1).expand(t, hh, d)
        elif gates is not None:
            a = gates[:, :, :1].expand(t, hh, d)
            k = k * gates[:, :, 1:2]
        else:
            a = torch.exp(F.logsigmoid(z.float() + z_bias.float()) / tau).view(t, hh, d)
        o = torch.empty(t, hh, dv, dtype=torch.float32)
        cu, pos, slots = sb.cu.tolist(), sb.positions.tolist(), sb.state_slots.tolist()
        for b in range(sb.num_seqs):
            lo, hi = cu[b], cu[b + 1]
            if hi == lo:
                continue
            s = state[slots[b]].clone() if pos[lo] > 0 else torch.zeros(hh, dv, d)
            for i in range(lo, hi):
                s = s * a[i][:, None, :] + v[i][:, :, None] * k[i][:, None, :]
                o[i] = torch.einsum("hvd,hd->hv", s, q[i])
            state[slots[b]] = s
        return o if gates is None else o * gates[:, :, 2:3]
    if d > MAX_KEY_DIM:
        raise ValueError(f"decay_scan: key size {d} > {MAX_KEY_DIM}")
    _ck(proj, "proj")
    _ck(state, "state", torch.float32)
    if decay is not None:
        _ck(decay, "decay", torch.float32)
    elif gates is not None:
        _ck(gates, "gates", torch.float32)
    else:
        _ck(z, "z", proj.dtype)
        _ck(z_bias, "z_bias", torch.float32)
    o = torch.empty(t, hh, dv, dtype=torch.float32, device=proj.device)
    _k().la_scan(o.data_ptr(), proj.data_ptr(), proj.shape[1], int(qcol), int(kcol), int(vcol), _ptr(decay), _ptr(z),
                 _ptr(z_bias), 1.0 / float(tau), float(q_scale), 1 if act == "silu" else 0, _ptr(gates), state.data_ptr(),
                 sb.cu.data_ptr(), sb.positions.data_ptr(), sb.state_slots.data_ptr(), sb.num_seqs, sb.max_q_len, hh, d,
                 dv, _f32flag(proj), _stream())
    return o


def memory_scan(proj: torch.Tensor, qcol: int, kcol: int, vcol: int, icol: int, fcol: int, spec: MatrixMemorySpec,
                i_bias: torch.Tensor, f_bias: torch.Tensor, state: torch.Tensor, n_state: torch.Tensor,
                m_state: torch.Tensor, sb: SeqBatch, q_scale: float = 1.0) -> torch.Tensor:
    """The exponentially gated matrix memory over a varlen batch: :func:`memory_gates` then :func:`decay_scan` (decode
    steps, float32, sizes that are no multiple of 8), or -- bfloat16 prompts -- blocks of 64 tokens on the matrix cores
    (csrc/kernels/memory.hip).  Returns o [T, heads, vdim] float32."""
    hh, d, dv = spec.heads, spec.dim, spec.vdim
    blocks = proj.is_cuda and proj.dtype == torch.bfloat16 and sb.max_q_len >= MEMORY_BLOCK_MIN and d <= MAX_KEY_DIM and \
        all(x % 8 == 0 for x in (d, dv, qcol, kcol, vcol, proj.shape[1]))
    if not blocks:
        g = memory_gates(proj, qcol, kcol, icol, fcol, spec, i_bias, f_bias, n_state, m_state, sb, q_scale)
        return decay_scan(proj, qcol, kcol, vcol, spec, state, sb, q_scale=q_scale, gates=g)
    if state.shape[1:] != (hh, dv, d) or n_state.shape[1:] != (hh, d) or m_state.shape[1:] != (hh,) or proj.shape[1] < max(
            qcol + hh * d, kcol + hh * d, vcol + hh * dv, icol + hh, fcol + hh) or i_bias.numel() != hh or f_bias.numel() != hh:
        raise ValueError("memory_scan: shape mismatch")
    _ck(proj, "proj")
    for nm, x in (("i_bias", i_bias), ("f_bias", f_bias), ("state", state), ("n_state", n_state), ("m_state", m_state)):
        _ck(x, nm, torch.float32)
    o = torch.empty(proj.shape[0], hh, dv, dtype=torch.float32, device=proj.device)
    ws = None
    if _k().ml_chunk_cols(sb.num_seqs, hh, d, dv) < dv:          # a head's columns on several workgroups
        ws = torch.empty(sb.num_seqs * hh * (d + 1), dtype=torch.float32, device=proj.device)
    _k().ml_chunk(o.data_ptr(), proj.data_ptr(), proj.shape[1], int(qcol), int(kcol), int(vcol), int(icol), int(fcol),
                  i_bias.data_ptr(), f_bias.data_ptr(), float(spec.cap), float(q_scale), float(spec.den_eps), state.data_ptr(),
                  n_state.data_ptr(), m_state.data_ptr(), _ptr(ws), sb.cu.data_ptr(), sb.positions.data_ptr(),
                  sb.state_slots.data_ptr(), sb.num_seqs, hh, d, dv, _stream())
    return o


def memory_mixer(proj: torch.Tensor, qcol: int, kcol: int, vcol: int, gcol: int, icol: int, fcol: int,
                 spec: MatrixMemorySpec, i_bias: torch.Tensor, f_bias: torch.Tensor, norm: torch.Tensor, state: torch.Tensor,
                 n_state: torch.Tensor, m_state: torch.Tensor, sb: SeqBatch, eps: float, q_scale: float = 1.0) -> torch.Tensor:
    """The mixer between its input and output projections: :func:`memory_scan`, every head's o over its root mean
    square, times ``norm`` [heads vdim], times sigmoid of the ``proj`` columns at ``gcol`` -- steps of one token per
    sequence in one launch.  Returns [T, heads vdim] in ``proj``'s dtype."""
    hh, d, dv = spec.heads, spec.dim, spec.vdim
    if not (proj.is_cuda and sb.max_q_len == 1 and d % 4 == 0 and d <= MAX_KEY_DIM and dv <= MEMORY_STEP_MAX_VDIM):
        o = memory_scan(proj, qcol, kcol, vcol, icol, fcol, spec, i_bias, f_bias, state, n_state, m_state, sb, q_scale)
        return gated_norm(o, proj, gcol, norm, eps, groups=hh, gate_act="sigmoid")
    if state.shape[1:] != (hh, dv, d) or n_state.shape[1:] != (hh, d) or m_state.shape[1:] != (hh,) or proj.shape[1] < max(
            qcol + hh * d, kcol + hh * d, vcol + hh * dv, gcol + hh * dv, icol + hh, fcol + hh) or i_bias.numel() != hh or \
            f_bias.numel() != hh or norm.numel() != hh * dv:
        raise ValueError("memory_mixer: shape mismatch")
    _ck(proj, "proj")
    _ck(norm, "norm", proj.dtype)
    for nm, x in (("i_bias", i_bias), ("f_bias", f_bias), ("state", state), ("n_state", n_state), ("m_state", m_state)):
        _ck(x, nm, torch.float32)
    y = torch.empty(proj.shape[0], hh * dv, dtype=proj.dtype, device=proj.device)
    _k().ml_step(y.data_ptr(), proj.data_ptr(), proj.shape[1], int(qcol), int(kcol), int(vcol), int(gcol), int(icol), int(fcol),
                 i_bias.data_ptr(), f_bias.data_ptr(), float(spec.cap), float(q_scale), float(spec.den_eps), state.data_ptr(),
                 n_state.data_ptr(), m_state.data_ptr(), norm.data_ptr(), float(eps), sb.cu.data_ptr(), sb.positions.data_ptr(),
                 sb.state_slots.data_ptr(), sb.num_seqs, sb.max_q_len, hh, d, dv, _f32flag(proj), _stream())
    return y


def gated_norm(o: torch.Tensor, gate: torch.Tensor, gcol: int, w: torch.Tensor, eps: float, groups: int,
               gate_act: str = "silu") -> torch.Tensor:
    """o [T, C] float32 in ``groups`` equal groups of channels -> o / sqrt(mean_group(o^2) + eps) * w *
    act(gate[:, gcol + c]) as [T, C] in ``gate``'s dtype.  ``w`` has one group's channels (shared by the groups) or all
    C (with several groups: a weight per group).
    ``gate_act``: "silu" (g sigmoid(g)) or "sigmoid"."""
    from .delta import gated_head_norm
    t, c = o.shape[0], o[0].numel()
    if c % groups or w.numel() not in (c, c // groups):
        raise ValueError("gated_norm: groups do not fit")
    return gated_head_norm(o.view(t, groups, c // groups), gate, gcol,
                           w.view(groups, c // groups) if groups > 1 and w.numel() == c else w, eps, gate_act=gate_act)
