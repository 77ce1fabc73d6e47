"""The Kupedra decoder (several residual streams, attention normed after its rotation, distance-biased attention
beside an exponentially gated matrix memory, clipped-GLU experts weighted over all logits, a looped span of layers)
against the plain float64 oracle of tests/oracle_kupedra.py: every mechanism alone, then the engine -- whole
prompts, token-by-token decoding, prompt portions down to two tokens, batches of unequal requests, blocks and state
slots that are freed and used again, keys just inside and just outside the distance buckets, keys and memory
writes far back, the first tokens, long decoding, and greedy generation through the scheduler.  Each case runs on
the CPU path in float32 and, marked gpu, on the HIP kernels in float32 and bfloat16.
"""
import json
import math

import numpy as np
import pytest
import torch

import oracle_kupedra as O
from distributed_llms_amd.config import ModelConfig
from distributed_llms_amd.engine.sequence import SamplingParams
from distributed_llms_amd.models import make_stage
from distributed_llms_amd.ops import hyper as hc
from distributed_llms_amd.ops import linattn as la
from distributed_llms_amd.ops import moe
from distributed_llms_amd.ops import seqmix as sm
from test_fekizen import (TARGETS, _atol, _dev, _np, _paged, _round, _sb, make_engine, prompts_for, replay, row_errs)


def _attn(heads, kv_heads, dim, vdim, scale, dims, mlp, base=10000.0, factor=None):
    rot = {"base": base, "dims": dims}
    if factor:
        rot["scaling"] = {"factor": factor}
    return {"type": "attention", "mlp": mlp, "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
                                                       "scale": scale, "rot": rot}}


def _left(heads, kv_heads, dim, vdim, scale, far, rows, coef=None, every=0):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "bias_max": far, "rows": rows}
    if coef is not None:
        m["q_temp"] = {"coef": coef, "every": every}
    return m


def _right(heads, dim, vdim, cap):
    return {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}


def _par(left, right, mlp):
    return {"type": "parallel", "mixer": {"left": left, "right": right}, "mlp": mlp}


def _moe(experts, top, ff, limit, shared=0, shared_limit=1.0):
    return {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": {"experts": experts, "top": top},
            "shared": {"ff": shared, "limit": shared_limit} if shared else None}


def cfg_a():
    """Layers that differ from one another: key and value sizes apart, a rotated part shorter than the head, scaled
    and unscaled frequencies, several bias tables, a loop that starts after the first layer, a layer without a
    feed-forward and one without a shared expert."""
    return {"architecture": "Kupedra", "vocab": 200, "width": 96, "norm": {"eps": 1e-6}, "embedding": {"scale": 3.0},
            "streams": 4, "logit_scale": 0.7, "loop": {"start": 1, "stop": 3, "times": 2},
            "layers": [
                _par(_left(6, 2, 24, 16, 0.25, 60, 12, 0.4, 16), _right(3, 16, 24, 8.0), _moe(6, 2, 48, 1.5, 64, 2.5)),
                _attn(4, 2, 24, 40, 0.3, 16, _moe(5, 3, 40, 2.0), factor=4.0),
                _par(_left(3, 1, 16, 24, 0.2, 200, 32, 0.2, 50), _right(2, 24, 40, 12.0), None),
                _attn(3, 3, 16, 16, 0.5, 16, _moe(4, 1, 32, 3.0, 32, 0.5), base=500.0),
            ]}


def cfg_b():
    """Degenerate sizes: one stream, one head, one expert, every expert per token, a two-row bias table, a
    temperature period of one, odd widths, a loop over every layer that runs once."""
    return {"architecture": "Kupedra", "vocab": 131, "width": 72, "norm": {"eps": 1e-5}, "embedding": {"scale": 1.0},
            "streams": 1, "logit_scale": 1.0, "loop": {"start": 0, "stop": 3, "times": 1},
            "layers": [
                _par(_left(1, 1, 12, 12, 0.3, 3, 2, 0.5, 1), _right(1, 8, 8, 1.0), _moe(3, 3, 24, 0.7)),
                _attn(1, 1, 10, 14, 0.4, 2, _moe(1, 1, 16, 9.0, 8, 1.0)),
                _par(_left(5, 5, 8, 6, 0.35, 9, 6), _right(2, 70, 6, 30.0), None),
            ]}


def cfg_c():
    """Sizes that the matrix-core attention kernels and the grouped expert kernels take; no loop."""
    return {"architecture": "Kupedra", "vocab": 160, "width": 128, "norm": {"eps": 1e-6}, "embedding": {"scale": 1.7},
            "streams": 2, "logit_scale": 1.5,
            "layers": [
                _par(_left(4, 2, 64, 64, 0.12, 128, 16, 0.1, 32), _right(2, 32, 128, 10.0), _moe(8, 2, 128, 2.0, 128, 3.0)),
                _attn(4, 1, 32, 64, 0.3, 32, _moe(8, 2, 128, 1.0, 128, 1.0), factor=2.0),
                _par(_left(4, 1, 32, 32, 0.2, 50, 8), _right(1, 128, 64, 15.0), None),
            ]}


CONFIGS = {"a": cfg_a, "b": cfg_b, "c": cfg_c}


def oracle(cfg, sd, tokens, taps=None):
    """(logits, decided): ``decided`` [T] marks the tokens none of whose expert choices was a close call in any layer."""
    margins = []
    want = O.forward(cfg, _np(sd), np.array(tokens), taps, margins)
    ok = np.ones(len(tokens), dtype=bool)
    for m in margins:
        ok &= m > 0.2
    return want, ok


def assert_close(got, want, target, what=""):
    """float32: every position within 2e-4, 2e-5 at the median (a wrong key, weight or state shows at 1e-2 and
    more).  bfloat16, at the tokens whose expert choices are no close calls (rounded activations may turn those the
    other way, which is no fault, and which later tokens see through the mixers): 6e-2 at the median, 0.2 at all
    but one token in eight.  The bfloat16 kernels are held to rounding one by one above."""
    want, decided = want
    e = row_errs(got, want)
    if target[1] == torch.float32:
        assert np.median(e) < 2e-5 and e.max() < 2e-4, (what, float(np.median(e)), float(e.max()), int(e.argmax()))
    elif decided.any():
        d = e[decided]
        over = int((d > 0.2).sum())
        assert np.median(d) < 6e-2 and over <= max(1, len(d) // 8), (what, len(d), float(np.median(d)), over, float(d.max()))


def _t(rng, dtype, *shape, scale=1.0, off=0.0):
    return torch.from_numpy((off + scale * rng.standard_normal(shape)).astype(np.float32)).to(dtype)


def _d(x):
    return x.detach().cpu().double().numpy()


# ------------------------------------------------------------------------------ mechanisms alone
@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("streams,width", [(1, 96), (2, 72), (3, 33), (4, 512), (5, 40), (9, 260), (16, 1100)])
def test_streams_are_mixed_from_the_old_ones(target, streams, width):
    """Embedding into every stream; the write of one output, and of two normed apart, while ALL streams are mixed
    from the old ones (indexed from, to); the next read in the same call and alone; a read with ones."""
    device, dtype = _dev(target)
    rng = np.random.default_rng(streams)
    t, eps = 5, 1e-5
    table = _t(rng, dtype, 30, width)
    ids = torch.tensor([3, 29, 0, 7, 7], dtype=torch.int32, device=device)
    x = hc.embed_streams(ids, table.to(device), streams, 2.5)
    assert x.shape == (t, streams, width) and x.dtype == torch.float32
    for s in range(streams):
        np.testing.assert_allclose(_d(x[:, s]), _d(table)[[3, 29, 0, 7, 7]] * 2.5, rtol=1e-6)
    x0 = torch.from_numpy(rng.standard_normal((t, streams, width)).astype(np.float32))
    f = lambda *s: torch.from_numpy(rng.standard_normal(s).astype(np.float32))
    mix, w_out, w_in = f(streams, streams), f(streams), f(streams)
    o1, o2 = _t(rng, dtype, t, width, scale=5.0), _t(rng, dtype, t, width, scale=0.02)
    w1, w2 = _t(rng, dtype, width, scale=0.3, off=1.0), _t(rng, dtype, width, scale=0.3, off=1.0)
    dv = lambda a: a.to(device)

    def want(y):
        hcw = {"in": np.zeros(streams), "out": _d(w_out), "mix": _d(mix)}
        new = O.hyper_connected(_d(x0).transpose(1, 0, 2), hcw, lambda u: y)
        return new.transpose(1, 0, 2), O.rms(np.einsum("s,tsw->tw", _d(w_in), new.transpose(1, 0, 2)), eps) * 1.3
    for kw, y in (({}, _d(o1)),
                  ({"w_o": dv(w1), "o2": dv(o2), "w_o2": dv(w2), "coef": 0.5},
                   0.5 * (O.rms(_d(o1), eps) * _d(w1) + O.rms(_d(o2), eps) * _d(w2)))):
        wx, wh = want(y)
        xg, h = hc.stream_step(dv(x0.clone()), dv(mix), dv(w_out), dv(o1), eps, nxt=(dv(w_in), 1.3), **kw)
        np.testing.assert_allclose(_d(xg), wx, atol=3e-5 * max(1.0, np.abs(wx).max()))
        assert h.dtype == dtype
        np.testing.assert_allclose(_d(h), wh, atol=_atol(dtype, 1e-4, 4e-2))
        xg, h = hc.stream_step(dv(x0.clone()), dv(mix), dv(w_out), dv(o1), eps, **kw)
        assert h is None
        np.testing.assert_allclose(_d(xg), wx, atol=3e-5 * max(1.0, np.abs(wx).max()))
    if streams > 1:      # the other index order, and streams mixed one after the other, are far away
        assert np.abs(np.einsum("ts,btw->bsw", _d(mix).T, _d(x0)) - np.einsum("ts,btw->bsw", _d(mix), _d(x0))).max() > 0.1
    h = hc.stream_read(dv(x0.clone()), dv(torch.ones(streams)), 0.8, eps, dtype)
    np.testing.assert_allclose(_d(h), O.rms(_d(x0).sum(1), eps) * 0.8, atol=_atol(dtype, 1e-4, 3e-2))


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("shape", [(4, 2, 24, 16, 16), (3, 1, 16, 24, 8), (2, 2, 64, 64, 64), (5, 5, 10, 4, 4), (2, 1, 12, 9, 0),
                                   (20, 4, 128, 128, 128), (3, 1, 136, 8, 136), (6, 2, 40, 40, 30)])
@pytest.mark.parametrize("norm_last", [False, True])
def test_head_norm_rotation_and_query_factors(target, shape, norm_last):
    """The attention input stage: an RMS norm per head before (weighted) or after (unweighted) the rotation of
    adjacent pairs by divided frequencies, a factor per head and one that steps up with the position (positions just
    before and just after a step), values appended unchanged; a small eps against tiny heads, so that norming
    before or after and the eps inside the root both show."""
    device, dtype = _dev(target)
    h, g, d, dv, dims = shape
    rng = np.random.default_rng(d + dims)
    pos = [0, 1, 6, 7, 8, 14, 15, 1000, 20000]
    t, pad, eps, bs = len(pos), 8, 1e-2, 16
    x = _t(rng, dtype, t, pad + h * d + g * (d + dv) + 8, scale=0.3)
    slots = [5 * bs + 3, 2 * bs, 2 * bs + 1, 7 * bs + 15, bs, 3 * bs + 8, 4 * bs + 15, 6 * bs, 8 * bs + 2]
    kc = torch.zeros(9, g, bs, d, dtype=dtype, device=device)
    vc = torch.zeros(9, g, dv, bs, dtype=dtype, device=device)
    rot = {"base": 3000.0, "dims": dims, "scaling": {"factor": 3.0}}
    freqs = sm.rotary_frequencies(dims, 3000.0, 3.0).to(device) if dims else None
    qw, kw = (None, None) if norm_last else (_t(rng, dtype, d, scale=0.3, off=1.0), _t(rng, dtype, d, scale=0.3, off=1.0))
    mul = torch.from_numpy(rng.uniform(0.5, 2.0, h).astype(np.float32))
    qt = {"coef": 0.4, "every": 8}
    dvc = lambda a: None if a is None else a.to(device)
    q = sm.head_norm_rope(x.to(device), pad, dvc(qw), dvc(kw), freqs, eps, kc, vc,
                          torch.tensor(slots, dtype=torch.int32, device=device),
                          torch.tensor(pos, dtype=torch.int32, device=device), h, g, d, dv, norm_last=norm_last,
                          q_mul=mul.to(device), q_temp=(0.4, 8))
    xd = _d(x)

    def prep(a, w, p):
        turn = (lambda z: O.rotate_pairs(z, rot, first_pos=p)) if dims else (lambda z: z)
        return O.rms(turn(a), eps) if norm_last else turn(O.rms(a, eps) * _d(w))
    for i, p in enumerate(pos):
        f = O.query_temperature(np.array([p]), qt)[0]
        wq = prep(xd[i, pad:pad + h * d].reshape(1, h, d), qw, p)[0] * f * _d(mul)[:, None]
        wk = prep(xd[i, pad + h * d:pad + (h + g) * d].reshape(1, g, d), kw, p)[0]
        tol = (2e-3 if p > 100 else 2e-5) if dtype == torch.float32 else 2e-2      # float32 angles far out
        s = slots[i]
        np.testing.assert_allclose(_d(q[i]), wq, atol=tol * np.abs(wq).max())
        np.testing.assert_allclose(_d(kc[s // bs, :, s % bs]), wk, atol=tol * np.abs(wk).max())
        v0 = pad + (h + g) * d
        np.testing.assert_array_equal(_d(vc[s // bs, :, :, s % bs]), xd[i, v0:v0 + g * dv].reshape(g, dv))
    # the factor steps at (p + 1) / every
    f = O.query_temperature(np.array(pos), qt)
    assert f[2] == 1.0 and f[3] > 1.2 and f[3] == f[4] == f[5] and f[6] > f[5]


def test_bucket_borders_are_exact():
    """Every distance's row against the closed form, on tables whose borders fall between integers; and ON integers
    (far / half a power of two), where the row must change exactly there."""
    for rows, far in ((12, 60), (32, 200), (8, 50), (6, 9), (2, 3), (16, 97), (32, 128), (10, 2000), (7, 30)):
        th = sm.bucket_thresholds(rows, far)
        assert len(th) == rows and th == sorted(th)
        for n in range(2 * far):
            row = max(r for r in range(rows) if th[r] <= n)
            x = n and n >= rows // 2 and math.log(n / (rows // 2)) / math.log(far / (rows // 2)) * (rows - rows // 2)
            if x and abs(x - round(x)) < 1e-9:
                continue                                  # on a border: below
            assert row == O.bucket(n, rows, far), (rows, far, n)
    th = sm.bucket_thresholds(16, 128)                    # 8 * 2^(k / 2): rows 10, 12, 14 start at 16, 32, 64
    assert th[10] == 16 and th[12] == 32 and th[14] == 64 and th[8] == 8
    rel = torch.arange(16.0)[:, None].repeat(1, 2)
    b = sm.distance_bias_table(rel, 128)
    assert b.shape == (2, th[-1] + 1) and b[0, 15] == 9 and b[0, 16] == 10 and b[1, -1] == 15
    with pytest.raises(ValueError):
        sm.bucket_thresholds(16, 8)


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("shape", [(4, 2, 24, 16, 16, 12, 60), (6, 3, 64, 40, 32, 16, 128), (3, 1, 12, 9, 16, 2, 3),
                                   (20, 1, 128, 128, 32, 32, 5000), (2, 2, 40, 136, 32, 8, 1000), (4, 4, 256, 64, 32, 6, 20)])
def test_distance_bias_and_sink(target, shape):
    """Attention with a bias per bucket of distances and a sink.  (a) Random inputs: whole sequence, a late portion,
    decoded tokens.  (b) One bucket's bias stands out: a query attends to exactly the keys of that bucket -- the
    nearest and farthest of them show, their neighbours outside do not -- in a prompt and decoded, for the first
    bucket, those at the borders and the open-ended last.  (c) The bias is not scaled and the sink gets none: a
    zero sink adds one to the denominator, a huge one takes the weight away."""
    device, dtype = _dev(target)
    h, g, d, dv, bs, rows, far = shape
    rng = np.random.default_rng(h * d + far)
    n, scale, nb = 170, 0.15, 30
    q, k, v = (rng.standard_normal((n, a, b)).astype(np.float32) for a, b in ((h, d), (g, d), (g, dv)))
    sink = rng.standard_normal(h).astype(np.float32)
    rel = rng.standard_normal((rows, h)).astype(np.float32)
    table = list(rng.permutation(np.arange(1, nb))[:-(-n // bs)])
    T = lambda a: torch.from_numpy(a).to(dtype)
    bt = torch.tensor([table], dtype=torch.int32, device=device)
    tol = _atol(dtype)
    kk, vv, qq = T(k), T(v), T(q)
    caches = _paged(kk, vv, table, nb, bs, dtype, device)

    def run(qx, rl, sk, lo, p, decode):
        b = sm.distance_bias_table(torch.from_numpy(rl).to(device), far)
        return sm.window_attention(qx[lo:p + 1].contiguous().to(device), *caches, bt, _sb([(lo, p + 1 - lo)], device), 1 << 30,
                                   scale, num_decode=None if decode else 0, sinks=torch.from_numpy(sk).to(device), bias=b,
                                   max_ctx=p + 1).float().cpu().numpy()

    def want(qx, rl, sk):
        bias = np.stack([rl[O.bucket(m, rows, far)] for m in range(n)]).astype(np.float64)
        return O.softmax_attention(_d(qx), _d(kk), _d(vv), scale, sk.astype(np.float64), bias)
    w = want(qq, rel, sink)
    np.testing.assert_allclose(run(qq, rel, sink, 0, n - 1, False), w, rtol=tol, atol=tol)
    np.testing.assert_allclose(run(qq, rel, sink, 101, n - 1, False), w[101:], rtol=tol, atol=tol)
    for p in (0, 1, rows // 2 - 1, rows // 2, min(n - 1, far), n - 1):
        np.testing.assert_allclose(run(qq, rel, sink, p, p, True), w[p:p + 1], rtol=tol, atol=tol)
    # (b) a query of zeros: the scores are the biases alone
    q0 = torch.zeros_like(qq)
    buckets = [O.bucket(m, rows, far) for m in range(n)]
    for row in sorted({0, rows // 2 - 1, rows // 2, buckets[n - 1] - 1, buckets[n - 1]}):
        if row < 0:
            continue
        r2 = np.full((rows, h), -30.0, dtype=np.float32)
        r2[row] = 20.0
        p = n - 1
        hit = [p - m for m in range(n) if buckets[m] == row]
        mean = _d(vv)[hit].mean(0).repeat(h // g, 0)
        for lo, decode in ((p - 3, False), (p, True)):
            got = run(q0, r2, np.full(h, -30.0, dtype=np.float32), lo, p, decode)[-1]
            np.testing.assert_allclose(got, mean, rtol=tol, atol=tol)
        for off in (min(hit) - 1, max(hit) + 1):                # one key more than the bucket's would show
            if 0 <= off <= p:
                more = _d(vv)[hit + [off]].mean(0).repeat(h // g, 0)
                assert np.abs(more - mean).max() > (1e-2 if len(hit) < 60 else 3e-3)
    # (c)
    none = np.zeros((rows, h), dtype=np.float32)
    got = run(q0, none, np.zeros(h, dtype=np.float32), 0, 9, False)
    for i in range(10):
        np.testing.assert_allclose(got[i], _d(vv)[:i + 1].sum(0).repeat(h // g, 0) / (i + 2), rtol=tol, atol=tol)
    got = run(q0, none + 7.0, np.full(h, 7.0 + math.log(3.0), dtype=np.float32), 3, 3, True)[0]
    np.testing.assert_allclose(got, _d(vv)[:4].sum(0).repeat(h // g, 0) / 7.0, rtol=tol, atol=tol)
    assert np.abs(run(qq, rel, np.full(h, 60.0, dtype=np.float32), n - 1, n - 1, True)).max() < 1e-6


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("decode", [False, True])
def test_far_key_behind_a_long_context(target, decode):
    """One key 1500 positions back matches the query, beyond the last bias border: it owns the row (several cache
    blocks, key runs on separate workgroups when decoded); with the last bucket's bias far down it does not."""
    device, dtype = _dev(target)
    h, g, d, bs, n = 4, 1, 32, 32, 1600
    rng = np.random.default_rng(1)
    q, k, v = (torch.from_numpy(rng.standard_normal(s).astype(np.float32) * f).to(dtype)
               for s, f in (((n, h, d), 0.1), ((n, g, d), 0.1), ((n, g, d), 1.0)))
    k[99], q[n - 1] = 0.0, 0.0
    k[99, :, 3], q[n - 1, :, 3] = 12.0, 12.0
    table = list(rng.permutation(np.arange(1, 60))[:n // bs])
    caches = _paged(k, v, table, 60, bs, dtype, device)
    bt = torch.tensor([table], dtype=torch.int32, device=device)
    for last, owned in ((1.0, True), (-80.0, False)):
        rel = torch.zeros(8, h)
        rel[7] = last
        b = sm.distance_bias_table(rel, 64).to(device)
        lo = n - 1 if decode else n - 40
        o = sm.window_attention(q[lo:].contiguous().to(device), *caches, bt, _sb([(lo, n - lo)], device), 1 << 30, 0.3,
                                num_decode=None if decode else 0, sinks=torch.zeros(h, device=device), bias=b, max_ctx=n)
        dist = (o[-1].float().cpu() - v[99].float()).abs().max().item()
        assert (dist < 2e-2) == owned, (last, dist)


def _gate_case(rng, n, hh, case):
    zi, zf = rng.standard_normal((n, hh)), 3.0 + rng.standard_normal((n, hh))
    if case == "loud":                    # large input gates now and then, some tokens that forget everything
        zi[::7] += 9.0
        zf[::11] -= 12.0
    if case == "quiet":                   # input gates far below zero: the maximum stays where it started
        zi -= 8.0
    return zi, zf


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("sizes", [(3, 16, 24), (2, 48, 32), (1, 128, 128), (1, 8, 8), (2, 200, 20), (4, 20, 72), (2, 64, 130),
                                   (1, 256, 72)])
@pytest.mark.parametrize("case", ["mild", "loud", "quiet"])
def test_matrix_memory_through_state_slots(target, sizes, case):
    """Exponential gates with a running maximum that starts at zero, the normaliser and its floor: the whole
    sequence (over several 64-token blocks), then portions of one to many tokens -- short ones go token by token, long
    ones in blocks where sizes allow -- and a batch of two sequences through state slots, one of them in a slot an
    earlier owner left full."""
    device, dtype = _dev(target)
    hh, d, dv = sizes
    rng = np.random.default_rng(hh * d + dv)
    n, pad, cap = 151, 8, 11.0
    qk, vv = hh * d, hh * dv
    x = _t(rng, dtype, n, -(-(pad + 2 * qk + vv + 2 * hh) // 8) * 8, scale=0.8)
    ci = pad + 2 * qk + vv
    zi, zf = _gate_case(rng, n, hh, case)
    ib, fb = rng.standard_normal(hh), rng.standard_normal(hh)
    x[:, ci:ci + hh] = torch.from_numpy(zi - ib).to(dtype)
    x[:, ci + hh:ci + 2 * hh] = torch.from_numpy(zf - fb).to(dtype)
    sp = la.MatrixMemorySpec(hh, d, dv, cap=cap)
    xd = _d(x)
    ib32, fb32 = (torch.from_numpy(a.astype(np.float32)).to(device) for a in (ib, fb))
    ig = O.capped(xd[:, ci:ci + hh] + ib.astype(np.float32), cap)
    fg = O.log_sigmoid(O.capped(xd[:, ci + hh:ci + 2 * hh] + fb.astype(np.float32), cap))
    q = xd[:, pad + qk:pad + 2 * qk].reshape(n, hh, d) * d ** -0.5         # q after k: the columns are arguments
    k, v = xd[:, pad:pad + qk].reshape(n, hh, d), xd[:, pad + 2 * qk:ci].reshape(n, hh, dv)
    scan_want = lambda s: np.stack([O.memory_scan(q[s, a], k[s, a], v[s, a], ig[s, a], fg[s, a]) for a in range(hh)], 1)
    want = scan_want(slice(0, n))
    # bf16 inputs are exact here: all math is float32.  A read-out whose normaliser nearly cancels amplifies
    # rounding: errors count against the row's own size
    def check(got, ref):
        e = np.abs(got - ref).max(-1) / (np.abs(ref).max(-1) + 0.05 * np.abs(ref).max())
        assert e.max() < 2e-3 and np.median(e) < (2e-5 if dtype == torch.float32 else 1e-4), (e.max(), np.median(e))

    def scan(rows, sb, st):
        xx = x[rows].contiguous().to(device)
        return la.memory_scan(xx, pad + qk, pad, pad + 2 * qk, ci, ci + hh, sp, ib32, fb32, st["s"], st["n"], st["m"], sb,
                              q_scale=d ** -0.5).cpu().numpy()

    full = lambda *s: torch.full((4,) + s, 5.0, dtype=torch.float32, device=device)       # an earlier owner's content
    st = {"s": full(hh, dv, d), "n": full(hh, d), "m": full(hh)}
    check(scan(slice(0, n), _sb([(0, n)], device, slots=[3]), st), want)
    got, at = [], 0
    for c in [1, 2, 1, 9, 8, 17, 3, 66, 2, 42]:          # blocks start inside earlier blocks' tokens
        got.append(scan(slice(at, at + c), _sb([(at, c)], device, slots=[1]), st))
        at += c
    assert at == n
    check(np.concatenate(got), want)
    scan(slice(0, 70), _sb([(0, 70)], device, slots=[2]), st)
    rows = torch.cat([torch.arange(70, n), torch.arange(0, 6)])
    o = scan(rows, _sb([(70, n - 70), (0, 6)], device, slots=[2, 3]), st)
    check(o[:n - 70], want[70:])
    check(o[n - 70:], want[:6])
    if case == "quiet":      # a maximum that started at minus infinity would lift the first tokens' read-out
        late = ig[0] < fg[0]
        assert late.all() and np.abs(want[0]).max() < 0.2 * np.abs(v[0]).max()


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("d,dv", [(8, 72), (16, 136), (10, 72)])
def test_matrix_memory_many_heads(target, d, dv):
    """Enough heads that long chunks take the forms with several value columns per lane and 128 per workgroup; two
    unequal sequences."""
    device, dtype = _dev(target)
    hh, n = 132, 40
    rng = np.random.default_rng(5)
    qk, vv = hh * d, hh * dv
    x = _t(rng, dtype, n, 2 * qk + vv + 2 * hh, scale=0.8)
    ci = 2 * qk + vv
    sp = la.MatrixMemorySpec(hh, d, dv, cap=6.0)
    zero = torch.zeros(hh, device=device)
    xd = _d(x)
    ig = O.capped(xd[:, ci:ci + hh], 6.0)
    fg = O.log_sigmoid(O.capped(xd[:, ci + hh:], 6.0))
    q, k, v = (xd[:, a:b].reshape(n, hh, -1) for a, b in ((0, qk), (qk, 2 * qk), (2 * qk, ci)))
    st = {"s": torch.zeros(3, hh, dv, d, device=device), "n": torch.zeros(3, hh, d, device=device),
          "m": torch.zeros(3, hh, device=device)}
    sb = _sb([(0, 23), (0, 17)], device, slots=[2, 1])
    o = la.memory_scan(x.to(device), 0, qk, 2 * qk, ci, ci + hh, sp, zero, zero, st["s"], st["n"], st["m"], sb).cpu().numpy()
    for lo, hi in ((0, 23), (23, 40)):
        for a in range(0, hh, 7):
            w = O.memory_scan(q[lo:hi, a], k[lo:hi, a], v[lo:hi, a], ig[lo:hi, a], fg[lo:hi, a])
            e = np.abs(o[lo:hi, a] - w).max(-1) / (np.abs(w).max(-1) + 0.05 * np.abs(w).max())
            assert e.max() < 2e-3, (a, e.max())


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("sizes", [(3, 16, 24), (2, 48, 40), (1, 128, 128), (2, 200, 20), (4, 20, 72), (1, 256, 9), (2, 30, 16)])
def test_matrix_memory_decoding_with_norm_and_gate(target, sizes):
    """The whole mixer between its projections, token by token for two sequences of unequal age and one that
    starts anew in a slot an earlier owner left full, after a prompt portion that went through the other forms."""
    device, dtype = _dev(target)
    hh, d, dv = sizes
    rng = np.random.default_rng(d + dv)
    n, qk, vv, eps = 40, hh * d, hh * dv, 1e-5
    ci = 2 * qk + 2 * vv
    xs = [_t(rng, dtype, n, -(-(ci + 2 * hh) // 8) * 8, scale=0.8) for _ in range(3)]
    ib, fb = (torch.from_numpy(rng.standard_normal(hh).astype(np.float32)) for _ in range(2))
    fb += 2.0
    w = _t(rng, dtype, vv, scale=0.4, off=1.0)
    sp = la.MatrixMemorySpec(hh, d, dv, cap=7.0)

    def want(x):
        xd = _d(x)
        q, k, v, g = (xd[:, a:b].reshape(n, hh, -1) for a, b in ((0, qk), (qk, 2 * qk), (2 * qk, 2 * qk + vv), (2 * qk + vv, ci)))
        ig = O.capped(xd[:, ci:ci + hh] + _d(ib), 7.0)
        fg = O.log_sigmoid(O.capped(xd[:, ci + hh:ci + 2 * hh] + _d(fb), 7.0))
        o = np.stack([O.memory_scan(q[:, a] * d ** -0.5, k[:, a], v[:, a], ig[:, a], fg[:, a]) for a in range(hh)], 1)
        return O.rms(o, eps).reshape(n, vv) * _d(w) * O.sigmoid(g.reshape(n, vv)), np.abs(o).max(-1).min(-1)
    full = lambda *s: torch.full((4,) + s, 5.0, dtype=torch.float32, device=device)
    st = (full(hh, dv, d), full(hh, d), full(hh))

    def run(x, sb):
        return _d(la.memory_mixer(x.contiguous().to(device), 0, qk, 2 * qk, 2 * qk + vv, ci, ci + hh, sp, ib.to(device),
                                  fb.to(device), w.to(device), *st, sb, eps, q_scale=d ** -0.5))
    refs = [want(x) for x in xs]

    def check(got, ref, rows):                   # rows whose read-out is not nearly cancelled in some head
        ok = ref[1][rows] > 0.02
        assert ok.any()
        np.testing.assert_allclose(got[ok], ref[0][rows][ok], atol=(1e-3 if dtype == torch.float32 else 3e-2) * np.abs(ref[0]).max())
    a = run(torch.cat([xs[0][:20], xs[1][:3]]), _sb([(0, 20), (0, 3)], device, slots=[1, 3]))
    check(a[:20], refs[0], slice(0, 20))
    steps = [run(torch.stack([xs[0][20 + i], xs[1][3 + i], xs[2][i]]), _sb([(20 + i, 1), (3 + i, 1), (i, 1)], device, slots=[1, 3, 2]))
             for i in range(20)]
    for j, lo in enumerate((20, 3, 0)):
        check(np.stack([s[j] for s in steps]), refs[j], slice(lo, lo + 20))


@pytest.mark.parametrize("target", TARGETS)
def test_a_write_far_back_is_read_from_the_memory(target):
    """A key written 300 tokens ago under a loud input gate is still read by a matching query, as one portion and
    token by token through the slot; with forget gates of one half it is gone."""
    device, dtype = _dev(target)
    n, d, dv = 301, 16, 8
    rng = np.random.default_rng(0)
    x = (rng.standard_normal((n, 2 * d + dv + 8)) * 0.01).astype(np.float32)
    x[0, d], x[n - 1, 0] = 4.0, 4.0
    x[0, 2 * d:2 * d + dv] = np.arange(1, dv + 1)
    x[:, 2 * d + dv] = -4.0
    x[0, 2 * d + dv] = 6.0
    for logit, seen in ((9.0, True), (0.0, False)):
        x[:, 2 * d + dv + 1] = logit
        xx = torch.from_numpy(x).to(dtype).to(device)
        sp = la.MatrixMemorySpec(1, d, dv, cap=15.0)
        zero = torch.zeros(1, device=device)
        st = {"s": torch.zeros(2, 1, dv, d, device=device), "n": torch.zeros(2, 1, d, device=device),
              "m": torch.zeros(2, 1, device=device)}

        def run(lo, hi, slot):
            sb = _sb([(lo, hi - lo)], device, slots=[slot])
            return la.memory_scan(xx[lo:hi], 0, d, 2 * d, 2 * d + dv, 2 * d + dv + 1, sp, zero, zero, st["s"], st["n"], st["m"],
                                  sb)[-1, 0].cpu().numpy()
        whole = run(0, n, 1)
        for i in range(n):
            last = run(i, i + 1, 0)
        np.testing.assert_allclose(last, whole, atol=1e-3, rtol=1e-3)
        assert (np.abs(whole - np.arange(1, dv + 1)).max() < 0.3) == seen, whole


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("hh,dv", [(3, 8), (2, 24), (2, 128), (2, 600)])
def test_output_norm_with_a_weight_per_head(target, hh, dv):
    """Every head over its own root mean square, then one weight vector over all heads and a sigmoid gate."""
    device, dtype = _dev(target)
    rng = np.random.default_rng(dv)
    t = 7
    o = torch.from_numpy((rng.standard_normal((t, hh * dv)) * np.repeat([9.0, 0.1, 1.0][:hh], dv)).astype(np.float32))
    gate, w = _t(rng, dtype, t, 8 + hh * dv), _t(rng, dtype, hh * dv, scale=0.5, off=1.0)
    y = la.gated_norm(o.to(device), gate.to(device), 8, w.to(device), 1e-6, groups=hh, gate_act="sigmoid")
    want = O.rms(_d(o).reshape(t, hh, dv), 1e-6).reshape(t, -1) * _d(w) * O.sigmoid(_d(gate)[:, 8:])
    np.testing.assert_allclose(_d(y), want, atol=_atol(dtype, 2e-5, 3e-2) * np.abs(want).max())


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("sizes", [(96, 6, 2, 48, 64), (128, 8, 2, 128, 128), (256, 8, 3, 256, 128), (72, 3, 3, 24, 0), (128, 4, 1, 128, 40)])
@pytest.mark.parametrize("tokens", [1, 5, 70, 300])
def test_clipped_experts_weighted_over_all_logits(target, sizes, tokens):
    """Weights are the softmax over ALL experts, not renormalised; gate and up are clipped on their own sides with
    different limits for the experts and the shared one, whose sigmoid gate is one number per token."""
    device, dtype = _dev(target)
    width, e, top, ff, fs = sizes
    rng = np.random.default_rng(width + tokens)
    mlp = _moe(e, top, ff, 0.8, fs, 1.7)
    w = {"router": _t(rng, torch.float32, e, width, scale=4.0 * width ** -0.5)}
    for j in range(e):
        for nm, s in (("gate", (ff, width)), ("up", (ff, width)), ("down", (width, ff))):
            w[f"e{j}.{nm}"] = _t(rng, dtype, *s, scale=2.0 * s[1] ** -0.5)
    rows = [w["router"]]
    if fs:
        for nm, s in (("gate", (fs, width)), ("up", (fs, width)), ("down", (width, fs))):
            w[f"shared.{nm}"] = _t(rng, dtype, *s, scale=2.0 * s[1] ** -0.5)
        w["shared.sg"] = _t(rng, torch.float32, 1, width, scale=2.0 * width ** -0.5)
        rows.append(w["shared.sg"])
    h = _t(rng, dtype, tokens, width)
    margins = []
    want = O.moe_ff(_d(h), {k: _d(v) for k, v in w.items()}, mlp, margins)
    gu = torch.stack([torch.cat([w[f"e{j}.gate"], w[f"e{j}.up"]], 0) for j in range(e)], 0)
    dn = torch.stack([w[f"e{j}.down"] for j in range(e)], 0)
    dv = lambda a: a.to(device)
    got = moe.softmax_top_ffn(dv(h), dv(torch.cat(rows, 0)), None, dv(gu), dv(dn), top,
                              dv(torch.cat([w["shared.gate"], w["shared.up"]], 0)) if fs else None,
                              dv(w["shared.down"]) if fs else None, over_all=True, limit=0.8, shared_limit=1.7)
    ok = margins[0] > 1e-3                                   # a tie may fall either way
    scale = np.abs(want).max()
    np.testing.assert_allclose(_d(got)[ok], want[ok], atol=(2e-5 if dtype == torch.float32 else 2e-2) * scale)
    if top < e:              # renormalised weights would show
        z = _d(h) @ _d(w["router"]).T
        assert np.median([O.route(r, top)[1].sum() for r in z]) < 0.995


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("tokens,width,ff", [(1, 256, 128), (3, 72, 24), (33, 512, 1024), (200, 2048, 256), (700, 256, 256),
                                             (8192, 128, 1024)])
def test_dense_clipped_glu(target, tokens, width, ff):
    """Gate clipped from above only, up from both sides and shifted by one: decode sizes (in the split-K reduction),
    prompt sizes (in the persistent GEMM's epilogue) and sizes that take neither."""
    device, dtype = _dev(target)
    rng = np.random.default_rng(ff)
    x, w = _t(rng, dtype, tokens, width), _t(rng, dtype, 2 * ff, width, scale=2.0 * width ** -0.5)
    got = _d(moe.linear_clipped_glu(x.to(device), w.to(device), 1.1))
    rows = np.unique(np.linspace(0, tokens - 1, 80).astype(int))
    want = O.clipped_expert(_d(x)[rows], {"gate": _d(w)[:ff], "up": _d(w)[ff:], "down": np.eye(ff)}, 1.1)
    np.testing.assert_allclose(got[rows], want, atol=2e-5 if dtype == torch.float32 else 3e-2)
    g = _d(x)[rows] @ _d(w)[:ff].T
    assert (g > 1.1).any() and (g < -1.1).any() and want.min() < -0.1


# ------------------------------------------------------------------------------ the engine
@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("name", ["a", "b", "c"])
def test_whole_prompts_and_layers(target, name, tmp_path):
    """Whole prompts in one step, alone and three at once; the sum of the streams after every layer run (a looped
    layer counts once per pass) against the oracle's."""
    cfg = CONFIGS[name]()
    sd = _round(O.make_weights(cfg, seed=3), target[1])
    eng = make_engine(cfg, sd, target, tmp_path)
    p = prompts_for(cfg, [97, 1, 30], seed=5)
    taps = []
    want = {n: oracle(cfg, sd, t, taps if n == "r2" else None) for n, t in p.items()}
    eng.runner.stage.taps = got_taps = []
    got = replay(eng, [[("r2", 30)]], {"r2": p["r2"]})
    eng.runner.stage.taps = None
    assert len(got_taps) == len(taps) == len(O.layer_runs(cfg))
    if target[1] == torch.float32:
        for a, b in zip(got_taps, taps):
            np.testing.assert_allclose(a.cpu().numpy(), b, atol=2e-4 * max(1.0, np.abs(b).max()))
    assert_close(got["r2"], want["r2"], target, "alone")
    got = replay(eng, [[("r0", 97), ("r1", 1), ("r2", 30)]], p)
    for n in p:
        assert_close(got[n], want[n], target, n)


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("name", ["a", "b", "c"])
def test_decode_and_portions_match_the_whole(target, name, tmp_path):
    """Token-by-token decoding after a prompt (90 steps over several cache blocks, temperature steps and bias
    buckets), portions of changing sizes down to two tokens and one, and decoding from the very first token."""
    cfg = CONFIGS[name]()
    sd = _round(O.make_weights(cfg, seed=4), target[1])
    eng = make_engine(cfg, sd, target, tmp_path)
    p = prompts_for(cfg, [150], seed=7)
    want = oracle(cfg, sd, p["r0"])
    got = replay(eng, [[("r0", 60)]] + [[("r0", 1)]] * 90, p)
    assert_close(got["r0"], want, target, "decode")
    sizes = [2, 3, 1, 31, 2, 33, 5, 64, 2, 7]
    assert sum(sizes) == 150
    got = replay(eng, [[("r0", s)] for s in sizes], p)
    assert_close(got["r0"], want, target, "portions")
    got = replay(eng, [[("r0", 1)]] * 40, {"r0": p["r0"][:40]})
    assert_close(got["r0"], (want[0][:40], want[1][:40]), target, "from the first token")


@pytest.mark.parametrize("target", TARGETS)
def test_mixed_batches_and_reused_blocks_and_slots(target, tmp_path):
    """Up to four unequal requests per step, portions beside single tokens; finished requests give their
    blocks and their state slot to new ones (a pool sized for the live tokens only, four slots for seven
    requests).  Every request matches its own whole-sequence oracle: the batch, the pool and the slots do
    not show."""
    cfg = cfg_a()
    sd = _round(O.make_weights(cfg, seed=5), target[1])
    eng = make_engine(cfg, sd, target, tmp_path, max_tokens=288, max_requests=4)
    lens = [70, 9, 33, 64, 20, 50, 3]
    prompts = prompts_for(cfg, lens, seed=9)
    names = list(prompts)
    at = {n: 0 for n in names}
    waiting, live, schedule = list(names), [], []
    rng = np.random.default_rng(0)
    while waiting or live:
        while waiting and len(live) < 4:
            live.append(waiting.pop(0))
        step = []
        for n in list(live):
            left = len(prompts[n]) - at[n]
            c = min(left, int(rng.choice([1, 1, 2, 3, 17, 32])))
            if rng.random() < 0.15 and len(live) > 1:
                continue                                # left out of this step, goes on later
            step.append((n, c))
            at[n] += c
            if at[n] == len(prompts[n]):
                live.remove(n)
        if step:
            schedule.append(step)
    got = replay(eng, schedule, prompts)
    assert eng.bm.num_free() == eng.bm.num_blocks - 1            # all given back (block 0 is the scratch block)
    for n in names:
        assert_close(got[n], oracle(cfg, sd, prompts[n]), target, n)


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("name,graphs", [("a", False), ("c", True)])
def test_greedy_generation_through_the_scheduler(target, name, graphs, tmp_path):
    """LLMEngine.generate (scheduler, continuous batching, sampler; for the model whose experts the grouped
    kernels take, decode steps replayed from HIP graphs) on three prompts at once: every generated token is
    the argmax of the oracle's logits for the sequence so far (where the oracle's top two are not within
    rounding of each other and, in bfloat16, no expert choice of the token is a close call; earlier tokens' close calls
    may still turn one such token in five)."""
    cfg = CONFIGS[name]()
    sd = _round(O.make_weights(cfg, seed=6), target[1])
    eng = make_engine(cfg, sd, target, tmp_path, graphs=graphs)
    prompts = list(prompts_for(cfg, [5, 40, 17], seed=11).values())
    outs = eng.generate(prompts, SamplingParams(max_new_tokens=24, ignore_eos=True))
    margin = 1e-3 if target[1] == torch.float32 else 0.3
    checked = wrong = 0
    for p, o in zip(prompts, outs):
        assert len(o) == 24
        logits, decided = oracle(cfg, sd, p + o)
        for i, tok in enumerate(o):
            row = logits[len(p) + i - 1]
            top = np.sort(row)[-2:]
            if top[1] - top[0] > margin * cfg["logit_scale"] and (target[1] == torch.float32 or decided[len(p) + i - 1]):
                checked += 1
                wrong += tok != int(row.argmax())
    assert checked > (36 if target[1] == torch.float32 else 12)
    assert wrong <= (0 if target[1] == torch.float32 else checked // 5), (wrong, checked)


def random_config(seed):
    """A model whose every size is drawn: widths, streams, head counts and groupings, key / value sizes, rotated
    parts, bias tables, caps, limits, expert counts, layer count and order, the looped span."""
    rng = np.random.default_rng(3000 + seed)
    pick = lambda xs: xs[int(rng.integers(len(xs)))]
    layers = []
    for _ in range(int(rng.integers(2, 5))):
        e = pick([1, 2, 3, 5, 8, 12])
        mlp = pick([None, "moe", "moe"]) and _moe(e, pick([t for t in (1, 2, 3, 4, 6) if t <= e]), pick([16, 40, 64, 128]),
                                                  float(rng.uniform(0.3, 4.0)), pick([0, 24, 64, 128]), float(rng.uniform(0.3, 4.0)))
        g = pick([1, 2, 3])
        hh, d, dv = g * pick([1, 2, 3, 4]), pick([8, 16, 20, 32, 40, 64, 80, 128]), pick([8, 12, 24, 32, 64, 128])
        scale = float(rng.uniform(0.05, 0.4))
        if rng.random() < 0.5:
            layers.append(_attn(hh, g, d, dv, scale, pick([r for r in (2, 4, 8, 16, 20, 64, 128) if r <= d]), mlp,
                                base=float(pick([100.0, 10000.0, 1e6])), factor=pick([None, 2.0, 10.0])))
        else:
            rows = pick([2, 4, 8, 10, 32])
            left = _left(hh, g, d, dv, scale, rows // 2 + pick([1, 7, 50, 300]), rows,
                         *pick([(None, 0), (0.3, 10), (0.1, 64), (-0.2, 1)]))
            layers.append(_par(left, _right(pick([1, 2, 3]), pick([8, 16, 24, 32, 48, 64, 128]), pick([8, 16, 40, 64, 128]),
                                            float(pick([2.0, 8.0, 20.0]))), mlp))
    cfg = {"architecture": "Kupedra", "vocab": pick([97, 128, 200, 333]), "width": pick([64, 72, 96, 128, 160, 256]),
           "norm": {"eps": pick([1e-6, 1e-5, 1e-4])}, "embedding": {"scale": float(pick([0.25, 1.0, 8.0]))},
           "streams": pick([1, 2, 3, 4, 6]), "logit_scale": float(pick([0.125, 1.0, 2.0])), "layers": layers}
    if rng.random() < 0.7:
        start = int(rng.integers(0, len(layers)))
        cfg["loop"] = {"start": start, "stop": int(rng.integers(start + 1, len(layers) + 1)), "times": int(rng.integers(1, 4))}
    return cfg


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("seed", range(8))
def test_drawn_models_on_a_mixed_schedule(target, seed, tmp_path):
    """Models of drawn sizes: three unequal requests, portions of changing size beside single tokens, a
    fourth request that takes over freed blocks and a freed slot; each equals its whole-sequence oracle."""
    cfg = random_config(seed)
    sd = _round(O.make_weights(cfg, seed=0), target[1])
    eng = make_engine(cfg, sd, target, tmp_path, max_tokens=320, max_requests=3)
    prompts = prompts_for(cfg, [75, 18, 110, 40], seed=seed)
    schedule = [[("r0", 33), ("r1", 2)], [("r0", 1), ("r1", 16), ("r2", 64)], [("r0", 1), ("r2", 3)], [("r0", 30), ("r2", 1)],
                [("r2", 2), ("r0", 1)], [("r0", 9), ("r2", 39), ("r3", 7)], [("r3", 1), ("r2", 1)], [("r3", 32)]]
    got = replay(eng, schedule, prompts)
    assert eng.bm.num_free() == eng.bm.num_blocks - 1
    for n, p in prompts.items():
        assert_close(got[n], oracle(cfg, sd, p), target, (seed, n))


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("case", ["attention only", "parallel only, all looped", "no rotation, loop on the last layer"])
def test_unusual_layer_orders(target, case, tmp_path):
    """Models without any recurrent state, with every layer inside a loop of three passes, with a loop over the last
    layer only and heads that do not turn: two requests in portions beside single tokens."""
    base = {"architecture": "Kupedra", "vocab": 101, "width": 64, "norm": {"eps": 1e-6}, "embedding": {"scale": 4.0},
            "streams": 2, "logit_scale": 0.5}
    if case == "attention only":
        cfg = dict(base, layers=[_attn(2, 1, 16, 8, 0.3, 16, _moe(4, 2, 16, 2.0, 16)), _attn(1, 1, 8, 24, 0.5, 4, None)])
    elif case == "parallel only, all looped":
        cfg = dict(base, loop={"start": 0, "stop": 2, "times": 3},
                   layers=[_par(_left(2, 1, 16, 16, 0.2, 40, 8), _right(1, 8, 8, 5.0), None),
                           _par(_left(2, 2, 8, 8, 0.3, 20, 4, 0.2, 8), _right(2, 8, 16, 9.0), _moe(3, 1, 8, 1.0))])
    else:
        cfg = dict(base, loop={"start": 2, "stop": 3, "times": 2},
                   layers=[_attn(2, 2, 16, 8, 0.3, 8, None),
                           _par(_left(4, 2, 16, 8, 0.2, 70, 10), _right(1, 8, 8, 5.0), _moe(2, 2, 8, 3.0, 8)),
                           _attn(1, 1, 8, 8, 0.4, 0, None)])
    sd = _round(O.make_weights(cfg, seed=1), target[1])
    eng = make_engine(cfg, sd, target, tmp_path, max_tokens=256, max_requests=3)
    p = prompts_for(cfg, [70, 33], seed=2)
    got = replay(eng, [[("r0", 40), ("r1", 2)], [("r0", 1), ("r1", 31)], [("r0", 29)]], p)
    for n in p:
        assert_close(got[n], oracle(cfg, sd, p[n]), target, (case, n))


def test_config_round_trip_and_registry(tmp_path):
    from distributed_llms_amd.config import get_model_config
    from distributed_llms_amd.models.hybrid import layer_runs
    from distributed_llms_amd.models.kupedra import KupedraStage, model_shapes
    cfg = cfg_a()
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    m = get_model_config(str(tmp_path))
    assert m.arch == "kupedra" and m.num_layers == 4 and m.hidden_size == 96 and m.embed_scale == 3.0 and m.streams == 4
    assert m.logit_scale == 0.7 and m.needs_seq_index and m.needs_state_slots
    back = ModelConfig.from_hf_config(m.to_hf_config())
    assert (back.layers, back.norm_eps, back.loop, back.embed_scale, back.streams, back.logit_scale) == (
        m.layers, m.norm_eps, m.loop, 3.0, 4, 0.7)
    assert [i for i, _ in layer_runs(m)] == O.layer_runs(cfg)
    st = make_stage(m)
    assert isinstance(st, KupedraStage)
    sd = O.make_weights(cfg)
    assert {k: tuple(v.shape) for k, v in sd.items()} == model_shapes(m, {k: torch.from_numpy(v) for k, v in sd.items()})
    assert st.num_layers == 6                                  # every run has a K / V pair of its own
    for bad in ({"type": "lightning"}, {"mlp": {"kind": "dense", "ff": 8}}):
        c = cfg_a()
        c["layers"][0].update(bad)
        with pytest.raises(ValueError):
            ModelConfig.from_hf_config(c)
    c = cfg_a()
    c["layers"][1]["mixer"]["rot"]["dims"] = 32               # wider than the head
    with pytest.raises(ValueError):
        make_stage(ModelConfig.from_hf_config(c))
    c = cfg_a()
    c["loop"]["stop"] = 9
    with pytest.raises(ValueError):
        ModelConfig.from_hf_config(c)
    c = cfg_a()
    c["streams"] = 99
    with pytest.raises(ValueError):
        make_stage(ModelConfig.from_hf_config(c))
    assert get_model_config("tiny-kupedra").arch == "kupedra"
    make_stage(get_model_config("tiny-kupedra")).init_synthetic(0)


@pytest.mark.parametrize("target", [t for t in TARGETS if "gpu" in t.id])
def test_decode_graphs_replay_like_eager_steps(target, tmp_path):
    """Decode steps replayed from captured HIP graphs (several replays, eager prompt steps and
    synchronisations between them) give the logits of eager decode steps, recurrent state included."""
    if target[1] != torch.bfloat16:
        pytest.skip("the float32 expert path reads row counts on the host: it decodes eagerly")
    cfg = cfg_c()
    sd = _round(O.make_weights(cfg, seed=8), target[1])
    p = prompts_for(cfg, [60, 23], seed=3)
    sched = [[("r0", 45), ("r1", 13)]] + [[("r0", 1), ("r1", 1)]] * 10
    eager = replay(make_engine(cfg, sd, target, tmp_path, graphs=False), sched, p)
    eng = make_engine(cfg, sd, target, tmp_path, graphs=True)
    assert eng.runner.graphs is not None
    graphed = replay(eng, sched, p)
    for n in p:
        np.testing.assert_allclose(graphed[n], eager[n], rtol=1e-3, atol=1e-3)


def test_trace_run_program_loads_a_model_folder(tmp_path):
    """bin/trace_run on a folder with config.json + model.safetensors (bfloat16): the registry picks the
    stage by the config, the checkpoint loader reads the tensors (the bias table's rows from their shapes), steps
    with portions beside single tokens answer with the wanted logits (CPU path, float32)."""
    import os
    import subprocess
    import sys
    from safetensors.torch import save_file
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    cfg = cfg_a()
    sd = {k: torch.from_numpy(v).to(torch.bfloat16) for k, v in O.make_weights(cfg, seed=21).items()}
    for l in cfg["layers"]:                      # a model folder names no row count: the tensors do
        if l["type"] == "parallel":
            del l["mixer"]["left"]["rows"]
    model = tmp_path / "model"
    model.mkdir()
    (model / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.contiguous() for k, v in sd.items()}, str(model / "model.safetensors"))
    rng = np.random.default_rng(3)
    toks = {"a": rng.integers(0, cfg["vocab"], 50).tolist(), "b": rng.integers(0, cfg["vocab"], 21).tolist()}
    steps = [
        {"step": 0, "entries": [{"id": "a", "tokens": toks["a"][:30], "want": [0, 29]}], "end": []},
        {"step": 1, "entries": [{"id": "a", "tokens": toks["a"][30:31], "want": [0]},
                                {"id": "b", "tokens": toks["b"][:20], "want": [19]}], "end": []},
        {"step": 2, "entries": [{"id": "b", "tokens": toks["b"][20:], "want": []}], "end": ["b"]},
        {"step": 3, "entries": [{"id": "a", "tokens": toks["a"][31:], "want": [18]}], "end": ["a"]},
    ]
    out = tmp_path / "out"
    p = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", str(model), "--dtype", "float32",
                        "--out", str(out), "--max-tokens", "128", "--device", "cpu"],
                       input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=600)
    assert p.returncode == 0, p.stderr[-2000:]
    assert [l for l in p.stdout.splitlines() if l.startswith("done")] == [f"done {i}" for i in range(4)]
    assert not (out / "2.f32").exists()                       # nothing wanted in step 2
    f64 = {k: v.double().numpy() for k, v in sd.items()}
    ref = {n: O.forward(cfg_a(), f64, t) for n, t in toks.items()}
    got = {i: np.fromfile(out / f"{i}.f32", dtype="<f4").reshape(-1, cfg["vocab"]) for i in (0, 1, 3)}
    assert row_errs(got[0], ref["a"][[0, 29]]).max() < 1e-4
    assert row_errs(got[1], np.stack([ref["a"][30], ref["b"][19]])).max() < 1e-4
    assert row_errs(got[3], ref["a"][[49]]).max() < 1e-4
