"""The Basopel decoder (layer norms before and after every sublayer, distance-biased windows whose first tokens stay
visible, chunked attention with capped scores, latent attention with element gates, values shared between layers, gelu
GLUs, a tied head) against the plain float64 oracle of tests/oracle_basopel.py: every mechanism alone, then the engine
-- whole prompts, token-by-token decoding, prompt portions down to two tokens, batches of unequal requests, blocks
that are freed and used again, keys just inside and just outside windows, chunks and the kept first tokens, the
first tokens, long decoding, and greedy generation through the scheduler.  Each case runs on the CPU path in float32
and, marked gpu, on the HIP kernels in float32 and bfloat16.
"""
import json

import numpy as np
import pytest
import torch

import oracle_basopel as O
from distributed_llms_amd import ops
from distributed_llms_amd.config import ModelConfig
from distributed_llms_amd.engine.sequence import SamplingParams
from distributed_llms_amd.models import make_stage
from distributed_llms_amd.ops import gemm
from distributed_llms_amd.ops import latent as lat
from distributed_llms_amd.ops import seqmix as sm
from test_fekizen import (TARGETS, _atol, _dev, _np, _paged, _round, _sb, make_engine, prompts_for, replay, row_errs)


def _attn(heads, kv_heads, dim, vdim, scale, size, keep, far, rows, ff=0, v_mix=True):
    return {"type": "attention", "mlp": {"kind": "dense", "ff": ff} if ff else None, "mixer": {
        "heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "bias_max": far, "rows": rows,
        "mask": {"size": size, "keep_first": keep}, "v_mix": v_mix}}


def _two(heads, kv_heads, dim, vdim, scale, chunk, cap, dims, ff=0, base=10000.0, factor=None, v_mix=True):
    rot = {"base": base, "dims": dims}
    if factor:
        rot["scaling"] = {"factor": factor}
    return {"type": "attention_2", "mlp": {"kind": "dense", "ff": ff} if ff else None, "mixer": {
        "heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "softcap": cap, "rot": rot,
        "mask": {"size": chunk}, "v_mix": v_mix}}


def _lat(heads, dim, rot_dim, vdim, rank, scale, size, ff=0, base=10000.0):
    return {"type": "latent_attention", "mlp": {"kind": "dense", "ff": ff} if ff else None, "mixer": {
        "heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": rank, "scale": scale, "mask": {"size": size},
        "rot": {"base": base, "dims": rot_dim}}}


def _model(vocab, width, layers, scale=5.0, eps=1e-6):
    return {"architecture": "Basopel", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": scale},
            "layers": layers}


def cfg_a():
    """Layers that differ from one another: windows, chunks and kept tokens that are no multiple of a cache block or of
    each other, several bias tables, a latent layer first, values shared from a biased window to chunked layers and back,
    one layer between them that does not take part, a layer without a feed-forward."""
    return _model(200, 96, [
        _lat(4, 16, 8, 24, 40, 0.2, 33, 128),
        _attn(6, 2, 24, 16, 0.25, 20, 3, 60, 12, 160),
        _two(4, 2, 24, 16, 0.3, 24, 15.0, 16, 96, factor=4.0),
        _two(2, 1, 16, 40, 0.2, 37, 30.0, 16, 64, base=500.0, v_mix=False),
        _attn(2, 1, 16, 32, 0.4, 9, 5, 200, 32),
        _lat(3, 12, 4, 16, 24, 0.3, 50, 48, base=100.0),
        _two(4, 4, 8, 8, 0.5, 10, 8.0, 4, 40),
    ])


def cfg_b():
    """Degenerate sizes: one head, a window of one, no kept tokens and more kept tokens than the window holds, a two-row
    bias table, chunks of one and two, head sizes and widths that are no multiple of 8."""
    return _model(131, 70, [
        _attn(1, 1, 12, 9, 0.3, 1, 0, 3, 2, 24),
        _two(3, 3, 10, 3, 0.4, 2, 5.0, 2, 33),
        _lat(1, 5, 2, 7, 11, 0.3, 1),
        _attn(5, 5, 8, 6, 0.35, 2, 17, 9, 6, 16, v_mix=False),
        _two(1, 1, 6, 9, 0.3, 1, 100.0, 6),
        _attn(3, 1, 14, 9, 0.3, 40, 1, 500, 10),
    ], scale=1.0, eps=1e-5)


def cfg_c():
    """Sizes that the matrix-core attention kernels and the framework's own GEMMs take."""
    return _model(160, 256, [
        _two(4, 2, 64, 64, 0.12, 48, 20.0, 32, 256, factor=2.0),
        _attn(4, 1, 64, 128, 0.12, 40, 4, 100, 16, 256),
        _lat(4, 32, 32, 64, 96, 0.12, 72, 384),
        _two(2, 1, 128, 128, 0.09, 70, 30.0, 128, 128),
    ], scale=16.0)


CONFIGS = {"a": cfg_a, "b": cfg_b, "c": cfg_c}


def assert_close(got, want, target, what=""):
    """float32: every position within 2e-4, 2e-5 at the median (a wrong key, weight or bias shows at 1e-2 and more).
    bfloat16: 3e-2 at the median, 0.1 at all but one position in twenty, 0.4 at all."""
    e = row_errs(got, want)
    if target[1] == torch.float32:
        assert np.median(e) < 2e-5 and e.max() < 2e-4, (what, float(np.median(e)), float(e.max()), int(e.argmax()))
    else:
        over = int((e > 0.1).sum())
        assert np.median(e) < 3e-2 and over <= max(1, len(e) // 20) and e.max() < 0.4, (
            what, float(np.median(e)), over, float(e.max()), int(e.argmax()))


def _t(rng, dtype, *shape, scale=1.0, off=0.0):
    return torch.from_numpy((off + scale * rng.standard_normal(shape)).astype(np.float32)).to(dtype)


def _d(x):
    return x.detach().cpu().double().numpy()


# ------------------------------------------------------------------------------ mechanisms alone
@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("width", [33, 70, 96, 260, 1000, 1100, 2560, 4097, 8192, 12288])
def test_layer_norms_around_a_sublayer(target, width):
    """The layer norm of a stream with a mean far from zero, and the close of a sublayer: the output's own layer norm
    (projection bias inside it) added to the stream, the next sublayer's norm of the NEW stream; an eps that matters."""
    device, dtype = _dev(target)
    rng = np.random.default_rng(width)
    t, eps = 5, 0.3
    x0 = torch.from_numpy((30.0 + rng.standard_normal((t, width))).astype(np.float32))
    o = _t(rng, dtype, t, width, scale=0.5, off=2.0)
    w1, w2, wn = (_t(rng, dtype, width, scale=0.3, off=1.0) for _ in range(3))
    b1, b2, bn, ob = (_t(rng, dtype, width) for _ in range(4))
    dv = lambda a: a.to(device)
    y = sm.layer_norm_f32(dv(x0), dv(w1), dv(b1), eps, dtype)
    assert y.dtype == dtype
    np.testing.assert_allclose(_d(y), O.layer_norm(_d(x0), _d(w1), _d(b1), eps), atol=_atol(dtype, 1e-4, 4e-2))
    for bias in (None, ob):
        new = _d(x0) + O.layer_norm(_d(o) + (0.0 if bias is None else _d(ob)), _d(w2), _d(b2), eps)
        kw = {} if bias is None else {"bias": dv(ob)}
        x, h = sm.post_layer_norm_add(dv(x0.clone()), dv(o), dv(w2), dv(b2), eps, w_next=dv(wn), b_next=dv(bn), **kw)
        np.testing.assert_allclose(_d(x), new, atol=2e-5)
        assert h.dtype == dtype
        np.testing.assert_allclose(_d(h), O.layer_norm(new, _d(wn), _d(bn), eps), atol=_atol(dtype, 1e-4, 4e-2))
        x, h = sm.post_layer_norm_add(dv(x0.clone()), dv(o), dv(w2), dv(b2), eps, **kw)
        assert h is None
        np.testing.assert_allclose(_d(x), new, atol=2e-5)


@pytest.mark.gpu
@pytest.mark.parametrize("tokens,width,k", [(1, 256, 1024), (32, 2560, 2048), (7, 1024, 7680), (200, 512, 4096), (3, 4096, 4096),
                                            (1, 128, 8192)])
def test_layer_norm_sums_split_products(tokens, width, k):
    """The close of a sublayer on a split-K product that is not reduced yet, against the same on the reduced one."""
    device, dtype = _dev(("cuda", torch.bfloat16))
    rng = np.random.default_rng(k)
    a, w = _t(rng, dtype, tokens, k).to(device), _t(rng, dtype, width, k, scale=k ** -0.5).to(device)
    part = ops.linear(a, w, defer=True)
    assert isinstance(part, gemm.SplitKPartial)
    whole = part.materialize()
    np.testing.assert_allclose(_d(whole), _d(a) @ _d(w).T, atol=3e-2)
    x0 = torch.from_numpy(rng.standard_normal((tokens, width)).astype(np.float32)).to(device)
    ws = [_t(rng, dtype, width, scale=0.3, off=1.0).to(device) for _ in range(4)]
    ob = _t(rng, dtype, width).to(device)
    got = sm.post_layer_norm_add(x0.clone(), part, ws[0], ws[1], 1e-5, bias=ob, w_next=ws[2], b_next=ws[3])
    want = sm.post_layer_norm_add(x0.clone(), whole, ws[0], ws[1], 1e-5, bias=ob, w_next=ws[2], b_next=ws[3])
    np.testing.assert_allclose(_d(got[0]), _d(want[0]), atol=1e-5)
    np.testing.assert_allclose(_d(got[1]), _d(want[1]), atol=3e-2)


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("whole", [False, True])
@pytest.mark.parametrize("shape", [(4, 2, 24, 16, 16), (3, 1, 16, 24, 8), (2, 2, 64, 48, 64), (5, 5, 10, 4, 4), (2, 1, 12, 9, 2),
                                   (16, 4, 128, 128, 64), (3, 1, 136, 8, 136)])
def test_input_stages_with_biases_and_shared_values(target, whole, shape):
    """Projection biases enter before the norms (per head, or over the whole projection with a half-split rotation by
    divided frequencies) and into the values; the first layer's values are handed on as cached, a later layer's are
    blended with them and the blend is what its cache holds.  A small eps, tiny heads: the eps inside the root shows."""
    device, dtype = _dev(target)
    h, g, d, dv, dims = shape
    rng = np.random.default_rng(d + dims)
    pos = [0, 1, 6, 7, 8, 14, 15, 1000, 20000]
    t, pad, eps, bs = len(pos), 8, 1e-2, 16
    nq, nk, nv = h * d, g * d, g * dv
    x = _t(rng, dtype, t, pad + nq + nk + nv + 8, scale=0.3)
    bias = _t(rng, dtype, nq + nk + nv, scale=0.3)
    slots = [5 * bs + 3, 2 * bs, 2 * bs + 1, 7 * bs + 15, bs, 3 * bs + 8, 4 * bs + 15, 6 * bs, 8 * bs + 2]
    rot = {"base": 3000.0, "dims": dims, "scaling": {"factor": 3.0}}
    freqs = sm.rotary_frequencies(dims, 3000.0, 3.0).to(device)
    qw, kw = ((_t(rng, dtype, n, scale=0.3, off=1.0) for n in ((nq, nk) if whole else (d, d))))
    first = torch.full((t, nv), 9.0, dtype=dtype, device=device)
    xd = _d(x)[:, pad:pad + nq + nk + nv] + _d(bias)
    dvc = lambda a: a.to(device)
    si, pi = (torch.tensor(a, dtype=torch.int32, device=device) for a in (slots, pos))
    for lam in (None, 0.3):
        kc = torch.zeros(9, g, bs, d, dtype=dtype, device=device)
        vc = torch.zeros(9, g, dv, bs, dtype=dtype, device=device)
        mix = sm.ValueMix(first, lam)
        if whole:
            q = sm.rownorm_rope(dvc(x), pad, dvc(qw), dvc(kw), freqs, eps, kc, vc, si, pi, h, g, d, dv, bias=dvc(bias), v_mix=mix)
        else:
            q = sm.head_norm_rope(dvc(x), pad, dvc(qw), dvc(kw), None, eps, kc, vc, si, pi, h, g, d, dv, bias=dvc(bias), v_mix=mix)
        v = O.mix_values(xd[:, nq + nk:], None if lam is None else _d(first), lam)
        for i, p in enumerate(pos):
            if whole:
                wq = O.rotate_halves((O.rms(xd[i:i + 1, :nq], eps) * _d(qw)).reshape(1, h, d), rot, first_pos=p)[0]
                wk = O.rotate_halves((O.rms(xd[i:i + 1, nq:nq + nk], eps) * _d(kw)).reshape(1, g, d), rot, first_pos=p)[0]
            else:
                wq = O.rms(xd[i, :nq].reshape(h, d), eps) * _d(qw)
                wk = O.rms(xd[i, nq:nq + nk].reshape(g, d), eps) * _d(kw)
            tol = (2e-3 if p > 100 and whole else 2e-5) if dtype == torch.float32 else 2e-2      # float32 angles far out
            s = slots[i]
            np.testing.assert_allclose(_d(q[i]), wq, atol=tol * np.abs(wq).max())
            np.testing.assert_allclose(_d(kc[s // bs, :, s % bs]), wk, atol=tol * np.abs(wk).max())
            np.testing.assert_allclose(_d(vc[s // bs, :, :, s % bs]), v[i].reshape(g, dv), atol=_atol(dtype, 2e-6, 1e-2))
        if lam is None:
            np.testing.assert_allclose(_d(first), v, atol=_atol(dtype, 2e-6, 1e-2))


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("whole", [False, True])
@pytest.mark.parametrize("offset", [0, 3])
def test_values_of_long_prompts(target, whole, offset):
    """Enough tokens that values are appended eight tokens at a time: runs that fill aligned eighths of blocks, runs
    that start inside one, a block border, a last incomplete run; with and without another layer's values."""
    device, dtype = _dev(target)
    h, g, d, dv, bs, n = 2, 2, 16, 24, 32, 1101
    rng = np.random.default_rng(offset)
    nq, nk, nv = h * d, g * d, g * dv
    x, bias = _t(rng, dtype, n, nq + nk + nv), _t(rng, dtype, nq + nk + nv)
    table = rng.permutation(np.arange(1, 40))
    slots = np.array([table[(j + offset) // bs] * bs + (j + offset) % bs for j in range(n)], dtype=np.int32)
    first = _t(rng, dtype, n, nv)
    w = torch.ones(nq if whole else d, dtype=dtype, device=device)
    v0 = _d(x)[:, nq + nk:] + _d(bias)[nq + nk:]
    for mix, want in ((None, v0), (sm.ValueMix(first.to(device), 0.25), 0.75 * v0 + 0.25 * _d(first)),
                      (sm.ValueMix(torch.zeros(n, nv, dtype=dtype, device=device)), v0)):
        kc = torch.zeros(40, g, bs, d, dtype=dtype, device=device)
        vc = torch.zeros(40, g, dv, bs, dtype=dtype, device=device)
        si = torch.from_numpy(slots).to(device)
        pi = torch.arange(n, dtype=torch.int32, device=device)
        f = sm.rotary_frequencies(8, 100.0).to(device)
        fn = (lambda **k: sm.rownorm_rope(x.to(device), 0, w, w, f, 1e-6, kc, vc, si, pi, h, g, d, dv, **k)) if whole else (
            lambda **k: sm.head_norm_rope(x.to(device), 0, w, w, None, 1e-6, kc, vc, si, pi, h, g, d, dv, **k))
        fn(bias=bias.to(device), v_mix=mix)
        got = _d(vc)[slots // bs, :, :, slots % bs].reshape(n, nv)
        np.testing.assert_allclose(got, want, atol=_atol(dtype, 2e-6, 3e-2))
        assert np.count_nonzero(_d(vc)) == np.count_nonzero(got)                      # nothing beside the slots
        if mix is not None and mix.lam is None:
            np.testing.assert_array_equal(_d(mix.first), got)


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("shape", [(4, 2, 24, 16, 16, 20, 3), (6, 3, 64, 40, 32, 33, 40), (3, 1, 12, 9, 16, 1, 1), (20, 1, 128, 128, 32, 64, 6),
                                   (2, 2, 40, 136, 32, 31, 0), (4, 4, 256, 64, 32, 100, 32), (2, 1, 16, 16, 8, 5, 200)])
@pytest.mark.parametrize("biased", [False, True])
def test_windows_with_kept_first_tokens(target, shape, biased):
    """A window beside which the first tokens stay visible, each key once, at its true distance.  (a) Random inputs:
    whole sequence, a late portion, decoded tokens around every edge.  (b) One key stands out so that it owns the row if
    it is visible: the oldest key inside the window and the next older one, the last kept token and the one after
    it -- in a prompt and decoded, while the window still covers the kept tokens and far beyond them."""
    device, dtype = _dev(target)
    h, g, d, dv, bs, size, keep = shape
    rng = np.random.default_rng(h * d + size)
    n, scale, nb, rows, far = 170, 0.15, 40, 8, 50
    q, k, v = (rng.standard_normal((n, a, b)).astype(np.float32) for a, b in ((h, d), (g, d), (g, dv)))
    rel = rng.standard_normal((rows, h)).astype(np.float32)
    table = list(rng.permutation(np.arange(1, nb))[:-(-n // bs)])
    T = lambda a: torch.from_numpy(a).to(dtype)
    bt = torch.tensor([table], dtype=torch.int32, device=device)
    tol = _atol(dtype)
    kk, vv, qq = T(k), T(v), T(q)
    bias = np.stack([rel[O.bucket(m, rows, far)] for m in range(n)]).astype(np.float64) if biased else None

    def run(qx, caches, lo, p, decode):
        kw = {"bias": sm.distance_bias_table(torch.from_numpy(rel).to(device), far)} if biased else {}
        return sm.window_attention(qx[lo:p + 1].contiguous().to(device), *caches, bt, _sb([(lo, p + 1 - lo)], device), size, scale,
                                   num_decode=None if decode else 0, max_ctx=p + 1, keep_first=keep, **kw).float().cpu().numpy()
    caches = _paged(kk, vv, table, nb, bs, dtype, device)
    w = O.softmax_attention(_d(qq), _d(kk), _d(vv), scale, lambda i: O.window_keys(i, size, keep), bias=bias)
    np.testing.assert_allclose(run(qq, caches, 0, n - 1, False), w, rtol=tol, atol=tol)
    np.testing.assert_allclose(run(qq, caches, 101, n - 1, False), w[101:], rtol=tol, atol=tol)
    edges = {0, 1, keep - 1, keep, keep + 1, size - 1, size, size + 1, size + keep - 1, size + keep, n - 1}
    for p in sorted(p for p in edges if 0 <= p < n):
        np.testing.assert_allclose(run(qq, caches, p, p, True), w[p:p + 1], rtol=tol, atol=tol)
    # (b)
    for p in sorted({n - 1, min(n - 1, size + keep), min(n - 1, size)}):
        for j in sorted({p - size + 1, p - size, keep - 1, keep, 0}):
            if not 0 <= j <= p:
                continue
            k2, q2 = k.copy() * 0.1, q.copy() * 0.1
            k2[j], q2[p] = 0.0, 0.0
            k2[j, :, 1], q2[p, :, 1] = 16.0, 16.0
            c2 = _paged(T(k2), vv, table, nb, bs, dtype, device)
            seen = p - j < size or j < keep
            assert seen == (j in O.window_keys(p, size, keep))
            for lo, decode in ((max(0, p - 3), False), (p, True)):
                got = run(T(q2), c2, lo, p, decode)[-1]
                dist = np.abs(got - _d(vv)[j].repeat(h // g, 0)).max()
                assert (dist < 3e-2) == seen, (p, j, decode, dist)


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("decode", [False, True])
def test_kept_tokens_far_behind_a_long_context(target, decode):
    """A kept token 1600 positions back owns the row (key runs on separate workgroups when decoded); the token after the
    kept ones does not; a huge negative bias in the last bucket, its true distance, takes it away."""
    device, dtype = _dev(target)
    h, g, d, bs, n, keep = 4, 1, 32, 32, 1620, 5
    rng = np.random.default_rng(1)
    for j, last, owned in ((4, 1.0, True), (5, 1.0, False), (0, 1.0, True), (4, -80.0, False)):
        q, k, v = (torch.from_numpy(rng.standard_normal(s).astype(np.float32) * f).to(dtype)
                   for s, f in (((n, h, d), 0.1), ((n, g, d), 0.1), ((n, g, d), 1.0)))
        k[j], q[n - 1] = 0.0, 0.0
        k[j, :, 3], q[n - 1, :, 3] = 12.0, 12.0
        table = list(rng.permutation(np.arange(1, 60))[:-(-n // bs)])
        caches = _paged(k, v, table, 60, bs, dtype, device)
        bt = torch.tensor([table], dtype=torch.int32, device=device)
        rel = torch.zeros(8, h)
        rel[7] = last
        lo = n - 1 if decode else n - 40
        o = sm.window_attention(q[lo:].contiguous().to(device), *caches, bt, _sb([(lo, n - lo)], device), 900, 0.3,
                                num_decode=None if decode else 0, bias=sm.distance_bias_table(rel, 64).to(device), max_ctx=n,
                                keep_first=keep)
        dist = (o[-1].float().cpu() - v[j].float()).abs().max().item()
        assert (dist < 2e-2) == owned, (j, last, dist)


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("shape", [(4, 2, 24, 16, 16, 20), (3, 3, 64, 48, 32, 37), (2, 1, 12, 9, 16, 1), (20, 4, 128, 128, 32, 64),
                                   (6, 1, 40, 136, 32, 31)])
def test_chunks_with_caps_sinks_and_head_gates(target, shape):
    """Capped scores inside fixed chunks counted from position 0, an uncapped sink, one sigmoid gate per head from
    columns of a wider projection.  (a) Random inputs: whole sequence, a portion cut inside a chunk, decoded tokens at
    both sides of a border.  (b) A key that stands out: a chunk's first position shows, the one before it does not.
    (c) A sink that stands out is not capped; closed gates close."""
    device, dtype = _dev(target)
    h, g, d, dv, bs, size = shape
    rng = np.random.default_rng(h * d + size)
    n, scale, nb, cap, col = 130, 0.4, 40, 6.0, 8
    q, k, v = (rng.standard_normal((n, a, b)).astype(np.float32) for a, b in ((h, d), (g, d), (g, dv)))
    sink = rng.standard_normal(h).astype(np.float32)
    gate = _t(rng, dtype, n, col + h + 3, scale=2.0)
    table = list(rng.permutation(np.arange(1, nb))[:-(-n // bs)])
    T = lambda a: torch.from_numpy(a).to(dtype)
    bt = torch.tensor([table], dtype=torch.int32, device=device)
    tol = _atol(dtype)
    kk, vv, qq = T(k), T(v), T(q)

    def run(qx, caches, lo, p, decode, sk=sink, gt=gate):
        return sm.window_attention(qx[lo:p + 1].contiguous().to(device), *caches, bt, _sb([(lo, p + 1 - lo)], device), 1 << 30,
                                   scale, num_decode=None if decode else 0, max_ctx=p + 1, chunk=size, softcap=cap,
                                   sinks=torch.from_numpy(sk).to(device), gate=gt[lo:p + 1].contiguous().to(device),
                                   gate_col=col).float().cpu().numpy()
    caches = _paged(kk, vv, table, nb, bs, dtype, device)
    w = O.softmax_attention(_d(qq), _d(kk), _d(vv), scale, lambda i: O.chunk_keys(i, size), cap=cap, sink=sink.astype(np.float64))
    w = w * O.sigmoid(_d(gate)[:, col:col + h])[:, :, None]
    np.testing.assert_allclose(run(qq, caches, 0, n - 1, False), w, rtol=tol, atol=tol)
    np.testing.assert_allclose(run(qq, caches, 77, n - 1, False), w[77:], rtol=tol, atol=tol)
    for p in sorted({0, 1, size - 1, size, size + 1, 2 * size - 1, 2 * size, n - 1} & set(range(n))):
        np.testing.assert_allclose(run(qq, caches, p, p, True), w[p:p + 1], rtol=tol, atol=tol)
    opened = torch.full_like(gate, 60.0)
    low = np.full(h, -60.0, dtype=np.float32)
    for p in sorted({size, 2 * size - 1, n - 1} & set(range(n))):
        start = p - p % size
        for j in (start, start - 1):
            if j < 0:
                continue
            k2, q2 = k * 0.0, q * 0.0
            k2[j, :, 1], q2[p, :, 1] = 30.0, 30.0
            c2 = _paged(T(k2), vv, table, nb, bs, dtype, device)
            ref = O.softmax_attention(_d(T(q2))[:p + 1], _d(T(k2)), _d(vv), scale, lambda i: O.chunk_keys(i, size), cap=cap, sink=low)[p]
            hid = _d(vv)[start:p + 1].mean(0).repeat(h // g, 0)
            assert (np.abs(ref - hid).max() < 1e-9) == (j < start or p == start)
            for lo, decode in ((max(0, p - 3), False), (p, True)):
                np.testing.assert_allclose(run(T(q2), c2, lo, p, decode, low, opened)[-1], ref, rtol=tol, atol=tol)
    big = np.full(h, 60.0, dtype=np.float32)
    assert np.abs(run(qq, caches, n - 1, n - 1, True, big, opened)).max() < 1e-6
    assert np.abs(run(qq, caches, n - 4, n - 1, False, sink, -opened)).max() < 1e-6
    assert np.abs(run(qq, caches, n - 1, n - 1, True, sink, -opened)).max() < 1e-6


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("sizes", [(4, 16, 8, 24, 40, 20), (2, 32, 32, 64, 96, 33), (3, 10, 6, 7, 11, 9), (1, 24, 16, 40, 64, 1),
                                   (6, 128, 64, 128, 192, 70)])
def test_latent_attention_without_a_query_latent(target, sizes):
    """The whole mixer: queries, latent, shared key part and element gates from one projection, half-split rotation of
    the queries' last dimensions and the key part, a sliding window, a sink -- whole, in portions (short and long ones
    take different kernels) and decoded."""
    device, dtype = _dev(target)
    h, d, dr, dv, r, size = sizes
    rng = np.random.default_rng(d + r)
    n, width, bs, nb, eps = 150, 64, 32, 12, 1e-4
    sp = lat.LatentSpec(heads=h, dim=d, vdim=dv, rank=r, q_rank=0, scale=(d + dr) ** -0.5, rot_dim=dr, gated=True,
                        gate_elements=True, rot_half=True)
    w = {"q": _t(rng, dtype, sp.q_cols, width, scale=0.3), "dkv": _t(rng, dtype, r + dr, width, scale=0.2),
         "dkv.norm": _t(rng, dtype, r, scale=0.3, off=1.0), "uk": _t(rng, dtype, h * d, r, scale=r ** -0.5),
         "uv": _t(rng, dtype, h * dv, r, scale=r ** -0.5), "sink": _t(rng, torch.float32, h), "g": _t(rng, dtype, h * dv, width, scale=0.3),
         "o": _t(rng, dtype, width, h * dv, scale=(h * dv) ** -0.5)}
    x = _t(rng, dtype, n, width)
    m = {"heads": h, "dim": d, "rot_dim": dr, "vdim": dv, "kv_rank": r, "scale": sp.scale, "mask": {"size": size},
         "rot": {"base": 1000.0, "dims": dr}}
    want = O.latent_attention(_d(x), {k: _d(v) for k, v in w.items()}, m, eps)
    assert sp.down_width == sp.q_cols + r + dr + h * dv
    down = torch.cat([w["q"], w["dkv"], w["g"]], 0)
    down = torch.cat([down, torch.zeros(-down.shape[0] % 16, width, dtype=dtype)], 0)
    ww = {"down": down, "c_norm": w["dkv.norm"], "uk": w["uk"].view(h, d, r), "uv_t": w["uv"].view(h, dv, r).transpose(1, 2).contiguous(),
          "o": w["o"], "sinks": w["sink"]}
    ww = {k: v.to(device) for k, v in ww.items()}
    freqs = sm.rotary_frequencies(dr, 1000.0).to(device)
    table = rng.permutation(np.arange(1, nb))[:-(-n // bs)]
    bt = torch.tensor([table.tolist()], dtype=torch.int32, device=device)
    for sizes_ in ([150], [66, 1, 1, 70, 2, 1, 9], [2, 3, 1, 31, 33, 64, 16]):
        kc = torch.zeros(nb, 1, bs, r + dr, dtype=dtype, device=device)
        vc = torch.zeros(nb, 1, r, bs, dtype=dtype, device=device)
        at, got = 0, []
        for c in sizes_:
            slots = torch.tensor([table[j // bs] * bs + j % bs for j in range(at, at + c)], dtype=torch.int32, device=device)
            got.append(_d(lat.latent_attention(x[at:at + c].to(device), ww, sp, freqs, eps, kc, vc, slots, bt, _sb([(at, c)], device),
                                               num_decode=1 if c == 1 and at else 0, window=size, max_ctx=at + c)))
            at += c
        assert at == n
        np.testing.assert_allclose(np.concatenate(got), want, rtol=0, atol=_atol(dtype, 3e-5, 4e-2) * np.abs(want).max())


@pytest.mark.parametrize("target", TARGETS)
def test_half_split_rotation_far_out(target):
    """Rotated query and key parts at far positions, 4 of 6 dimensions turning in pairs (i, i + 2)."""
    device, dtype = _dev(target)
    sp = lat.LatentSpec(heads=2, dim=4, vdim=4, rank=8, q_rank=0, scale=1.0, rot_dim=6, rot_half=True)
    freqs = sm.rotary_frequencies(4, 10000.0).to(device)
    rng = np.random.default_rng(0)
    pos = np.array([0, 1, 31, 4097, 60001], dtype=np.int32)
    n = len(pos)
    down = _t(rng, dtype, n, sp.gate_col)
    pt = torch.from_numpy(pos).to(device)
    kc = torch.zeros(1, 1, 8, 14, dtype=dtype, device=device)
    vc = torch.zeros(1, 1, 8, 8, dtype=dtype, device=device)
    one = torch.ones(8, dtype=dtype, device=device)
    dd = down.to(device)
    assert lat.latent_prep(dd, sp, None, one, freqs, 1e-6, kc, vc, torch.arange(n, dtype=torch.int32, device=device), pt) is None
    uk = _t(rng, dtype, 2, 4, 8)
    many = [lat.latent_queries(dd[:, :20], uk.to(device), sp, freqs, pt),
            lat.latent_queries(dd[:, :20].repeat(20, 1), uk.to(device), sp, freqs, pt.repeat(20))[-n:]]     # both kernels
    rot = {"base": 10000.0, "dims": 4}
    for t in range(n):
        tol = _atol(dtype, 2e-5, 3e-2) + 4 * (4e-3 * pos[t] / 6e4 + 1e-5)       # float32 angles
        q = _d(down)[t:t + 1, :20].reshape(1, 2, 10)
        for qf in many:
            np.testing.assert_allclose(_d(qf)[t, :, 8:], O.rotate_halves(q[:, :, 4:], rot, first_pos=int(pos[t]))[0], atol=tol)
            np.testing.assert_allclose(_d(qf)[t, :, :8], np.einsum("hd,hdr->hr", q[0, :, :4], _d(uk)), atol=_atol(dtype, 2e-5, 6e-2))
        k = O.rotate_halves(_d(down)[t:t + 1, None, 28:34], rot, first_pos=int(pos[t]))[0, 0]
        np.testing.assert_allclose(_d(kc)[0, 0, t, 8:], k, atol=tol)


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("tokens,width,ff", [(1, 256, 128), (3, 72, 24), (5, 64, 33), (33, 512, 1024), (200, 2048, 256), (700, 256, 256),
                                             (8192, 128, 1024)])
def test_gelu_glu(target, tokens, width, ff):
    """The gated unit with the tanh form of gelu: decode sizes (in the split-K reduction), prompt sizes (in the persistent
    GEMM's epilogue) and sizes that take neither; gates far out on both sides."""
    device, dtype = _dev(target)
    rng = np.random.default_rng(ff)
    x, w = _t(rng, dtype, tokens, width), _t(rng, dtype, 2 * ff, width, scale=2.0 * width ** -0.5)
    x[0] *= 12.0
    got = _d(sm.linear_gelu_glu(x.to(device), w.to(device)))
    rows = np.unique(np.linspace(0, tokens - 1, 80).astype(int))
    g, u = _d(x)[rows] @ _d(w)[:ff].T, _d(x)[rows] @ _d(w)[ff:].T
    want = O.gelu_tanh(g) * u
    tol = 1e-5 if dtype == torch.float32 else 2e-2
    size = np.abs(g).max(-1, keepdims=True) * np.abs(u).max(-1, keepdims=True)      # of a row's products
    assert (np.abs(got[rows] - want) <= tol * size).all()
    assert g.min() < -8 and g.max() > 8
    erf = torch.nn.functional.gelu(torch.from_numpy(g)).numpy() * u
    assert np.abs(erf - want).max() > 2e-4                     # the erf form is another function


# ------------------------------------------------------------------------------ the engine
@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("name", ["a", "b", "c"])
def test_whole_prompts_and_layers(target, name, tmp_path):
    """Whole prompts in one step, alone and three at once; the residual stream after every layer against the oracle's."""
    cfg = CONFIGS[name]()
    sd = _round(O.make_weights(cfg, seed=3), target[1])
    eng = make_engine(cfg, sd, target, tmp_path)
    p = prompts_for(cfg, [130, 1, 30], seed=5)
    taps = []
    want = {n: O.forward(cfg, _np(sd), t, taps if n == "r2" else None) for n, t in p.items()}
    eng.runner.stage.taps = got_taps = []
    got = replay(eng, [[("r2", 30)]], {"r2": p["r2"]})
    eng.runner.stage.taps = None
    assert len(got_taps) == len(taps) == len(cfg["layers"])
    if target[1] == torch.float32:
        for a, b in zip(got_taps, taps):
            np.testing.assert_allclose(a.cpu().numpy(), b, atol=2e-4 * max(1.0, np.abs(b).max()))
    assert_close(got["r2"], want["r2"], target, "alone")
    got = replay(eng, [[("r0", 130), ("r1", 1), ("r2", 30)]], p)
    for n in p:
        assert_close(got[n], want[n], target, n)


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("name", ["a", "b", "c"])
def test_decode_and_portions_match_the_whole(target, name, tmp_path):
    """Token-by-token decoding after a prompt (110 steps over several blocks, windows and chunks), portions of changing
    sizes down to two tokens and one, and decoding from the very first token."""
    cfg = CONFIGS[name]()
    sd = _round(O.make_weights(cfg, seed=4), target[1])
    eng = make_engine(cfg, sd, target, tmp_path)
    p = prompts_for(cfg, [150], seed=7)
    want = O.forward(cfg, _np(sd), p["r0"])
    got = replay(eng, [[("r0", 40)]] + [[("r0", 1)]] * 110, p)
    assert_close(got["r0"], want, target, "decode")
    sizes = [2, 3, 1, 31, 2, 33, 5, 64, 2, 7]
    assert sum(sizes) == 150
    got = replay(eng, [[("r0", s)] for s in sizes], p)
    assert_close(got["r0"], want, target, "portions")
    got = replay(eng, [[("r0", 2)]] * 75, p)
    assert_close(got["r0"], want, target, "two at a time")
    got = replay(eng, [[("r0", 1)]] * 60, {"r0": p["r0"][:60]})
    assert_close(got["r0"], want[:60], target, "from the first token")


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("block_size", [16, 64])
def test_mixed_batches_and_reused_blocks(target, block_size, tmp_path):
    """Up to four unequal requests per step, portions beside single tokens; finished requests give their blocks to new
    ones (a pool sized for the live tokens only).  Every request matches its own whole-sequence oracle: the batch and
    the pool do not show."""
    cfg = cfg_a()
    sd = _round(O.make_weights(cfg, seed=5), target[1])
    eng = make_engine(cfg, sd, target, tmp_path, max_tokens=384, max_requests=4, block_size=block_size)
    prompts = prompts_for(cfg, [90, 9, 33, 64, 20, 70, 3], seed=9)
    at = {n: 0 for n in prompts}
    waiting, live, schedule = list(prompts), [], []
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
    for n in prompts:
        assert_close(got[n], O.forward(cfg, _np(sd), prompts[n]), target, n)


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("name,graphs", [("a", False), ("c", True)])
def test_greedy_generation_through_the_scheduler(target, name, graphs, tmp_path):
    """LLMEngine.generate (scheduler, continuous batching, sampler, decode steps replayed from HIP graphs) on three
    prompts at once: every generated token is the argmax of the oracle's logits for the sequence so far (where the
    oracle's top two are not within rounding of each other)."""
    cfg = CONFIGS[name]()
    sd = _round(O.make_weights(cfg, seed=6), target[1])
    eng = make_engine(cfg, sd, target, tmp_path, graphs=graphs)
    prompts = list(prompts_for(cfg, [5, 60, 17], seed=11).values())
    outs = eng.generate(prompts, SamplingParams(max_new_tokens=24, ignore_eos=True))
    checked = 0
    for p, o in zip(prompts, outs):
        assert len(o) == 24
        logits = O.forward(cfg, _np(sd), p + o)
        for i, tok in enumerate(o):
            row = logits[len(p) + i - 1]
            top = np.sort(row)[-2:]
            if top[1] - top[0] > (1e-3 if target[1] == torch.float32 else 0.15) * row.std():
                checked += 1
                assert tok == int(row.argmax()), (i, float(top[1] - top[0]))
    assert checked > 36


def random_config(seed):
    """A model whose every size is drawn: widths, head counts and groupings, key / value sizes, rotated parts, windows,
    chunks, kept tokens, bias tables, caps, latents, who shares values, layer count and order."""
    rng = np.random.default_rng(4000 + seed)
    pick = lambda xs: xs[int(rng.integers(len(xs)))]
    layers = []
    shared = pick([12, 24, 32, 64, 96])                  # kv_heads * vdim of the layers that share values
    for _ in range(int(rng.integers(2, 6))):
        kind = pick(["attention", "attention_2", "latent_attention"])
        ff = pick([0, 16, 40, 128, 256])
        scale = float(rng.uniform(0.05, 0.4))
        if kind == "latent_attention":
            layers.append(_lat(pick([1, 2, 3, 8]), pick([8, 12, 16, 32, 64]), pick([2, 8, 16, 32]), pick([8, 12, 24, 80]),
                               pick([16, 20, 40, 64, 128]), scale, pick([1, 7, 32, 45, 100]), ff, base=float(pick([100.0, 1e4, 5e5]))))
            continue
        mix = bool(rng.random() < 0.7)
        g = pick([1, 2, 4]) if mix else pick([1, 2, 3])
        dv = shared // g if mix else pick([8, 12, 24, 64, 128])
        hh, d = g * pick([1, 2, 3, 4]), pick([8, 16, 20, 32, 40, 64, 80, 128])
        if kind == "attention":
            rows = pick([2, 4, 8, 10, 32])
            layers.append(_attn(hh, g, d, dv, scale, pick([1, 8, 31, 50, 96]), pick([0, 1, 4, 33]), rows // 2 + pick([1, 7, 50, 300]), rows,
                                ff, v_mix=mix))
        else:
            layers.append(_two(hh, g, d, dv, scale, pick([1, 16, 30, 64, 200]), float(pick([3.0, 20.0, 50.0])),
                               pick([r for r in (2, 4, 8, 16, 20, 64, 128) if r <= d]), ff, base=float(pick([100.0, 1e4, 1e6])),
                               factor=pick([None, 2.0, 10.0]), v_mix=mix))
    return _model(pick([97, 128, 200, 333]), pick([64, 70, 96, 128, 160, 256]), layers, scale=float(pick([0.25, 1.0, 8.0])),
                  eps=pick([1e-6, 1e-5, 1e-4]))


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("seed", range(10))
def test_drawn_models_on_a_mixed_schedule(target, seed, tmp_path):
    """Models of drawn sizes: three unequal requests, portions of changing size beside single tokens, a fourth request
    that takes over freed blocks; each equals its whole-sequence oracle."""
    cfg = random_config(seed)
    sd = _round(O.make_weights(cfg, seed=0), target[1])
    eng = make_engine(cfg, sd, target, tmp_path, max_tokens=320, max_requests=3)
    prompts = prompts_for(cfg, [75, 18, 110, 40], seed=seed)
    schedule = [[("r0", 33), ("r1", 2)], [("r0", 1), ("r1", 16), ("r2", 64)], [("r0", 1), ("r2", 3)], [("r0", 30), ("r2", 1)],
                [("r2", 2), ("r0", 1)], [("r0", 9), ("r2", 39), ("r3", 7)], [("r3", 1), ("r2", 1)], [("r3", 32)]]
    got = replay(eng, schedule, prompts)
    assert eng.bm.num_free() == eng.bm.num_blocks - 1
    for n, p in prompts.items():
        assert_close(got[n], O.forward(cfg, _np(sd), p), target, (seed, n))


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("case", ["latent only", "one sharing layer", "chunked layers first and last"])
def test_unusual_layer_orders(target, case, tmp_path):
    """Models without any sharing layer, with one that has no partner, and with the sharing layers far apart."""
    if case == "latent only":
        cfg = _model(101, 64, [_lat(2, 16, 8, 8, 24, 0.3, 30, 32), _lat(1, 8, 2, 24, 16, 0.4, 7)])
    elif case == "one sharing layer":
        cfg = _model(101, 64, [_two(2, 1, 16, 8, 0.3, 16, 9.0, 8, 32, v_mix=False), _attn(2, 2, 8, 8, 0.3, 12, 2, 30, 8, 16),
                               _two(2, 2, 8, 16, 0.3, 50, 9.0, 8, v_mix=False)])
    else:
        cfg = _model(101, 64, [_two(2, 1, 16, 16, 0.3, 16, 9.0, 8), _lat(2, 16, 8, 8, 24, 0.3, 30, 32),
                               _attn(2, 2, 8, 24, 0.3, 12, 2, 30, 8, 16, v_mix=False), _two(4, 2, 8, 8, 0.3, 20, 9.0, 8, 16)])
    sd = _round(O.make_weights(cfg, seed=1), target[1])
    eng = make_engine(cfg, sd, target, tmp_path, max_tokens=256, max_requests=3)
    p = prompts_for(cfg, [70, 33], seed=2)
    got = replay(eng, [[("r0", 40), ("r1", 2)], [("r0", 1), ("r1", 31)], [("r0", 29)]], p)
    for n in p:
        assert_close(got[n], O.forward(cfg, _np(sd), p[n]), target, (case, n))


def test_shared_values_show_in_the_logits():
    """The oracle itself: the blend, and whose values enter it, are far above the tests' bounds."""
    cfg = cfg_a()
    sd = O.make_weights(cfg, seed=3)
    toks = prompts_for(cfg, [60])["r0"]
    want = O.forward(cfg, sd, toks)
    for name in ("l2.mix.vmix", "l4.mix.vmix", "l6.mix.vmix"):
        assert row_errs(O.forward(cfg, dict(sd, **{name: sd[name] + 0.1}), toks), want).max() > 5e-3
    first = dict(sd, **{"l1.mix.vmix": sd["l1.mix.vmix"] + 0.1})          # the first sharing layer's weight is not used
    assert row_errs(O.forward(cfg, first, toks), want).max() == 0.0


def test_config_round_trip_and_registry(tmp_path):
    from distributed_llms_amd.config import get_model_config
    from distributed_llms_amd.models.basopel import BasopelStage, model_shapes
    cfg = cfg_a()
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    m = get_model_config(str(tmp_path))
    assert m.arch == "basopel" and m.num_layers == 7 and m.hidden_size == 96 and m.embed_scale == 5.0 and m.tie_embeddings
    assert m.needs_seq_index and not m.needs_state_slots
    back = ModelConfig.from_hf_config(m.to_hf_config())
    assert (back.layers, back.norm_eps, back.embed_scale) == (m.layers, m.norm_eps, 5.0)
    st = make_stage(m)
    assert isinstance(st, BasopelStage) and st.num_layers == 7
    sd = O.make_weights(cfg)
    assert {k: tuple(v.shape) for k, v in sd.items()} == model_shapes(m, {k: torch.from_numpy(v) for k, v in sd.items()})
    per_token = sum(torch.Size(a).numel() + torch.Size(b).numel() for a, b in st.cache_shapes(1).values())
    assert m.kv_bytes_per_token(2) == 2 * per_token
    for bad in ({"type": "lightning"}, {"mlp": {"kind": "moe", "ff": 8}}):
        c = cfg_a()
        c["layers"][0].update(bad)
        with pytest.raises(ValueError):
            ModelConfig.from_hf_config(c)
    for i, path, val in ((2, "rot.dims", 32), (0, "rot.dims", 10), (1, "kv_heads", 4), (1, "mask.size", 0), (6, "vdim", 16)):
        c = cfg_a()
        d = c["layers"][i]["mixer"]
        *head, leaf = path.split(".")
        for k in head:
            d = d[k]
        d[leaf] = val
        with pytest.raises(ValueError):
            make_stage(ModelConfig.from_hf_config(c))
    short = {k: torch.from_numpy(v) for k, v in sd.items() if k != "l3.mix.o.b"}
    with pytest.raises(KeyError):
        make_stage(m).load_hf_state(short)
    assert get_model_config("tiny-basopel").arch == "basopel"
    make_stage(get_model_config("tiny-basopel")).init_synthetic(0)


@pytest.mark.parametrize("target", [t for t in TARGETS if "gpu" in t.id])
def test_decode_graphs_replay_like_eager_steps(target, tmp_path):
    """Decode steps replayed from captured HIP graphs (several replays, eager prompt steps and synchronisations between
    them) give the logits of eager decode steps."""
    cfg = cfg_c()
    sd = _round(O.make_weights(cfg, seed=8), target[1])
    p = prompts_for(cfg, [60, 53], seed=3)
    sched = [[("r0", 45), ("r1", 38)]] + [[("r0", 1), ("r1", 1)]] * 7 + [[("r0", 3), ("r1", 2)]] + [[("r0", 1), ("r1", 1)]] * 5
    eager = replay(make_engine(cfg, sd, target, tmp_path, graphs=False), sched, p)
    eng = make_engine(cfg, sd, target, tmp_path, graphs=True)
    assert eng.runner.graphs is not None
    graphed = replay(eng, sched, p)
    for n in p:
        np.testing.assert_allclose(graphed[n], eager[n], rtol=1e-3, atol=1e-3)


def test_trace_run_program_loads_a_model_folder(tmp_path):
    """bin/trace_run on a folder with config.json + model.safetensors (bfloat16): the registry picks the stage by the
    config, the checkpoint loader reads the tensors (a bias table's rows from its shape), steps with portions beside
    single tokens answer with the wanted logits (CPU path, float32)."""
    import os
    import subprocess
    import sys
    from safetensors.torch import save_file
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    cfg = cfg_a()
    sd = {k: torch.from_numpy(v).to(torch.bfloat16) for k, v in O.make_weights(cfg, seed=21).items()}
    for l in cfg["layers"]:                      # a model folder names no row count: the tensors do
        l["mixer"].pop("rows", None)
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
    ref = {n: O.forward(cfg, f64, t) for n, t in toks.items()}
    got = {i: np.fromfile(out / f"{i}.f32", dtype="<f4").reshape(-1, cfg["vocab"]) for i in (0, 1, 3)}
    assert row_errs(got[0], ref["a"][[0, 29]]).max() < 1e-4
    assert row_errs(got[1], np.stack([ref["a"][30], ref["b"][19]])).max() < 1e-4
    assert row_errs(got[3], ref["a"][[49]]).max() < 1e-4
