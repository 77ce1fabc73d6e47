"""A plain, slow float64 implementation of the Basopel decoder, one function per mechanism, written from the model's
equations and sharing no code with distributed_llms_amd: whole sequences only, Python loops, no cache, no batching.
The tests compare the engine against it.

The model: layer norms (weight and bias) before and after every sublayer around a residual stream; three kinds of
token mixer -- "attention" (biased projections, per-head query / key norms, a learned bias per distance bucket, a
sliding window beside which the first tokens stay visible), "latent_attention" (keys and values are up-projections
of one small normed vector per token, a rotated key part common to all heads, a sliding window, a sink, an
elementwise output gate) and "attention_2" (biased projections, norms over the whole query / key projections, a
half-split rotation with divided frequencies, capped scores inside fixed chunks of positions, a sink, a gate per
head); in layers that ask for it the values are blended with those of the first such layer.  Feed-forward: a gated
unit with the tanh form of gelu.  The output projection is the embedding table.

Checkpoint names: embed, final.norm, final.norm.b, l<i>.norm1|norm1b|norm2|norm2b (each with a '.b'), l<i>.mix.*,
l<i>.mlp.gate|up|down.  Linear weights are [out, in].
"""
import math

import numpy as np


def rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps)


def layer_norm(x, w, b, eps):
    c = x - x.mean(-1, keepdims=True)
    return c / np.sqrt((c * c).mean(-1, keepdims=True) + eps) * w + b


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def sub(w, prefix):
    """The tensors under ``prefix`` with the prefix taken off."""
    return {k[len(prefix):]: v for k, v in w.items() if k.startswith(prefix)}


def rotate_halves(x, rot, first_pos=0):
    """x [T, heads, D]: dimension i < dims / 2 turns with dimension i + dims / 2 by p base^(-2i / dims) / factor."""
    out = x.copy()
    n = rot["dims"] // 2
    factor = (rot.get("scaling") or {}).get("factor", 1.0)
    p = (first_pos + np.arange(x.shape[0]))[:, None]
    for i in range(n):
        a = p * (rot["base"] ** (-2.0 * i / rot["dims"]) / factor)
        u, v = x[:, :, i], x[:, :, i + n]
        out[:, :, i] = u * np.cos(a) - v * np.sin(a)
        out[:, :, i + n] = v * np.cos(a) + u * np.sin(a)
    return out


def bucket(n, rows, far):
    """Row of the distance-bias table for a key ``n`` positions back: one row per distance up to half the
    table, then rows whose width grows geometrically until ``far``; everything beyond shares the last row."""
    half = rows // 2
    if n < half:
        return n
    return min(rows - 1, half + math.floor(math.log(n / half) / math.log(far / half) * (rows - half)))


# ------------------------------------------------------------------------------ which keys a query sees
def window_keys(i, size, keep=0):
    """Keys of position i: the last ``size`` positions and the first ``keep`` of the sequence."""
    return [j for j in range(i + 1) if i - j < size or j < keep]


def chunk_keys(i, size):
    return [j for j in range(i + 1) if j // size == i // size]


def softmax_attention(q, k, v, scale, keys, cap=0.0, bias=None, sink=None):
    """q [T, H, D], k [T, G, D], v [T, G, Dv]; ``keys(i)``: the positions that query i sees; ``bias`` [T, H]: added to
    the scaled score of a key n positions back; ``cap``: s <- cap tanh(s / cap); ``sink`` [H]: exp(sink) joins the
    denominator."""
    t, hh, _ = q.shape
    rep = hh // k.shape[1]
    out = np.zeros((t, hh, v.shape[2]))
    for i in range(t):
        js = np.array(keys(i))
        for a in range(hh):
            s = (k[js, a // rep] @ q[i, a]) * scale
            if cap:
                s = cap * np.tanh(s / cap)
            if bias is not None:
                s = s + bias[i - js, a]
            top = s.max() if sink is None else max(s.max(), sink[a])
            e = np.exp(s - top)
            den = e.sum() + (0.0 if sink is None else math.exp(sink[a] - top))
            out[i, a] = (e @ v[js, a // rep]) / den
    return out


def mix_values(v, first, lam):
    """(1 - lam) v + lam first, row by row of the value projection; ``first`` None: this is the first layer that mixes."""
    return v if first is None else (1.0 - lam) * v + lam * first.reshape(v.shape)


# ------------------------------------------------------------------------------ mixers
def attention(h, w, m, eps, v_first=None):
    """Returns (output [T, W], the layer's values [T, G, vdim] as attended)."""
    t = h.shape[0]
    hh, g, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms((h @ w["q"].T + w["q.b"]).reshape(t, hh, d), eps) * w["q.norm"]
    k = rms((h @ w["k"].T + w["k.b"]).reshape(t, g, d), eps) * w["k.norm"]
    v = (h @ w["v"].T + w["v.b"]).reshape(t, g, dv)
    if m.get("v_mix"):
        v = mix_values(v, v_first, w["vmix"])
    bias = np.stack([w["rel"][bucket(n, w["rel"].shape[0], m["bias_max"])] for n in range(t)])
    o = softmax_attention(q, k, v, m["scale"], lambda i: window_keys(i, m["mask"]["size"], m["mask"]["keep_first"]), bias=bias)
    return o.reshape(t, hh * dv) @ w["o"].T, v


def attention_2(h, w, m, eps, v_first=None):
    t = h.shape[0]
    hh, g, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rotate_halves((rms(h @ w["q"].T + w["q.b"], eps) * w["q.norm"]).reshape(t, hh, d), m["rot"])
    k = rotate_halves((rms(h @ w["k"].T + w["k.b"], eps) * w["k.norm"]).reshape(t, g, d), m["rot"])
    v = (h @ w["v"].T + w["v.b"]).reshape(t, g, dv)
    if m.get("v_mix"):
        v = mix_values(v, v_first, w["vmix"])
    o = softmax_attention(q, k, v, m["scale"], lambda i: chunk_keys(i, m["mask"]["size"]), cap=m["softcap"], sink=w["sink"])
    o = o * sigmoid(h @ w["g"].T)[:, :, None]
    return o.reshape(t, hh * dv) @ w["o"].T + w["o.b"], v


def latent_attention(h, w, m, eps):
    t = h.shape[0]
    hh, d, dr, dv, r = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    q = (h @ w["q"].T).reshape(t, hh, d + dr)
    dkv = h @ w["dkv"].T
    c = rms(dkv[:, :r], eps) * w["dkv.norm"]
    kr = rotate_halves(dkv[:, None, r:], m["rot"])
    q = np.concatenate([q[:, :, :d], rotate_halves(q[:, :, d:], m["rot"])], -1)
    k = np.concatenate([(c @ w["uk"].T).reshape(t, hh, d), np.repeat(kr, hh, 1)], -1)
    v = (c @ w["uv"].T).reshape(t, hh, dv)
    o = softmax_attention(q, k, v, m["scale"], lambda i: window_keys(i, m["mask"]["size"]), sink=w["sink"])
    return (o.reshape(t, hh * dv) * sigmoid(h @ w["g"].T)) @ w["o"].T


def feed_forward(h, w):
    return (gelu_tanh(h @ w["gate"].T) * (h @ w["up"].T)) @ w["down"].T


# ------------------------------------------------------------------------------ the model
def forward(cfg, sd, tokens, taps=None):
    """Logits [T, vocab] of one whole sequence.  ``sd``: checkpoint name -> float64 array.  ``taps``: a list that
    receives the residual stream after every layer."""
    eps = cfg["norm"]["eps"]
    x = sd["embed"][np.asarray(tokens)] * cfg["embedding"]["scale"]
    v_first = None
    for i, layer in enumerate(cfg["layers"]):
        w, m = sub(sd, f"l{i}."), layer["mixer"]
        wm = sub(w, "mix.")
        norm = lambda z, name: layer_norm(z, w[name], w[name + ".b"], eps)
        h = norm(x, "norm1")
        if layer["type"] == "latent_attention":
            o = latent_attention(h, wm, m, eps)
        else:
            o, v = (attention if layer["type"] == "attention" else attention_2)(h, wm, m, eps, v_first)
            if m.get("v_mix") and v_first is None:
                v_first = v
        x = x + norm(o, "norm1b")
        if layer.get("mlp"):
            x = x + norm(feed_forward(norm(x, "norm2"), sub(w, "mlp.")), "norm2b")
        if taps is not None:
            taps.append(x.copy())
    return layer_norm(x, sd["final.norm"], sd["final.norm.b"], eps) @ sd["embed"].T


def shapes(cfg):
    """Checkpoint name -> shape.  ``mixer.rows`` (default 8) is the row count of a distance-bias table."""
    w = cfg["width"]
    s = {"embed": (cfg["vocab"], w), "final.norm": (w,), "final.norm.b": (w,)}
    for i, layer in enumerate(cfg["layers"]):
        p, m, mlp = f"l{i}.", layer["mixer"], layer.get("mlp")
        for n in ("norm1", "norm1b") + (("norm2", "norm2b") if mlp else ()):
            s.update({p + n: (w,), p + n + ".b": (w,)})
        a, hh = p + "mix.", m["heads"]
        if layer["type"] == "latent_attention":
            s.update({a + "q": (hh * (m["dim"] + m["rot_dim"]), w), a + "dkv": (m["kv_rank"] + m["rot_dim"], w),
                      a + "dkv.norm": (m["kv_rank"],), a + "uk": (hh * m["dim"], m["kv_rank"]),
                      a + "uv": (hh * m["vdim"], m["kv_rank"]), a + "sink": (hh,), a + "g": (hh * m["vdim"], w)})
        else:
            for n, rows in (("q", hh * m["dim"]), ("k", m["kv_heads"] * m["dim"]), ("v", m["kv_heads"] * m["vdim"])):
                s.update({a + n: (rows, w), a + n + ".b": (rows,)})
            whole = layer["type"] == "attention_2"
            s.update({a + "q.norm": (hh * m["dim"] if whole else m["dim"],),
                      a + "k.norm": (m["kv_heads"] * m["dim"] if whole else m["dim"],)})
            s.update({a + "sink": (hh,), a + "g": (hh, w), a + "o.b": (w,)} if whole else {a + "rel": (m.get("rows", 8), hh)})
            if m.get("v_mix"):
                s[a + "vmix"] = ()
        s[a + "o"] = (w, hh * m["vdim"])
        if mlp:
            s.update({p + "mlp.gate": (mlp["ff"], w), p + "mlp.up": (mlp["ff"], w), p + "mlp.down": (w, mlp["ff"])})
    return s


def make_weights(cfg, seed=0):
    """Random float64 weights under the checkpoint names: projections ~ N(0, 1 / fan_in), norm weights around one,
    biases, distance biases and sinks of moderate size, values mixed about half and half."""
    rng = np.random.default_rng(seed)
    sd = {}
    for name, shape in shapes(cfg).items():
        leaf = name.rsplit(".", 1)[-1]
        if leaf in ("norm", "norm1", "norm2", "norm1b", "norm2b"):
            t = 1.0 + 0.2 * rng.standard_normal(shape)
        elif leaf == "b":
            t = 0.3 * rng.standard_normal(shape)
        elif leaf in ("rel", "sink"):
            t = rng.standard_normal(shape)
        elif leaf == "vmix":
            t = rng.uniform(0.3, 0.7)
        elif name == "embed":
            t = rng.standard_normal(shape) / shape[-1] ** 0.5
        else:
            t = rng.standard_normal(shape) / shape[-1] ** 0.5
        sd[name] = np.asarray(t, dtype=np.float64)
    return sd
