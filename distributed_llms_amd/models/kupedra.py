"""Kupedra: a pre-norm layer-list decoder whose residual state is several float32 streams (hyper-connections), with
two kinds of layer -- rotated softmax attention, and distance-biased softmax attention beside an exponentially
gated matrix memory -- mixtures of clipped-GLU experts, and a span of layers that may run several times with the
same weights.

``config.json`` keys (read by ``config._from_kupedra``): ``width``, ``vocab``, ``norm.eps``, ``embedding.scale``,
``streams``, ``logit_scale``, optionally ``loop`` (``start``, ``stop``, ``times``), and ``layers``: per layer ``type``,
``mixer``, ``mlp``.

  type "attention": ``heads``, ``kv_heads``, ``dim`` (q / k), ``vdim``, ``scale``, ``rot`` (``base``, ``dims``, optional
      ``scaling.factor`` that divides every frequency; dimensions 2i and 2i + 1 of a head turn together).  q and k are
      divided by their root mean square per head AFTER the rotation; the scores of a head are multiplied by its
      ``temp``; one is added to the softmax denominator (a sink whose score is 0).
  type "parallel": two mixers on the same input, each output RMS-normed over the model width with a weight of its
      own, then averaged.
      ``left`` -- attention: ``heads``, ``kv_heads``, ``dim``, ``vdim``, ``scale``; q and k normed per head with weights
      shared by the heads, no rotation; ``q_temp`` (``coef``, ``every``): q times 1 + coef ln(floor((p + 1) / every) + 1);
      ``bias_max``: a learned bias per bucket of distances is added to the scaled score (the table's rows come from its
      tensor); a learned sink per head.
      ``right`` -- matrix memory: ``heads``, ``dim``, ``vdim``, ``gate_cap``.  q = W_q h dim^-1/2, k, v; log gates
      i = cap tanh((W_i h + b_i) / cap), f = log_sigmoid(cap tanh((W_f h + b_f) / cap)); with the running maximum
      m <- max(f + m, i): S <- e^(f + m' - m) S + e^(i - m) k v^T, n likewise with k alone,
      o = S^T q / (max(|n.q|, e^-m) + 1e-6); o over its root mean square per head, times a weight over all heads, times
      sigmoid(W_g h), then the output projection.
  mlp: None or {"kind": "moe", "expert": {"ff", "limit"}, "router": {"experts", "top"}, "shared": {"ff", "limit"} |
      None}: clipped-GLU experts, float32 router logits, the ``top`` largest, weighted by the softmax over ALL experts
      (not renormalised); the shared expert is scaled by a sigmoid gate per token.

One layer: h = rms(sum_s in_s x_s) g, x_t <- sum_s mix[s, t] x_s + out_t mixer(h); then the same with the
feed-forward; g is one number.  The streams start as embed[token] * scale, each; the model ends with
rms(sum_s x_s) g, the head and ``logit_scale``.

Checkpoint names: ``embed``, ``final.norm``, ``head``; per layer ``l<i>.``: ``norm1``, ``norm2`` (scalars),
``hc1.in|out|mix``, ``hc2.*``; ``mix.q|k|v|temp|o`` (attention); ``mix.left.q|k|v|q.norm|k.norm|rel|sink|o|out``,
``mix.right.q|k|v|g|o|norm|i|i.b|f|f.b|out`` (parallel); ``mlp.router``, ``mlp.e<j>.gate|up|down``,
``mlp.shared.gate|up|down|sg``.  Linear weights are [out, in].

What a sequence keeps between steps, per layer RUN (a looped layer counts once per pass): paged K / V (one block
table for all, from the engine's BlockManager) and in parallel layers a state slot: the float32 matrices
[heads, vdim, dim], normalisers [heads, dim] and maxima [heads].  Streams, norms, angles, scores and softmax
weights, router logits, gates and states are float32 also when activations are bfloat16.
"""
from __future__ import annotations

from typing import Any, Dict, Optional

import torch

from .. import ops
from ..config import ModelConfig
from ..ops import hyper as hc
from ..ops import linattn as la
from ..ops import moe
from ..ops import seqmix as sm
from .hybrid import LayerListStage, layer_runs
from .stage import BatchMeta
from .weights import tensor_seed

DEFAULT_BIAS_ROWS = 32       # synthetic weights only: a checkpoint's tensors give the rows of the distance-bias table
MEMORY_EPS = 1e-6            # added to the matrix memory's divisor
PROJ_ALIGN = 16              # rows of the fused input projection are padded to a multiple of this (aligned row pieces)


def memory_spec(layer: Dict[str, Any]) -> la.MatrixMemorySpec:
    m = layer["mixer"]["right"]
    return la.MatrixMemorySpec(heads=int(m["heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]), cap=float(m["gate_cap"]),
                               den_eps=MEMORY_EPS)


def attn_mixer(layer: Dict[str, Any]) -> Dict[str, Any]:
    """The sizes of the layer's softmax attention (every layer has one)."""
    return layer["mixer"] if layer["type"] == "attention" else layer["mixer"]["left"]


def layer_shapes(width: int, streams: int, layer: Dict[str, Any], rows: Optional[int] = None) -> Dict[str, tuple]:
    """Checkpoint tensor name (without the ``l<i>.`` prefix) -> shape (``rows``: of the distance-bias table)."""
    a = attn_mixer(layer)
    p = "mix." if layer["type"] == "attention" else "mix.left."
    s: Dict[str, tuple] = {p + "q": (a["heads"] * a["dim"], width), p + "k": (a["kv_heads"] * a["dim"], width),
                           p + "v": (a["kv_heads"] * a["vdim"], width), p + "o": (width, a["heads"] * a["vdim"])}
    if layer["type"] == "attention":
        s["mix.temp"] = (a["heads"],)
    else:
        sp = memory_spec(layer)
        qk, vv = sp.heads * sp.dim, sp.heads * sp.vdim
        rows = rows or int(a.get("rows", DEFAULT_BIAS_ROWS))
        s.update({p + "q.norm": (a["dim"],), p + "k.norm": (a["dim"],), p + "rel": (rows, a["heads"]), p + "sink": (a["heads"],),
                  "mix.left.out": (width,), "mix.right.out": (width,),
                  "mix.right.q": (qk, width), "mix.right.k": (qk, width), "mix.right.v": (vv, width),
                  "mix.right.g": (vv, width), "mix.right.o": (width, vv), "mix.right.norm": (vv,),
                  "mix.right.i": (sp.heads, width), "mix.right.i.b": (sp.heads,),
                  "mix.right.f": (sp.heads, width), "mix.right.f.b": (sp.heads,)})
    mlp = layer.get("mlp")
    for q in (1, 2) if mlp else (1,):
        s.update({f"norm{q}": (), f"hc{q}.in": (streams,), f"hc{q}.out": (streams,), f"hc{q}.mix": (streams, streams)})
    if mlp:
        e, f = mlp["router"]["experts"], mlp["expert"]["ff"]
        s["mlp.router"] = (e, width)
        for j in range(e):
            s.update({f"mlp.e{j}.gate": (f, width), f"mlp.e{j}.up": (f, width), f"mlp.e{j}.down": (width, f)})
        if mlp.get("shared"):
            fs = mlp["shared"]["ff"]
            s.update({"mlp.shared.gate": (fs, width), "mlp.shared.up": (fs, width), "mlp.shared.down": (width, fs),
                      "mlp.shared.sg": (1, width)})
    return s


def model_shapes(cfg: ModelConfig, sd: Optional[Dict[str, torch.Tensor]] = None) -> Dict[str, tuple]:
    """Every checkpoint tensor's shape; with ``sd`` the distance-bias rows are read from its ``rel`` tensors."""
    w = cfg.hidden_size
    s = {"embed": (cfg.vocab_size, w), "final.norm": (), "head": (cfg.vocab_size, w)}
    for i, layer in enumerate(cfg.layers):
        rel = None if sd is None else sd.get(f"l{i}.mix.left.rel")
        rows = int(rel.shape[0]) if rel is not None and rel.dim() == 2 else None
        s.update({f"l{i}.{n}": shp for n, shp in layer_shapes(w, cfg.streams, layer, rows).items()})
    return s


def synth_state_dict(cfg: ModelConfig, seed: int = 0, dtype=torch.float32) -> Dict[str, torch.Tensor]:
    """Seeded random weights under the checkpoint names (CPU): projections ~ N(0, 1 / fan_in), norm weights and
    temperatures around one, stream mixes near the identity, forget gates that keep the memory for a while, the
    router wide enough that choices are not close calls, an embedding whose scaled rows have unit size."""
    sd = {}
    for name, shape in model_shapes(cfg).items():
        g = torch.Generator().manual_seed(tensor_seed(seed, 0, name))
        leaf = name.rsplit(".", 1)[-1]
        r = torch.randn(shape, generator=g)
        if leaf in ("norm1", "norm2", "norm", "temp") or (leaf == "out" and ".mix." in name):
            t = 1.0 + 0.2 * r
        elif leaf in ("in", "out"):
            t = (1.0 if leaf == "out" else 1.0 / shape[0]) + 0.1 * r
        elif leaf == "mix":
            t = 0.9 * torch.eye(shape[0]) + 0.1 / shape[0] * r
        elif leaf in ("sink", "rel"):
            t = r
        elif name.endswith("f.b"):
            t = 3.0 + r
        elif name.endswith("i.b"):
            t = 0.5 * r
        elif leaf == "router":
            t = 3.0 * r / shape[-1] ** 0.5
        elif name == "embed":
            t = r / cfg.embed_scale
        else:
            t = r / shape[-1] ** 0.5
        sd[name] = t.to(dtype)
    return sd


class KupedraStage(LayerListStage):
    """All layers of a Kupedra model on one device (see the module docstring)."""

    @staticmethod
    def layer_param_count(width: int, layer: Dict[str, Any]) -> int:
        return sum(int(torch.Size(s).numel()) for s in layer_shapes(width, 1, layer).values())

    @staticmethod
    def kv_elements_per_token(cfg: ModelConfig) -> int:
        """K + V elements a token adds over all layer runs."""
        ms = [attn_mixer(cfg.layers[i]) for i, _ in layer_runs(cfg)]
        return sum(m["kv_heads"] * (m["dim"] + m["vdim"]) for m in ms)

    def __init__(self, cfg: ModelConfig, layer_start: int = 0, layer_end: Optional[int] = None, device="cpu",
                 dtype=torch.bfloat16, units: Optional[tuple] = None, tp=None, unit_group: int = 2):
        super().__init__(cfg, layer_start, layer_end, device, dtype, units, tp, unit_group)
        if not 1 <= cfg.streams <= hc.MAX_STREAMS or cfg.hidden_size > hc.MAX_WIDTH:
            raise ValueError(f"1 .. {hc.MAX_STREAMS} streams of width <= {hc.MAX_WIDTH}")
        self.runs = layer_runs(cfg)
        self.mspec: Dict[int, la.MatrixMemorySpec] = {}         # parallel layer -> its matrix memory
        self.freqs: Dict[int, Optional[torch.Tensor]] = {}      # attention layer -> [dims / 2] f32
        for i, l in enumerate(self.specs):
            m = attn_mixer(l)
            if m["heads"] % m["kv_heads"]:
                raise ValueError(f"layer {i}: attention heads / kv_heads do not fit")
            if l["type"] == "attention":
                r = m.get("rot")
                if r and (r["dims"] % 2 or r["dims"] > m["dim"]):
                    raise ValueError(f"layer {i}: rot.dims does not fit")
                self.freqs[i] = None
                if r and r["dims"]:
                    factor = float((r.get("scaling") or {}).get("factor", 1.0))
                    self.freqs[i] = sm.rotary_frequencies(int(r["dims"]), float(r["base"]), factor).to(self.device)
            else:
                self.mspec[i] = sp = memory_spec(l)
                if sp.dim > la.MAX_KEY_DIM:
                    raise ValueError(f"layer {i}: key size {sp.dim} > {la.MAX_KEY_DIM}")
            mlp = l.get("mlp")
            if mlp and not 1 <= mlp["router"]["top"] <= min(16, mlp["router"]["experts"]):
                raise ValueError(f"layer {i}: router top does not fit")

    # ------------------------------------------------------------------ weights
    def load_hf_state(self, sd: Dict[str, torch.Tensor]) -> "KupedraStage":
        """From checkpoint-named tensors: ONE input projection per layer (attention q | k | v; parallel: then the
        matrix memory's q | k | v | g | i | f), rows padded with zeros to a multiple of PROJ_ALIGN; gate | up stacked per
        expert; the shared expert's gate as one more router row; the distance biases expanded to one entry per
        distance; what feeds float32 math directly (router rows, sinks, temperatures, gate biases, stream weights)
        is float32."""
        want = model_shapes(self.cfg, sd)
        for n, shp in want.items():
            if n not in sd:
                raise KeyError(f"checkpoint lacks {n}")
            if tuple(sd[n].shape) != tuple(shp):
                raise ValueError(f"{n}: shape {tuple(sd[n].shape)}, config says {tuple(shp)}")
        cv = lambda t: t.to(device=self.device, dtype=self.dtype).contiguous()
        f32 = lambda t: t.to(device=self.device, dtype=torch.float32).contiguous()

        def fused(names):
            t = torch.cat([sd[n] for n in names], 0)
            pad = -t.shape[0] % PROJ_ALIGN
            return cv(torch.cat([t, t.new_zeros(pad, t.shape[1])], 0) if pad else t)
        self.embed = {"embed": cv(sd["embed"])}
        self.final_gain = float(sd["final.norm"])
        self.head = {"lm_head": cv(sd["head"]), "in": torch.ones(self.cfg.streams, device=self.device)}
        self.layers = []
        for i, layer in enumerate(self.specs):
            p = f"l{i}."
            mlp = layer.get("mlp")
            w: Dict[str, Any] = {}
            for q in (1, 2) if mlp else (1,):
                w[f"gain{q}"] = float(sd[p + f"norm{q}"])
                for k in ("in", "out", "mix"):
                    w[f"hc{q}_{k}"] = f32(sd[p + f"hc{q}.{k}"])
            m = attn_mixer(layer)
            if layer["type"] == "attention":
                w["w_in"] = fused([p + "mix." + x for x in "qkv"])
                w["wo"], w["temp"] = cv(sd[p + "mix.o"]), f32(sd[p + "mix.temp"])
                w["sinks"] = torch.zeros(m["heads"], dtype=torch.float32, device=self.device)   # exp(0): the added one
            else:
                pl, pr = p + "mix.left.", p + "mix.right."
                w["w_in"] = fused([pl + x for x in "qkv"] + [pr + x for x in "qkvgif"])
                w["q_norm"], w["k_norm"] = cv(sd[pl + "q.norm"]), cv(sd[pl + "k.norm"])
                w["bias"] = sm.distance_bias_table(f32(sd[pl + "rel"]), m["bias_max"])
                w["sinks"] = f32(sd[pl + "sink"])
                w["wo_left"], w["wo_right"] = cv(sd[pl + "o"]), cv(sd[pr + "o"])
                w["mix_norm"] = cv(sd[pr + "norm"])
                w["i_b"], w["f_b"] = f32(sd[pr + "i.b"]), f32(sd[pr + "f.b"])
                w["out_left"], w["out_right"] = cv(sd[pl + "out"]), cv(sd[pr + "out"])
            if mlp:
                e = mlp["router"]["experts"]
                rows = [sd[p + "mlp.router"]] + ([sd[p + "mlp.shared.sg"]] if mlp.get("shared") else [])
                w["router"] = f32(torch.cat(rows, 0))
                w["e_gu"] = cv(torch.stack([torch.cat([sd[p + f"mlp.e{j}.gate"], sd[p + f"mlp.e{j}.up"]], 0)
                                            for j in range(e)], 0))
                w["e_down"] = cv(torch.stack([sd[p + f"mlp.e{j}.down"] for j in range(e)], 0))
                if mlp.get("shared"):
                    w["s_gu"] = cv(torch.cat([sd[p + "mlp.shared.gate"], sd[p + "mlp.shared.up"]], 0))
                    w["s_down"] = cv(sd[p + "mlp.shared.down"])
            self.layers.append(w)
        return self

    def init_synthetic(self, seed: int = 0) -> "KupedraStage":
        return self.load_hf_state(synth_state_dict(self.cfg, seed))

    # ------------------------------------------------------------------ cache and state
    def cache_shapes(self, block_size: int) -> Dict[Any, tuple]:
        """Per layer RUN the attention's paged pair k [NB, G, BS, dim], v [NB, G, vdim, BS] (transposed inside a block)."""
        out = {}
        for r, (i, _) in enumerate(self.runs):
            m = attn_mixer(self.specs[i])
            out[r] = ((m["kv_heads"], block_size, m["dim"]), (m["kv_heads"], m["vdim"], block_size))
        return out

    def allocate_state(self, num_slots: int):
        """State pools, one row per BlockManager state slot, per RUN of a parallel layer, float32: the matrices
        [slots, heads, vdim, dim], the normalisers [slots, heads, dim] and the running maxima [slots, heads]."""
        self.num_state_slots = num_slots
        self.state = []
        for i, _ in self.runs:
            sp, st = self.mspec.get(i), {}
            if sp is not None:
                z = lambda *shape: torch.zeros(num_slots, *shape, dtype=torch.float32, device=self.device)
                st = {"s": z(sp.heads, sp.vdim, sp.dim), "n": z(sp.heads, sp.dim), "m": z(sp.heads)}
            self.state.append(st)
        return self.state

    def state_bytes_per_slot(self) -> int:
        sps = [self.mspec[i] for i, _ in self.runs if i in self.mspec]
        return sum(4 * sp.heads * (sp.vdim * sp.dim + sp.dim + 1) for sp in sps)

    @property
    def graph_capturable(self) -> bool:
        """Whether a decode step runs without a host round trip.  Experts whose sizes the grouped
        kernels do not take (and float32) read the per-expert row counts on the host, which a HIP-graph
        capture cannot record: such a model decodes with eager launches."""
        for l in self.specs:
            mlp = l.get("mlp")
            if mlp and (self.dtype != torch.bfloat16 or self.cfg.hidden_size % 128 or mlp["expert"]["ff"] % 128):
                return False
        return True

    # ------------------------------------------------------------------ forward
    def _attend(self, r: int, q: torch.Tensor, m, w, meta: BatchMeta, sb: sm.SeqBatch) -> torch.Tensor:
        kc, vc = self.kv.caches[r]
        nd = meta.num_decode if meta.is_prefill else meta.num_seqs
        a = sm.window_attention(q, kc, vc, meta.block_tables, sb, 1 << 30, float(m["scale"]), num_decode=nd,
                                sinks=w["sinks"], bias=w.get("bias"),
                                max_ctx=meta.max_ctx_d if (meta.is_prefill and nd) else meta.max_ctx)
        return a.view(a.shape[0], -1)

    def _attention(self, r: int, i: int, h: torch.Tensor, w, meta: BatchMeta, sb: sm.SeqBatch) -> torch.Tensor:
        m = self.specs[i]["mixer"]
        kc, vc = self.kv.caches[r]
        q = sm.head_norm_rope(ops.linear(h, w["w_in"]), 0, None, None, self.freqs[i], self.cfg.norm_eps, kc, vc,
                              meta.slot_mapping, sb.positions, m["heads"], m["kv_heads"], m["dim"], m["vdim"],
                              norm_last=True, q_mul=w["temp"])
        return ops.linear(self._attend(r, q, m, w, meta, sb), w["wo"])

    def _parallel(self, r: int, i: int, h: torch.Tensor, w, meta: BatchMeta, sb: sm.SeqBatch):
        """Both mixers on the same input: (attention output, matrix memory output), each [T, W]."""
        m, sp, st = self.specs[i]["mixer"]["left"], self.mspec[i], self.state[r]
        kc, vc = self.kv.caches[r]
        proj = ops.linear(h, w["w_in"])
        qt = m.get("q_temp")
        q = sm.head_norm_rope(proj, 0, w["q_norm"], w["k_norm"], None, self.cfg.norm_eps, kc, vc, meta.slot_mapping,
                              sb.positions, m["heads"], m["kv_heads"], m["dim"], m["vdim"],
                              q_temp=(float(qt["coef"]), int(qt["every"])) if qt else None)
        a = self._attend(r, q, m, w, meta, sb)
        qc = m["heads"] * m["dim"] + m["kv_heads"] * (m["dim"] + m["vdim"])     # first column of q | k | v | g | i | f
        qk, vv = sp.heads * sp.dim, sp.heads * sp.vdim
        kcol, vcol, gcol, icol = qc + qk, qc + 2 * qk, qc + 2 * qk + vv, qc + 2 * (qk + vv)
        y = la.memory_mixer(proj, qc, kcol, vcol, gcol, icol, icol + sp.heads, sp, w["i_b"], w["f_b"], w["mix_norm"], st["s"],
                            st["n"], st["m"], sb, self.cfg.norm_eps, q_scale=sp.dim ** -0.5)
        return ops.linear(a, w["wo_left"]), ops.linear(y, w["wo_right"])

    def _ff(self, h: torch.Tensor, w, mlp) -> torch.Tensor:
        sh = mlp.get("shared")
        return moe.softmax_top_ffn(h, w["router"], None, w["e_gu"], w["e_down"], int(mlp["router"]["top"]), w.get("s_gu"),
                                   w.get("s_down"), over_all=True, limit=float(mlp["expert"]["limit"]),
                                   shared_limit=float(sh["limit"]) if sh else None)

    @torch.inference_mode()
    def forward(self, inp: torch.Tensor, meta: BatchMeta) -> torch.Tensor:
        if self.kv is None or self.state is None:
            raise RuntimeError("allocate_kv() and allocate_state() before forward()")
        cfg, eps = self.cfg, self.cfg.norm_eps
        sb = self._seq_batch(meta)
        x = hc.embed_streams(inp, self.embed["embed"], cfg.streams, cfg.embed_scale)
        first = self.layers[self.runs[0][0]]
        h = hc.stream_read(x, first["hc1_in"], first["gain1"], eps, self.dtype)
        last = len(self.runs) - 1
        for r, (i, _) in enumerate(self.runs):
            spec, w = self.specs[i], self.layers[i]
            mlp = spec.get("mlp")
            nxt = None
            if r < last:
                wn = self.layers[self.runs[r + 1][0]]
                nxt = (wn["hc1_in"], wn["gain1"])
            after = (w["hc2_in"], w["gain2"]) if mlp else nxt
            if spec["type"] == "attention":
                x, h = hc.stream_step(x, w["hc1_mix"], w["hc1_out"], self._attention(r, i, h, w, meta, sb), eps, nxt=after)
            else:
                left, right = self._parallel(r, i, h, w, meta, sb)
                x, h = hc.stream_step(x, w["hc1_mix"], w["hc1_out"], left, eps, w_o=w["out_left"], o2=right,
                                      w_o2=w["out_right"], coef=0.5, nxt=after)
            if mlp:
                x, h = hc.stream_step(x, w["hc2_mix"], w["hc2_out"], self._ff(h, w, mlp), eps, nxt=nxt)
            if self.taps is not None:
                self.taps.append(x.sum(1))
        if meta.logits_idx is not None:
            x = x.index_select(0, meta.logits_idx)
        hf = hc.stream_read(x, self.head["in"], self.final_gain, eps, self.dtype)
        return sm.softcap_f32(ops.linear(hf, self.head["lm_head"]), 0.0, scale=cfg.logit_scale)
