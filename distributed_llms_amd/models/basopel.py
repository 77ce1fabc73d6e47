"""Basopel: a layer-list decoder with a layer norm before and after every sublayer, three kinds of token mixer -- a
distance-biased window whose first tokens stay visible, latent attention inside a window, chunked attention with capped
scores --, values shared between layers, gelu GLU feed-forwards and a head tied to the embedding.

``config.json`` keys (read by ``config._from_basopel``): ``width``, ``vocab``, ``norm.eps``, ``embedding.scale`` and ``layers``:
per layer ``type``, ``mixer``, ``mlp`` (None or {"kind": "dense", "ff"}).

  type "attention": ``heads``, ``kv_heads``, ``dim`` (q / k), ``vdim``, ``scale``, ``bias_max``, ``mask`` (``size``,
      ``keep_first``), ``v_mix``.  Biased q / k / v projections, q and k RMS-normed per head, no rotation; a learned bias per
      bucket of distances is added to the scaled score (the table's rows come from its tensor); a query sees the last
      ``size`` positions and the first ``keep_first`` of the sequence.
  type "attention_2": ``heads``, ``kv_heads``, ``dim``, ``vdim``, ``scale``, ``softcap``, ``mask.size`` (chunks of positions),
      ``rot`` (``base``, ``dims``, optional ``scaling.factor`` that divides every frequency; half-split pairs), ``v_mix``.  Biased
      q / k / v / o projections, q and k RMS-normed over all heads at once, capped scores, a learned sink per head, a
      sigmoid gate per head.
  type "latent_attention": ``heads``, ``dim``, ``rot_dim``, ``vdim``, ``kv_rank``, ``scale``, ``mask.size`` (window), ``rot``
      (half-split pairs of the rotated part).  Keys and values are up-projections of one RMS-normed latent per token, one
      rotated key part serves every head; a learned sink per head; a sigmoid gate per output element.
  ``v_mix``: from the second such layer on the values are (1 - vmix) v + vmix v_first, v_first the values of the first
      such layer (of either softmax type) for the same token; the cache holds the blend.

One layer: x += ln(mixer(ln(x))), x += ln(ff(ln(x))); the model ends with a layer norm and the embedding table.

Checkpoint names: ``embed``, ``final.norm`` (+ ``.b``); per layer ``l<i>.``: ``norm1|norm1b|norm2|norm2b`` (+ ``.b``);
``mix.q|k|v`` (+ ``.b``), ``mix.q.norm|k.norm``, ``mix.rel`` or ``mix.sink|g|o.b``, ``mix.vmix``, ``mix.o``; latent layers
``mix.q|dkv|dkv.norm|uk|uv|sink|g|o``; ``mlp.gate|up|down``.  Linear weights are [out, in].

What a sequence keeps between steps is paged only, behind one block table: per softmax layer a K / V pair, per latent
layer the latent and the rotated key part in the two layouts the attention kernels read (ops/latent.py).  The residual
stream, norms, angles, scores, biases and softmax weights are float32 also when activations are bfloat16.
"""
from __future__ import annotations

from typing import Any, Dict, Optional

import torch

from .. import ops
from ..config import ModelConfig
from ..ops import latent as lat
from ..ops import seqmix as sm
from .hybrid import LayerListStage
from .stage import BatchMeta
from .weights import tensor_seed

DEFAULT_BIAS_ROWS = 32       # synthetic weights only: a checkpoint's tensors give the rows of the distance-bias table
PROJ_ALIGN = 16              # rows of a fused input projection are padded to a multiple of this (aligned row pieces)
LATENT = "latent_attention"


def latent_spec(layer: Dict[str, Any]) -> lat.LatentSpec:
    m = layer["mixer"]
    return lat.LatentSpec(heads=int(m["heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]), rank=int(m["kv_rank"]), q_rank=0,
                          scale=float(m["scale"]), rot_dim=int(m["rot_dim"]), gated=True, gate_elements=True, rot_half=True)


def layer_shapes(width: int, layer: Dict[str, Any], rows: Optional[int] = None) -> Dict[str, tuple]:
    """Checkpoint tensor name (without the ``l<i>.`` prefix) -> shape (``rows``: of the distance-bias table)."""
    m, mlp = layer["mixer"], layer.get("mlp")
    s: Dict[str, tuple] = {}
    for n in ("norm1", "norm1b") + (("norm2", "norm2b") if mlp else ()):
        s.update({n: (width,), n + ".b": (width,)})
    h, vd = m["heads"], m["heads"] * m["vdim"]
    if layer["type"] == LATENT:
        sp = latent_spec(layer)
        s.update({"mix.q": (sp.q_cols, width), "mix.dkv": (sp.key_width, width), "mix.dkv.norm": (sp.rank,),
                  "mix.uk": (h * sp.dim, sp.rank), "mix.uv": (vd, sp.rank), "mix.sink": (h,), "mix.g": (vd, width)})
    else:
        nq, nk, nv = h * m["dim"], m["kv_heads"] * m["dim"], m["kv_heads"] * m["vdim"]
        for n, r in (("q", nq), ("k", nk), ("v", nv)):
            s.update({f"mix.{n}": (r, width), f"mix.{n}.b": (r,)})
        if layer["type"] == "attention":
            s.update({"mix.q.norm": (m["dim"],), "mix.k.norm": (m["dim"],),
                      "mix.rel": (rows or int(m.get("rows", DEFAULT_BIAS_ROWS)), h)})
        else:
            s.update({"mix.q.norm": (nq,), "mix.k.norm": (nk,), "mix.sink": (h,), "mix.g": (h, width), "mix.o.b": (width,)})
        if m.get("v_mix"):
            s["mix.vmix"] = ()
    s["mix.o"] = (width, vd)
    if mlp:
        s.update({"mlp.gate": (mlp["ff"], width), "mlp.up": (mlp["ff"], width), "mlp.down": (width, mlp["ff"])})
    return s


def model_shapes(cfg: ModelConfig, sd: Optional[Dict[str, torch.Tensor]] = None) -> Dict[str, tuple]:
    """Every checkpoint tensor's shape; with ``sd`` the distance-bias rows are read from its ``rel`` tensors."""
    w = cfg.hidden_size
    s = {"embed": (cfg.vocab_size, w), "final.norm": (w,), "final.norm.b": (w,)}
    for i, layer in enumerate(cfg.layers):
        rel = None if sd is None else sd.get(f"l{i}.mix.rel")
        rows = int(rel.shape[0]) if rel is not None and rel.dim() == 2 else None
        s.update({f"l{i}.{n}": shp for n, shp in layer_shapes(w, layer, rows).items()})
    return s


def synth_state_dict(cfg: ModelConfig, seed: int = 0, dtype=torch.float32) -> Dict[str, torch.Tensor]:
    """Seeded random weights under the checkpoint names (CPU): projections and the embedding ~ N(0, 1 / width), norm
    weights around one, biases small, distance biases and sinks of moderate size, values blended about half and half."""
    sd = {}
    for name, shape in model_shapes(cfg).items():
        g = torch.Generator().manual_seed(tensor_seed(seed, 0, name))
        leaf = name.rsplit(".", 1)[-1]
        r = torch.randn(shape, generator=g)
        if leaf in ("norm", "norm1", "norm1b", "norm2", "norm2b"):
            t = 1.0 + 0.2 * r
        elif leaf == "b":
            t = 0.1 * r
        elif leaf in ("rel", "sink"):
            t = r
        elif leaf == "vmix":
            t = 0.5 + 0.1 * r
        else:
            t = r / shape[-1] ** 0.5
        sd[name] = t.to(dtype)
    return sd


class BasopelStage(LayerListStage):
    """All layers of a Basopel model on one device (see the module docstring)."""

    @staticmethod
    def layer_param_count(width: int, layer: Dict[str, Any]) -> int:
        return sum(int(torch.Size(s).numel()) for s in layer_shapes(width, layer).values())

    @staticmethod
    def kv_elements_per_token(cfg: ModelConfig) -> int:
        # a latent is held twice (row-major for the scores, transposed for the weighted sum)
        return sum(2 * latent_spec(l).rank + latent_spec(l).rot_dim if l["type"] == LATENT
                   else l["mixer"]["kv_heads"] * (l["mixer"]["dim"] + l["mixer"]["vdim"]) for l in cfg.layers)

    def __init__(self, cfg: ModelConfig, layer_start: int = 0, layer_end: Optional[int] = None, device="cpu",
                 dtype=torch.bfloat16, units: Optional[tuple] = None, tp=None, unit_group: int = 2):
        super().__init__(cfg, layer_start, layer_end, device, dtype, units, tp, unit_group)
        if cfg.hidden_size > sm.LAYER_NORM_MAX_WIDTH:
            raise ValueError(f"width <= {sm.LAYER_NORM_MAX_WIDTH}")
        self.lspec: Dict[int, lat.LatentSpec] = {}              # latent layer -> its sizes
        self.freqs: Dict[int, Optional[torch.Tensor]] = {}      # rotated layer -> [dims / 2] f32 (None: nothing turns)
        mixing = []
        for i, l in enumerate(self.specs):
            m = l["mixer"]
            if l["type"] == LATENT:
                self.lspec[i] = latent_spec(l)
            elif m["heads"] % m["kv_heads"]:
                raise ValueError(f"layer {i}: attention heads / kv_heads do not fit")
            elif m.get("v_mix"):
                mixing.append(i)
            if l["type"] != "attention":
                r = m.get("rot") or {"dims": 0, "base": 1.0}
                if r["dims"] % 2 or r["dims"] > (m["rot_dim"] if l["type"] == LATENT else m["dim"]):
                    raise ValueError(f"layer {i}: rot.dims does not fit")
                factor = float((r.get("scaling") or {}).get("factor", 1.0))
                f = sm.rotary_frequencies(int(r["dims"]), float(r["base"]), factor).to(self.device)
                self.freqs[i] = f if r["dims"] or l["type"] != LATENT else None
            mask = m.get("mask") or {}
            if int(mask.get("size", 1)) < 1 or int(mask.get("keep_first", 0)) < 0:
                raise ValueError(f"layer {i}: mask sizes")
        if len({self.specs[i]["mixer"]["kv_heads"] * self.specs[i]["mixer"]["vdim"] for i in mixing}) > 1:
            raise ValueError("layers that share values need equal kv_heads * vdim")
        self.mix_first = mixing[0] if len(mixing) > 1 else None      # the layer whose values others read
        self.mixing = set(mixing) if len(mixing) > 1 else set()

    # ------------------------------------------------------------------ weights
    def load_hf_state(self, sd: Dict[str, torch.Tensor]) -> "BasopelStage":
        """From checkpoint-named tensors: ONE input projection per layer (q | k | v, then the head gates; latent layers q |
        latent | shared key part | element gates), rows padded with zeros to a multiple of PROJ_ALIGN; the biases of q | k |
        v in one vector; gate | up fused; uk as [H, dim, rank], uv transposed ([H, rank, vdim]); the distance biases
        expanded to one entry per distance; sinks float32; the head is the embedding table."""
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
        self.head = {"final_norm": cv(sd["final.norm"]), "final_norm_b": cv(sd["final.norm.b"])}
        self.layers = []
        for i, layer in enumerate(self.specs):
            p, q = f"l{i}.", f"l{i}.mix."
            m, mlp = layer["mixer"], layer.get("mlp")
            w: Dict[str, Any] = {}
            for n in ("norm1", "norm1b") + (("norm2", "norm2b") if mlp else ()):
                w[n], w[n + "_b"] = cv(sd[p + n]), cv(sd[p + n + ".b"])
            if layer["type"] == LATENT:
                sp = self.lspec[i]
                w["mix"] = {"down": fused([q + "q", q + "dkv", q + "g"]), "c_norm": cv(sd[q + "dkv.norm"]),
                            "uk": cv(sd[q + "uk"].view(sp.heads, sp.dim, sp.rank)),
                            "uv_t": cv(sd[q + "uv"].view(sp.heads, sp.vdim, sp.rank).transpose(1, 2)),
                            "o": cv(sd[q + "o"]), "sinks": f32(sd[q + "sink"])}
            else:
                two = layer["type"] == "attention_2"
                w["w_in"] = fused([q + x for x in (("q", "k", "v", "g") if two else ("q", "k", "v"))])
                w["b_in"] = cv(torch.cat([sd[q + x + ".b"] for x in "qkv"], 0))
                w["q_norm"], w["k_norm"], w["wo"] = cv(sd[q + "q.norm"]), cv(sd[q + "k.norm"]), cv(sd[q + "o"])
                if two:
                    w["sinks"], w["bo"] = f32(sd[q + "sink"]), cv(sd[q + "o.b"])
                else:
                    w["bias"] = sm.distance_bias_table(f32(sd[q + "rel"]), m["bias_max"])
                if m.get("v_mix"):
                    w["vmix"] = float(sd[q + "vmix"])
            if mlp:
                w["w_gu"] = cv(torch.cat([sd[p + "mlp.gate"], sd[p + "mlp.up"]], 0))
                w["w_down"] = cv(sd[p + "mlp.down"])
            self.layers.append(w)
        return self

    def init_synthetic(self, seed: int = 0) -> "BasopelStage":
        return self.load_hf_state(synth_state_dict(self.cfg, seed))

    def lm_head_weight(self, full: bool = False) -> torch.Tensor:
        return self.embed["embed"]

    # ------------------------------------------------------------------ cache
    def cache_shapes(self, block_size: int) -> Dict[Any, tuple]:
        """Per layer k [NB, G, BS, dim], v [NB, G, vdim, BS] (transposed inside a block); latent layers k [NB, 1, BS, rank +
        rot_dim] (latent | shared rotated key part), v [NB, 1, rank, BS] (the latent again)."""
        out = {}
        for i, l in enumerate(self.specs):
            m = l["mixer"]
            if l["type"] == LATENT:
                out[i] = ((1, block_size, self.lspec[i].key_width), (1, self.lspec[i].rank, block_size))
            else:
                out[i] = ((m["kv_heads"], block_size, m["dim"]), (m["kv_heads"], m["vdim"], block_size))
        return out

    def allocate_state(self, num_slots: int):
        self.num_state_slots = num_slots
        self.state = []
        return self.state

    # ------------------------------------------------------------------ forward
    def _softmax_mixer(self, i: int, h: torch.Tensor, w, meta: BatchMeta, sb: sm.SeqBatch, nd: int, max_ctx,
                       v_mix: Optional[sm.ValueMix]):
        spec = self.specs[i]
        m, eps = spec["mixer"], self.cfg.norm_eps
        hh, g, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        kc, vc = self.kv.caches[i]
        size = int((m.get("mask") or {}).get("size") or 0)          # no mask entry: plain causal attention
        proj = ops.linear(h, w["w_in"])
        if spec["type"] == "attention":
            q = sm.head_norm_rope(proj, 0, w["q_norm"], w["k_norm"], None, eps, kc, vc, meta.slot_mapping, sb.positions, hh, g,
                                  d, dv, bias=w["b_in"], v_mix=v_mix)
            a = sm.window_attention(q, kc, vc, meta.block_tables, sb, size or 1 << 30, float(m["scale"]), num_decode=nd,
                                    max_ctx=max_ctx, bias=w["bias"],
                                    keep_first=int((m.get("mask") or {}).get("keep_first") or 0))
        else:
            q = sm.rownorm_rope(proj, 0, w["q_norm"], w["k_norm"], self.freqs[i], eps, kc, vc, meta.slot_mapping, sb.positions,
                                hh, g, d, dv, bias=w["b_in"], v_mix=v_mix)
            a = sm.window_attention(q, kc, vc, meta.block_tables, sb, 1 << 30, float(m["scale"]), num_decode=nd,
                                    max_ctx=max_ctx, chunk=size, softcap=float(m.get("softcap") or 0.0), sinks=w["sinks"],
                                    gate=proj, gate_col=hh * d + g * (d + dv))
        return ops.linear(a.view(a.shape[0], -1), w["wo"], defer=True)

    def _value_mix(self, i: int, first: Optional[torch.Tensor], tokens: int) -> Optional[sm.ValueMix]:
        if i not in self.mixing:
            return None
        if i == self.mix_first:
            m = self.specs[i]["mixer"]
            return sm.ValueMix(torch.empty(tokens, m["kv_heads"] * m["vdim"], dtype=self.dtype, device=self.device))
        return sm.ValueMix(first, self.layers[i]["vmix"])

    @torch.inference_mode()
    def forward(self, inp: torch.Tensor, meta: BatchMeta) -> torch.Tensor:
        if self.kv is None:
            raise RuntimeError("allocate_kv() before forward()")
        cfg, eps = self.cfg, self.cfg.norm_eps
        sb = self._seq_batch(meta)
        nd = meta.num_decode if meta.is_prefill else meta.num_seqs
        max_ctx = meta.max_ctx_d if (meta.is_prefill and nd) else meta.max_ctx
        x = sm.embedding_f32(inp, self.embed["embed"], cfg.embed_scale)
        h = sm.layer_norm_f32(x, self.layers[0]["norm1"], self.layers[0]["norm1_b"], eps, self.dtype)
        v_first = None                    # the values that later layers read, from the first layer that shares them
        for i, (spec, w) in enumerate(zip(self.specs, self.layers)):
            nxt = (None, None)
            if i + 1 < len(self.layers):
                nxt = (self.layers[i + 1]["norm1"], self.layers[i + 1]["norm1_b"])
            if spec["type"] == LATENT:
                kc, vc = self.kv.caches[i]
                o = lat.latent_attention(h, w["mix"], self.lspec[i], self.freqs[i], eps, kc, vc, meta.slot_mapping,
                                         meta.block_tables, sb, num_decode=nd, max_ctx=max_ctx, defer=True,
                                         window=int((spec["mixer"].get("mask") or {}).get("size") or 1 << 30))
            else:
                vm = self._value_mix(i, v_first, inp.numel())
                if vm is not None and vm.lam is None:
                    v_first = vm.first
                o = self._softmax_mixer(i, h, w, meta, sb, nd, max_ctx, vm)
            after = (w["norm2"], w["norm2_b"]) if spec.get("mlp") else nxt
            x, h = sm.post_layer_norm_add(x, o, w["norm1b"], w["norm1b_b"], eps, bias=w.get("bo"), w_next=after[0],
                                          b_next=after[1])
            if spec.get("mlp"):
                y = ops.linear(sm.linear_gelu_glu(h, w["w_gu"]), w["w_down"], defer=True)
                x, h = sm.post_layer_norm_add(x, y, w["norm2b"], w["norm2b_b"], eps, w_next=nxt[0], b_next=nxt[1])
            if self.taps is not None:
                self.taps.append(x.clone())
        if meta.logits_idx is not None:
            x = x.index_select(0, meta.logits_idx)
        hf = sm.layer_norm_f32(x, self.head["final_norm"], self.head["final_norm_b"], eps, self.dtype)
        return sm.softcap_f32(ops.linear(hf, self.embed["embed"]), 0.0)
