"""Kikurax: sigmoid attention beside a gated delta rule, Mamba-2 scans and
rotary softmax attention on an fp32 residual.

A layer is pre-norm,

    x += mixer(norm1(x));   x += experts(norm2(x))       (experts may be absent)

with norms on `groups` equal consecutive parts of the width, each divided by
its own root mean square. Three kinds of mixer:

* an averaged pair — unrotated attention whose weights are sigmoids of the
  scores (a bias per head, no normalisation over keys; unit-RMS q and k, a
  query factor that grows with the logarithm of the position, an elementwise
  sigmoid gate on the attended heads) beside a gated delta rule (a decay per
  head and key channel from a low-rank projection, short convolutions on q, k
  and v, unit q and k, per-head norm and a low-rank sigmoid gate); each output
  is RMS-normed over the width and the two are averaged;
* Mamba-2 — one decay per head and token on a [state, vdim] memory, B and C
  shared by groups of heads, the gate before a norm on equal parts;
* attention — biased projections, rotary q/k with wavelength-scaled
  frequencies, then unit RMS per head, a temperature per head, a tanh score
  cap, a softmax with one more term e^0 in its denominator, and values
  blended with the first blending layer's.

Feed-forward: a mixture of clamped gated experts; the choice and the weights
(softmax over the chosen logits) come from biased fp32 router logits. The
output head is the embedding table.

MI355X mapping, in the manner of the other hybrid families:

- plain-tensor weights; everything that reads the mixer's input is ONE GEMM
  per layer (segments at 16-byte boundaries, the convolved segments first so
  one kernel convolves them together); the delta rule's two low-rank
  projections are small GEMMs on slices of its output;
- the residual stays fp32; closing a sublayer and opening the next (add,
  grouped norm) is one kernel;
- keys and values go through the paged cache and the block table for prompt
  portions and single tokens alike; one kernel per token does the per-head
  norms, rotation, query factors, value blend and scatter (a norm without a
  weight commutes with the rotation; the factors of q ride on it); the paged
  attention kernels of the other families take the sigmoid weights, the
  elementwise gate, the cap and the zero-score sink as options;
- convolution tails, the delta rule's [dim, vdim] and the scan's [state, vdim]
  memories live in per-sequence state slots, fp32; the scan runs on the
  diagonal-decay recurrence kernel of the other families in its scalar-gate
  mode, the delta rule on a kernel of its own;
- a step's expert mixture runs sorted by expert on vendor GEMMs, or, inside
  captured decode graphs, as one batched GEMM pair over all experts.
"""

from __future__ import annotations

import math
from typing import Dict, List, Optional, Union

import torch
import torch.nn.functional as F

from llmq_amd import ops
from llmq_amd.engine.forward_meta import DecodeMeta, MixedMeta, PrefillMeta
from llmq_amd.engine.kv_cache import KVCache
from llmq_amd.engine.model_specs import KikuraxSpec
from llmq_amd.engine.models.rotary import scaled_inv_freq


class KikuraxLayerWeights:
    def __init__(self) -> None:
        self.t: Dict[str, torch.Tensor] = {}     # packed / checkpoint-shaped tensors
        self.seg: Dict[str, tuple] = {}          # name -> (first row, rows) in t["in"]
        self.conv_cols = 0                       # leading columns of the packed projection the conv reads
        self.inv_freq: Optional[torch.Tensor] = None   # fp32 rotary table
        self.rate: Optional[torch.Tensor] = None       # fp32 [H] = exp(A_log)
        self.zero_sink: Optional[torch.Tensor] = None  # fp32 [H] zeros
        self.lam = 0.0                                 # value blend


def _align8(n: int) -> int:
    return -(-n // 8) * 8


class KikuraxLM:
    #: HIP extension groups this family runs on
    ext_groups = ("hybrid",)
    #: prompt portions attend through the block table (no gathered copy)
    paged_prefill = True
    #: mixed steps run their decode and prefill segments one after the other
    #: (the expert GEMMs pick stream-k kernels at some shapes; those must not
    #: share the chip with a second stream's kernels)
    overlap_mixed = False

    def __init__(self, spec: KikuraxSpec, device: torch.device, dtype: torch.dtype,
                 tp_rank: int = 0, tp_size: int = 1):
        if tp_size != 1:
            raise NotImplementedError("the hybrid families run on one GPU per replica")
        self.spec = spec
        self.device = device
        self.dtype = dtype
        self.tp_rank, self.tp_size = tp_rank, tp_size
        self.layers: List[KikuraxLayerWeights] = []
        self.embedding: Optional[torch.Tensor] = None
        self.final_norm: Optional[torch.Tensor] = None
        self.first_v_mix = spec.first_v_mix()
        self.taps: Optional[List[torch.Tensor]] = None  # stream after each layer (debug)
        self._alloc()

    @property
    def lm_head(self) -> torch.Tensor:
        return self.embedding

    # -- layout the engine asks for ---------------------------------------

    def kv_layout(self):
        out = []
        for ls in self.spec.layers:
            m = ls.mixer
            a = m.left if m.kind == "parallel" else m
            out.append(None if m.kind == "mamba2" else (a.kv_heads, a.dim, a.vdim))
        return out

    def state_layout(self):
        out = []
        for ls, lw in zip(self.spec.layers, self.layers):
            m = ls.mixer
            if m.kind == "attention":
                out.append(None)
            elif m.kind == "mamba2":
                out.append([(m.heads, m.state, m.vdim), (m.conv - 1, lw.conv_cols)])
            else:
                r = m.right
                out.append([(r.heads, r.dim, r.vdim), (r.conv - 1, lw.conv_cols)])
        return out

    # -- weights ---------------------------------------------------------

    def _empty(self, *shape, dtype=None) -> torch.Tensor:
        return torch.empty(*shape, device=self.device, dtype=dtype or self.dtype)

    def _alloc(self) -> None:
        s = self.spec
        W = s.hidden_size
        f32 = torch.float32
        self.embedding = self._empty(s.vocab_size, W)
        self.final_norm = self._empty(W)
        for ls in s.layers:
            lw = KikuraxLayerWeights()
            m, t = ls.mixer, lw.t
            t["norm1"] = self._empty(W)
            conv, taps = [], 0               # segments a short convolution reads, in front
            if m.kind == "attention":
                rest = [("q", m.heads * m.dim), ("k", m.kv_heads * m.dim),
                        ("v", m.kv_heads * m.vdim)]
                t["temp"] = self._empty(m.heads, dtype=f32)
                if m.v_mix:
                    t["vmix"] = self._empty((), dtype=f32)
                t["o"] = self._empty(W, m.heads * m.vdim)
            elif m.kind == "mamba2":
                bc = m.groups * m.state
                conv, taps = [("x", m.inner), ("B", bc), ("C", bc)], m.conv
                rest = [("z", m.inner), ("dt", m.heads)]
                for name in ("dt_bias", "A_log", "D"):
                    t[name] = self._empty(m.heads, dtype=f32)
                t["norm"] = self._empty(m.inner)
                t["o"] = self._empty(W, m.inner)
            else:
                a, r = m.left, m.right
                conv = [("dq", r.kv_heads * r.dim), ("dk", r.kv_heads * r.dim),
                        ("dv", r.heads * r.vdim)]
                taps = r.conv
                rest = [("q", a.heads * a.dim), ("k", a.kv_heads * a.dim),
                        ("v", a.kv_heads * a.vdim), ("g", a.heads * a.vdim),
                        ("a1", r.decay_rank), ("g1", r.gate_rank), ("b", r.heads)]
                t["pb"] = self._empty(a.heads, dtype=f32)
                t["o"] = self._empty(W, a.heads * a.vdim)
                t["left_out"] = self._empty(W)
                t["a2"] = self._empty(r.heads * r.dim, r.decay_rank)
                t["g2"] = self._empty(r.heads * r.vdim, r.gate_rank)
                t["dt_bias"] = self._empty(r.heads * r.dim, dtype=f32)
                t["A_log"] = self._empty(r.heads, dtype=f32)
                t["d_norm"] = self._empty(r.vdim)
                t["d_o"] = self._empty(W, r.heads * r.vdim)
                t["right_out"] = self._empty(W)
            at = 0
            for name, n in conv + rest:
                lw.seg[name] = (at, n)
                at += _align8(n)
            lw.conv_cols = sum(_align8(n) for _, n in conv)
            t["in"] = self._empty(at, W).zero_()
            if m.kind == "attention":
                t["in_b"] = self._empty(at).zero_()
            if conv:
                t["conv_w"] = self._empty(lw.conv_cols, taps, dtype=f32).zero_()
            if m.kind == "mamba2":
                t["conv_b"] = self._empty(lw.conv_cols, dtype=f32).zero_()
            if ls.moe:
                e = ls.moe
                t["norm2"] = self._empty(W)
                t["router"] = self._empty(e.experts, W, dtype=f32)
                t["router_b"] = self._empty(e.experts, dtype=f32)
                t["e_gate_up"] = self._empty(e.experts, 2 * e.ff, W)
                t["e_down"] = self._empty(e.experts, W, e.ff)
            self.layers.append(lw)

    @torch.no_grad()
    def finalize(self) -> None:
        """Derive what the kernels read from the loaded tensors."""
        for ls, lw in zip(self.spec.layers, self.layers):
            m = ls.mixer
            if m.kind == "attention":
                if m.rot.dims:
                    lw.inv_freq = scaled_inv_freq(m.rot.base, m.rot.dims,
                                                  m.rot_scaling).to(self.device)
                lw.zero_sink = torch.zeros(m.heads, dtype=torch.float32, device=self.device)
                lw.lam = float(lw.t["vmix"]) if m.v_mix else 0.0
            else:
                lw.rate = torch.exp(lw.t["A_log"])

    @torch.no_grad()
    def random_init(self, seed: int = 0, fast: bool = False) -> None:
        if fast and self.device.type == "cuda":
            gen = torch.Generator(device=self.device).manual_seed(seed)

            def fill(t: torch.Tensor, std: float, mean: float = 0.0) -> None:
                t.normal_(mean, std, generator=gen)
        else:
            gen = torch.Generator(device="cpu").manual_seed(seed)

            def fill(t: torch.Tensor, std: float, mean: float = 0.0) -> None:
                cpu = torch.randn(t.shape, generator=gen, dtype=torch.float32) * std + mean
                t.copy_(cpu.to(t.dtype))

        W = self.spec.hidden_size
        fill(self.embedding, 1.0)
        fill(self.final_norm, 0.1, 1.0)
        for lw in self.layers:
            keep = torch.zeros(lw.t["in"].shape[0], dtype=torch.bool)
            for at, n in lw.seg.values():
                keep[at:at + n] = True
            keep = keep.to(self.device)
            for name, t in lw.t.items():
                if name in ("norm1", "norm2", "norm", "d_norm", "D"):
                    fill(t, 0.1, 1.0)
                elif name in ("left_out", "right_out"):
                    fill(t, 0.05, 0.5)
                elif name == "temp":
                    fill(t, 0.2, 1.2)
                elif name == "vmix":
                    t.fill_(0.4)
                elif name == "pb":
                    fill(t, 0.3, -3.0)
                elif name == "A_log":
                    fill(t, 0.5)
                elif name == "dt_bias":
                    fill(t, 0.5, -3.0)
                elif name == "router_b":
                    fill(t, 0.1)
                elif name in ("in", "in_b", "conv_w", "conv_b"):
                    fill(t, 1.0 / math.sqrt(W) if name == "in" else 0.3 if name == "in_b" else 0.5)
                    t[~keep[:t.shape[0]]] = 0
                else:
                    fill(t, 1.0 / math.sqrt(t.shape[-1]))
        self.finalize()

    def named_tensors(self) -> Dict[str, torch.Tensor]:
        out = {"embedding": self.embedding, "final_norm": self.final_norm}
        for i, lw in enumerate(self.layers):
            for name, t in lw.t.items():
                out[f"layers.{i}.{name}"] = t
        return out

    def weight_bytes(self) -> int:
        return sum(t.numel() * t.element_size() for t in self.named_tensors().values())

    # -- mixers ----------------------------------------------------------

    @staticmethod
    def _cols(p: torch.Tensor, lw: KikuraxLayerWeights, name: str) -> torch.Tensor:
        at, n = lw.seg[name]
        return p[:, at:at + n]

    def _heads(self, p, lw, name: str, heads: int) -> torch.Tensor:
        return self._cols(p, lw, name).unflatten(1, (heads, -1))

    def _attend(self, q, kc, vc, a, meta, gate=None, **extra):
        def sl(rows):
            return None if gate is None else gate[rows]

        if meta.is_prefill:
            return ops.window_attn_prefill(
                q, kc, vc, a.vdim, meta.block_tables, meta.cu_seqlens, meta.q_start,
                meta.max_seqlen, 0, a.scale, gate=gate, **extra)
        if meta.is_mixed:
            nd, pm, dm = meta.n_decode, meta.prefill, meta.decode
            att_d = ops.window_attn_decode(
                q[:nd], kc, vc, a.vdim, dm.block_tables, dm.context_lens, 0, a.scale,
                gate=sl(slice(None, nd)), **extra)
            att_p = ops.window_attn_prefill(
                q[nd:], kc, vc, a.vdim, pm.block_tables, pm.cu_seqlens, pm.q_start, pm.max_seqlen,
                0, a.scale, gate=sl(slice(nd, None)), **extra)
            return torch.cat([att_d, att_p], dim=0)
        return ops.window_attn_decode(
            q, kc, vc, a.vdim, meta.block_tables, meta.context_lens, 0, a.scale, gate=gate, **extra)

    def _rotary_attention(self, p, lw, a, i, v_first, positions, kv_cache, meta):
        q = self._heads(p, lw, "q", a.heads)
        v = self._heads(p, lw, "v", a.kv_heads)
        kc, vc = kv_cache.k[i], kv_cache.v[i]
        ops.qkv_norm_rope_cache(
            q, self._heads(p, lw, "k", a.kv_heads), v, None, None, lw.inv_freq, a.rot.dims,
            positions, kc, vc, meta.slot_mapping, self.spec.rms_eps, qk_unit_norm=True,
            head_scale=lw.t["temp"], v_first=v_first if a.v_mix else None, mix=lw.lam)
        att = self._attend(q, kc, vc, a, meta, sink=lw.zero_sink, softcap=a.softcap)
        return F.linear(att.flatten(1), lw.t["o"]), v

    def _sigmoid_attention(self, p, lw, a, i, positions, kv_cache, meta):
        q = self._heads(p, lw, "q", a.heads)
        kc, vc = kv_cache.k[i], kv_cache.v[i]
        ops.qkv_norm_rope_cache(
            q, self._heads(p, lw, "k", a.kv_heads), self._heads(p, lw, "v", a.kv_heads), None, None,
            None, 0, positions, kc, vc, meta.slot_mapping, self.spec.rms_eps, qk_unit_norm=True,
            temp_coef=a.temp_coef, temp_every=a.temp_every)
        att = self._attend(q, kc, vc, a, meta, gate=self._cols(p, lw, "g"), sigmoid=True,
                           wbias=lw.t["pb"])
        return F.linear(att.flatten(1), lw.t["o"])

    def _delta_rule(self, p, lw, r, i, kv_cache, meta):
        rm = meta.recurrent
        S, tail = kv_cache.recurrent.state[i]
        x = ops.causal_conv_silu(p[:, :lw.conv_cols], lw.t["conv_w"], None, tail,
                                 rm.cu, rm.slots, rm.fresh)
        z = F.linear(self._cols(p, lw, "a1"), lw.t["a2"]).unflatten(1, (r.heads, r.dim))
        o = ops.gated_delta_rule(
            self._heads(x, lw, "dq", r.kv_heads), self._heads(x, lw, "dk", r.kv_heads),
            self._heads(x, lw, "dv", r.heads), z, lw.t["dt_bias"], lw.rate, self._cols(p, lw, "b"),
            S, rm.cu, rm.slots, rm.fresh, r.dim ** -0.5)
        gate = F.linear(self._cols(p, lw, "g1"), lw.t["g2"])
        y = ops.gla_out_norm_gate(o, lw.t["d_norm"], gate, self.spec.rms_eps, self.dtype,
                                  sigmoid=True)
        return F.linear(y, lw.t["d_o"])

    def _mamba2(self, p, lw, m, i, kv_cache, meta):
        rm = meta.recurrent
        S, tail = kv_cache.recurrent.state[i]
        xbc = ops.causal_conv_silu(p[:, :lw.conv_cols], lw.t["conv_w"], lw.t["conv_b"], tail,
                                   rm.cu, rm.slots, rm.fresh)
        x = self._cols(xbc, lw, "x")
        o = ops.ssd_scan(
            x.unflatten(1, (m.heads, m.vdim)), self._heads(xbc, lw, "B", m.groups),
            self._heads(xbc, lw, "C", m.groups), self._cols(p, lw, "dt"), lw.t["dt_bias"], lw.rate,
            S, rm.cu, rm.slots, rm.fresh)
        y = ops.ssd_out_gate_norm(o, x, lw.t["D"], self._cols(p, lw, "z"), lw.t["norm"],
                                  self.spec.rms_eps, m.norm_groups, self.dtype)
        return F.linear(y, lw.t["o"])

    def _moe(self, h, lw, e, meta):
        logits = F.linear(h.float(), lw.t["router"], lw.t["router_b"])
        # softmax over all, then the chosen divided by their sum: the softmax
        # over the chosen logits alone
        idx, w = ops.softmax_topk(logits, e.top, 1.0, renorm=True)
        decode_only = not (meta.is_prefill or meta.is_mixed)
        return ops.moe_experts(h, idx, w, lw.t["e_gate_up"], lw.t["e_down"], sync_free=decode_only,
                               act="clamp_swish", limit=e.limit, weight_output=True)

    # -- forward ---------------------------------------------------------

    @torch.no_grad()
    def forward(
        self,
        input_ids: torch.Tensor,
        positions: torch.Tensor,
        kv_cache: KVCache,
        meta: Union[PrefillMeta, DecodeMeta, MixedMeta],
    ) -> torch.Tensor:
        s = self.spec
        eps, groups = s.rms_eps, s.norm_groups
        n = len(self.layers)
        res = F.embedding(input_ids, self.embedding).float().mul_(s.embedding_scale)
        first = self.layers[0].t["norm1"] if n else self.final_norm
        h = ops.rmsnorm_cast(res, first, eps, 0.0, self.dtype, groups)
        v_first = None       # values of the first blending layer, this step's rows
        for i, (ls, lw) in enumerate(zip(s.layers, self.layers)):
            m = ls.mixer
            p = F.linear(h, lw.t["in"], lw.t.get("in_b"))
            if m.kind == "attention":
                y, v = self._rotary_attention(p, lw, m, i, v_first, positions, kv_cache, meta)
                if i == self.first_v_mix:
                    v_first = v
            elif m.kind == "mamba2":
                y = self._mamba2(p, lw, m, i, kv_cache, meta)
            else:
                yl = self._sigmoid_attention(p, lw, m.left, i, positions, kv_cache, meta)
                yr = self._delta_rule(p, lw, m.right, i, kv_cache, meta)
                y = ops.dual_norm_mean(yl, lw.t["left_out"], yr, lw.t["right_out"], eps)
            w_next = self.layers[i + 1].t["norm1"] if i + 1 < n else self.final_norm
            if ls.moe:
                h = ops.scaled_add_norm(res, y, None, 1.0, 0.0, lw.t["norm2"], eps, self.dtype,
                                        groups)
                y = self._moe(h, lw, ls.moe, meta)
            h = ops.scaled_add_norm(res, y, None, 1.0, 0.0, w_next, eps, self.dtype, groups)
            if self.taps is not None:
                self.taps.append(res.clone())
        return h

    @torch.no_grad()
    def compute_logits(self, hidden: torch.Tensor) -> torch.Tensor:
        """final-normed hidden [N, width] -> logits [N, vocab] fp32."""
        return F.linear(hidden, self.embedding).float()
