"""Zarisun: windowed attention on convolved keys, a gated delta rule and
latent attention with shared caches, on an fp32 residual.

The sublayers read the stream itself; only their outputs are normed,

    x += rmsnorm(mixer(x)) * w1;   x += rmsnorm(ff(x)) * w2     (ff may be absent)

Three kinds of mixer:

* attention — q and k pass a short causal convolution per channel; the values
  are the keys as they leave it. q and k are then RMS-normed over the whole
  projection and rotated (adjacent pairs, frequencies and amplitude of a
  stretched context); a window, exp(sink_head) in the softmax denominator, and
  a sigmoid gate per head on the attended values;
* delta — a gated delta rule with one decay per head and token: convolutions
  with SiLU on q, k and v, unit q and k, an RMS norm per head and a SiLU gate
  on the read-out;
* latent attention — keys and values expanded per head from a normed latent,
  one rotated key part shared by all heads, with sink and gate as above. A
  layer may attend over the rows another layer cached.

Feed-forward: dense, SiLU-gated. The output head is the embedding table times
a constant.

MI355X mapping, in the manner of the other hybrid families:

- plain-tensor weights; everything that reads the mixer's input is ONE GEMM
  per layer (segments at 16-byte boundaries, the convolved segments first);
- the residual stays fp32; a sublayer's output norm, its residual add and the
  rounded copy the next sublayer reads are one kernel;
- one kernel per token does the whole-row norms, the rotation and the cache
  scatter of raw and finished keys; for single tokens it runs the convolution
  and advances its tail as well;
- latent attention runs in the absorbed form over [latent ‖ rotated key] rows
  (the query is mapped into the latent straight into the packed query, W_uv is
  applied to the attended latent); a layer that shares a cache packs only its
  queries;
- the paged attention kernels of the other families take window, sink and gate
  as options; with one kv head for all query heads a decode step runs on the
  matrix cores;
- convolution tails and the delta rule's [dim, vdim] memories live in
  per-sequence state slots, fp32; the delta rule runs on the kernel of the
  other families in its one-decay-per-head mode.
"""

from __future__ import annotations

import math
from typing import Dict, List, Optional, Union

import torch
import torch.nn.functional as F

from llmq_amd import ops
from llmq_amd.engine.forward_meta import DecodeMeta, MixedMeta, PrefillMeta
from llmq_amd.engine.kv_cache import KVCache
from llmq_amd.engine.model_specs import ZarisunSpec
from llmq_amd.engine.models.rotary import yarn_inv_freq


class ZarisunLayerWeights:
    def __init__(self) -> None:
        self.t: Dict[str, torch.Tensor] = {}     # packed / checkpoint-shaped tensors
        self.seg: Dict[str, tuple] = {}          # name -> (first row, rows) in t["in"]
        self.conv_cols = 0                       # leading columns of the packed projection the conv reads
        self.inv_freq: Optional[torch.Tensor] = None   # fp32 rotary table
        self.amplitude = 1.0                           # factor on cos and sin
        self.rate: Optional[torch.Tensor] = None       # fp32 [H] = exp(A_log)


def _align8(n: int) -> int:
    return -(-n // 8) * 8


class ZarisunLM:
    #: HIP extension groups this family runs on
    ext_groups = ("hybrid",)
    #: prompt portions attend through the block table (no gathered copy)
    paged_prefill = True
    #: mixed steps run their decode and prefill segments one after the other
    #: (projection GEMMs pick stream-k kernels at some shapes; those must not
    #: share the chip with a second stream's kernels)
    overlap_mixed = False

    def __init__(self, spec: ZarisunSpec, device: torch.device, dtype: torch.dtype,
                 tp_rank: int = 0, tp_size: int = 1):
        if tp_size != 1:
            raise NotImplementedError("the hybrid families run on one GPU per replica")
        self.spec = spec
        self.device = device
        self.dtype = dtype
        self.tp_rank, self.tp_size = tp_rank, tp_size
        self.layers: List[ZarisunLayerWeights] = []
        self.embedding: Optional[torch.Tensor] = None
        self.final_norm: Optional[torch.Tensor] = None
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
            if m.kind == "attention":
                out.append((m.kv_heads, m.dim, m.dim))
            elif m.kind == "latent_attention" and m.kv_from is None:
                out.append((1, m.kv_rank + m.rot_dim, 0))
            else:
                out.append(None)
        return out

    def state_layout(self):
        out = []
        for ls, lw in zip(self.spec.layers, self.layers):
            m = ls.mixer
            if m.kind == "attention":
                out.append([(m.conv - 1, lw.conv_cols)])
            elif m.kind == "delta":
                out.append([(m.heads, m.dim, m.vdim), (m.conv - 1, lw.conv_cols)])
            else:
                out.append(None)
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
            lw = ZarisunLayerWeights()
            m, t = ls.mixer, lw.t
            t["norm1"] = self._empty(W)
            conv = []                        # segments a short convolution reads, in front
            if m.kind == "attention":
                conv = [("q", m.heads * m.dim), ("k", m.kv_heads * m.dim)]
                rest = [("g", m.heads)]
                t["q_norm"] = self._empty(m.heads * m.dim)
                t["k_norm"] = self._empty(m.kv_heads * m.dim)
                t["sink"] = self._empty(m.heads, dtype=f32)
            elif m.kind == "delta":
                conv = [("q", m.kv_heads * m.dim), ("k", m.kv_heads * m.dim),
                        ("v", m.heads * m.vdim)]
                rest = [("g", m.heads * m.vdim), ("b", m.heads), ("a", m.heads)]
                for name in ("A_log", "dt_bias"):
                    t[name] = self._empty(m.heads, dtype=f32)
                t["norm"] = self._empty(m.vdim)
            else:
                rest = [("q", m.heads * (m.dim + m.rot_dim))]
                if m.kv_from is None:
                    rest.append(("dkv", m.kv_rank + m.rot_dim))
                    t["dkv_norm"] = self._empty(m.kv_rank)
                rest.append(("g", m.heads))
                t["uk"] = self._empty(m.heads, m.dim, m.kv_rank)     # [H, dim, R]
                t["uv"] = self._empty(m.heads, m.kv_rank, m.vdim)    # [H, R, vdim]
                t["sink"] = self._empty(m.heads, dtype=f32)
            t["o"] = self._empty(W, m.heads * m.vdim)
            at = 0
            for name, n in conv + rest:
                lw.seg[name] = (at, n)
                at += _align8(n)
            lw.conv_cols = sum(_align8(n) for _, n in conv)
            t["in"] = self._empty(at, W).zero_()
            if conv:
                t["conv_w"] = self._empty(lw.conv_cols, m.conv, dtype=f32).zero_()
            if ls.ff:
                t["norm2"] = self._empty(W)
                t["gate_up"] = self._empty(2 * ls.ff, W)
                t["down"] = self._empty(W, ls.ff)
            self.layers.append(lw)

    @torch.no_grad()
    def finalize(self) -> None:
        """Derive what the kernels read from the loaded tensors."""
        for ls, lw in zip(self.spec.layers, self.layers):
            m = ls.mixer
            if m.kind == "delta":
                lw.rate = torch.exp(lw.t["A_log"])
                continue
            if m.rot.dims:
                lw.inv_freq = yarn_inv_freq(m.rot.base, m.rot.dims, m.rot_scaling).to(self.device)
            lw.amplitude = m.rot_scaling.amplitude if m.rot_scaling else 1.0

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
                if name in ("q_norm", "k_norm", "dkv_norm", "norm"):
                    fill(t, 0.1, 1.0)
                elif name in ("norm1", "norm2"):
                    fill(t, 0.05, 0.5)
                elif name == "sink":
                    fill(t, 1.0)
                elif name == "A_log":
                    fill(t, 0.5)
                elif name == "dt_bias":
                    fill(t, 0.5, -3.0)
                elif name in ("in", "conv_w"):
                    fill(t, 1.0 / math.sqrt(W) if name == "in" else 0.5)
                    t[~keep[:t.shape[0]]] = 0
                elif name == "uv":
                    fill(t, 1.0 / math.sqrt(t.shape[1]))
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
    def _cols(p: torch.Tensor, lw: ZarisunLayerWeights, name: str) -> torch.Tensor:
        at, n = lw.seg[name]
        return p[:, at:at + n]

    def _heads(self, p, lw, name: str, heads: int) -> torch.Tensor:
        return self._cols(p, lw, name).unflatten(1, (heads, -1))

    @staticmethod
    def _attend(q, kc, vc, dv, m, meta, gate, sink):
        if meta.is_prefill:
            return ops.window_attn_prefill(
                q, kc, vc, dv, meta.block_tables, meta.cu_seqlens, meta.q_start, meta.max_seqlen,
                m.window, m.scale, gate=gate, sink=sink)
        if meta.is_mixed:
            nd, pm, dm = meta.n_decode, meta.prefill, meta.decode
            att_d = ops.window_attn_decode(
                q[:nd], kc, vc, dv, dm.block_tables, dm.context_lens, m.window, m.scale,
                gate=gate[:nd], sink=sink)
            att_p = ops.window_attn_prefill(
                q[nd:], kc, vc, dv, pm.block_tables, pm.cu_seqlens, pm.q_start, pm.max_seqlen,
                m.window, m.scale, gate=gate[nd:], sink=sink)
            return torch.cat([att_d, att_p], dim=0)
        return ops.window_attn_decode(
            q, kc, vc, dv, meta.block_tables, meta.context_lens, m.window, m.scale, gate=gate,
            sink=sink)

    def _conv_key_attention(self, p, lw, m, i, positions, kv_cache, meta):
        rm = meta.recurrent
        tail, = kv_cache.recurrent.state[i]
        single = not (meta.is_prefill or meta.is_mixed)
        if single:              # one row per sequence: the norm kernel convolves
            x, conv = p, (lw.t["conv_w"], tail, rm.slots, rm.fresh, lw.seg["q"][0], lw.seg["k"][0])
        else:
            x, conv = ops.causal_conv_silu(p[:, :lw.conv_cols], lw.t["conv_w"], None, tail, rm.cu,
                                           rm.slots, rm.fresh, silu=False), None
        q = self._heads(x, lw, "q", m.heads)
        kc, vc = kv_cache.k[i], kv_cache.v[i]
        ops.rownorm_rope_cache(
            q, self._heads(x, lw, "k", m.kv_heads), lw.t["q_norm"], lw.t["k_norm"], lw.inv_freq,
            m.rot.dims, positions, kc, vc, meta.slot_mapping, self.spec.rms_eps, lw.amplitude, conv)
        att = self._attend(q, kc, vc, m.dim, m, meta, self._cols(p, lw, "g"), lw.t["sink"])
        return F.linear(att.flatten(1), lw.t["o"])

    def _latent_attention(self, p, lw, m, i, positions, kv_cache, meta):
        T = p.shape[0]
        H, D, R = m.heads, m.dim, m.kv_rank
        q = self._heads(p, lw, "q", H)
        own = m.kv_from is None
        kc = kv_cache.k[self.spec.cache_layer(i)]
        # the unrotated query part mapped into the latent space, per head,
        # straight into the packed query's first R channels
        qf = torch.empty(T, H, R + m.rot_dim, dtype=p.dtype, device=p.device)
        torch.bmm(q[:, :, :D].transpose(0, 1), lw.t["uk"], out=qf[:, :, :R].transpose(0, 1))
        ops.latent_rope_pack(
            q, None, self._cols(p, lw, "dkv") if own else None, lw.t["dkv_norm"] if own else None,
            lw.inv_freq, positions, kc if own else None, meta.slot_mapping, D, m.rot.dims,
            m.rot.layout == "interleaved", self.spec.rms_eps, lw.amplitude, out=qf)
        ctx = self._attend(qf, kc, None, R, m, meta, self._cols(p, lw, "g"), lw.t["sink"])
        # values: W_uv on the attended latent, per head
        o = torch.empty(T, H, m.vdim, dtype=p.dtype, device=p.device)
        torch.bmm(ctx.transpose(0, 1), lw.t["uv"], out=o.transpose(0, 1))
        return F.linear(o.flatten(1), lw.t["o"])

    def _delta_rule(self, p, lw, m, i, kv_cache, meta):
        rm = meta.recurrent
        S, tail = kv_cache.recurrent.state[i]
        x = ops.causal_conv_silu(p[:, :lw.conv_cols], lw.t["conv_w"], None, tail,
                                 rm.cu, rm.slots, rm.fresh)
        o = ops.gated_delta_rule(
            self._heads(x, lw, "q", m.kv_heads), self._heads(x, lw, "k", m.kv_heads),
            self._heads(x, lw, "v", m.heads), self._cols(p, lw, "a"), lw.t["dt_bias"], lw.rate,
            self._cols(p, lw, "b"), S, rm.cu, rm.slots, rm.fresh, m.dim ** -0.5)
        y = ops.gla_out_norm_gate(o, lw.t["norm"], self._cols(p, lw, "g"), self.spec.rms_eps,
                                  self.dtype)
        return F.linear(y, lw.t["o"])

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
        eps, last = s.rms_eps, len(self.layers) - 1
        h = F.embedding(input_ids, self.embedding)
        res = h.to(torch.float32, copy=True)
        for i, (ls, lw) in enumerate(zip(s.layers, self.layers)):
            m = ls.mixer
            p = F.linear(h, lw.t["in"])
            if m.kind == "attention":
                y = self._conv_key_attention(p, lw, m, i, positions, kv_cache, meta)
            elif m.kind == "delta":
                y = self._delta_rule(p, lw, m, i, kv_cache, meta)
            else:
                y = self._latent_attention(p, lw, m, i, positions, kv_cache, meta)
            # the sublayers read the stream itself; the head reads its norm
            w_end = self.final_norm if i == last else None
            h = ops.sandwich_norm_res32(y, res, lw.t["norm1"], None if ls.ff else w_end, eps, 0.0)
            if ls.ff:
                y = F.linear(ops.act_and_mul(F.linear(h, lw.t["gate_up"])), lw.t["down"])
                h = ops.sandwich_norm_res32(y, res, lw.t["norm2"], w_end, eps, 0.0)
            if self.taps is not None:
                self.taps.append(res.clone())
        return h

    @torch.no_grad()
    def compute_logits(self, hidden: torch.Tensor) -> torch.Tensor:
        """final-normed hidden [N, width] -> logits [N, vocab] fp32."""
        # the constant rides on the GEMM, before its output's one rounding
        zero = hidden.new_zeros(1)
        return torch.addmm(zero, hidden, self.embedding.t(), beta=0.0,
                           alpha=self.spec.logit_scale).float()
