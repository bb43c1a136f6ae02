"""Modepel: sandwich-normed layers of gated attention with an added one in the softmax and
blended values, or of a matrix-memory recurrence, with polynomial-norm feed-forwards or routed
experts some of which are the identity, on the kernels of csrc/kernels/mix_*.hip.

The residual stream x is fp32.  Every norm is an RMS norm with one number g:

  x = embed[token]
  per layer:
    x += norm1b(mixer(norm1(x)))
    x += norm2b(ff(norm2(x)))                 (layers with a feed-forward)
  logits = head . norm_final(x)

A sublayer's output norm, the residual update and the next sublayer's input norm are one kernel
(gain_sandwich), which also adds the parts of a mixture that need no product of their own: the
shared expert times the sigmoid of its logit, and the identity experts' share of the input.

attention   q | k | v | gate in one product (biases on q, k, v).  One kernel adds the biases,
  rotates the first rot_dims of every head of q and k (half split), blends the values of every
  v_mix layer but the first with that layer's values of the same token,
  v <- (1 - lambda) v + lambda v_first (kept in fp32 for the step), and writes k and v into the
  pages.  Causal softmax with exp(0) = 1 added to the denominator: a sink whose logit is 0; the
  output times sigmoid(gate), one gate per output, inside the attention kernel.
mlstm   q | k | v | gate in one product, input- and forget-gate logits in another (fp32 out).
  Per head S <- a S + b k v^T, n <- a n + b k with stabilised exponential gates and the read-out
  S^T q / (max(|n . q|, e^-m) + 1e-6); o / rms(o) per head * w * sigmoid(gate).
feed-forward   W_down polynorm(W_up h), or experts W_down (silu(W_gate h) * W_up h) chosen by
  a grouped softmax router over real and identity experts.
"""
from __future__ import annotations

import torch

from .. import ops
from ..parallel.tp import SINGLE, TPContext
from .config import LayeredConfig
from .moe import MoEBuffers, grouped_ok, moe_mlp
from .weights import init_modepel_weights


class ModepelLM:
    stateful = True            # sequences own a state slot (matrix memories)

    def __init__(self, cfg: LayeredConfig, device, tp: TPContext = SINGLE, seed: int = 0,
                 weights: dict | None = None, dtype=torch.bfloat16, moe_ep: bool = False):
        if tp.enabled:
            raise ValueError("layer-list models run at TP = 1")
        self.cfg = cfg
        self.tp = tp
        self.device = torch.device(device)
        self.dtype = dtype
        self.w = weights if weights is not None else init_modepel_weights(cfg, self.device, dtype, seed)
        self.vocab_start = 0
        self.vocab_local = self.w["lm_head"].shape[0]
        # the kernels of this model take no per-head decode work list: one entry per row
        self.hq = self.hkv = 1
        self.kv_k = self.kv_v = self.layer_state = None
        self.norms_folded = False
        if dtype == torch.float32:
            torch.backends.cuda.matmul.allow_tf32 = False
        self._moe_bufs: dict = {}
        self._seq_ids = None
        mixing = [i for i, ly in enumerate(cfg.layers) if ly.mixer.v_mix]
        self.first_mix = mixing[0] if mixing else -1
        self.any_mix = len(mixing) > 1
        self.recurrent = any(ly.mixer.kind == "mlstm" for ly in cfg.layers)
        for ly, lw in zip(cfg.layers, self.w["layers"]):
            m, f = ly.mixer, ly.mlp
            if m.kind == "window_attention":
                lw["inv_freq"], _ = ops.rotary_scaled_freq(m.rot_dims, m.rot_base, m.rot_scaling,
                                                           self.device)
            # the alignment behind the grouped expert GEMMs takes 64 segments, one of which
            # holds the identity pairs
            lw["grouped"] = bool(f is not None and f.kind == "moe" and self.device.type == "cuda"
                                 and dtype == torch.bfloat16 and f.experts + (f.identity > 0) <= 64
                                 and grouped_ok(lw["w13"], lw["w2e"]))

    # engine hooks shared with the other decoders
    def fold_norms(self) -> bool:
        return False

    def tile_decode_weights(self, mode: str | None = None) -> int:
        return 0

    def attach_kv_cache(self, k_pools, v_pools, state=None, layer_state=None) -> None:
        """Per attention layer: K pool [num_blocks, G, block, dim] and V pool [.., vdim];
        layer_state[i] of an mlstm layer: "S" [2*slots, H, dim, vdim], "n" [2*slots, H, dim], "m"
        [2*slots, H], fp32."""
        assert len(k_pools) == self.cfg.n_layers
        self.kv_k, self.kv_v, self.layer_state = k_pools, v_pools, layer_state

    def _decode_work(self, n: int):
        """(sequence index, query block 0) per decode-section sequence; views of two tensors
        that only grow (never inside a graph capture: the warm-up run sizes them)."""
        if self._seq_ids is None or self._seq_ids[0].numel() < n:
            size = max(1024, 2 * n)
            self._seq_ids = (torch.arange(size, dtype=torch.int32, device=self.device),
                             torch.zeros(size, dtype=torch.int32, device=self.device))
        return self._seq_ids[0][:n], self._seq_ids[1][:n]

    def _run_rows(self, m):
        """First row of every scheduled run of the step (decode section, then prefill section;
        -1 for a sequence without rows: padding of a graph step), for the recurrence's grid."""
        if self.device.type != "cuda" or not self.recurrent:
            return None
        parts = []
        if m.dec_q_len is not None and m.dec_q_len.numel():
            parts.append(torch.where(m.dec_q_len > 0, m.dec_q_start, -1))
        if m.pf_q_len is not None and m.pf_q_len.numel():
            parts.append(torch.where(m.pf_q_len > 0, m.pf_q_start + m.num_decode, -1))
        if not parts:
            return None
        return (parts[0] if len(parts) == 1 else torch.cat(parts)).to(torch.int32)

    def weight_bytes(self) -> int:
        tot = sum(v.numel() * v.element_size() for v in self.w.values() if isinstance(v, torch.Tensor))
        for lw in self.w["layers"]:
            tot += sum(t.numel() * t.element_size() for t in lw.values() if isinstance(t, torch.Tensor))
        return tot

    # ------------------------------------------------------------------ mixers
    def _attention(self, li, mx, lw, h, m, v_first):
        T, D, dt, dev = m.num_tokens, m.num_decode, self.dtype, h.device
        H, G, dim, vd = mx.heads, mx.kv_heads, mx.dim, mx.vdim
        kc, vc = self.kv_k[li], self.kv_v[li]
        pr = ops.matmul_nt(h, lw["proj"])
        gate = pr[:, H * dim + G * (dim + vd):]
        q = torch.empty((T, H, dim), dtype=torch.float32, device=dev)
        v_in = v_first if mx.v_mix and li != self.first_mix else None
        v_out = None
        if self.any_mix and li == self.first_mix:
            v_out = v_first = torch.empty((T, G * vd), dtype=torch.float32, device=dev)
        ops.qk_norm_rotary_append(pr, lw["proj_b"], None, None, False, 0, self.cfg.rms_eps,
                                  m.positions[:T], lw["inv_freq"], 1.0, 0, 0, m.slot_mapping[:T], kc, vc,
                                  H, G, dim, dim, vd, 0, q, v_in, lw["vmix"], v_out)
        attn = torch.empty((T, H * vd), dtype=dt, device=dev)
        if D > 0:
            ids, zeros = self._decode_work(m.dec_q_len.shape[0])
            ops.attn_keep_window(q[:D], kc, vc, vd, m.dec_block_tables, m.dec_q_start, m.dec_q_len,
                                 m.dec_kv_len, ids, zeros, lw["sink"], gate[:D], attn[:D], mx.scale,
                                 short_rows=ops.TALK_DECODE_MAX_ROWS)
        if T > D:
            ops.attn_keep_window(q[D:], kc, vc, vd, m.pf_block_tables, m.pf_q_start, m.pf_q_len,
                                 m.pf_kv_len, m.work_seq, m.work_qblk, lw["sink"], gate[D:T],
                                 attn[D:T], mx.scale)
        return ops.matmul_nt(attn, lw["o"]), v_first

    def _mlstm(self, li, mx, lw, h, rows):
        T, H, dim, vd = h.shape[0], mx.heads, mx.dim, mx.vdim
        rs, rb, rf, pos, runs = rows
        st = self.layer_state[li]
        pr = ops.matmul_nt(h, lw["proj"])
        z = ops.matmul_nt(h, lw["zif"], out_dtype=torch.float32)
        a, b = H * dim, 2 * H * dim
        y = ops.mlstm_recurrence(pr[:, :a], pr[:, a:b], pr[:, b:b + H * vd], z, lw["zif_b"], mx.gate_cap,
                                 mx.scale, pr[:, b + H * vd:], lw["gn"], self.cfg.rms_eps, st["S"],
                                 st["n"], st["m"], rs, rb, rf, pos,
                                 torch.empty((T, H * vd), dtype=self.dtype, device=h.device), runs)
        return ops.matmul_nt(y, lw["o"])

    # ------------------------------------------------------------ feed-forward
    def _moe_buffers(self, T: int, f, d: int) -> MoEBuffers:
        cap = 1
        while cap < T:
            cap *= 2
        key = (cap, f.top, f.experts, f.identity > 0, f.ff)
        if key not in self._moe_bufs:
            self._moe_bufs[key] = MoEBuffers.allocate(cap, f.top, f.experts + (f.identity > 0), d, f.ff,
                                                      self.device, self.dtype)
        return self._moe_bufs[key]

    def _moe(self, f, lw, h) -> dict:
        """The mixture as gain_sandwich takes it: the experts' weighted sum, the shared expert
        with its logits, the identity experts' weights with their input."""
        T, dev, n = h.shape[0], h.device, f.experts + f.identity
        z = ops.matmul_nt(h, lw["router"], out_dtype=torch.float32)     # router logits | shared logit
        out = {}
        ident = None
        if f.identity:
            ident = torch.empty((T,), dtype=torch.float32, device=dev)
            out.update(h_in=h, h_weight=ident)
        if f.shared_ff:
            sh = ops.matmul_nt(ops.silu_mul_any(ops.matmul_nt(h, lw["shared_gu"])), lw["shared_down"])
            out.update(y2=sh, y2_logit=z[:, n])

        def route(w, i):
            ops.moe_route_softmax(z, lw["correction"], f.experts, f.top, f.groups, f.keep,
                                  f.router_scale, i, w, ident)

        if lw["grouped"]:
            # the sparse decoder's alignment, grouped MFMA GEMMs and combine behind this router
            out["y"] = moe_mlp(h, lw["router"][:f.experts], lw["w13"], lw["w2e"], f.top,
                               self._moe_buffers(T, f, h.shape[1]), routing=route,
                               spare=f.identity > 0)
            return out
        ids = torch.empty((T, f.top), dtype=torch.int32, device=dev)
        wts = torch.empty((T, f.top), dtype=torch.float32, device=dev)
        route(wts, ids)
        out["y"] = ops.moe_experts(h, ids, wts, lw["w13"], lw["w2e"], None,
                                   torch.empty((T, h.shape[1]), dtype=torch.float32, device=dev))
        return out

    def _mlp(self, f, lw, h) -> dict:
        if f.kind == "moe":
            return self._moe(f, lw, h)
        up = ops.matmul_nt(h, lw["up"])
        return {"y": ops.matmul_nt(ops.poly_norm_rows(up, lw["poly"], self.cfg.rms_eps, up), lw["down"])}

    # ------------------------------------------------------------------ forward
    def forward(self, m, taps: list | None = None) -> torch.Tensor:
        """Logits [rows, V] (fp32) of the step.  ``taps``: a list that receives the residual
        stream after every layer (debugging / layer-wise tests)."""
        cfg, w = self.cfg, self.w
        T, eps, dt = m.num_tokens, cfg.rms_eps, self.dtype
        rows = (m.extra["row_state"], m.extra["row_back"], m.extra["row_fwd"], m.positions[:T],
                self._run_rows(m))
        x = ops.embed_rows(m.input_ids[:T], w["embed"])
        h = torch.empty((T, cfg.hidden), dtype=dt, device=x.device)
        ops.gain_sandwich(x, g_pre=w["layers"][0]["norm1"], eps=eps, out=h)
        v_first = None
        for li, ly in enumerate(cfg.layers):
            lw, mx, f = w["layers"][li], ly.mixer, ly.mlp
            last = li + 1 == cfg.n_layers
            nxt = w["final_norm"] if last else w["layers"][li + 1]["norm1"]
            if mx.kind == "mlstm":
                y = self._mlstm(li, mx, lw, h, rows)
            else:
                y, v_first = self._attention(li, mx, lw, h, m, v_first)
            post = lw["norm1b"]
            parts = {"y": y}
            if f is not None:
                ops.gain_sandwich(x, g_post=post, g_pre=lw["norm2"], eps=eps, out=h, **parts)
                parts, post = self._mlp(f, lw, h), lw["norm2b"]
            # the last layer's kernel applies the final norm
            ops.gain_sandwich(x, g_post=post, g_pre=nxt, eps=eps, out=h, **parts)
            if taps is not None:
                taps.append(x.clone())
        hn = h if m.logits_idx is None else h.index_select(0, m.logits_idx.long())
        return ops.matmul_nt(hn, w["lm_head"], out_dtype=torch.float32)
