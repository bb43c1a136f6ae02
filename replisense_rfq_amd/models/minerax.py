"""Minerax: layers of softcapped attention and the channel-wise gated delta rule side by side, or
of windowed latent attention with a rotated key part, around several residual streams, with gated
tanh-gelu feed-forwards, on the kernels of csrc/kernels/mix_*.hip.

Every row holds S residual streams x_1 .. x_S (fp32):

  x_s = embed[token] for all s
  per sublayer (mixer, feed-forward):
    u = sum_s in[s] x_s;  y = sublayer(layer_norm(u) w)
    x_t <- sum_s mix[s, t] x_s + out[t] y        with the previous streams on the right
  logits = head . (layer_norm(sum_s x_s) w_final) * logit_scale

The update of the streams, the next sublayer's weighted sum and its norm are one kernel
(streams_norm), which also starts the streams from the embedding table.  Mixers:

parallel   the projections of both sides in one product.
  left   one kernel (qk_norm_rotary_append) convolves q, k and v over time (the last taps - 1
    projected rows are per-sequence state), norms q and k over the whole projection, rotates
    the first rot_dims of every head (half split) and writes k and v into the pages; causal
    softmax over cap * tanh(score / cap).
  right   q, k, v pass a causal convolution + silu, q and k become unit vectors; gated delta rule
    with a decay per key channel (gated_linear_recurrence); o / rms(o) * w * sigmoid(gate).
  Both sides write their halves of one row, already times left_scale and right_scale, and the two
  output projections are one product.
latent_attention   q | dkv | gate in one product; the page row is [normed latent | rotated key
  part] (neighbouring pairs); scores and weighted sums in the latent space inside a sliding
  window, softmax with a sink; W_uv per head, then sigmoid(gate) per output while the heads are
  laid side by side (gate_heads).
"""
from __future__ import annotations

import torch

from .. import ops
from ..parallel.tp import SINGLE, TPContext
from .config import LayeredConfig
from .weights import init_minerax_weights

UNIT_EPS = 1e-6            # q, k of the delta rule: y / sqrt(sum(y^2) + UNIT_EPS)


class MineraxLM:
    stateful = True            # sequences own a state slot (recurrent matrices, convolution inputs)

    def __init__(self, cfg: LayeredConfig, device, tp: TPContext = SINGLE, seed: int = 0,
                 weights: dict | None = None, dtype=torch.bfloat16, moe_ep: bool = False):
        if tp.enabled:
            raise ValueError("layer-list models run at TP = 1")
        self.cfg = cfg
        self.tp = tp
        self.device = torch.device(device)
        self.dtype = dtype
        self.w = weights if weights is not None else init_minerax_weights(cfg, self.device, dtype, seed)
        self.vocab_start = 0
        self.vocab_local = self.w["lm_head"].shape[0]
        # the kernels of this model take no per-head decode work list: one entry per row
        self.hq = self.hkv = 1
        self.kv_k = self.kv_v = self.layer_state = None
        self.norms_folded = False
        if dtype == torch.float32:
            torch.backends.cuda.matmul.allow_tf32 = False
        self._seq_ids = None
        self.recurrent = any(ly.mixer.kind == "parallel" for ly in cfg.layers)
        # (layer, 1: mixer | 2: feed-forward) in the order they run
        self.sublayers = [(i, q) for i, ly in enumerate(cfg.layers)
                          for q in ((1, 2) if ly.mlp is not None else (1,))]
        for ly, lw in zip(cfg.layers, self.w["layers"]):
            m = ly.mixer.paged
            lw["inv_freq"], lw["rot_mult"] = ops.rotary_scaled_freq(m.rot_dims, m.rot_base,
                                                                    m.rot_scaling, self.device)

    # engine hooks shared with the other decoders
    def fold_norms(self) -> bool:
        return False

    def tile_decode_weights(self, mode: str | None = None) -> int:
        return 0

    def attach_kv_cache(self, k_pools, v_pools, state=None, layer_state=None) -> None:
        """Per layer: K pool [num_blocks, G, block, dim] and V pool [.., vdim] (parallel), or one pool
        [num_blocks, 1, block, kv_rank + rot_dim] (latent attention); layer_state[i] of a parallel
        layer: "0.conv" [2*slots, taps-1, channels] of the attention, "1.conv" and "1.S" [2*slots,
        H, dim, vdim] of the delta rule, fp32."""
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
    def _attend(self, m, mx, q, kc, vc, vdim, sink, out, out_mult=1.0):
        """Both sections of the step through attn_keep_window."""
        T, D = m.num_tokens, m.num_decode
        if D > 0:
            ids, zeros = self._decode_work(m.dec_q_len.shape[0])
            ops.attn_keep_window(q[:D], kc, vc, vdim, m.dec_block_tables, m.dec_q_start, m.dec_q_len,
                                 m.dec_kv_len, ids, zeros, sink, None, out[:D], mx.scale, mx.window,
                                 short_rows=ops.TALK_DECODE_MAX_ROWS, softcap=mx.softcap,
                                 out_mult=out_mult)
        if T > D:
            ops.attn_keep_window(q[D:], kc, vc, vdim, m.pf_block_tables, m.pf_q_start, m.pf_q_len,
                                 m.pf_kv_len, m.work_seq, m.work_qblk, sink, None, out[D:T], mx.scale,
                                 mx.window, softcap=mx.softcap, out_mult=out_mult)

    def _parallel(self, li, mx, lw, h, m, rows):
        T, dt, dev, eps = m.num_tokens, self.dtype, h.device, self.cfg.rms_eps
        (a, b), st, seg = mx.parts, self.layer_state[li], lw["seg"]
        rs, rb, rf, pos, runs = rows
        pr = ops.matmul_nt(h, lw["proj"])

        def cols(name):
            at, n = seg[name]
            return pr[:, at:at + n]

        na, nb = a.heads * a.vdim, b.heads * b.vdim
        y = torch.empty((T, na + nb), dtype=dt, device=dev)
        # attention
        q = torch.empty((T, a.heads, a.dim), dtype=torch.float32, device=dev)
        ops.qk_norm_rotary_append(pr, None, lw["qn"], lw["kn"], True, a.dim, eps, pos, lw["inv_freq"],
                                  lw["rot_mult"], 0, 0, m.slot_mapping[:T], self.kv_k[li], self.kv_v[li],
                                  a.heads, a.kv_heads, a.dim, a.dim, a.vdim, 0, q,
                                  conv=(lw["conv_l"], st["0.conv"], rs, rb, rf))
        self._attend(m, a, q, self.kv_k[li], self.kv_v[li], a.vdim, None, y[:, :na], mx.part_scales[0])
        # delta rule
        G, nk = b.kv_heads, b.kv_heads * b.dim
        qkv = torch.empty((T, seg["right"][1]), dtype=torch.float32, device=dev)
        ops.conv_act_heads(cols("right"), lw["conv_r"], st["1.conv"], rs, rb, rf, pos, 2 * G, b.dim,
                           UNIT_EPS, qkv)
        z = ops.matmul_nt(cols("a1"), lw["a2"], out_dtype=torch.float32)
        gate = ops.matmul_nt(cols("g1"), lw["g2"])
        ops.gated_linear_recurrence(
            qkv[:, :nk].unflatten(1, (G, b.dim)), qkv[:, nk:2 * nk].unflatten(1, (G, b.dim)),
            qkv[:, 2 * nk:].unflatten(1, (b.heads, b.vdim)), z, lw["rate"], lw["zbias"], 1.0, cols("b"),
            gate, True, lw["gn"], eps, b.scale, st["1.S"], rs, rb, rf, pos, y[:, na:], runs)
        return ops.matmul_nt(y, lw["o"])

    def _latent_attention(self, li, mx, lw, h, m):
        T, dt, dev = m.num_tokens, self.dtype, h.device
        H, dim, rd, R, vd = mx.heads, mx.dim, mx.rot_dim, mx.kv_rank, mx.vdim
        pool = self.kv_k[li]
        pr = ops.matmul_nt(h, lw["proj"])                   # q | dkv | gate
        nq, (g0, gn) = H * (dim + rd), lw["seg"]["g"]
        # one (R + rd)-wide fp32 query per head: the plain part carried into the latent space (read
        # as the projection left it) beside the rotated part
        q = torch.empty((T, H, R + rd), dtype=torch.float32, device=dev)
        qn = pr[:, :nq].unflatten(1, (H, dim + rd))[:, :, :dim].transpose(0, 1)
        ops.bmm_f32(qn, lw["uk"], out=q[:, :, :R].transpose(0, 1))
        ops.qk_norm_rotary_append(pr, None, None, lw["dkv_norm"], False, R, self.cfg.rms_eps,
                                  m.positions[:T], lw["inv_freq"], lw["rot_mult"], dim, R,
                                  m.slot_mapping[:T], pool, None, H, 1, dim + rd, R + rd, 0, 2, q[:, :, R:],
                                  neighbours=mx.rot_neighbours)
        lat = torch.empty((T, H * R), dtype=dt, device=dev)
        self._attend(m, mx, q, pool, pool, R, lw["sink"], lat)
        ov = torch.bmm(lat.view(T, H, R).transpose(0, 1), lw["uv_t"])               # [H, T, vdim]
        y = ops.gate_heads(ov, pr[:, g0:g0 + gn], torch.empty((T, H * vd), dtype=dt, device=dev))
        return ops.matmul_nt(y, lw["o"])

    def _mlp(self, lw, h):
        return ops.matmul_nt(ops.gelu_glu_rows(ops.matmul_nt(h, lw["gate_up"])), lw["down"])

    # ------------------------------------------------------------------ forward
    def forward(self, m, taps: list | None = None) -> torch.Tensor:
        """Logits [rows, V] (fp32) of the step.  ``taps``: a list that receives the sum of the
        residual streams after every layer (debugging / layer-wise tests)."""
        cfg, w = self.cfg, self.w
        T, eps = m.num_tokens, cfg.rms_eps
        rows = (m.extra["row_state"], m.extra["row_back"], m.extra["row_fwd"], m.positions[:T],
                self._run_rows(m))
        x = torch.empty((T, cfg.streams, cfg.hidden), dtype=torch.float32, device=self.device)
        h = torch.empty((T, cfg.hidden), dtype=self.dtype, device=self.device)
        subs, lws = self.sublayers, w["layers"]
        ops.streams_norm(x, w_in=lws[0]["hc1_in"], w=lws[0]["norm1"], eps=eps, out=h,
                         ids=m.input_ids[:T], table=w["embed"])
        for n, (li, q) in enumerate(subs):
            lw, mx = lws[li], cfg.layers[li].mixer
            if q == 2:
                y = self._mlp(lw, h)
            elif mx.kind == "parallel":
                y = self._parallel(li, mx, lw, h, m, rows)
            else:
                y = self._latent_attention(li, mx, lw, h, m)
            last = n + 1 == len(subs)
            if last:                   # the streams' sum through the final norm
                w_in, wn = w["stream_sum"], w["final_norm"]
            else:
                nl, nq = subs[n + 1]
                w_in, wn = lws[nl][f"hc{nq}_in"], lws[nl][f"norm{nq}"]
            ops.streams_norm(x, y, lw[f"hc{q}_mix"], lw[f"hc{q}_out"], w_in, wn, eps, out=h,
                             keep=not last or taps is not None)
            if taps is not None and (last or subs[n + 1][0] != li):
                taps.append(x.sum(1))
        hn = h if m.logits_idx is None else h.index_select(0, m.logits_idx.long())
        return ops.matmul_nt(hn, w["lm_head"], out_dtype=torch.float32)
