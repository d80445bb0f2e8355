"""Lizesun decoder: pre-norm layers whose norm is a Dynamic Tanh (no mean, no variance) and whose mixer is
a delta rule with a decay per key channel, attention inside chunks of the sequence with values mixed
across layers, or a parallel pair — windowed attention with kept first tokens and a learned sink beside
a matrix memory with exponential gates — summed with two constants; the feed-forward squares a ReLU.

Per layer (the same code for prompts, portions of prompts, single decoded tokens and any mix of them in
one batch; only the attention launch and the scan differ):

    h     = add_tanh_norm(x, pending)           H18 (HIP): residual add + tanh(alpha x) * w + b
    proj  = h @ W_in^T                          one GEMM for every projection that reads h
    channel_delta:
      s     = channel_delta_prep(proj)          C10 (HIP): short convolutions, silu, unit vectors, step
                                                size, low-rank decay path
      o     = state_scan(s)                     C5 (HIP): the recurrence, state in registers
      pending = head_norm_gate(o, proj_g1 @ W_g2^T) @ Wo^T          C6 (HIP)
    attention:
      q     = qk_prep(proj)                     H2 (HIP): biases, per-head norms with weights, values mixed
                                                with the first such layer's; keys / values -> paged cache
      pending = gqa_attention(q) @ Wo^T         H19 / H3 (HIP): chunks, soft cap, one gate per head
    parallel:
      q     = qk_prep(proj)                     H2: rotation in halves, then the norms
      cat[:, :left] = gqa_attention(q)          H19 / H3: window, kept first keys, learned sinks, scaled result
      s     = memory_prep(proj)                 C11 (HIP): gates, running maximum, weighted keys
      o     = state_scan(s)                     C5: the state and, as one more column, its normaliser
      cat[:, left:] = head_norm_gate(o)         C6: read-out divided, per-head norm, weight, gate, scale
      pending = cat @ [Wo_left | Wo_right]^T    one GEMM for both halves
    h     = add_tanh_norm(x, pending)           H18
    pending = relu2(h @ Wup^T) @ Wdown^T        C8 (HIP) between two GEMMs

The residual stream, every norm, positions and angles, scores and softmax, the convolution states,
decays, step sizes, gates, unit vectors and the whole recurrences are fp32 whatever the model dtype;
GEMM operands, the activations between them and the key / value cache take the model dtype.
"""
from __future__ import annotations

from typing import Dict, Optional

import torch
import torch.nn.functional as F

from ..ops import hybrid as Hy
from ..parallel.tp import TPInfo
from .config import DeltaSpec, GroupedAttentionSpec, MatrixMemorySpec, ModelConfig, ParallelSpec, attention_of
from .goganex import GoganexModel
from .llama import AttnMeta


class LizesunModel(GoganexModel):
    """Shares the row bookkeeping, attention tile maps, scan chunk lists, split-key workspaces and decode
    GEMMs of :class:`GoganexModel`; the layers, the cache and the forward are its own."""
    _DEC_LINEARS = ("w_in", "w_out", "mix.g2", "mlp.up", "mlp.down")

    def __init__(self, cfg: ModelConfig, weights: Dict[str, torch.Tensor], device, dtype=torch.bfloat16,
                 tp: Optional[TPInfo] = None):
        self.cfg = cfg
        self.w = weights
        self.tp = tp or TPInfo()
        if self.tp.size > 1:
            raise ValueError(f"{cfg.name}: tensor parallelism is not supported for this architecture")
        self.device = torch.device(device)
        self.dtype = dtype
        if dtype == torch.float32:      # true fp32 products: no reduced-precision matrix mode
            torch.backends.cuda.matmul.allow_tf32 = False
            torch.backends.cudnn.allow_tf32 = False
        self.n_heads, self.n_kv_heads, self.head_dim = cfg.n_heads, cfg.n_kv_heads, cfg.head_dim
        f32 = torch.float32
        mixing = [i for i, ls in enumerate(cfg.layers) if isinstance(ls.mixer, GroupedAttentionSpec) and ls.mixer.v_mix]
        self.first_mix = mixing[0] if mixing else None      # the layer whose values the later ones mix in
        self.layers: Dict[int, Dict[str, torch.Tensor]] = {}
        for i, ls in enumerate(cfg.layers):
            p, m = f"l{i}.", ls.mixer
            lw = {k[len(p):]: v for k, v in weights.items() if k.startswith(p)}
            if isinstance(m, DeltaSpec):
                names = ["q", "k", "v", "b", "a1", "g1"]
            elif isinstance(m, ParallelSpec):
                names = ["left.q", "left.k", "left.v", "right.q", "right.k", "right.v", "right.g", "right.i", "right.f"]
            else:
                names = ["q", "k", "v", "g"]
            off: Dict[str, int] = {}
            at, parts = 0, []
            for n in names:
                off[n] = at
                parts.append(lw.pop("mix." + n))
                at += parts[-1].shape[0]
            if at % 16:                 # whole tiles of the decode GEMM: zero rows that nothing reads
                parts.append(parts[0].new_zeros(16 - at % 16, cfg.hidden))
            lw["w_in"], lw["off"] = torch.cat(parts).contiguous(), off
            fp = []
            if isinstance(m, DeltaSpec):
                lw["w_out"] = lw.pop("mix.o")
                lw["conv_w"] = torch.cat([lw.pop(f"mix.{n}.conv") for n in "qkv"]).to(f32).contiguous()
                lw["neg_rate"] = -torch.exp(lw.pop("mix.A_log").to(f32)).contiguous()
                lw["a2_t"] = lw.pop("mix.a2").to(f32).t().contiguous()          # [rank, heads * dim]
                lw["gate_rank"] = lw["mix.g2"].shape[1]
                fp += ["mix.dt_bias", "mix.norm"]
            elif isinstance(m, ParallelSpec):
                lw["w_out"] = torch.cat([lw.pop("mix.left.o"), lw.pop("mix.right.o")], 1).contiguous()
                lw["freq"] = Hy.rotary_halves_table(m.left.rot, self.device)[0]
                fp += ["mix.left.sink", "mix.right.norm", "mix.right.i.b", "mix.right.f.b"]
            else:
                lw["w_out"] = lw.pop("mix.o")
                lw["lam"] = float(lw.pop("mix.vmix")) if m.v_mix else 0.0
                fp += ["mix.q.b", "mix.k.b", "mix.v.b", "mix.q.norm", "mix.k.norm"]
            for n in ("norm1", "norm2"):
                if n in lw:
                    lw[n + ".alpha"] = float(lw[n + ".alpha"])
                    fp += [n, n + ".b"]
            for n in fp:
                lw[n] = lw[n].to(f32).contiguous()
            self.layers[i] = lw
        self.final_norm, self.final_bias = (weights[n].to(f32).contiguous() for n in ("final.norm", "final.norm.b"))
        self.final_alpha = float(weights["final.norm.alpha"])
        self._dec = None
        self._split_ws = None
        self._static = {}
        self._ws = {}

    # ---- cache ------------------------------------------------------------------------------------
    def cache_shapes(self):
        return [(a.kv_heads, a.dim, a.vdim) if a is not None else None for a in map(attention_of, self.cfg.layers)]

    def make_cache(self, num_blocks: int, block_size: int, device, dtype, n_slots: int):
        from ..engine.kv_cache import GroupedKVCache
        rec, short, gates = [], [], []
        for ls in self.cfg.layers:
            m = ls.mixer.right if isinstance(ls.mixer, ParallelSpec) else ls.mixer
            rec.append(getattr(m, "state_size", 0))
            short.append((m.conv_channels, m.conv) if isinstance(m, DeltaSpec) else None)
            gates.append(m.heads if isinstance(m, MatrixMemorySpec) else 0)
        return GroupedKVCache(self.cache_shapes(), self.cfg.hidden, rec, num_blocks, block_size, device, dtype,
                              n_slots=n_slots, shift_layers=[False] * len(rec), short_conv=short, gate_heads=gates)

    def cache_bytes_per_block(self, block_size: int, dtype_bytes: int) -> int:
        return max(1, sum(sh[0] * (sh[1] + sh[2]) for sh in self.cache_shapes() if sh is not None)) * block_size * dtype_bytes

    # ---- forward ----------------------------------------------------------------------------------
    def _mask_splits(self, a: GroupedAttentionSpec, rows: int, kt: int) -> int:
        """Key ranges per decoded row: as many as fill the chip, but no more than the key tiles a row's
        window (with its kept first keys) or chunk can touch."""
        splits = self.decode_splits(rows, a.kv_heads)
        span = a.window or a.chunk
        if splits > 1 and span > 0:
            splits = max(1, min(splits, (span + kt - 1) // kt + 1 + (a.keep_first + kt - 1) // kt))
        return splits

    def _attend(self, q, a: GroupedAttentionSpec, l, kv, meta, b, decode, **kw):
        T = q.shape[0]
        plan = Hy.attention_plan(a, T, kv.block_size, self.dtype, decode) if q.is_cuda else None
        splits = self._mask_splits(a, T, plan.key_tile) if decode and plan is not None else 1
        return Hy.gqa_attention(q, kv.k_layer(l), kv.v_layer(l), meta.block_tables, b.cu_q, b.start_pos, a.scale, None, 0.0,
                                tiles=self._tiles(meta, plan.rows, b) if plan is not None else None, plan=plan,
                                num_splits=splits, workspace=self._workspace(T, a, splits), out_dtype=self.dtype,
                                window=a.window, keep_first=a.keep_first, chunk=a.chunk, softcap=a.softcap, **kw)

    def _attention(self, proj, a: GroupedAttentionSpec, lw, l, first, positions, kv, meta, b, decode):
        off = lw["off"]
        mix = None
        if a.v_mix and first is not None:
            mix = (first[0], first[1]["off"]["v"], first[1]["mix.v.b"], lw["lam"])
        q = Hy.qk_prep(proj, a, off["q"], off["k"], off["v"], None, self.cfg.norm_eps, positions, kv.k_layer(l),
                       kv.v_layer(l), meta.slot_mapping, self.dtype, q_weight=lw["mix.q.norm"], k_weight=lw["mix.k.norm"],
                       q_bias=lw["mix.q.b"], k_bias=lw["mix.k.b"], v_bias=lw["mix.v.b"], mix=mix)
        return self._attend(q, a, l, kv, meta, b, decode, gate=proj, gate_off=off["g"], gate_heads=True)

    def _parallel(self, proj, m: ParallelSpec, lw, l, positions, kv, meta, b, decode):
        """Both halves of a parallel mixer into one activation buffer [T, left | right]."""
        a, r, off = m.left, m.right, lw["off"]
        nl, nr = a.heads * a.vdim, r.heads * r.vdim
        cat = torch.empty(proj.shape[0], nl + nr, dtype=self.dtype, device=proj.device)
        q = Hy.qk_prep(proj, a, off["left.q"], off["left.k"], off["left.v"], lw["freq"], self.cfg.norm_eps, positions,
                       kv.k_layer(l), kv.v_layer(l), meta.slot_mapping, self.dtype)
        self._attend(q, a, l, kv, meta, b, decode, sinks=lw["mix.left.sink"], out_scale=m.left_scale, out_buf=cat, out_off=0)
        q, k, w, v, floors = Hy.memory_prep(proj, r, off["right.q"], off["right.k"], off["right.v"], off["right.i"],
                                            off["right.f"], lw["mix.right.i.b"], lw["mix.right.f.b"], kv.gmax[l], b.cu_q,
                                            b.start_pos, b.slots, step=decode)
        chunks = self._scan_chunks(meta, b) if proj.is_cuda and not decode else None
        o = Hy.state_scan(q, k, v, w, None, None, None, kv.rec[l], b.cu_q, b.start_pos, b.slots, r.heads, r.dim, r.vdim + 1,
                          chunks=chunks)
        return Hy.head_norm_gate(o, lw["mix.right.norm"], r.vdim, proj, off["right.g"], "sigmoid", self.cfg.norm_eps,
                                 m.right_scale, cat, nl, floors=floors)

    def _delta(self, proj, m: DeltaSpec, lw, l, positions, kv, meta, b, decode, skinny):
        off = lw["off"]
        four, v = Hy.channel_delta_prep(proj, m, off["q"], off["b"], off["a1"], lw["a2_t"], lw["conv_w"], kv.sconv[l],
                                        lw["neg_rate"], lw["mix.dt_bias"], b.row_seq, positions, b.start_pos, b.slots,
                                        shift_state=decode)
        if not decode:
            Hy.conv_state_update(proj, off["q"], m.conv_channels, kv.sconv[l], 0, b.cu_q, b.start_pos, b.slots)
        o = Hy.state_scan(four[0], four[1], v, four[2], four[1], four[3], None, kv.rec[l], b.cu_q, b.start_pos, b.slots,
                          m.heads, m.dim, m.vdim, chunks=self._scan_chunks(meta, b) if proj.is_cuda and not decode else None)
        low = proj[:, off["g1"]:off["g1"] + lw["gate_rank"]]
        gate = self._linear(low.contiguous() if skinny else low, l, "mix.g2", skinny)
        out = torch.empty(proj.shape[0], m.heads * m.vdim, dtype=self.dtype, device=proj.device)
        return Hy.head_norm_gate(o, lw["mix.norm"], m.vdim, gate, 0, "sigmoid", self.cfg.norm_eps, 1.0, out, 0)

    def forward(self, ids: torch.Tensor, positions: torch.Tensor, kv, meta: AttnMeta,
                hidden: Optional[torch.Tensor] = None, keep_layers: Optional[list] = None) -> torch.Tensor:
        """Logits [rows, vocab] fp32: every row of a decode step, ``meta.last_rows`` of a varlen
        step (all rows when it is None). ``keep_layers``: a list that receives the residual stream
        after every layer (debugging / tests)."""
        cfg, adt = self.cfg, self.dtype
        T = ids.shape[0]
        b = self._rows(positions, meta)
        decode = meta.kind == "decode"
        skinny = decode and T <= 32 and ids.is_cuda and self.use_skinny and bool(self.decode_weights())
        x = F.embedding(ids, self.w["embed"]).float()
        if cfg.embed_scale != 1.0:
            x = x * cfg.embed_scale
        pend = first = None         # a sublayer output whose add is still to come; the first mixing layer's projection
        for l, ls in enumerate(cfg.layers):
            lw, m = self.layers[l], ls.mixer
            h = Hy.add_tanh_norm(x, pend, lw["norm1.alpha"], lw["norm1"], lw["norm1.b"], adt)
            proj = self._linear(h, l, "w_in", skinny)
            if isinstance(m, DeltaSpec):
                o = self._delta(proj, m, lw, l, positions, kv, meta, b, decode, skinny)
            elif isinstance(m, ParallelSpec):
                o = self._parallel(proj, m, lw, l, positions, kv, meta, b, decode)
            else:
                o = self._attention(proj, m, lw, l, first, positions, kv, meta, b, decode)
                if l == self.first_mix:
                    first = (proj, lw)
            pend = self._linear(o, l, "w_out", skinny)
            if ls.ff:
                h = Hy.add_tanh_norm(x, pend, lw["norm2.alpha"], lw["norm2"], lw["norm2.b"], adt)
                pend = self._linear(Hy.relu2(self._linear(h, l, "mlp.up", skinny), adt), l, "mlp.down", skinny)
            if keep_layers is not None:
                x.add_(pend.float())
                pend = None
                keep_layers.append(x.clone())
        if not decode and meta.last_rows is not None:
            x = x.index_select(0, meta.last_rows)
            pend = pend.index_select(0, meta.last_rows) if pend is not None else None
        xn = Hy.add_tanh_norm(x, pend, self.final_alpha, self.final_norm, self.final_bias, adt)
        return F.linear(xn, self.w["head"]).float()
