"""Vurizen decoder: pre-norm layers (layer norms with bias) whose mixer is a windowed latent attention
— over cached rows of its own or over those of an earlier layer — or a gated linear attention, and
whose feed-forward is a mixture of sigmoid-routed gated experts chosen among the best groups. Every
sublayer output is multiplied by a learned number per channel and one constant before it is added.

Per layer (the same code for prompts, portions of prompts, single decoded tokens and any mix of
them in one batch; only the attention launch and the scan differ):

    h     = add_layer_norm(x, pending)          H13 (HIP): pending output scaled per channel, added to
                                                the fp32 residual, layer norm
    proj  = h @ W_in^T                          one GEMM for every projection that reads h
    latent_attention:
      latent_prep(proj)                         L2 (HIP): latent norm, rotated key part -> the paged
                                                cache (not in a layer that reads another's rows)
      q_lat = q_nope . Wuk                      hipBLASLt (batched over heads; decode steps: L7 (HIP)):
                                                the query moves into latent space, so keys are the
                                                cached rows
      o_lat = latent_attention(q_lat, q_rot)    L3 (HIP): sliding window, all heads of a row share
                                                each staged key tile (bf16: MFMA)
      pending = (o_lat . Wuv) @ Wo^T            as q_lat, then the output GEMM
    gla:
      q, k, decay, v = gla_prep(proj)           C9 (HIP): low-rank decay path, decays in fp32
      o     = state_scan(q, k, v, decay)        C5 (HIP): the recurrence; long spans in parallel chunks
      pending = head_norm_gate(o) @ Wo^T        C6 (HIP): per-head norm, weight, silu gate
    h     = add_layer_norm(x, pending)          H13 (it also combines the experts' rows of the layer before)
    idx, wt = route_groups(h, Wrouter)          H11 (HIP): fp32 scores, correction, groups, choice
    pending = moe_experts(h, idx, wt)           H14 - H16 (HIP): rows sorted by expert and two grouped
                                                matrix-core launches; decode steps: an expert's
                                                weights read once for all rows that chose it

The residual stream, every norm, positions and angles, scores and softmax, the router, decays and the
whole recurrence are fp32 whatever the model dtype; GEMM operands, the activations between them and
the latent cache take the model dtype.
"""
from __future__ import annotations

from typing import Dict, Optional

import torch
import torch.nn.functional as F

from ..ops import hybrid as Hy
from ..ops import latent as L
from ..parallel.tp import TPInfo
from .config import GLASpec, LatentAttentionSpec, ModelConfig
from .goganex import GoganexModel
from .llama import AttnMeta


class VurizenModel(GoganexModel):
    """Shares the row bookkeeping, attention tile maps, scan chunk lists and decode GEMMs of
    :class:`GoganexModel`; the layers, the cache and the forward are its own."""
    _DEC_LINEARS = ("w_in", "mix.o")

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
        self.n_heads, self.n_kv_heads, self.head_dim = cfg.n_heads, 1, cfg.head_dim
        f32 = torch.float32
        self.layers: Dict[int, Dict[str, torch.Tensor]] = {}
        for i, ls in enumerate(cfg.layers):
            p, m = f"l{i}.", ls.mixer
            lw = {k[len(p):]: v for k, v in weights.items() if k.startswith(p)}
            off: Dict[str, int] = {}
            at, parts = 0, []
            for n in ("q", "k", "v", "g", "a1") if isinstance(m, GLASpec) else ("q", "dkv"):
                if "mix." + n in lw:
                    off[n] = at
                    parts.append(lw.pop("mix." + n))
                    at += parts[-1].shape[0]
            lw["w_in"] = torch.cat(parts).contiguous()
            lw["off"] = off
            if isinstance(m, GLASpec):
                lw["a2_t"] = lw.pop("mix.a2").to(f32).t().contiguous()        # [rank, heads * dim]
            else:
                # per-head up-projections: q_lat[h] = q_nope[h] @ uk_h[h], o[h] = o_lat[h] @ uv_ht[h]
                lw["uk_h"] = lw.pop("mix.uk").view(m.heads, m.dim, m.kv_rank).contiguous()
                lw["uv_h"] = lw.pop("mix.uv").view(m.heads, m.vdim, m.kv_rank).contiguous()
                lw["uk_ht"], lw["uv_ht"] = (lw[n].transpose(1, 2).contiguous() for n in ("uk_h", "uv_h"))
                lw["rot"] = L.rotary_table(m.rot, self.device)
            if ls.ff:
                E = ls.moe.experts
                lw["w_gu"] = torch.stack([torch.cat([lw.pop(f"mlp.e{e}.gate"), lw.pop(f"mlp.e{e}.up")])
                                          for e in range(E)]).contiguous()                                # [E, 2F, W]
                lw["w_down"] = torch.stack([lw.pop(f"mlp.e{e}.down") for e in range(E)]).contiguous()     # [E, W, F]
            for n in ("ls1", "ls2"):        # layer scale and the residual multiplier in one number per channel
                if n in lw:
                    lw[n] = (lw[n].to(f32) * cfg.residual_mult).contiguous()
            for n in ("norm1", "norm1.b", "norm2", "norm2.b", "mix.dkv.norm", "mix.norm", "mix.a2.b", "mlp.router",
                      "mlp.correction"):
                if n in lw:
                    lw[n] = lw[n].to(f32).contiguous()
            self.layers[i] = lw
        self.final_norm, self.final_bias = (weights[n].to(f32).contiguous() for n in ("final.norm", "final.norm.b"))
        self._dec = None
        self._split_ws = None
        self._static = {}
        self._ws = {}

    # ---- cache ------------------------------------------------------------------------------------
    def cache_row_dims(self):
        return [m.cache_row if isinstance(m, LatentAttentionSpec) and m.kv_from is None else None
                for m in (ls.mixer for ls in self.cfg.layers)]

    def make_cache(self, num_blocks: int, block_size: int, device, dtype, n_slots: int):
        from ..engine.kv_cache import LatentKVCache
        mixers = [ls.mixer for ls in self.cfg.layers]
        return LatentKVCache(self.cache_row_dims(), self.cfg.hidden, 0, num_blocks, block_size, device, dtype,
                             n_slots=n_slots, shared=[getattr(m, "kv_from", None) for m in mixers],
                             rec_widths=[m.state_size if isinstance(m, GLASpec) else 0 for m in mixers])

    def cache_bytes_per_block(self, block_size: int, dtype_bytes: int) -> int:
        return max(1, sum(r for r in self.cache_row_dims() if r)) * block_size * dtype_bytes

    # ---- forward ----------------------------------------------------------------------------------
    def _workspace(self, rows: int, m, splits: int) -> Optional[L.LatentWorkspace]:
        if splits <= 1:
            return None
        key = (rows, m.heads, m.kv_rank, splits)
        ws = self._ws.get(key)
        if ws is None:
            ws = self._ws[key] = L.LatentWorkspace(rows, m.heads, m.kv_rank, splits, self.device)
        return ws

    def _latent(self, proj, m: LatentAttentionSpec, lw, l, positions, kv, meta, b, decode):
        """Latent attention of ``proj`` -> the concatenated heads [T, heads * vdim]."""
        adt, T = self.dtype, proj.shape[0]
        rows = kv.layer_rows(l)
        if m.kv_from is None:
            L.latent_prep(proj, m, None, lw["mix.dkv.norm"], self.cfg.norm_eps, positions, rows, meta.slot_mapping, adt,
                          kv_off=lw["off"]["dkv"], table=lw["rot"])
        q = proj[:, :m.heads * (m.dim + m.rot_dim)].unflatten(1, (m.heads, m.dim + m.rot_dim))
        qn = q[:, :, :m.dim]
        few = decode and L.head_product_fits(qn, lw["uk_ht"]) and m.kv_rank % 8 == 0
        if few:
            q_lat = torch.empty(m.heads, T, m.kv_rank, dtype=adt, device=proj.device)
            L.head_product(qn, lw["uk_ht"], q_lat.transpose(0, 1))
        else:
            q_lat = torch.bmm(qn.transpose(0, 1), lw["uk_h"])
        splits = L.window_splits(self.decode_splits(T, 1), m.window) if decode else 1
        tiles = None
        if proj.is_cuda:
            tiles = self._tiles(meta, L.rows_per_tile(m.heads, m.kv_rank, m.rot_dim, adt), b)
        o_lat = L.latent_attention(q_lat, q, m, rows, meta.block_tables, b.cu_q, b.start_pos, None, tiles=tiles,
                                   num_splits=splits, workspace=self._workspace(T, m, splits), out_dtype=adt, table=lw["rot"])
        o = torch.empty(T, m.heads, m.vdim, dtype=adt, device=proj.device)
        if few:
            L.head_product(o_lat.transpose(0, 1), lw["uv_h"], o)
        else:
            torch.bmm(o_lat, lw["uv_ht"], out=o.transpose(0, 1))
        return o.view(T, m.heads * m.vdim)

    def _gla(self, proj, m: GLASpec, lw, l, kv, meta, b, decode):
        """Gated linear attention of ``proj`` -> the normed, gated heads [T, heads * vdim]."""
        off = lw["off"]
        q, k, dec, v = Hy.gla_prep(proj, m, off["q"], off["k"], off["v"], off["a1"], lw["a2_t"], lw["mix.a2.b"])
        chunks = self._scan_chunks(meta, b) if proj.is_cuda and not decode else None
        o = Hy.state_scan(q, k, v, dec, None, None, None, kv.rec[l], b.cu_q, b.start_pos, b.slots, m.heads, m.dim, m.vdim,
                          chunks=chunks)
        out = torch.empty(proj.shape[0], m.heads * m.vdim, dtype=self.dtype, device=proj.device)
        return Hy.head_norm_gate(o, lw["mix.norm"], m.vdim, proj, off["g"], "silu", self.cfg.norm_eps, 1.0, out, 0)

    def forward(self, ids: torch.Tensor, positions: torch.Tensor, kv, meta: AttnMeta,
                hidden: Optional[torch.Tensor] = None, keep_layers: Optional[list] = None) -> torch.Tensor:
        """Logits [rows, vocab] fp32: every row of a decode step, ``meta.last_rows`` of a varlen
        step (all rows when it is None). ``keep_layers``: a list that receives the residual stream
        after every layer (debugging / tests)."""
        cfg, adt = self.cfg, self.dtype
        eps = cfg.norm_eps
        T = ids.shape[0]
        b = self._rows(positions, meta)
        decode = meta.kind == "decode"
        skinny = decode and T <= 32 and ids.is_cuda and self.use_skinny and bool(self.decode_weights())
        x = F.embedding(ids, self.w["embed"]).float()
        pend = scale = None         # a sublayer output whose scaled add is still to come
        for l, ls in enumerate(cfg.layers):
            lw, m = self.layers[l], ls.mixer
            h = Hy.add_layer_norm(x, pend, scale, lw["norm1"], lw["norm1.b"], eps, adt)
            proj = self._linear(h, l, "w_in", skinny)
            if isinstance(m, GLASpec):
                o = self._gla(proj, m, lw, l, kv, meta, b, decode)
            else:
                o = self._latent(proj, m, lw, l, positions, kv, meta, b, decode)
            pend, scale = self._linear(o, l, "mix.o", skinny), lw["ls1"]
            if ls.ff:
                h = Hy.add_layer_norm(x, pend, scale, lw["norm2"], lw["norm2.b"], eps, adt)
                idx, wt = Hy.route_groups(h, lw["mlp.router"], ls.moe, lw["mlp.correction"])
                pend, scale = Hy.moe_experts(h, idx, wt, lw["w_gu"], lw["w_down"], adt, combine=False), lw["ls2"]
            if keep_layers is not None:
                x.add_((pend.combine(torch.float32) if isinstance(pend, Hy.ExpertRows) else pend.float()) * scale)
                pend = None
                keep_layers.append(x.clone())
        if not decode and meta.last_rows is not None:
            x = x.index_select(0, meta.last_rows)
            if isinstance(pend, Hy.ExpertRows):
                pend = pend.select(meta.last_rows)
            elif pend is not None:
                pend = pend.index_select(0, meta.last_rows)
        xn = Hy.add_layer_norm(x, pend, scale, self.final_norm, self.final_bias, eps, adt)
        return F.linear(xn, self.w["head"]).float()
