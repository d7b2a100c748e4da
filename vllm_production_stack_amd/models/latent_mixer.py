"""Latent attention over the paged pool, for models whose layers have it among their mixers.

A token's cache entry is its RMS-normed KV latent and the rotated key part shared by all heads
(``kv_rank + rot_dim`` values).  Keys and values are never expanded: a head's unrotated query is carried into
latent space (q W_uk, one batched matrix product), the attention kernel scores it against the entries and
returns the probability-weighted latent, and W_uv takes that to the head's value space.  All heads then share
one key/value stream per token.  Large prefill parts (``EXPAND_MIN_ROWS``) are the exception: there the 3.4 x
FLOPs of latent space outweigh what it saves, so values and unrotated keys of every head are expanded for the
step (one library product over the sequences' gathered entries) and the same tile kernel runs over per-head
entries.  Layers with a sliding window visit, and expand, only the pages that hold keys some row of the step sees.

Layers of such a model carry ``spec.mixer`` (LatentMixerSpec), ``w_uk`` [heads, dim, kv_rank], ``w_uv``
[heads, kv_rank, vdim], ``sink`` (fp32 [heads] or None), ``cache_offset``, ``cos_sin`` and ``w_vk`` (derived, None
until needed); layers without latent attention leave these None.
"""

from __future__ import annotations

import torch

from .. import ops
from ..engine.config import LatentMixerSpec
from ..ops.latent import NO_WINDOW
from ..ops.reference import PAGE
from .batch import BatchMeta

# Prefill parts of at least this many rows expand keys and values per head for the step (below, the
# expansion of the whole context costs more than latent space saves)
EXPAND_MIN_ROWS = 256


class LatentAttention:
    """Mixin of model classes (uses ``device``, ``dtype``, ``max_model_len``, ``layers`` and the dict ``_tables``)."""

    def _cos_sin(self, m: LatentMixerSpec) -> torch.Tensor:
        key = (m.rope_base, m.rope_dims)
        t = self._tables.get(key)
        if t is None:
            t = self._tables[key] = ops.build_cos_sin(m.rope_dims, self.max_model_len, m.rope_base, None,
                                                      device=self.device)
        return t

    # derived copies (rebuilt from the weights when needed): per head [W_uv; W_uk], the matrix that
    # expands latents into values and unrotated keys for large prefill parts
    def packed_tensors(self):
        for lw in self.layers:
            if lw.w_vk is not None:
                yield lw.w_vk

    def drop_packed(self) -> None:
        for lw in self.layers:
            lw.w_vk = None

    def _expands(self, m: LatentMixerSpec) -> bool:
        return (self.device.type == "cuda" and self.dtype == torch.bfloat16 and m.kv_rank % 8 == 0 and m.rot_dim % 8 == 0
                and ops.latent_expanded_supported(m.vdim, m.dim + m.rot_dim))

    # ------------------------------------------------------------------ batch description
    def plan_latent_prefill(self, meta: BatchMeta, q_lens: list[int], ctx_lens: list[int], to_dev, mixers) -> None:
        """Which sequence of the prefill part each prefill row belongs to, and the tile kernel's work lists."""
        seq: list[int] = []
        for i, n in enumerate(q_lens):
            seq.extend([i] * n)
        meta.pre_row_seq = to_dev(seq, torch.int32)
        meta.pre_lat_tiles = {}
        meta.pre_expand = {}
        if sum(q_lens) >= EXPAND_MIN_ROWS:
            for heads, window in sorted({(m.heads, m.window) for m in mixers if self._expands(m)}):
                meta.pre_expand[heads, window] = self._plan_expanded(q_lens, ctx_lens, heads, window)
        if self.device.type == "cuda" and self.dtype == torch.bfloat16:
            for heads in sorted({m.heads for m in mixers if ops.latent_mfma_supported(m.kv_rank, m.rot_dim)}):
                tiles = ops.build_latent_tiles(q_lens, ctx_lens, heads)
                meta.pre_lat_tiles[heads] = torch.from_numpy(tiles).pin_memory().to(self.device, non_blocking=True)

    def _plan_expanded(self, q_lens, ctx_lens, heads: int, window: int = 0) -> dict:
        """Layout of a step's expanded entries (one run of pages per prefill sequence and head, from the page of the
        first key its rows see within ``window``) and the tile list over them: 64 consecutive tokens of one head
        per tile."""
        import numpy as np

        first = [max(0, c - n - window + 1) // PAGE if window else 0 for n, c in zip(q_lens, ctx_lens)]
        n_pages = [(c + PAGE - 1) // PAGE - f for c, f in zip(ctx_lens, first)]
        width = max(f + npg for f, npg in zip(first, n_pages))
        bt = np.zeros((len(q_lens) * heads, width), dtype=np.int32)
        parts, base, row = [], [], 0
        total = 0
        for i, (n, ctx, f, npg) in enumerate(zip(q_lens, ctx_lens, first, n_pages)):
            base.append(total)
            for h in range(heads):
                bt[i * heads + h, f:f + npg] = total + h * npg + np.arange(npg)
            k = np.arange(0, n, 64, dtype=np.int64)
            for h in range(heads):
                parts.append(np.stack([np.full_like(k, i * heads + h), row + k, np.minimum(64, n - k), ctx - n + k,
                                       np.full_like(k, h), np.ones_like(k)], axis=1))
            total += heads * npg
            row += n
        tiles = np.concatenate(parts)
        tiles = tiles[np.argsort(-(tiles[:, 3] + tiles[:, 2]), kind="stable")].astype(np.int32)
        return {"first": first, "n_pages": n_pages, "base": base, "total": total,
                "bt": torch.from_numpy(bt).pin_memory().to(self.device, non_blocking=True),
                "tiles": torch.from_numpy(tiles).pin_memory().to(self.device, non_blocking=True)}

    def _expanded_prefill(self, lw, q: torch.Tensor, pool, meta: BatchMeta, plan: dict, out: torch.Tensor, offset: int):
        """Attention of the prefill rows with keys and values expanded per head for this step: the
        sequences' entries are gathered from the pool, one library product makes values and unrotated
        keys of every head, and the tile kernel runs over per-head entries value | unrotated key |
        rotated part.  640 / 2176 of the latent form's FLOPs per query-key pair at 128 + 64 / 128 channels and rank
        512."""
        m: LatentMixerSpec = lw.spec.mixer
        h, v, d, r, kr = m.heads, m.vdim, m.dim, m.rot_dim, m.kv_rank
        if lw.w_vk is None:
            lw.w_vk = torch.cat([lw.w_uv.transpose(1, 2), lw.w_uk], dim=1).reshape(h * (v + d), kr).contiguous()
        wide = v + d + r
        view = pool[:, offset:offset + PAGE * m.entry].view(pool.shape[0], PAGE, m.entry)
        exp = torch.empty((plan["total"], PAGE * wide), dtype=q.dtype, device=q.device)
        for s, (f, npg, base) in enumerate(zip(plan["first"], plan["n_pages"], plan["base"])):
            ent = view[meta.pre_block_tables[s, f:f + npg].long()]                 # [pages, 64, entry]
            vk = ops.linear(ent[:, :, :kr].reshape(npg * PAGE, kr), lw.w_vk)       # [keys, heads * (v + d)]
            dst = exp[base:base + h * npg].view(h, npg, PAGE, wide)
            dst[:, :, :, :v + d] = vk.view(npg, PAGE, h, v + d).permute(2, 0, 1, 3)
            dst[:, :, :, v + d:] = ent[:, :, kr:].unsqueeze(0)
        ops.latent_attention(None, q, exp, 0, plan["bt"], None, meta.positions[meta.num_decode:], lw.sink, m.scale,
                             out=out, tiles=plan["tiles"], window=m.window or NO_WINDOW)

    # ------------------------------------------------------------------ forward
    def latent_heads(self, lw, q: torch.Tensor, pool, meta: BatchMeta, cache_offset: int | None = None) -> torch.Tensor:
        """Head outputs [T, heads, vdim] (contiguous) of the step's query rows q [T, heads, dim + rot_dim] (rotated; a
        view of a wider projection will do).  The step's own cache entries are in the pool already, ``cache_offset``
        elements into its pages (for layers that share tensors but not entries; else the layer's own offset)."""
        m: LatentMixerSpec = lw.spec.mixer
        t = q.shape[0]
        nd = meta.num_decode
        offset = lw.cache_offset if cache_offset is None else cache_offset
        window = m.window or NO_WINDOW
        splits = getattr(meta, "dec_num_splits", 1) or 1
        if m.window:  # no key range shorter than two pages
            splits = max(1, min(splits, ((m.window + PAGE - 1) // PAGE + 1) // 2))
        plan = (getattr(meta, "pre_expand", None) or {}).get((m.heads, m.window)) if self._expands(m) else None
        if plan is not None and meta.num_prefill_seqs > 0:
            # large prefill part: per-head keys and values for this step; decode rows stay in latent space
            o = torch.empty((t, m.heads, m.vdim), dtype=q.dtype, device=q.device)
            self._expanded_prefill(lw, q[nd:], pool, meta, plan, o[nd:], offset)
            if nd > 0:
                q_lat = torch.bmm(q[:nd, :, :m.dim].transpose(0, 1), lw.w_uk).transpose(0, 1)
                o_lat = ops.latent_attention(q_lat, q[:nd, :, m.dim:], pool, offset, meta.dec_block_tables, None,
                                             meta.positions[:nd], lw.sink, m.scale, splits=splits, window=window)
                torch.bmm(o_lat.transpose(0, 1), lw.w_uv, out=o[:nd].transpose(0, 1))
            return o
        # [heads, T, dim] x [heads, dim, kv_rank]: the unrotated query in latent space
        q_lat = torch.bmm(q[:, :, :m.dim].transpose(0, 1), lw.w_uk).transpose(0, 1)
        q_rot = q[:, :, m.dim:]
        o_lat = torch.empty((t, m.heads, m.kv_rank), dtype=q.dtype, device=q.device)
        if nd > 0:
            ops.latent_attention(q_lat[:nd], q_rot[:nd], pool, offset, meta.dec_block_tables, None,
                                 meta.positions[:nd], lw.sink, m.scale, out=o_lat[:nd], splits=splits, window=window)
        if meta.num_prefill_seqs > 0:
            ops.latent_attention(q_lat[nd:], q_rot[nd:], pool, offset, meta.pre_block_tables,
                                 meta.pre_row_seq, meta.positions[nd:], lw.sink, m.scale, out=o_lat[nd:],
                                 tiles=(meta.pre_lat_tiles or {}).get(m.heads), window=window)
        # [heads, T, kv_rank] x [heads, kv_rank, vdim], stored as [T, heads, vdim]
        o = torch.empty((t, m.heads, m.vdim), dtype=q.dtype, device=q.device)
        torch.bmm(o_lat.transpose(0, 1), lw.w_uv, out=o.transpose(0, 1))
        return o
