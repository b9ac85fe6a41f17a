"""Latent attention of the layered models: what a layer with ONE cached row per token
[latent | rotated key part] needs beside its projections -- the grouped second copy of the
latents for the matrix-core kernels, the split of decode rows over workgroups, the step's
attention in the latent space -- shared by every model with such layers.
"""
from __future__ import annotations

import math
from typing import Optional

import torch

from ..ops import stream as sops
from .config import LatentAttentionSpec
from .transformer import AttnBatch


class LatentPaths:
    """Mixin: expects .device, .dtype, .max_model_len and .layers whose latent layers carry
    w_uk [H, R, D] and w_uv [H, V, R] (and w_uk_t / w_uv_t, filled by _derive_latent)."""

    _lat_ws: Optional[tuple] = None

    def _derive_latent(self) -> None:
        """The per-head weights with the contracted index first, for prompt-sized steps."""
        for lw in self.layers:
            if getattr(lw, "w_uk", None) is not None:
                lw.w_uk_t = lw.w_uk.transpose(1, 2).contiguous()
                lw.w_uv_t = lw.w_uv.transpose(1, 2).contiguous()

    def _grouped(self, m: LatentAttentionSpec, block_size: int) -> bool:
        """Does the layer keep the grouped second copy of its latents (the operand layout of
        the matrix-core attention kernels: bf16 on the GPU, sizes they are built for)?"""
        if self.device.type != "cuda" or self.dtype != torch.bfloat16 or block_size % 32:
            return False
        sops.load_native(required=True)
        return bool(torch.ops.akap_stream.latent_mfma_supported(m.kv_rank, m.rot_dim))

    def _latent_parts(self, rows: int, heads: int) -> int:
        """Key partitions of a decode row: static in the batch size and the model length
        (hipGraph-capturable).  One workgroup per (row, 32 heads, partition); about one
        workgroup per CU measured best (64 rows x 2112 keys, 16 heads, latent 512 + 64: 138 us
        unsplit, 64 us at 4 partitions, 80 at 8, 87 at 16), a partition never under 128 keys."""
        max_parts = max(1, math.ceil(self.max_model_len / 128))
        groups = max(1, rows * math.ceil(heads / 32))
        return min(max_parts, 64, max(1, math.ceil(256 / groups)))

    def _latent_workspace(self, rows: int, heads: int, kv_rank: int, parts: int):
        """Partial softmax state of the split decode: (max, sum) per (row, head, partition) and
        the unnormalised latent output.  Layers differ in heads and latent size, so both
        buffers are checked; a buffer that has to grow (eager steps only: the runner warms a
        bucket before capturing it) is kept alive, since captured graphs may still point at
        it."""
        n_ml, n_o = 2 * rows * heads * parts, rows * heads * parts * kv_rank
        if self._lat_ws is None or self._lat_ws[0].numel() < n_ml or self._lat_ws[1].numel() < n_o:
            if self._lat_ws is not None:
                self._lat_ws_kept = [*getattr(self, "_lat_ws_kept", ()), self._lat_ws]
                n_ml, n_o = max(n_ml, self._lat_ws[0].numel()), max(n_o, self._lat_ws[1].numel())
            self._lat_ws = (torch.empty(n_ml, dtype=torch.float32, device=self.device),
                            torch.empty(n_o, dtype=torch.float32, device=self.device))
        return self._lat_ws

    def _latent_attention(self, m: LatentAttentionSpec, o_lat, q_lat, q, batch: AttnBatch, cache,
                          groups) -> None:
        T = q.shape[0]
        nd = batch.num_decode if batch.is_prefill else T
        if nd:
            parts, ws = 1, None
            if groups is not None:
                parts = self._latent_parts(nd, m.heads)
                ws = self._latent_workspace(nd, m.heads, m.kv_rank, parts) if parts > 1 else None
            # the leading nd rows are contiguous slices of the head-major buffers only when
            # they are all rows; a mixed step's decode rows go through narrow copies
            if nd == T:
                sops.latent_attention_decode(o_lat, q_lat, q, m.dim, cache, groups,
                                             batch.block_tables[:nd], batch.seq_lens[:nd],
                                             batch.positions[:nd], m.scale, ws, parts)
            else:
                od = torch.empty(m.heads, nd, m.kv_rank, dtype=o_lat.dtype, device=o_lat.device)
                sops.latent_attention_decode(od, q_lat[:, :nd].contiguous(), q[:nd], m.dim, cache,
                                             groups, batch.block_tables[:nd], batch.seq_lens[:nd],
                                             batch.positions[:nd], m.scale, ws, parts)
                o_lat[:, :nd] = od
        if batch.is_prefill:
            sops.latent_attention_prefill(o_lat, q_lat, q, m.dim, cache, groups,
                                          batch.block_tables, batch.seq_lens, batch.q_start,
                                          batch.positions, batch.tile_seq, batch.tile_row,
                                          batch.tile_rows, m.scale, first_seq=nd)
