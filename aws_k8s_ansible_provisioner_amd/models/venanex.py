"""Venanex: a layered decoder over one fp32 residual stream (LayeredConfig, arch "venanex").

Sequential layers with a layer norm (mean taken off, weight, no bias) before AND after each
sublayer:  x <- x + norm1b(mixer(norm1 x)),  x <- x + norm2b(ff(norm2 x)).  Mixers:
"latent_attention" -- queries W_uq rms(W_dq h), one cached row [rms(W_dkv h)[:R] | rotated key
part] per token, rotate-half positions under YaRN scaling -- or "attention" -- differential
attention inside chunks of positions: two softmax maps per head over the same values, the second
taken off lambda times, each head divided by its root mean square, a sigmoid gate per output
entry.  Feed-forwards are routed: sigmoid scores, the best `top` experts, clamped gated units
whose routing weight multiplies the expert's INPUT, beside a shared expert with a gate of its own.
A span of layers can run several times with the same weights (own cache per pass); every pass
starts with x <- W [x; embedding output].  The embedding table is the output head.

MI355X mapping.  Latent layers run like the framework's other latent design (models/latent.py:
attention in the latent space, the cache read once for all heads).  A differential layer projects
[q | k | v | gate] in one GEMM; the two maps' queries and keys of a head lie side by side, so a
cached key is one row of 2 D entries and the attention kernel reads each value fragment once for
both maps; difference, head norm and gate happen in that kernel's registers.  The post-norm, the
residual sum and the next sublayer's norm are one kernel; ahead of a pass it writes the stream
straight into the left half of the injection GEMM's input, whose right half holds the embedding.
Small batches (every decode step, hipGraph-captured) run ALL experts and the shared one as one
GEMM pair: the experts have no biases, so the routing weight on the input is a factor on both
projections, applied ahead of the clamps by the activation kernel (0 for experts not chosen), the
shared expert's gate a factor on its activation; prompt-sized batches run the grouped expert GEMMs
of the core library with the same units in their epilogue, or expert-sorted rows.
"""
from __future__ import annotations

import dataclasses
import math
from typing import Optional

import torch
import torch.nn.functional as F

from .. import ops
from ..ops import stream as sops
from ..parallel.state import ParallelState, get_state
from .config import AttentionSpec, LatentAttentionSpec, LayeredConfig, LayerSpec
from .latent import LatentPaths
from .routed import MOE_DENSE_ROWS, routed_sorted
from .transformer import AttnBatch


@dataclasses.dataclass
class DiffLatentLayerWeights:
    spec: LayerSpec
    norm1: torch.Tensor                     # fp32 [d]
    norm1b: torch.Tensor
    w_in: torch.Tensor                      # latent [dq | dkv]; differential [q | k | v | g]
    w_o: torch.Tensor                       # [d, H V]
    dq_norm: Optional[torch.Tensor] = None  # fp32 [q_rank]
    dkv_norm: Optional[torch.Tensor] = None
    w_uq: Optional[torch.Tensor] = None     # [H (D + r), q_rank]
    w_uk: Optional[torch.Tensor] = None     # [H, R, D]
    w_uv: Optional[torch.Tensor] = None     # [H, V, R]
    w_uk_t: Optional[torch.Tensor] = None   # the two with their last sizes exchanged (derived)
    w_uv_t: Optional[torch.Tensor] = None
    cos_sin: Optional[torch.Tensor] = None
    lam: Optional[torch.Tensor] = None      # fp32 [4, D]: lq1, lk1, lq2, lk2
    lam_value: float = 0.0                  # lambda (derived)
    norm2: Optional[torch.Tensor] = None
    norm2b: Optional[torch.Tensor] = None
    w_up: Optional[torch.Tensor] = None     # [E 2F + 2Fs, d]: per expert [gate | up], the shared one
    w_down: Optional[torch.Tensor] = None   # [d, E F + Fs]
    router: Optional[torch.Tensor] = None   # fp32 [E (+ 1), d]: the last row gates the shared expert
    w_down_e: Optional[torch.Tensor] = None     # [E, d, F]: the routed ones, made on first use
    w_loop: Optional[torch.Tensor] = None   # [d, 2 d], on the loop's first layer


class VenanexLM(LatentPaths):
    """Weights + forward of one replica (same surface as DecoderLM for the model runner)."""

    supports_v_tail = False
    gemm_tunable = True
    gemm_weight_names = ("w_in", "w_uq", "w_o", "w_up", "w_down", "w_loop")
    fused_gemm_chain = False
    dtypes = (torch.bfloat16, torch.float32)

    def __init__(self, cfg: LayeredConfig, device: torch.device | str = "cpu",
                 dtype: torch.dtype = torch.bfloat16, seed: int = 0,
                 pstate: Optional[ParallelState] = None, max_model_len: int = 4096,
                 full_then_shard: bool = False, init_std: float = 0.02):
        if dtype not in self.dtypes:
            raise ValueError(f"Venanex runs in bfloat16 or float32, not {dtype}")
        self.cfg = cfg
        self.device = torch.device(device)
        self.dtype = dtype
        self.ps = pstate or get_state()
        if self.ps.tp_size != 1:
            raise ValueError("Venanex: tensor parallelism is not implemented (tp must be 1)")
        if max_model_len > cfg.max_position:
            raise ValueError(f"max_model_len {max_model_len} exceeds max_position "
                             f"{cfg.max_position}")
        self.max_model_len = max_model_len
        self.init_std = init_std
        self.runs = cfg.layer_runs()
        a, b, times = cfg.loop if cfg.loop else (0, 0, 0)
        # layer runs that start a pass of the loop
        self.entries = {a + i * (b - a) for i in range(times)}
        self.hq, self.hkv, self.D = cfg.num_heads, max(1, cfg.num_kv_heads), cfg.head_dim
        self.ffn = cfg.intermediate_size
        self.vocab_start, self.vocab_end = 0, cfg.vocab_size
        self._tables: dict = {}
        self._ws: Optional[tuple] = None
        self._ws_kept: list = []
        self._seg_map: dict = {}
        self._init_weights(seed)

    # ------------------------------------------------------------------ weights
    def _table(self, rot) -> torch.Tensor:
        key = (rot.dims, rot.base, tuple(sorted((rot.scaling or {}).items())))
        if key not in self._tables:
            self._tables[key] = sops.rotary_table_yarn(max(self.max_model_len, 16), rot.dims,
                                                       rot.base, rot.scaling, device=self.device)
        return self._tables[key]

    @staticmethod
    def _slices(m) -> list:
        """(checkpoint suffix, rows) of the mixer's input projections, in w_in's order."""
        if isinstance(m, LatentAttentionSpec):
            return [("dq", m.q_rank), ("dkv", m.cache_dim)]
        return [("q", m.heads * m.key_dim), ("k", m.kv_heads * m.key_dim),
                ("v", m.kv_heads * m.vdim), ("g", m.heads * m.vdim)]

    def _init_weights(self, seed: int) -> None:
        cfg, d = self.cfg, self.cfg.hidden_size
        g = torch.Generator(device="cpu")
        g.manual_seed(seed)
        f32 = torch.float32

        def rand(*shape, s=self.init_std, mean=0.0, dt=None):
            t = torch.empty(*shape, dtype=f32).normal_(mean, s, generator=g)
            return t.to(torch.bfloat16).to(dt or self.dtype).to(self.device)

        def gain(n):
            return rand(n, s=0.1, mean=1.0, dt=f32)

        self.embed = rand(cfg.vocab_size, d, s=1.0)
        self.layers: list[DiffLatentLayerWeights] = []
        for i, ls in enumerate(cfg.layer_specs):
            m = ls.mixer
            n = sum(rows for _, rows in self._slices(m))
            npad = -(-n // 256) * 256
            if npad > 1.05 * n:
                npad = -(-n // 8) * 8
            w_in = torch.zeros(npad, d, dtype=self.dtype, device=self.device)
            w_in[:n] = rand(n, d)
            lw = DiffLatentLayerWeights(spec=ls, norm1=gain(d), norm1b=gain(d), w_in=w_in,
                                        w_o=rand(d, m.heads * m.vdim))
            if isinstance(m, LatentAttentionSpec):
                sq, sr = m.q_rank ** -0.5, m.kv_rank ** -0.5
                lw.dq_norm, lw.dkv_norm = gain(m.q_rank), gain(m.kv_rank)
                lw.w_uq = rand(m.heads * (m.dim + m.rot_dim), m.q_rank, s=sq)
                lw.w_uk = rand(m.heads, m.kv_rank, m.dim, s=sr)
                lw.w_uv = rand(m.heads, m.vdim, m.kv_rank, s=sr)
                lw.cos_sin = self._table(m.rot)
            else:
                lw.lam = rand(4, m.dim, s=0.1, dt=f32)
            ml = ls.mlp
            if ml is not None:
                E = ml.router.experts
                lw.norm2, lw.norm2b = gain(d), gain(d)
                lw.w_up = rand(E * 2 * ml.ff + 2 * ml.shared_ff, d)
                lw.w_down = rand(d, E * ml.ff + ml.shared_ff)
                lw.router = rand(E + (1 if ml.shared_gate else 0), d, s=4 * self.init_std, dt=f32)
            if cfg.loop_inject and i == cfg.loop[0]:
                lw.w_loop = rand(d, 2 * d)
            self.layers.append(lw)
        self.final_norm = gain(d)
        self._derive()

    def _derive(self) -> None:
        """What the forward reads instead of the stored tensors."""
        self._derive_latent()
        for lw in self.layers:
            lw.w_down_e = None
            if lw.lam is not None:
                lq1, lk1, lq2, lk2 = lw.lam.double().cpu()
                lw.lam_value = (math.exp(float((lq1 * lk1).sum()))
                                - math.exp(float((lq2 * lk2).sum())) + lw.spec.mixer.diff)

    def _names(self, i: int, lw: DiffLatentLayerWeights):
        """(checkpoint name, destination view, layout of the checkpoint tensor) of layer i."""
        p, m = f"l{i}.", lw.spec.mixer
        same = lambda t: t  # noqa: E731
        out, o = [(p + "norm1", lw.norm1, same), (p + "norm1b", lw.norm1b, same),
                  (p + "mix.o", lw.w_o, same)], 0
        for name, rows in self._slices(m):
            out.append((p + "mix." + name, lw.w_in[o:o + rows], same))
            o += rows
        if isinstance(m, LatentAttentionSpec):
            H, D, V, R = m.heads, m.dim, m.vdim, m.kv_rank
            out += [(p + "mix.dq.norm", lw.dq_norm, same), (p + "mix.dkv.norm", lw.dkv_norm, same),
                    (p + "mix.uq", lw.w_uq, same),
                    # [H D, R] -> [H, R, D] and [H V, R] -> [H, V, R]: both contiguous in the
                    # index their product contracts over
                    (p + "mix.uk", lw.w_uk,
                     lambda t: self._want(t, (H * D, R)).reshape(H, D, R).transpose(1, 2)),
                    (p + "mix.uv", lw.w_uv, lambda t: self._want(t, (H * V, R)).reshape(H, V, R))]
        else:
            out += [(p + "mix." + n, lw.lam[j], same)
                    for j, n in enumerate(("lq1", "lk1", "lq2", "lk2"))]
        ml = lw.spec.mlp
        if ml is not None:
            E, F_, Fs = ml.router.experts, ml.ff, ml.shared_ff
            out += [(p + "norm2", lw.norm2, same), (p + "norm2b", lw.norm2b, same),
                    (p + "mlp.router", lw.router[:E], same)]
            for e in range(E):
                u = e * 2 * F_
                out += [(p + f"mlp.e{e}.gate", lw.w_up[u:u + F_], same),
                        (p + f"mlp.e{e}.up", lw.w_up[u + F_:u + 2 * F_], same),
                        (p + f"mlp.e{e}.down", lw.w_down[:, e * F_:(e + 1) * F_], same)]
            if Fs:
                u = E * 2 * F_
                out += [(p + "mlp.shared.gate", lw.w_up[u:u + Fs], same),
                        (p + "mlp.shared.up", lw.w_up[u + Fs:u + 2 * Fs], same),
                        (p + "mlp.shared.down", lw.w_down[:, E * F_:E * F_ + Fs], same)]
            if ml.shared_gate:
                out.append((p + "mlp.shared.sg", lw.router[E:], same))
        if lw.w_loop is not None:
            out.append(("loop.in", lw.w_loop, same))
        return out

    @staticmethod
    def _want(t: torch.Tensor, shape: tuple) -> torch.Tensor:
        if tuple(t.shape) != shape:
            raise ValueError(f"checkpoint shape {tuple(t.shape)} does not fit the config "
                             f"(wanted {shape})")
        return t

    def _all_names(self):
        same = lambda t: t  # noqa: E731
        out = [("embed", self.embed, same), ("final.norm", self.final_norm, same)]
        for i, lw in enumerate(self.layers):
            out += self._names(i, lw)
        return out

    def state_dict(self) -> dict:
        """The weights under the checkpoint's names."""
        sd = {}
        for i, lw in enumerate(self.layers):
            m = lw.spec.mixer
            if isinstance(m, LatentAttentionSpec):
                sd[f"l{i}.mix.uk"] = lw.w_uk.transpose(1, 2).reshape(m.heads * m.dim,
                                                                     m.kv_rank).clone()
                sd[f"l{i}.mix.uv"] = lw.w_uv.reshape(m.heads * m.vdim, m.kv_rank).clone()
        for name, t, _ in self._all_names():
            if name not in sd:
                sd[name] = t.clone()
        return sd

    def load_state_dict(self, sd: dict) -> None:
        """Checkpoint tensors (bf16 safetensors) into the fused layout; shapes are checked
        against the config."""
        for name, dst, layout in self._all_names():
            if name not in sd:
                raise KeyError(f"checkpoint has no tensor {name!r}")
            src = layout(sd[name])
            if tuple(src.shape) != tuple(dst.shape):
                raise ValueError(f"{name}: checkpoint shape {tuple(sd[name].shape)} does not fit "
                                 f"the config (wanted {tuple(dst.shape)} after layout)")
            dst.copy_(src.to(dst.dtype))
        self._derive()

    @property
    def graph_safe(self) -> bool:
        return True

    def weight_bytes(self) -> int:
        seen = [self.embed, self.final_norm]
        for lw in self.layers:
            seen += [getattr(lw, f.name) for f in dataclasses.fields(lw)
                     if f.name not in ("cos_sin", "w_uk_t", "w_uv_t", "w_down_e")
                     and isinstance(getattr(lw, f.name), torch.Tensor)]
        return sum(t.numel() * t.element_size() for t in seen)

    # ------------------------------------------------------------------ cache
    def prefill_tile_plan(self) -> tuple:
        """(q rows per token, rows per tile, rows per tile of short steps) of the scheduler's
        prefill tile map."""
        return 1, 128, 0

    def kv_block_bytes(self, block_size: int, kv_dtype: str = "auto") -> int:
        es = torch.empty(0, dtype=self.dtype).element_size()
        n = 0
        for i in self.runs:
            m = self.cfg.layer_specs[i].mixer
            if isinstance(m, LatentAttentionSpec):
                n += block_size * es * (m.cache_dim
                                        + (m.kv_rank if self._grouped(m, block_size) else 0))
            else:
                n += block_size * es * m.kv_heads * (m.key_dim + m.vdim)
        return n

    def allocate_kv_segments(self, num_blocks: int, block_size: int, kv_dtype: str = "auto",
                             max_segment_bytes: Optional[int] = None) -> list:
        """Per layer run.  Latent: rows [NB, BS, R + r] and, where the matrix-core kernels run, the
        latents again as [NB, BS / 8, R, 8].  Differential: K [NB, G, BS, 2 D] (a token's two keys
        side by side) and V [NB, G, BS / 8, Dv, 8] (groups of 8 tokens, dimension-major inside a
        group).  Zero-filled, the model's dtype."""
        if kv_dtype not in ("auto", "bf16", "bfloat16"):
            raise ValueError("Venanex: the KV cache is kept in the model's dtype (no fp8)")
        if block_size % 8:
            raise ValueError("Venanex: the block size must be a multiple of 8")

        def zeros(*shape):
            segs.append(torch.zeros(num_blocks, *shape, dtype=self.dtype, device=self.device))
            return len(segs) - 1

        segs, self._seg_map = [], {}
        for r, i in enumerate(self.runs):
            m = self.cfg.layer_specs[i].mixer
            if isinstance(m, LatentAttentionSpec):
                a, b = zeros(block_size, m.cache_dim), None
                if self._grouped(m, block_size):
                    b = zeros(block_size // 8, m.kv_rank, 8)
            else:
                a = zeros(m.kv_heads, block_size, m.key_dim)
                b = zeros(m.kv_heads, block_size // 8, m.vdim, 8)
            self._seg_map[r] = (a, b)
        return segs

    def allocate_kv_cache(self, num_blocks: int, block_size: int, kv_dtype: str = "auto"):
        return self.allocate_kv_segments(num_blocks, block_size, kv_dtype)

    def cache_views(self, kv, block_size: int):
        segs = list(kv)
        pairs = [self._seg_map[r] for r in range(len(self.runs))]
        return [segs[a] for a, _ in pairs], [segs[b] if b is not None else None for _, b in pairs]

    # ------------------------------------------------------------------ forward
    def _linear(self, x: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
        if self.dtype == torch.bfloat16:
            return ops.linear(x, w)
        return F.linear(x, w)

    def _workspace(self, rows: int, parts: int):
        """Partial softmax state of split differential decode rows (two maps per head); a buffer
        that has to grow (eager steps only: the runner warms a bucket before capturing it) is kept
        alive, since captured graphs may still point at it."""
        att = [ls.mixer for ls in self.cfg.layer_specs if isinstance(ls.mixer, AttentionSpec)]
        heads, dim = 2 * max(a.heads for a in att), max(a.vdim for a in att)
        need = rows * parts
        if self._ws is None or self._ws[0] < need:
            if self._ws is not None:
                self._ws_kept.append(self._ws)
            self._ws = (need, sops.decode_workspace(rows, heads, dim, parts, self.device))
        return self._ws[1]

    def _latent(self, lw: DiffLatentLayerWeights, m: LatentAttentionSpec, h, batch: AttnBatch,
                rows, groups) -> torch.Tensor:
        T, dt, dev = h.shape[0], self.dtype, self.device
        H, D, rd, R = m.heads, m.dim, m.rot_dim, m.kv_rank
        proj = self._linear(h, lw.w_in)                              # [T, dq | dkv]
        cq = torch.empty(T, m.q_rank, dtype=dt, device=dev)
        sops.latent_prep(proj, cq, rows, batch.positions, batch.slots, lw.cos_sin, lw.dq_norm,
                         lw.dkv_norm, m.q_rank, R, rd, 0, m.q_rank, self.cfg.rms_eps, groups,
                         half=True)
        q = self._linear(cq, lw.w_uq).view(T, H, D + rd)
        sops.rotate_heads_(q, batch.positions, lw.cos_sin, D, half=True)
        q_lat = sops.head_matmul(q[:, :, :D].transpose(0, 1), lw.w_uk, lw.w_uk_t)   # [H, T, R]
        o_lat = torch.empty(H, T, R, dtype=dt, device=dev)
        self._latent_attention(m, o_lat, q_lat, q, batch, rows, groups)
        o = sops.head_matmul(o_lat, lw.w_uv, lw.w_uv_t, token_major=True)
        return self._linear(o.transpose(0, 1).reshape(T, H * m.vdim), lw.w_o)

    def _differential(self, lw: DiffLatentLayerWeights, m: AttentionSpec, h, batch: AttnBatch,
                      kc, vc) -> torch.Tensor:
        T = h.shape[0]
        proj = self._linear(h, lw.w_in)                              # [T, q | k | v | g]
        nq, nk, nv, ng = (rows for _, rows in self._slices(m))
        sops.head_norm_cache(proj, proj.new_empty(T, 0, m.key_dim), kc, vc, batch.slots, 0, m.kv_heads,
                             m.key_dim, m.vdim, 0, nq, nq + nk, self.cfg.rms_eps, False, False)
        att = torch.empty(T, m.heads * m.vdim, dtype=self.dtype, device=self.device)
        g0 = nq + nk + nv
        sops.diff_attention(att, proj[:, :nq], kc, vc, batch, proj[:, g0:g0 + ng], m.heads,
                            lw.lam_value, m.diff, m.scale, m.chunk, self.cfg.rms_eps,
                            self.max_model_len, self._workspace)
        return self._linear(att, lw.w_o)

    def _grouped_ok(self, h2: torch.Tensor, ff: int) -> bool:
        """Can the core library's grouped expert GEMMs run this layer (bf16 on the GPU, the
        library loaded -- a replay engine that returns logits alone runs without it --, both
        reduction depths multiples of 64)?"""
        return (h2.is_cuda and self.dtype == torch.bfloat16 and ops.native_loaded()
                and h2.shape[1] % 64 == 0 and ff % 64 == 0)

    def _feed_forward(self, lw: DiffLatentLayerWeights, h2: torch.Tensor, small: bool):
        """The feed-forward of h2 [T, d] as one or two addends (the second may be None)."""
        ml = lw.spec.mlp
        rt, F_, Fs = ml.router, ml.ff, ml.shared_ff
        T, d = h2.shape
        E = rt.experts
        sg = None
        if ml.shared_gate:
            ids, w, sg = sops.route_sigmoid(h2, lw.router, rt.top, gates=1)
        else:
            ids, w = sops.route_sigmoid(h2, lw.router, rt.top)
        if small:
            gu = self._linear(h2, lw.w_up)                   # every expert and the shared one
            act = torch.empty(T, E * F_ + Fs, dtype=gu.dtype, device=gu.device)
            sops.clamped_glu(gu, act, ml.limit, ids, w, E, Fs, ml.shared_limit, sg)
            return self._linear(act, lw.w_down), None

        def expert(e: int, rows: torch.Tensor) -> torch.Tensor:
            gu = F.linear(rows, lw.w_up[e * 2 * F_:(e + 1) * 2 * F_])
            u = torch.empty(rows.shape[0], F_, dtype=gu.dtype, device=gu.device)
            sops.clamped_glu(gu, u, ml.limit)
            return F.linear(u, lw.w_down[:, e * F_:(e + 1) * F_])

        if self._grouped_ok(h2, F_):
            # prompt-sized batches on an engine that has the core library: the framework's
            # grouped expert GEMMs (device-side sort and tile map, the clamped units in the
            # epilogue, no host round trip); they take the down-projections per expert, [E, d, F]
            if lw.w_down_e is None:
                lw.w_down_e = lw.w_down[:, :E * F_].reshape(d, E, F_).permute(1, 0, 2).contiguous()
            routed = ops.fused_moe(h2, lw.w_up[:E * 2 * F_].view(E, 2 * F_, d), lw.w_down_e, w,
                                   ids, clamp=(ml.limit, sops.CLAMPED_ALPHA))
        else:
            routed = routed_sorted(h2, ids, w, E, E, expert, weigh=rt.weigh)
        if not Fs:
            return routed, None
        gu = self._linear(h2, lw.w_up[E * 2 * F_:])
        u = torch.empty(T, Fs, dtype=gu.dtype, device=gu.device)
        sops.clamped_glu(gu, u, 0.0, None, None, 0, Fs, ml.shared_limit, sg)
        return self._linear(u, lw.w_down[:, E * F_:]), routed

    def forward(self, input_ids: torch.Tensor, batch: AttnBatch, k_caches, v_caches
                ) -> torch.Tensor:
        cfg, dt, dev = self.cfg, self.dtype, self.device
        T, d = input_ids.shape[0], cfg.hidden_size
        eps = cfg.rms_eps
        small = (not batch.is_prefill) or T <= MOE_DENSE_ROWS
        e = sops.embed_scaled(input_ids, self.embed, 1.0)            # fp32 [T, d]
        x = torch.empty_like(e)                                      # the stream
        cat = None
        if self.entries:
            # input of the injection GEMM: [stream | embedding output]
            cat = torch.empty(T, 2 * d, dtype=dt, device=dev)
            cat[:, d:].copy_(e)

        def sublayer_input(r: int):
            """(weights of the norm ahead of layer run r or None, its destination)."""
            if r == len(self.runs):
                return self.final_norm, torch.empty(T, d, dtype=dt, device=dev)
            if r in self.entries:
                return None, cat[:, :d]
            return self.layers[self.runs[r]].norm1, torch.empty(T, d, dtype=dt, device=dev)

        nw, h = sublayer_input(0)
        sops.stream_layer_norm_step(x, e, None, None, nw, eps, h, fresh=True)
        for r, li in enumerate(self.runs):
            lw = self.layers[li]
            m = lw.spec.mixer
            if r in self.entries:
                y = self._linear(cat, lw.w_loop)
                h = torch.empty(T, d, dtype=dt, device=dev)
                sops.stream_layer_norm_step(x, y, None, None, lw.norm1, eps, h, fresh=True)
            if isinstance(m, LatentAttentionSpec):
                y = self._latent(lw, m, h, batch, k_caches[r], v_caches[r])
            else:
                y = self._differential(lw, m, h, batch, k_caches[r], v_caches[r])
            if lw.spec.mlp is not None:
                h = torch.empty(T, d, dtype=dt, device=dev)
                sops.stream_layer_norm_step(x, y, None, lw.norm1b, lw.norm2, eps, h)
                ya, yb = self._feed_forward(lw, h, small)
                nw, h = sublayer_input(r + 1)
                sops.stream_layer_norm_step(x, ya, yb, lw.norm2b, nw, eps, h)
            else:
                nw, h = sublayer_input(r + 1)
                sops.stream_layer_norm_step(x, y, None, lw.norm1b, nw, eps, h)
        return h

    def compute_logits(self, h: torch.Tensor) -> torch.Tensor:
        return F.linear(h, self.embed)
