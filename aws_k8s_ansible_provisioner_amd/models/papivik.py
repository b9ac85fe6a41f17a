"""Papivik: a layered decoder over one fp32 residual stream whose sublayers read the stream
itself and norm only their OUTPUT (LayeredConfig, arch "papivik"):  x <- x + norm1(mixer(x)),
x <- x + norm2(ff(x)).  Three kinds of mixer, all with a recurrent matrix state per head and
live sequence (fp32, kept in the scheduler's sequence slots): "mlstm" -- matrix memory with
exponential, soft-capped input and forget gates, a normaliser and a running maximum;
"lightning" -- linear attention over silu-activated q, k, v with a fixed decay per head;
"parallel" -- a grouped-query softmax attention (short causal convolutions on q, k, v, per-head
q / k norms, partial rotate-half rotation) beside a gated delta rule (convolved and activated
q, k, v, unit q and k, a step size and a decay per head and token), summed with two constants.
Feed-forwards are dense with one gelu, or absent.

MI355X mapping.  One GEMM per mixer in and one out, through ops.linear like the other layered
models.  A parallel layer projects [q | k | v of both mixers | gate | step size | decay] at once;
ONE convolution launch serves both mixers' q, k, v (silu from the delta rule's first channel on,
a shorter kernel padded with zero taps), and both write side by side into one buffer, so the
weighted sum of the two outputs happens in the output GEMM's fp32 accumulator: the left
constant rides in the fp32 weights of the value convolution (the attention's output is linear
in the values), the right one in the head norm's weights.  The
recurrences have one set of kernels: prompt portions in chunks of 64 tokens on the matrix cores
with the fp32 state in accumulators, single rows in one launch from q, k, v to the normed and
gated heads, and a scan for other sizes and types.  The post-norm, the residual
sum and the copy of the stream that the next sublayer reads (or the model's output norm) are
one kernel.  Decode steps are sync-free and allocation-stable, so the runner captures them in
hipGraphs.
"""
from __future__ import annotations

import dataclasses
from typing import Optional

import torch
import torch.nn.functional as F

from .. import ops
from ..ops import stream as sops
from ..parallel.state import ParallelState, get_state
from .config import LayeredConfig, LayerSpec, MatrixMemorySpec, ParallelMixerSpec
from .transformer import AttnBatch


@dataclasses.dataclass
class PostNormLayerWeights:
    spec: LayerSpec
    norm1: torch.Tensor                     # fp32 [d]
    w_in: torch.Tensor                      # all projections of the mixer's input
    w_o: torch.Tensor                       # [d, heads' outputs]; parallel: [left | right]
    hnorm: torch.Tensor                     # fp32: the heads' output norm as stored
    hnorm_k: Optional[torch.Tensor] = None  # fp32 [H V]: what the kernel multiplies by
    decay: Optional[torch.Tensor] = None    # fp32 [H] (lightning)
    gate_b: Optional[torch.Tensor] = None   # fp32 [2, H]: mLSTM i.b, f.b; delta A_log, dt_bias
    conv: Optional[tuple] = None            # fp32 q, k, v, q, k, v taps as stored
    conv_k: Optional[torch.Tensor] = None   # fp32 [C, taps]: the same, stacked
    q_norm: Optional[torch.Tensor] = None   # fp32 [D]
    k_norm: Optional[torch.Tensor] = None
    cos_sin: Optional[torch.Tensor] = None
    norm2: Optional[torch.Tensor] = None
    w_up: Optional[torch.Tensor] = None
    w_down: Optional[torch.Tensor] = None


class PapivikLM:
    """Weights + forward of one replica (same surface as DecoderLM for the model runner)."""

    supports_v_tail = False
    gemm_tunable = True
    gemm_weight_names = ("w_in", "w_o", "w_up", "w_down")
    fused_gemm_chain = False
    dtypes = (torch.bfloat16, torch.float32)
    # convolution inputs and recurrent states of a live sequence sit in one of the scheduler's
    # sequence slots: the runner sizes the slot pool and turns prefix caching off
    state_slots = True

    def __init__(self, cfg: LayeredConfig, device: torch.device | str = "cpu",
                 dtype: torch.dtype = torch.bfloat16, seed: int = 0,
                 pstate: Optional[ParallelState] = None, max_model_len: int = 4096,
                 full_then_shard: bool = False, init_std: float = 0.02):
        if dtype not in self.dtypes:
            raise ValueError(f"Papivik runs in bfloat16 or float32, not {dtype}")
        self.cfg = cfg
        self.device = torch.device(device)
        self.dtype = dtype
        self.ps = pstate or get_state()
        if self.ps.tp_size != 1:
            raise ValueError("Papivik: tensor parallelism is not implemented (tp must be 1)")
        if max_model_len > cfg.max_position:
            raise ValueError(f"max_model_len {max_model_len} exceeds max_position "
                             f"{cfg.max_position}")
        self.max_model_len = max_model_len
        self.init_std = init_std
        self.runs = cfg.layer_runs()
        self.hq, self.hkv, self.D = cfg.num_heads, max(1, cfg.num_kv_heads), cfg.head_dim
        self.ffn = cfg.intermediate_size
        self.vocab_start, self.vocab_end = 0, cfg.vocab_size
        self._tables: dict = {}
        self.state: Optional[list] = None
        self._ws: Optional[tuple] = None
        self._ws_kept: list = []
        self._seg_map: dict = {}
        self._init_weights(seed)

    # ------------------------------------------------------------------ weights
    def _table(self, rot) -> Optional[torch.Tensor]:
        if rot is None or rot.dims <= 0:
            return None
        key = (rot.dims, rot.base)
        if key not in self._tables:
            self._tables[key] = sops.rotary_table(max(self.max_model_len, 16), rot.dims, rot.base,
                                                  None, device=self.device)
        return self._tables[key]

    @staticmethod
    def _slices(m) -> list:
        """(checkpoint suffix, rows) of the mixer's input projections, in w_in's order."""
        if isinstance(m, ParallelMixerSpec):
            a, r = m.left, m.right
            return [("left.q", a.heads * a.dim), ("left.k", a.kv_heads * a.dim),
                    ("left.v", a.kv_heads * a.vdim), ("right.q", r.qk_heads * r.dim),
                    ("right.k", r.qk_heads * r.dim), ("right.v", r.heads * r.vdim),
                    ("right.g", r.heads * r.vdim), ("right.b", r.heads), ("right.a", r.heads)]
        out = [("q", m.heads * m.dim), ("k", m.heads * m.dim), ("v", m.heads * m.vdim),
               ("g", m.heads * m.vdim)]
        if isinstance(m, MatrixMemorySpec):
            out += [("i", m.heads), ("f", m.heads)]
        return out

    @classmethod
    def _offsets(cls, m) -> dict:
        off, o = {}, 0
        for name, rows in cls._slices(m):
            off[name] = o
            o += rows
        return off

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
        self.layers: list[PostNormLayerWeights] = []
        for ls in cfg.layer_specs:
            m = ls.mixer
            n = sum(rows for _, rows in self._slices(m))
            npad = -(-n // 256) * 256
            if npad > 1.05 * n:
                npad = -(-n // 8) * 8
            w_in = torch.zeros(npad, d, dtype=self.dtype, device=self.device)
            w_in[:n] = rand(n, d)
            if isinstance(m, ParallelMixerSpec):
                a, r = m.left, m.right
                rows = [x for _, x in self._slices(m)[:6]]
                lw = PostNormLayerWeights(
                    spec=ls, norm1=gain(d), w_in=w_in,
                    w_o=rand(d, a.heads * a.vdim + r.heads * r.vdim), hnorm=gain(r.vdim),
                    gate_b=torch.stack([rand(r.heads, s=0.5, dt=f32),
                                        rand(r.heads, s=0.5, mean=-2.0, dt=f32)]),
                    conv=tuple(rand(x, a.conv if i < 3 else r.conv, s=0.5, dt=f32)
                               for i, x in enumerate(rows)),
                    q_norm=gain(a.dim), k_norm=gain(a.dim), cos_sin=self._table(a.rot))
            else:
                lw = PostNormLayerWeights(spec=ls, norm1=gain(d), w_in=w_in,
                                          w_o=rand(d, m.heads * m.vdim),
                                          hnorm=gain(m.heads * m.vdim))
                if isinstance(m, MatrixMemorySpec):
                    lw.gate_b = torch.stack([rand(m.heads, s=0.5, dt=f32),
                                             rand(m.heads, s=0.5, mean=3.0, dt=f32)])
                else:
                    lw.decay = torch.tensor(m.decay, dtype=f32, device=self.device)
            if ls.mlp is not None:
                lw.norm2 = gain(d)
                lw.w_up, lw.w_down = rand(ls.mlp.ff, d), rand(d, ls.mlp.ff)
            self.layers.append(lw)
        self.final_norm = gain(d)
        self.lm_head = rand(cfg.vocab_size, d)
        self._derive()

    def _derive(self) -> None:
        """What the kernels read instead of the stored tensors: the convolution taps of both
        mixers stacked (padded to the longer one, the left constant on the values' taps) and the
        head norm's weights per output column (times the right constant)."""
        for lw in self.layers:
            m = lw.spec.mixer
            if not isinstance(m, ParallelMixerSpec):
                lw.hnorm_k = lw.hnorm
                continue
            taps = max(m.left.conv, m.right.conv)
            parts = [F.pad(w, (taps - w.shape[1], 0)) for w in lw.conv]
            parts[2] = parts[2] * m.left_scale
            lw.conv_k = torch.cat(parts).contiguous()
            lw.hnorm_k = (lw.hnorm * m.right_scale).repeat(m.right.heads).contiguous()

    def _names(self, i: int, lw: PostNormLayerWeights):
        """(checkpoint name, destination view) of layer i."""
        p, m = f"l{i}.", lw.spec.mixer
        out, o = [(p + "norm1", lw.norm1)], 0
        for name, rows in self._slices(m):
            out.append((p + "mix." + name, lw.w_in[o:o + rows]))
            o += rows
        if isinstance(m, ParallelMixerSpec):
            na = m.left.heads * m.left.vdim
            out += [(p + f"mix.{n}.conv", w) for (n, _), w in zip(self._slices(m), lw.conv)]
            out += [(p + "mix.left.q.norm", lw.q_norm), (p + "mix.left.k.norm", lw.k_norm),
                    (p + "mix.left.o", lw.w_o[:, :na]), (p + "mix.right.o", lw.w_o[:, na:]),
                    (p + "mix.right.norm", lw.hnorm), (p + "mix.right.A_log", lw.gate_b[0]),
                    (p + "mix.right.dt_bias", lw.gate_b[1])]
        else:
            out += [(p + "mix.o", lw.w_o), (p + "mix.norm", lw.hnorm)]
            if isinstance(m, MatrixMemorySpec):
                out += [(p + "mix.i.b", lw.gate_b[0]), (p + "mix.f.b", lw.gate_b[1])]
        if lw.spec.mlp is not None:
            out += [(p + "norm2", lw.norm2), (p + "mlp.up", lw.w_up), (p + "mlp.down", lw.w_down)]
        return out

    def _all_names(self):
        out = [("embed", self.embed), ("final.norm", self.final_norm), ("head", self.lm_head)]
        for i, lw in enumerate(self.layers):
            out += self._names(i, lw)
        return out

    def state_dict(self) -> dict:
        """The weights under the checkpoint's names."""
        return {name: t.clone() for name, t in self._all_names()}

    def load_state_dict(self, sd: dict) -> None:
        """Checkpoint tensors (bf16 safetensors) into the fused layout; shapes are checked
        against the config."""
        for name, dst in self._all_names():
            if name not in sd:
                raise KeyError(f"checkpoint has no tensor {name!r}")
            src = sd[name]
            if tuple(src.shape) != tuple(dst.shape):
                raise ValueError(f"{name}: checkpoint shape {tuple(src.shape)} does not fit the "
                                 f"config (wanted {tuple(dst.shape)})")
            dst.copy_(src.to(dst.dtype))
        self._derive()

    @property
    def graph_safe(self) -> bool:
        return True

    def weight_bytes(self) -> int:
        seen = [self.embed, self.final_norm, self.lm_head]
        for lw in self.layers:
            seen += [getattr(lw, f.name) for f in dataclasses.fields(lw)
                     if f.name not in ("cos_sin", "hnorm_k", "conv_k")
                     and isinstance(getattr(lw, f.name), torch.Tensor)]
            seen += list(lw.conv or ())
        return sum(t.numel() * t.element_size() for t in seen)

    # ------------------------------------------------------------------ cache and state
    def prefill_tile_plan(self) -> tuple:
        """(q rows per token, rows per tile, rows per tile of short steps) of the scheduler's
        prefill tile map (the attention's; the recurrences take their grids from the sequence
        starts)."""
        return 1, 128, 0

    def _attentions(self):
        for r, i in enumerate(self.runs):
            m = self.cfg.layer_specs[i].mixer
            if isinstance(m, ParallelMixerSpec):
                yield r, m.left

    def kv_block_bytes(self, block_size: int, kv_dtype: str = "auto") -> int:
        es = torch.empty(0, dtype=self.dtype).element_size()
        return max(es, sum(block_size * es * a.kv_heads * (a.dim + a.vdim)
                           for _, a in self._attentions()))

    def allocate_kv_segments(self, num_blocks: int, block_size: int, kv_dtype: str = "auto",
                             max_segment_bytes: Optional[int] = None) -> list:
        """Per layer run with an attention: K [NB, G, BS, D] (token-major rows) and V
        [NB, G, BS / 8, Dv, 8] (groups of 8 tokens, dimension-major inside a group: what a
        matrix-core operand contracts over is one 16-byte load), zero-filled, in the model's
        dtype.  The other mixers cache nothing per token (a model without attention gets one
        placeholder so the pool has a dtype)."""
        if kv_dtype not in ("auto", "bf16", "bfloat16"):
            raise ValueError("Papivik: the KV cache is kept in the model's dtype (no fp8)")
        if block_size % 8:
            raise ValueError("Papivik: the block size must be a multiple of 8")
        segs, self._seg_map = [], {}
        for r, a in self._attentions():
            self._seg_map[r] = len(segs)
            segs.append(torch.zeros(num_blocks, a.kv_heads, block_size, a.dim, dtype=self.dtype,
                                    device=self.device))
            segs.append(torch.zeros(num_blocks, a.kv_heads, block_size // 8, a.vdim, 8,
                                    dtype=self.dtype, device=self.device))
        if not segs:
            segs.append(torch.zeros(1, dtype=self.dtype, device=self.device))
        return segs

    def allocate_kv_cache(self, num_blocks: int, block_size: int, kv_dtype: str = "auto"):
        return self.allocate_kv_segments(num_blocks, block_size, kv_dtype)

    def cache_views(self, kv, block_size: int):
        segs = list(kv)
        ks, vs = [], []
        for r in range(len(self.runs)):
            j = self._seg_map.get(r)
            ks.append(segs[j] if j is not None else None)
            vs.append(segs[j + 1] if j is not None else None)
        return ks, vs

    def allocate_state(self, num_slots: int) -> None:
        """Per layer run and sequence slot: the transposed states [slots, H, V, D] (fp32); mLSTM
        also the normalisers [slots, H, D] and running maxima [slots, H]; parallel also the last
        taps - 1 convolution inputs of both mixers [slots, taps - 1, C] (activation type)."""
        n = max(1, num_slots)

        def zeros(*shape, dt=torch.float32):
            return torch.zeros(n, *shape, dtype=dt, device=self.device)

        self.state = []
        for i in self.runs:
            m = self.cfg.layer_specs[i].mixer
            if isinstance(m, ParallelMixerSpec):
                r, taps, C = m.right, *self._conv_shape(m)
                self.state.append((zeros(r.heads, r.vdim, r.dim),
                                   zeros(taps - 1, C, dt=self.dtype)))
            elif isinstance(m, MatrixMemorySpec):
                self.state.append((zeros(m.heads, m.vdim, m.dim), zeros(m.heads, m.dim),
                                   zeros(m.heads)))
            else:
                self.state.append((zeros(m.heads, m.vdim, m.dim),))

    @classmethod
    def _conv_shape(cls, m: ParallelMixerSpec) -> tuple:
        """(taps, channels) of a parallel layer's convolution."""
        return max(m.left.conv, m.right.conv), sum(rows for _, rows in cls._slices(m)[:6])

    def state_bytes_per_slot(self) -> int:
        es = torch.empty(0, dtype=self.dtype).element_size()
        n = 0
        for i in self.runs:
            m = self.cfg.layer_specs[i].mixer
            if isinstance(m, ParallelMixerSpec):
                taps, C = self._conv_shape(m)
                n += 4 * m.right.state_floats + es * (taps - 1) * C
            else:
                n += 4 * m.state_floats
        return n

    # ------------------------------------------------------------------ forward
    def _linear(self, x: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
        if self.dtype == torch.bfloat16:
            return ops.linear(x, w)
        return F.linear(x, w)

    def _workspace(self, rows: int, parts: int):
        """Partial softmax state of split decode attention; a buffer that has to grow (eager
        steps only: the runner warms a bucket before capturing it) is kept alive, since captured
        graphs may still point at it."""
        heads = max(a.heads for _, a in self._attentions())
        dim = max(a.vdim for _, a in self._attentions())
        need = rows * heads * parts
        if self._ws is None or self._ws[0] < need:
            if self._ws is not None:
                self._ws_kept.append(self._ws)
            self._ws = (need, sops.decode_workspace(rows, heads, dim, parts, self.device))
        return self._ws[1]

    def _parallel(self, lw: PostNormLayerWeights, m: ParallelMixerSpec, proj, batch: AttnBatch,
                  r: int, kc, vc, seq_slot, q_start, first) -> torch.Tensor:
        a, d = m.left, m.right
        T = proj.shape[0]
        off = self._offsets(m)
        S, conv_state = self.state[r]
        C = lw.conv_k.shape[0]
        qkv = torch.empty(T, C, dtype=self.dtype, device=self.device)
        sops.conv_silu(qkv, proj, 0, lw.conv_k, None, conv_state, seq_slot, batch.positions,
                       q_start, silu_from=off["right.q"])
        q = torch.empty(T, a.heads, a.dim, dtype=self.dtype, device=self.device)
        sops.head_norm_cache(qkv, q, kc, vc, batch.slots, a.heads, a.kv_heads, a.dim, a.vdim, 0,
                             off["left.k"], off["left.v"], self.cfg.rms_eps, a.head_norm, a.v_norm,
                             lw.q_norm, lw.k_norm, lw.cos_sin, batch.positions)
        na = a.heads * a.vdim
        buf = torch.empty(T, na + d.heads * d.vdim, dtype=self.dtype, device=self.device)
        sops.causal_attention(buf[:, :na], q, kc, vc, batch, a.scale, self.max_model_len,
                              self._workspace)
        sops.gated_delta(buf[:, na:], qkv, off["right.q"], off["right.k"], off["right.v"], proj,
                         off["right.g"], off["right.b"], off["right.a"], lw.gate_b[0],
                         lw.gate_b[1], S, lw.hnorm_k, seq_slot, batch.positions, q_start, d.heads,
                         d.qk_heads, d.dim, d.vdim, self.cfg.rms_eps, first)
        return buf

    def _mixer(self, lw: PostNormLayerWeights, h, batch: AttnBatch, r: int, kc, vc, seq_slot,
               q_start, first) -> torch.Tensor:
        m, eps = lw.spec.mixer, self.cfg.rms_eps
        proj = self._linear(h, lw.w_in)
        if isinstance(m, ParallelMixerSpec):
            buf = self._parallel(lw, m, proj, batch, r, kc, vc, seq_slot, q_start, first)
            return self._linear(buf, lw.w_o)
        off = self._offsets(m)
        buf = torch.empty(h.shape[0], m.heads * m.vdim, dtype=self.dtype, device=self.device)
        if isinstance(m, MatrixMemorySpec):
            sops.matrix_memory(buf, proj, off["q"], off["k"], off["v"], off["g"], off["i"],
                               off["f"], lw.gate_b[0], lw.gate_b[1], m.cap, self.state[r],
                               lw.hnorm_k, seq_slot, batch.positions, q_start, m.heads, m.dim,
                               m.vdim, eps, first)
        else:
            sops.linear_attention(buf, proj, off["q"], off["k"], off["v"], off["g"], lw.decay,
                                  self.state[r][0], lw.hnorm_k, seq_slot, batch.positions,
                                  q_start, m.heads, m.dim, m.vdim, eps, m.act, m.out_norm, m.gate,
                                  first)
        return self._linear(buf, lw.w_o)

    def forward(self, input_ids: torch.Tensor, batch: AttnBatch, k_caches, v_caches
                ) -> torch.Tensor:
        cfg, dt, dev = self.cfg, self.dtype, self.device
        T, d = input_ids.shape[0], cfg.hidden_size
        eps = cfg.rms_eps
        if self.state is None:
            raise RuntimeError("Papivik: allocate_state() must run before forward()")
        if batch.tail_slot is None:
            raise RuntimeError("Papivik: the batch carries no sequence slots")
        seq_slot = batch.tail_slot[:T]
        q_start = batch.q_start if batch.is_prefill else None
        first = batch.num_decode if batch.is_prefill else 0
        x = sops.embed_scaled(input_ids, self.embed, cfg.embed_scale)   # fp32: the stream
        h = x.to(dt) if dt != torch.float32 else x.clone()
        for r, li in enumerate(self.runs):
            lw = self.layers[li]
            out_w = self.final_norm if r + 1 == len(self.runs) else None
            has_ff = lw.spec.mlp is not None
            y = self._mixer(lw, h, batch, r, k_caches[r], v_caches[r], seq_slot, q_start, first)
            h = torch.empty(T, d, dtype=dt, device=dev)
            sops.stream_post_norm_add_norm(x, y, None, None, None, lw.norm1,
                                           None if has_ff else out_w, eps, h)
            if has_ff:
                up = self._linear(h, lw.w_up)
                act = torch.empty_like(up)
                sops.gelu_tanh(up, act)
                y = self._linear(act, lw.w_down)
                h = torch.empty(T, d, dtype=dt, device=dev)
                sops.stream_post_norm_add_norm(x, y, None, None, None, lw.norm2, out_w, eps, h)
        return h

    def compute_logits(self, h: torch.Tensor) -> torch.Tensor:
        return F.linear(h, self.lm_head)
