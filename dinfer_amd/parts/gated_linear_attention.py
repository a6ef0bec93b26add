"""Gated linear attention: a state S [dim, vdim] a head whose every key channel decays by a factor of its own, made from
the input through a small inner size.

With h the mixer's input, H heads:

    q, k = Wq h * dim^-1/2, Wk h  (H x dim)      v = Wv h  (H x vdim)
    a = sigmoid(W2 (W1 h) + b)^(1 / tau)         a decay in (0, 1)  (H x dim; W1 has `low` rows)
    S <- diag(a) S + k v^T;   o = S^T q                          (per head, token by token, S float32)
    y = Wo concat_h( o_h / rms(o_h) * w * silu(Wg h)_h )         (w: a gain of vdim entries that the heads share)

One product makes q | k | v | gate | W1 h; what follows up to the operand of Wo is float (csrc/linear_attention.hip: the
decays, then the recurrence, which reads q, k and v as the product left them; in steps whose portions are too few to fill
the chip it runs in chunks side by side). The state lives in the request's state slot (DeltaStateSpec without a
convolution); a request's first step (position 0) starts from zeros.
"""
from __future__ import annotations

import torch

from ..kernels import ops
from .base import CacheView, Mixer
from .linear import Linear
from .registry import MIXERS
from .spec import DeltaStateSpec, TensorSpec


@MIXERS.register("gated_linear_attention")
class GatedLinearAttention(Mixer):
    capturable = True            # every kernel reads slots, lengths and row counts from the batch's device buffers
    capturable_portions = True   # whether a step runs in chunks follows its counts alone

    NAMES = {"q": "q", "k": "k", "v": "v", "g": "g", "a1": "a1", "a2": "a2", "a2_bias": "a2.b", "norm": "norm", "o": "o"}

    def __init__(self, hidden: int, heads: int, dim: int, vdim: int, low: int, tau: float, norm_eps: float,
                 out_scale: float = 1.0, names: dict | None = None):
        if not (0 < dim <= ops.GLA_MAX_DIM and vdim > 0 and 0 < low <= ops.GLA_MAX_LOW and tau > 0):
            raise ValueError(f"gated linear attention: dim {dim}, vdim {vdim}, an inner decay size of {low} or tau {tau} has no "
                             f"kernel (dim up to {ops.GLA_MAX_DIM}, inner size up to {ops.GLA_MAX_LOW})")
        self.hidden, self.heads, self.dim, self.vdim, self.low = hidden, heads, dim, vdim, low
        self.tau, self.norm_eps, self.out_scale = float(tau), float(norm_eps), float(out_scale)
        self.names = dict(self.NAMES, **(names or {}))
        self.qk_size, self.v_size = heads * dim, heads * vdim
        self.v_off, self.g_off = 2 * self.qk_size, 2 * self.qk_size + self.v_size
        self.l_off = self.g_off + self.v_size
        self.proj = Linear(hidden, -(-(self.l_off + low) // 8) * 8)     # rows padded to 8 with zeros
        self.o = Linear(self.v_size, hidden)

    def cache_spec(self):
        return DeltaStateSpec(self.heads, self.dim, self.vdim, 0, 1)

    def tensors(self):
        n, Hd = self.names, self.hidden
        return {n["q"]: TensorSpec((self.qk_size, Hd)), n["k"]: TensorSpec((self.qk_size, Hd)),
                n["v"]: TensorSpec((self.v_size, Hd)), n["g"]: TensorSpec((self.v_size, Hd)),
                n["a1"]: TensorSpec((self.low, Hd)), n["a2"]: TensorSpec((self.qk_size, self.low)),
                n["a2_bias"]: TensorSpec((self.qk_size,), init="zeros"), n["norm"]: TensorSpec((self.vdim,), init="gain"),
                n["o"]: TensorSpec((Hd, self.v_size))}

    # ---- the middle part alone, for a mixer that joins several (parts/joined.py) ------------------
    @property
    def in_columns(self) -> int:
        return self.proj.out_features

    @property
    def out_columns(self) -> int:
        return self.v_size

    def out_weight(self, get) -> torch.Tensor:
        return get(self.names["o"], compute=True)

    def weight_rows(self, get) -> torch.Tensor:
        n = self.names
        w = torch.cat([get(n[k], compute=True) for k in ("q", "k", "v", "g", "a1")], dim=0)
        if w.shape[0] < self.proj.out_features:
            w = torch.cat([w, w.new_zeros(self.proj.out_features - w.shape[0], self.hidden)], dim=0)
        return w

    def load_small(self, get) -> None:
        n = self.names
        # small parameters in 32 bits (exact for a bfloat16 file): they enter the recurrence
        self.a2t = get(n["a2"]).float().t().contiguous()
        self.a2_bias = get(n["a2_bias"]).float().contiguous()
        self.norm_weight = get(n["norm"]).float().repeat(self.heads).contiguous()

    def load(self, get):
        self.proj.set_weight(self.weight_rows(get))
        self.load_small(get)
        self.o.set_weight(self.out_weight(get))

    def bind(self, ctx):
        ws = ctx.workspace
        self.proj_buf = ws.buffer("gla_proj", self.proj.out_features)
        self.gated_buf = ws.buffer("gla_gated", self.v_size)
        self.out_buf = ws.buffer("mixer_out", self.hidden)
        self.bind_core(ctx)

    def bind_core(self, ctx):
        ws = ctx.workspace
        self.decays = ws.buffer("gla_decays", self.qk_size, dtype=torch.float32)
        self.o_buf = ws.buffer("gla_o", self.v_size, dtype=torch.float32)
        places = ops.gla_places(ctx.max_tokens, ctx.max_reqs)
        self.notes = self.products = None
        if places > ctx.max_reqs + 1:      # (an engine whose longest step is shorter than a chunk cuts none)
            self.notes = ws.buffer("gla_notes", self.heads * self.vdim * self.dim, dtype=torch.float32, rows=places)
            self.products = ws.buffer("gla_products", self.qk_size, dtype=torch.float32, rows=places)

    def forward(self, x, batch, cache: CacheView):
        T = batch.num_tokens
        self.proj.forward(x, self.proj_buf, T, scratch=True)
        self.core(self.proj_buf, 0, self.gated_buf, 0, batch, cache)
        return self.o.forward(self.gated_buf, self.out_buf, T, scratch=True)

    def core(self, proj_buf, col, gated_buf, out_col, batch, cache: CacheView):
        """Everything between the two products: this mixer's columns start at `col` of proj_buf, the operand of the
        output product goes to column `out_col` of gated_buf."""
        T, qk, H = batch.num_tokens, self.qk_size, self.heads
        if not cache.owner:
            raise NotImplementedError("a recurrent mixer keeps a state a request: an entry that borrows a cache has none")
        ops.channel_decay(proj_buf, T, low_off=col + self.l_off, w2t=self.a2t, bias=self.a2_bias, tau=self.tau, out=self.decays)
        cut = self.notes is not None and ops.gla_cuts(T, batch.max_q_len, batch.num_reqs, H, self.vdim)
        ops.gla_recurrence(proj_buf[:, col:col + qk], proj_buf[:, col + qk:col + 2 * qk],
                           proj_buf[:, col + self.v_off:col + self.v_off + self.v_size], self.decays, cache.state, self.o_buf,
                           q_scale=self.dim ** -0.5, notes=self.notes, products=self.products, state_slots=batch.state_slots,
                           cu_seqlens=batch.cu_seqlens, seq_lens=batch.seq_lens, num_reqs=batch.num_reqs, tokens=T,
                           max_rows=batch.max_q_len, cut=cut, heads=H, dim=self.dim, vdim=self.vdim)
        ops.gated_group_norm(self.o_buf, proj_buf, col + self.g_off, gated_buf, T, groups=H, group=self.vdim,
                             eps=self.norm_eps, weight=self.norm_weight, col_off=out_col, out_scale=self.out_scale,
                             gate_first=False)
