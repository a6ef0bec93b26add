"""Lightning attention: linear attention with a fixed decay a head, activated queries, keys and values, and one norm over
all heads.

With x the mixer's input, H heads:

    q, k = silu(Wq x), silu(Wk x)  (H x dim)      v = silu(Wv x)  (H x vdim)
    S <- decay_h S + k v^T;   o = S^T q                              (per head, token by token, S float32 [dim, vdim])
    y = Wo ( o / rms(o) * w * sigmoid(Wg x) )                        (the root mean square over all heads' entries at once)

One product makes q | k | v | gate. The state lives in the request's state slot (DeltaStateSpec without a convolution); a
request's first step (position 0) starts from zeros. bfloat16 steps with prompt portions run in blocks of tokens on the
matrix cores (ops.lightning), steps whose portions bring a few rows token by token (ops.lightning_few), 32-bit prompts and
sizes those two do not take through ops.gla_recurrence with fixed decays.
"""
from __future__ import annotations

import torch

from ..kernels import ops
from .base import CacheView, Mixer
from .linear import Linear
from .registry import MIXERS
from .spec import DeltaStateSpec, TensorSpec

FEW_ROWS = 8      # the longest portion of a step up to which its tokens are taken one by one


@MIXERS.register("lightning")
class Lightning(Mixer):
    capturable = True            # every kernel reads slots, lengths and row counts from the batch's device buffers
    capturable_portions = True   # whether a step runs in chunks follows its counts alone

    NAMES = {"q": "q", "k": "k", "v": "v", "g": "g", "o": "o", "norm": "norm"}

    def __init__(self, hidden: int, heads: int, dim: int, vdim: int, decay, norm_eps: float, names: dict | None = None):
        decay = tuple(float(d) for d in decay)
        if len(decay) != heads or not all(0.0 < d <= 1.0 for d in decay):
            raise ValueError(f"lightning attention: one decay in (0, 1] a head ({heads}), got {decay!r}")
        if not (0 < dim <= ops.GLA_MAX_DIM and vdim > 0):
            raise ValueError(f"lightning attention: dim {dim} or vdim {vdim} has no kernel (dim up to {ops.GLA_MAX_DIM})")
        self.hidden, self.heads, self.dim, self.vdim, self.decay = hidden, heads, dim, vdim, decay
        self.norm_eps, self.names = float(norm_eps), dict(self.NAMES, **(names or {}))
        self.qk_size, self.v_size = heads * dim, heads * vdim
        self.g_off = 2 * self.qk_size + self.v_size
        self.proj = Linear(hidden, -(-(self.g_off + self.v_size) // 8) * 8)
        self.o = Linear(self.v_size, hidden)

    def cache_spec(self):
        return DeltaStateSpec(self.heads, self.dim, self.vdim, 0, 1)

    def tensors(self):
        n, Hd = self.names, self.hidden
        return {n["q"]: TensorSpec((self.qk_size, Hd)), n["k"]: TensorSpec((self.qk_size, Hd)),
                n["v"]: TensorSpec((self.v_size, Hd)), n["g"]: TensorSpec((self.v_size, Hd)),
                n["norm"]: TensorSpec((self.v_size,), init="gain"), n["o"]: TensorSpec((Hd, self.v_size))}

    def load(self, get):
        n = self.names
        w = torch.cat([get(n[k], compute=True) for k in ("q", "k", "v", "g")], dim=0)
        if w.shape[0] < self.proj.out_features:
            w = torch.cat([w, w.new_zeros(self.proj.out_features - w.shape[0], self.hidden)], dim=0)
        self.proj.set_weight(w)
        self.o.set_weight(get(n["o"], compute=True))
        self.gain = get(n["norm"]).float().contiguous()
        self.decay_vec = torch.tensor(self.decay, dtype=torch.float32, device=w.device)

    def bind(self, ctx):
        ws = ctx.workspace
        self.proj_buf = ws.buffer("lightning_proj", self.proj.out_features)
        self.o_buf = ws.buffer("lightning_o", self.v_size, dtype=torch.float32)
        self.gated_buf = ws.buffer("lightning_gated", self.v_size)
        self.out_buf = ws.buffer("mixer_out", self.hidden)
        self.blocks = ctx.dtype == torch.bfloat16 and ops.lightning_supports(self.dim, self.vdim, self.proj.out_features)
        places = (ops.lightning_places if self.blocks else ops.gla_places)(ctx.max_tokens, ctx.max_reqs)
        self.notes = self.products = None
        if places > ctx.max_reqs + 1:      # (an engine whose longest step is shorter than a chunk cuts none)
            self.notes = ws.buffer("lightning_notes", self.heads * self.vdim * self.dim, dtype=torch.float32, rows=places)
            if not self.blocks:
                self.products = ws.buffer("lightning_products", self.qk_size, dtype=torch.float32, rows=places)

    def forward(self, x, batch, cache: CacheView):
        T, qk, H = batch.num_tokens, self.qk_size, self.heads
        p = self.proj_buf
        if not cache.owner:
            raise NotImplementedError("a recurrent mixer keeps a state a request: an entry that borrows a cache has none")
        self.proj.forward(x, p, T, scratch=True)
        q, k, v = p[:, :qk], p[:, qk:2 * qk], p[:, 2 * qk:self.g_off]
        step = dict(state_slots=batch.state_slots, cu_seqlens=batch.cu_seqlens, seq_lens=batch.seq_lens, num_reqs=batch.num_reqs,
                    tokens=T, heads=H, dim=self.dim, vdim=self.vdim)
        if self.dim % 4 == 0 and batch.max_q_len <= FEW_ROWS:
            ops.lightning_few(q, k, v, self.decay_vec, cache.state, self.o_buf, **step)
        elif self.blocks:
            cut = self.notes is not None and ops.lightning_cuts(T, batch.max_q_len, batch.num_reqs, H, self.vdim)
            ops.lightning(q, k, v, self.decay_vec, cache.state, self.o_buf, notes=self.notes, cut=cut, max_rows=batch.max_q_len,
                          **step)
        else:
            cut = self.products is not None and ops.gla_cuts(T, batch.max_q_len, batch.num_reqs, H, self.vdim)
            ops.gla_recurrence(q, k, v, None, cache.state, self.o_buf, q_scale=1.0, notes=self.notes, products=self.products,
                               fixed=self.decay_vec, act=True, cut=cut, max_rows=batch.max_q_len, **step)
        ops.gated_group_norm(self.o_buf, p, self.g_off, self.gated_buf, T, groups=1, group=self.v_size, eps=self.norm_eps,
                             weight=self.gain, gate_first=False, gate="sigmoid")
        return self.o.forward(self.gated_buf, self.out_buf, T, scratch=True)
