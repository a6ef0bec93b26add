"""minGRU: a gated recurrence of single channels whose gates read the current token only.

With h the mixer's input and N channels:

    a = sigmoid(Wz h + bz);   u = Wx h + bx;   c = u + 1/2 where u >= 0, sigmoid(u) where u < 0
    S <- (1 - a) S + a c                       (channel by channel, token by token, S float32)
    y = Wo ( S * silu(Wg h) )

One product makes z | x | gate; what follows up to the operand of Wo is float and one kernel (csrc/scan.hip; longer
portions run in chunks side by side). The state, one float a channel, lives in the request's state slot; a request's first
step (position 0) starts from zeros.
"""
from __future__ import annotations

import torch

from ..kernels import ops
from .base import CacheView, Mixer
from .linear import Linear
from .registry import MIXERS
from .spec import StateSpec, TensorSpec


@MIXERS.register("min_gru")
class MinGRU(Mixer):
    capturable = True            # both kernels read slots, lengths and row counts from the batch's device buffers
    capturable_portions = True

    NAMES = {"z": "z", "z_bias": "z.b", "x": "x", "x_bias": "x.b", "g": "g", "o": "o"}

    def __init__(self, hidden: int, channels: int, names: dict | None = None):
        if channels <= 0:
            raise ValueError(f"minGRU: {channels} channels")
        self.hidden, self.channels = hidden, channels
        self.names = dict(self.NAMES, **(names or {}))
        self.step = -(-channels // 8) * 8            # columns of each third of the product, padded to 8 with zeros
        self.proj = Linear(hidden, 3 * self.step)
        self.o = Linear(self.step, hidden)

    def cache_spec(self):
        return StateSpec((self.channels,))

    def tensors(self):
        n, Hd, N = self.names, self.hidden, self.channels
        return {n["z"]: TensorSpec((N, Hd)), n["z_bias"]: TensorSpec((N,), init="zeros"), n["x"]: TensorSpec((N, Hd)),
                n["x_bias"]: TensorSpec((N,), init="zeros"), n["g"]: TensorSpec((N, Hd)), n["o"]: TensorSpec((Hd, N))}

    def load(self, get):
        n, pad = self.names, self.step - self.channels
        rows = []
        for k in ("z", "x", "g"):
            w = get(n[k], compute=True)
            rows.append(torch.cat([w, w.new_zeros(pad, self.hidden)], dim=0) if pad else w)
        self.proj.set_weight(torch.cat(rows, dim=0))
        o = get(n["o"], compute=True)
        self.o.set_weight(torch.cat([o, o.new_zeros(self.hidden, pad)], dim=1) if pad else o)
        self.z_bias = get(n["z_bias"]).float().contiguous()
        self.x_bias = get(n["x_bias"]).float().contiguous()

    def bind(self, ctx):
        ws = ctx.workspace
        self.proj_buf = ws.buffer("min_gru_proj", self.proj.out_features)
        self.gated_buf = ws.buffer("min_gru_gated", self.step)
        if self.step != self.channels:
            self.gated_buf.zero_()      # padding columns meet zero weights, but must hold numbers
        self.out_buf = ws.buffer("mixer_out", self.hidden)
        self.notes = ws.buffer("min_gru_notes", 2 * self.channels, dtype=torch.float32,
                               rows=ops.min_gru_places(ctx.max_tokens, ctx.max_reqs))

    def forward(self, x, batch, cache: CacheView):
        T, s = batch.num_tokens, self.step
        if not cache.owner:
            raise NotImplementedError("a recurrent mixer keeps a state a request: an entry that borrows a cache has none")
        self.proj.forward(x, self.proj_buf, T, scratch=True)
        ops.min_gru(self.proj_buf, self.gated_buf, z_off=0, x_off=s, g_off=2 * s, z_bias=self.z_bias, x_bias=self.x_bias,
                    state=cache.state, notes=self.notes, state_slots=batch.state_slots, cu_seqlens=batch.cu_seqlens,
                    seq_lens=batch.seq_lens, num_reqs=batch.num_reqs, tokens=T, max_rows=batch.max_q_len)
        return self.o.forward(self.gated_buf, self.out_buf, T, scratch=True)
