"""Several mixers side by side on the same input: y = sum_i scale_i * mixer_i(h).

The members' input products are one product (their weight rows stacked), and so are their output products: member
i writes scale_i times the operand of its output product into its columns of one buffer, and the members' output
weights lie side by side, so [Wo_1 | Wo_2] [s_1 a_1; s_2 a_2] = s_1 Wo_1 a_1 + s_2 Wo_2 a_2 comes out of one product
with one rounding. A member is any mixer that offers its middle part alone: `in_columns`, `out_columns`,
`weight_rows(get)`, `load_small(get)`, `out_weight(get)`, `bind_core(ctx)`, `core(in_buf, col, out_buf, out_col, batch,
cache)` and the constructor parameter `out_scale` (and `out_bias(get)`, where its output projection adds one). Their
caches are joined by name (JoinedSpec); tensors are read under `<member name>.<the member's own names>`.

out_norm_eps: every member's output is RMS-normed over the model's width by a gain of its own (`<member name>.out`) before
the sum, y = sum_i scale_i * rms(mixer_i(h)) * w_i with one scale for all. The output products are then one a member, into
columns of one buffer, and one kernel adds their biases, norms and sums them; where the block hands over the residual
stream and the norm that reads it next, the same kernel adds into the stream and norms it.
"""
from __future__ import annotations

import torch

from ..kernels import gemm, ops
from .base import CacheView, Carried, Mixer
from .linear import Linear
from .norm import GroupRMSNorm
from .registry import MIXERS
from .spec import JoinedSpec, TensorSpec


@MIXERS.register("joined")
class JoinedMixers(Mixer):
    def __init__(self, hidden: int, members: list, out_norm_eps: float | None = None):
        """members: [(name, PartSpec of a mixer, scale)]; with out_norm_eps the scales are equal."""
        self.hidden = hidden
        self.out_norm_eps = None if out_norm_eps is None else float(out_norm_eps)
        self.sum_scale = 1.0
        if self.out_norm_eps is not None:
            self.sum_scale = float(members[0][2])
            if len(members) > ops.JOINED_NORMS_MAX or any(float(m[2]) != self.sum_scale for m in members):
                raise ValueError(f"joined mixers with norms: up to {ops.JOINED_NORMS_MAX} members of one scale")
            members = [(name, spec, 1.0) for name, spec, _ in members]      # (a factor before a norm would vanish in it)
        self.members = []
        self.scales = [float(scale) for _, _, scale in members]
        col = out_col = 0
        for name, spec, scale in members:
            m = MIXERS.get(spec.kind)(hidden=hidden, **dict(spec.params, out_scale=float(scale)))
            if not hasattr(m, "core"):
                raise ValueError(f"mixer {spec.kind!r} does not offer its middle part alone and cannot be joined")
            self.members.append((name, m, col, out_col))
            col += -(-m.in_columns // 8) * 8
            out_col += -(-m.out_columns // 8) * 8
        self.proj = Linear(hidden, col)
        # with norms: an output product a member; without: one for all, the members' weights side by side
        self.o = Linear(out_col, hidden) if self.out_norm_eps is None else None
        self.outs = [] if self.o is not None else [Linear(-(-m.out_columns // 8) * 8, hidden) for _, m, _, _ in self.members]
        self.mid_columns = out_col
        self.bias = self.out_gains = None

    @property
    def carries_norms(self):
        return self.out_norm_eps is not None      # the kernel that sums the normed outputs takes an Into

    @property
    def capturable(self):
        return all(m.capturable for _, m, _, _ in self.members)

    @property
    def capturable_portions(self):
        return all(m.capturable_portions for _, m, _, _ in self.members)

    def cache_spec(self):
        return JoinedSpec({name: m.cache_spec() for name, m, _, _ in self.members})

    def tensors(self):
        t = {f"{name}.{n}": s for name, m, _, _ in self.members for n, s in m.tensors().items()}
        if self.out_norm_eps is not None:
            t.update({f"{name}.out": TensorSpec((self.hidden,), init="gain") for name, _, _, _ in self.members})
        return t

    def load(self, get):
        rows, cols, biases, gains = [], [], [], []
        for name, m, _, _ in self.members:
            sub = lambda n, _p=name + ".", **kw: get(_p + n, **kw)
            w = m.weight_rows(sub)
            pad = -(-w.shape[0] // 8) * 8 - w.shape[0]
            rows.append(torch.cat([w, w.new_zeros(pad, self.hidden)], dim=0) if pad else w)
            o = m.out_weight(sub)
            pad = -(-o.shape[1] // 8) * 8 - o.shape[1]
            cols.append(torch.cat([o, o.new_zeros(self.hidden, pad)], dim=1) if pad else o)
            m.load_small(sub)
            biases.append(m.out_bias(sub) if hasattr(m, "out_bias") else None)
            if self.out_norm_eps is not None:
                gains.append(sub("out").float())
        self.proj.set_weight(torch.cat(rows, dim=0))
        if self.o is None:
            for lin, w in zip(self.outs, cols):
                lin.set_weight(w)
            self.out_gains = torch.stack(gains).contiguous()
            if any(b is not None for b in biases):
                self.bias = torch.stack([torch.zeros_like(self.out_gains[0]) if b is None else b for b in biases]).contiguous()
            return
        self.o.set_weight(torch.cat(cols, dim=1))
        if any(b is not None for b in biases):      # sum_i scale_i bias_i, added to the one product's rows
            self.bias = sum(s * b for b, s in zip(biases, self.scales) if b is not None).contiguous()

    def bind(self, ctx):
        ws = ctx.workspace
        self.proj_buf = ws.buffer("joined_proj", self.proj.out_features)
        self.mid_buf = ws.buffer("joined_mid", self.mid_columns)
        self.out_buf = ws.buffer("mixer_out", self.hidden)
        if self.o is None:
            self.branch_step = -(-self.hidden // 8) * 8
            self.branch_buf = ws.buffer("joined_branches", len(self.members) * self.branch_step)
        if any(-(-m.out_columns // 8) * 8 != m.out_columns for _, m, _, _ in self.members):
            self.mid_buf.zero_()      # padding columns meet zero weights, but must hold numbers
        for _, m, _, _ in self.members:
            m.bind_core(ctx)

    def forward(self, x, batch, cache: CacheView, into=None):
        T = batch.num_tokens
        self.proj.forward(x, self.proj_buf, T, scratch=True)
        for name, m, col, out_col in self.members:
            m.core(self.proj_buf, col, self.mid_buf, out_col, batch, cache.child(name))
        if self.o is None:
            return self._normed_sum(T, into)
        y = self.o.forward(self.mid_buf, self.out_buf, T, scratch=True)
        if self.bias is not None:
            ops.add_rows(y, T, vec=self.bias)
        return y

    def _normed_sum(self, T, into):
        for i, ((_, m, _, out_col), lin) in enumerate(zip(self.members, self.outs)):
            c = i * self.branch_step
            gemm.matmul_nt(self.mid_buf[:, out_col:out_col + lin.in_features], lin.weight,
                           self.branch_buf[:, c:c + self.hidden], T, may_pad=True)
        kw = dict(eps=[self.out_norm_eps] * len(self.members), scale=self.sum_scale, bias=self.bias)
        if into is not None and into.stream.dtype == torch.float32 and isinstance(into.norm, GroupRMSNorm):
            n = into.norm
            ops.joined_norms(self.branch_buf, self.out_gains, T, stream=into.stream, out=into.buf, weight=n.weight,
                             norm_eps=n.eps, groups=n.groups, **kw)
            return Carried(None, None, 0, 0.0, self.hidden, n, into.stream, into.buf, T, ready=True)
        ops.joined_norms(self.branch_buf, self.out_gains, T, out=self.out_buf, **kw)
        return self.out_buf
