"""Lotelix: configuration -> ModelSpec.

embed * scale -> pre-norm blocks( mixer | routed feed-forward or none ) -> norm -> head, a 32-bit residual stream, norms in
groups (equal parts of a row, each divided by its own root mean square) with plain gains. Mixers: `mingru` (a gated
recurrence of single channels); `attention` (a sliding window, a learned sink a head, rotation of pairs (i, i + dims/2) with
slow frequencies slowed further, an output gate an entry, values mixed with those of the first layer that mixes); `parallel`
(a causal attention whose weights are sigmoids of the scores plus a bias a head, with norms of q and k over the whole
projection, biases and a rotation of pairs (2i, 2i + 1), beside a gated linear attention; half the sum of the two outputs,
each normed over the width first). Feed-forward: routed experts down(relu(up x)^2) chosen by sigmoid score, the score
multiplying the expert's input.
Tensor names: embed, l<i>.norm{1,2}, l<i>.mix.{z, z.b, x, x.b, g, o} or l<i>.mix.{q, k, v, sink, vmix, g, o} or
l<i>.mix.left.{q, k, v, o}(.b), l<i>.mix.left.{q.norm, k.norm, pb, out} and
l<i>.mix.right.{q, k, v, g, a1, a2, a2.b, norm, o, out}; l<i>.mlp.{router, e<j>.{up, down}}; final.norm, head.
"""
from __future__ import annotations

from ..config.lotelix import LotelixConfig
from ..config.registry import register_architecture
from ..parts.spec import LayerSpec, ModelSpec, RunEntry, part

OUTPUT_SHARE = 0.5     # of each half of a parallel layer


def _position(cfg: LotelixConfig, rot, style: str):
    if rot.dims == 0:
        return part("none")
    scaling = None
    if rot.scaling is not None:
        s = rot.scaling
        scaling = dict(kind="wavelength_bands", factor=s.factor, low=s.low, high=s.high, original=s.original)
    return part("rotary", theta=rot.base, max_positions=cfg.MAX_POSITIONS, rotary_dim=rot.dims, style=style, scaling=scaling)


def _mixer(cfg: LotelixConfig, i: int):
    l = cfg.layers[i]
    m = l.mixer
    if l.type == "mingru":
        return part("min_gru", channels=m.width)
    if l.type == "attention":
        mixes = None if not m.v_mix else "keep" if i == cfg.first_mixing_layer else "mix"
        return part("attention", heads=m.heads, kv_heads=m.kv_heads, head_dim=m.dim, v_dim=m.vdim,
                    position=_position(cfg, m.rot, "neox"), window=m.window, scale=m.scale, sink=True, gate="sigmoid",
                    value_mix=mixes, names={"q": "q", "k": "k", "v": "v", "o": "o", "sink": "sink", "g": "g", "value_mix": "vmix"})
    a, r = m.left, m.right
    left = part("attention", heads=a.heads, kv_heads=a.kv_heads, head_dim=a.dim, v_dim=a.vdim,
                position=_position(cfg, a.rot, "interleaved"), scale=a.scale, bias=True, out_bias=True, qk_row_eps=cfg.norm_eps,
                sigmoid_bias=True,
                names={"q": "q", "k": "k", "v": "v", "o": "o", "q_bias": "q.b", "k_bias": "k.b", "v_bias": "v.b",
                       "o_bias": "o.b", "q_norm": "q.norm", "k_norm": "k.norm", "sigmoid_bias": "pb"})
    right = part("gated_linear_attention", heads=r.heads, dim=r.dim, vdim=r.vdim, low=r.decay_rank, tau=r.tau,
                 norm_eps=cfg.norm_eps)
    return part("joined", members=[("left", left, OUTPUT_SHARE), ("right", right, OUTPUT_SHARE)], out_norm_eps=cfg.norm_eps)


def build_spec(cfg: LotelixConfig) -> ModelSpec:
    norm = part("group_rmsnorm", eps=cfg.norm_eps, groups=cfg.norm_groups, weight_name="")
    block = part("prenorm", mixer_prefix="mix.", ff_prefix="mlp.", norm_in="norm1", norm_post="norm2")
    layers = []
    for i, l in enumerate(cfg.layers):
        f = l.mlp
        ff = part("none") if f is None else part("moe", experts=f.experts, top=f.top, intermediate=f.ff, act="relu2", gated=False,
                                                 scores="sigmoid", weigh="input")
        layers.append(LayerSpec(block=block, mixer=_mixer(cfg, i), feed_forward=ff, norm=norm, prefix=f"l{i}."))
    return ModelSpec(
        architecture=cfg.ARCHITECTURE, vocab_size=cfg.vocab, hidden_size=cfg.width, max_positions=cfg.MAX_POSITIONS,
        layers=layers, run=[RunEntry(i) for i in range(len(layers))], final_norm=norm, final_norm_name="final.norm",
        embed_name="embed", head_name="head", tie_embeddings=False, eos_token_ids=(), embed_scale=cfg.embedding_scale,
        stream_dtype="float32")


register_architecture(LotelixConfig.ARCHITECTURE, LotelixConfig, build_spec)
