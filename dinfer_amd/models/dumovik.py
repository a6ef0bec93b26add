"""Dumovik: configuration -> ModelSpec.

embed -> blocks whose sublayers read the stream itself and whose outputs are normed (h += norm1(mixer(h)); h += norm2(ff(h)))
-> norm -> the embedding table as head. Layer norms with a gain and no bias, a 32-bit residual stream. Mixers:
`latent_attention` (one normed latent a token and a rotated key part shared by the heads, pairs (i, i + dims/2), causal, one
sigmoid gate an output entry); `attention` (norms of q and k over the whole projection, no positions, softly capped scores,
keys of the query's own chunk of positions; a layer with `kv_from` runs on the cache of the layer it names: a run entry that
borrows); `lightning` (a recurrent state with a fixed decay a head over silu-activated q, k and v). Feed-forwards: gated with
the tanh form of gelu, or routed experts with clamps, weighted by the softmax over the chosen logits.
Tensor names: embed, l<i>.norm{1,2}, l<i>.mix.{q, dkv, dkv.norm, uk, uv, g, o} or l<i>.mix.{q, k, v, q.norm, k.norm, o} or
l<i>.mix.{q, k, v, g, norm, o}; l<i>.mlp.{gate, up, down} or l<i>.mlp.{router, e<j>.{gate, up, down}}; final.norm.
"""
from __future__ import annotations

from ..config.dumovik import DumovikConfig
from ..config.registry import register_architecture
from ..parts.spec import LayerSpec, ModelSpec, RunEntry, part

EXPERT_SLOPE = 1.702     # of the sigmoid in an expert's gate


def _mixer(cfg: DumovikConfig, i: int):
    l = cfg.layers[i]
    m, eps = l.mixer, cfg.norm_eps
    if l.type == "latent_attention":
        position = part("rotary", theta=m.rot_base, max_positions=cfg.MAX_POSITIONS, rotary_dim=m.rot_dims, style="neox")
        return part("latent_attention", heads=m.heads, dim=m.dim, rot_dim=m.rot_dim, vdim=m.vdim, rank=m.kv_rank, scale=m.scale,
                    position=position, latent_norm=part("rmsnorm", eps=eps, weight_name=""), gated="entries")
    if l.type == "lightning":
        return part("lightning", heads=m.heads, dim=m.dim, vdim=m.vdim, decay=m.decay, norm_eps=eps)
    borrows = m.kv_from is not None
    return part("attention", heads=m.heads, kv_heads=m.kv_heads, head_dim=m.dim, v_dim=m.vdim, position=part("none"), scale=m.scale,
                qk_row_eps=eps, softcap=m.softcap, chunk=m.chunk, shares_cache=borrows,
                cache_window=m.chunk if borrows else cfg.kept_keys(i),
                names={"q": "q", "k": "k", "v": "v", "o": "o", "q_norm": "q.norm", "k_norm": "k.norm"})


def _feed_forward(f):
    if f is None:
        return part("none")
    if f.kind == "dense":
        return part("gated_mlp", intermediate=f.ff, act="gelu_tanh", names=("gate", "up", "down"))
    return part("moe", experts=f.experts, top=f.top, intermediate=f.ff, clamp=(f.limit, EXPERT_SLOPE))


def build_spec(cfg: DumovikConfig) -> ModelSpec:
    norm = part("layernorm", eps=cfg.norm_eps, bias=False, weight_name="")
    layers, run = [], []
    for i, l in enumerate(cfg.layers):
        layers.append(LayerSpec(block=part("outnorm"), mixer=_mixer(cfg, i), feed_forward=_feed_forward(l.mlp), norm=norm,
                                prefix=f"l{i}."))
        # layer i is run entry i, so a layer index names the entry whose cache is read
        run.append(RunEntry(i, l.mixer.kv_from if l.type == "attention" else None))
    return ModelSpec(
        architecture=cfg.ARCHITECTURE, vocab_size=cfg.vocab, hidden_size=cfg.width, max_positions=cfg.MAX_POSITIONS,
        layers=layers, run=run, final_norm=norm, final_norm_name="final.norm", embed_name="embed", head_name="head",
        tie_embeddings=True, eos_token_ids=(), stream_dtype="float32")


register_architecture(DumovikConfig.ARCHITECTURE, DumovikConfig, build_spec)
