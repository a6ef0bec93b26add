"""Dumovik without a GPU: the configuration and its refusals, tensor names of the model description, the caches its layers
ask for (and how far back one must keep keys that another layer reads), and the plain float64 model (plain_dumovik.py) pinned
by library functions and hand-worked cases."""
import copy
import json
import math

import pytest
import torch

import plain_dumovik as plain

F = torch.float64


def dense(layer, ff=40):
    return dict(layer, mlp=dict(kind="dense", ff=ff))


def routed(layer, experts=5, top=2, ff=24, limit=1.5):
    return dict(layer, mlp=dict(kind="moe", expert=dict(ff=ff, limit=limit), router=dict(experts=experts, top=top)))


def bare(layer):
    return dict(layer, mlp=None)


def lightning(**kw):
    return dict(type="lightning", mixer=dict(dict(heads=2, dim=16, vdim=24, decay=[0.5, 0.97]), **kw))


def latent(**kw):
    return dict(type="latent_attention", mixer=dict(dict(heads=3, dim=16, rot_dim=8, vdim=12, kv_rank=20, scale=0.2,
                                                         rot=dict(base=1000.0, dims=8)), **kw))


def attention(**kw):
    return dict(type="attention", mixer=dict(dict(heads=4, kv_heads=2, dim=16, vdim=8, scale=0.3, softcap=4.0, mask=dict(size=9)), **kw))


def config(**kw):
    return dict(dict(architecture="Dumovik", vocab=96, width=64, norm=dict(eps=1e-5),
                     layers=[dense(lightning()), routed(latent()), routed(attention()), dense(attention(kv_from=2, mask=dict(size=30))),
                             bare(attention(mask=dict(size=9)))]), **kw)


def parsed(cfg):
    from dinfer_amd.config.registry import architecture_of
    arch = architecture_of(cfg)
    return arch, arch.config_class.from_dict(cfg)


def changed(layer, path, value):
    out = copy.deepcopy(layer)
    d = out
    for k in path[:-1]:
        d = d[k]
    d[path[-1]] = value
    return out


def test_config_round_trip_and_refusals():
    from dinfer_amd.config.base import ConfigError
    arch, cfg = parsed(config())
    assert arch.name == "Dumovik" and cfg.vocab_size == 96 and cfg.hidden_size == 64
    assert type(cfg).from_dict(json.loads(json.dumps(cfg.to_dict()))) == cfg
    open_ = parsed(config(layers=[bare(attention(softcap=None, mask=None))]))[1]
    assert open_.layers[0].mixer.softcap is None and open_.kept_keys(0) is None
    assert type(open_).from_dict(open_.to_dict()) == open_
    bad = [dict(layers=[]), dict(norm=None), dict(layers=[dict(bare(lightning()), type="mamba")]), dict(width=0),
           dict(layers=[bare(lightning(decay=[0.5]))]), dict(layers=[bare(lightning(decay=[0.5, 1.5]))]),
           dict(layers=[bare(lightning(decay=[0.5, 0.0]))]), dict(layers=[bare(lightning(decay=[0.5, "x"]))]),
           dict(layers=[bare(attention(kv_heads=3))]), dict(layers=[bare(attention(softcap=-1.0))]),
           dict(layers=[bare(attention(mask=dict(size=0)))]), dict(layers=[bare(attention(kv_from=0))]),
           dict(layers=[bare(lightning()), bare(attention(kv_from=0))]),
           dict(layers=[bare(attention()), bare(attention(kv_from=0)), bare(attention(kv_from=1))]),
           dict(layers=[bare(attention()), bare(attention(kv_from=0, vdim=12))]),
           dict(layers=[bare(latent()), bare(latent(kv_from=0))]),
           dict(layers=[changed(bare(latent()), ["mixer", "rot", "dims"], 10)]), dict(layers=[changed(bare(latent()), ["mixer", "rot", "dims"], 3)]),
           dict(layers=[routed(lightning(), top=6)]), dict(layers=[routed(lightning(), limit=0.0)]),
           dict(layers=[dict(lightning(), mlp=dict(kind="wide", ff=8))])]
    for change in bad:
        with pytest.raises(ConfigError):
            parsed(config(**change))


def test_tensor_names_and_caches():
    from dinfer_amd.parts import DecoderModel
    arch, cfg = parsed(config())
    spec = arch.build_spec(cfg)
    assert spec.stream_dtype == "float32" and spec.tie_embeddings
    m = DecoderModel(spec)
    exp, optional = m.expected_tensors()
    assert optional == {"head"}          # (a file may carry the head again)
    assert {n: tuple(s.shape) for n, s in exp.items()} == {n: tuple(s) for n, s in plain.tensor_shapes(config()).items()}
    # (the latent layers' cache depends on the kernels chosen when a model is bound to a device)
    needs = DecoderModel(arch.build_spec(parsed(config(layers=[l for l in config()["layers"] if l["type"] != "latent_attention"][:1]
                                                      + [bare(lightning())] + config()["layers"][2:]))[1])).cache_needs()
    assert needs[0].group_key() is None and needs[0].slot_bytes(torch.bfloat16) == 2 * 16 * 24 * 4
    assert needs[2].window == 30 and needs[3] is None and needs[4].window == 9      # layer 3 looks further back than the owner
    assert needs[2].group_key() != needs[4].group_key()
    wide = config(layers=[bare(attention()), bare(attention(kv_from=0, mask=None)), bare(attention(kv_from=0, mask=dict(size=4)))])
    assert DecoderModel(arch.build_spec(parsed(wide)[1])).cache_needs()[0].window is None


def test_norms_and_activations_by_hand():
    x = torch.tensor([[3.0, 5.0, 4.0, 0.0]], dtype=F)
    w = torch.tensor([1.0, 2.0, 3.0, 4.0], dtype=F)
    assert torch.allclose(plain.layer_norm(x, w, 1e-3), torch.nn.functional.layer_norm(x, (4,), w, None, 1e-3))
    assert torch.allclose(plain.rms_norm(x, w, 0.5), x / math.sqrt(12.5 + 0.5) * w)
    z = torch.linspace(-4, 4, 33, dtype=F)
    assert torch.allclose(plain.gelu_tanh(z), torch.nn.functional.gelu(z, approximate="tanh"))
    assert torch.allclose(plain.silu(z), torch.nn.functional.silu(z))


def test_chunks_and_caps_by_hand():
    m = plain.visible(7, 3)
    assert m[5].tolist() == [False, False, False, True, True, True, False]
    assert m[3].tolist() == [False, False, False, True, False, False, False]          # a chunk's first position sees itself alone
    assert m[2].tolist() == [True, True, True, False, False, False, False]
    s = torch.tensor([-1e9, -0.01, 0.0, 3.0, 1e9], dtype=F)
    c = plain.soft_cap(s, 2.0)
    assert abs(c[0] + 2) < 1e-12 and abs(c[4] - 2) < 1e-12 and abs(c[3] - 2 * math.tanh(1.5)) < 1e-12 and c[2] == 0


def test_rotation_by_hand():
    x = torch.arange(1.0, 7.0, dtype=F).view(1, 1, 6).repeat(3, 1, 1)
    y = plain.rotate_halves(x, dict(base=100.0, dims=4))
    assert torch.equal(y[0], x[0]) and y[2, 0, 4:].tolist() == [5.0, 6.0]
    for i, (f, a, b) in enumerate(((1.0, 0, 2), (0.1, 1, 3))):
        u, v = x[2, 0, a].item(), x[2, 0, b].item()
        assert abs(y[2, 0, a].item() - (u * math.cos(2 * f) - v * math.sin(2 * f))) < 1e-12
        assert abs(y[2, 0, b].item() - (v * math.cos(2 * f) + u * math.sin(2 * f))) < 1e-12


def test_lightning_by_hand():
    """One head, decay 1/2, two tokens; the norm takes both value entries of the head at once."""
    eye = torch.eye(2, dtype=F)
    w = {"m.q": eye, "m.k": eye, "m.v": eye, "m.g": eye * 0.0, "m.o": eye, "m.norm": torch.tensor([1.0, 3.0], dtype=F)}
    h = torch.tensor([[1.0, 0.0], [2.0, -1.0]], dtype=F)
    a = plain.silu(h)
    S = torch.outer(a[0], a[0])
    o0 = S.T @ a[0]
    S = 0.5 * S + torch.outer(a[1], a[1])
    o1 = S.T @ a[1]
    want = torch.stack([o / o.pow(2).mean().sqrt() for o in (o0, o1)]) * w["m.norm"] * 0.5      # (the gate: sigmoid of zero)
    assert torch.allclose(plain.lightning(h, w, "m", dict(heads=1, dim=2, vdim=2, decay=[0.5]), 0.0), want)


def test_expert_and_router_by_hand():
    w = {"m.router": torch.tensor([[1.0, 0.0], [0.0, 1.0], [-1.0, 0.0]], dtype=F)}
    for e in range(3):
        w[f"m.e{e}.gate"], w[f"m.e{e}.up"] = torch.tensor([[1.0 + e, 0.0]], dtype=F), torch.tensor([[0.0, 4.0]], dtype=F)
        w[f"m.e{e}.down"] = torch.tensor([[1.0], [e]], dtype=F)
    h = torch.tensor([[2.0, -1.0]], dtype=F)
    f = dict(router=dict(experts=3, top=2), expert=dict(ff=1, limit=3.0))
    idx, share = plain.chosen_experts(h, w, "m", f)
    s = torch.softmax(torch.tensor([2.0, -1.0], dtype=F), 0)
    assert idx.tolist() == [[0, 1]] and torch.allclose(share, s[None])
    glu = lambda g, u: min(g, 3.0) / (1 + math.exp(-1.702 * min(g, 3.0))) * (max(-3.0, min(3.0, u)) + 1)
    y = [glu(2.0, -4.0), glu(4.0, -4.0)]                 # the second expert's gate and both values meet the limit
    assert torch.allclose(plain.routed_ff(h, w, "m", f), torch.tensor([[s[0] * y[0] + s[1] * y[1], s[1] * y[1]]], dtype=F))
    low = plain.expert(torch.tensor([-9.0, 0.0], dtype=F), w, "m.e0", 3.0)       # the gate has no lower limit
    assert torch.allclose(low[0], torch.tensor(-9.0 / (1 + math.exp(1.702 * 9.0)), dtype=F))


def test_a_layer_reads_the_keys_of_the_layer_it_names():
    cfg = config()
    w = plain.as_float64(plain.random_weights(cfg, 5))
    kept = {}
    h = torch.randn(12, 64, dtype=F, generator=torch.Generator().manual_seed(1))
    plain.mixer(h, w, cfg, 2, kept)
    k, v = kept[2]
    got = plain.mixer(h * 2, w, cfg, 3, kept)
    assert list(kept) == [2] and torch.equal(kept[2][0], k)
    assert torch.equal(got, plain.chunked_attention(h * 2, w, "l3.mix", cfg["layers"][3]["mixer"], 1e-5, k, v))
    assert not torch.allclose(got, plain.chunked_attention(h * 2, w, "l3.mix", cfg["layers"][2]["mixer"], 1e-5, k, v))


def test_latent_attention_against_expanded_keys():
    """The same through torch's attention on keys and values written out for every head."""
    cfg = config()
    m = cfg["layers"][1]["mixer"]
    w = plain.as_float64(plain.random_weights(cfg, 6))
    p, T, H = "l1.mix", 9, m["heads"]
    h = torch.randn(T, 64, dtype=F, generator=torch.Generator().manual_seed(2))
    q = (h @ w[p + ".q"].T).view(T, H, 24)
    d = h @ w[p + ".dkv"].T
    c = plain.rms_norm(d[:, :20], w[p + ".dkv.norm"], 1e-5)
    k = torch.cat([(c @ w[p + ".uk"].T).view(T, H, 16), plain.rotate_halves(d[:, None, 20:], m["rot"]).expand(T, H, 8)], -1)
    q = torch.cat([q[..., :16], plain.rotate_halves(q[..., 16:], m["rot"])], -1)
    v = (c @ w[p + ".uv"].T).view(T, H, 12)
    a = torch.nn.functional.scaled_dot_product_attention(q.transpose(0, 1), k.transpose(0, 1), v.transpose(0, 1), is_causal=True, scale=0.2)
    want = (a.transpose(0, 1).reshape(T, -1) * torch.sigmoid(h @ w[p + ".g"].T)) @ w[p + ".o"].T
    assert torch.allclose(plain.latent_attention(h, w, p, m, 1e-5), want)


def test_parts_refuse_what_they_do_not_do():
    from dinfer_amd.parts.registry import BLOCKS, FEED_FORWARDS, MIXERS
    from dinfer_amd.parts.spec import LayerSpec, part
    att = dict(hidden=32, heads=2, kv_heads=1, head_dim=8, position=part("none"))
    for kw in (dict(softcap=-1.0), dict(softcap=2.0, sigmoid_bias=True), dict(shares_cache=True, bias=True),
               dict(shares_cache=True, qk_norm=part("rmsnorm", eps=1e-5)), dict(chunk=8, cache_window=4), dict(cache_window=5),
               dict(chunk=8, keep_first=2),
               dict(shares_cache=True, position=part("rotary", theta=10.0, max_positions=9))):
        with pytest.raises(ValueError):
            MIXERS.get("attention")(**{**att, **kw})
    assert MIXERS.get("attention")(**att, chunk=8, cache_window=12).cache_spec().window == 12
    assert MIXERS.get("attention")(**att, chunk=8, window=5).cache_spec().window == 5
    for kw in (dict(clamp=(0.0, 1.0)), dict(clamp=(1.0, 1.0), gated=False), dict(clamp=(1.0, 1.0), shared_intermediate=8)):
        with pytest.raises(ValueError):
            FEED_FORWARDS.get("moe")(32, experts=4, top=1, intermediate=8, **kw)
    for kw in (dict(decay=[0.5]), dict(decay=[0.5, 0.0]), dict(dim=512)):
        with pytest.raises(ValueError):
            MIXERS.get("lightning")(32, **{**dict(heads=2, dim=8, vdim=8, decay=[0.5, 0.5], norm_eps=1e-5), **kw})
    with pytest.raises(ValueError):
        MIXERS.get("latent_attention")(32, heads=1, dim=8, rot_dim=8, vdim=8, rank=16, scale=1.0, gated="all", position=part("none"),
                                       latent_norm=part("rmsnorm", eps=1e-5))
    spec = LayerSpec(block=part("outnorm"), mixer=part("lightning", heads=1, dim=8, vdim=8, decay=[0.5], norm_eps=1e-5),
                     feed_forward=part("none"), norm=part("rmsnorm", eps=1e-5), prefix="l0.")
    with pytest.raises(ValueError):
        BLOCKS.get("outnorm")(hidden=32, layer=spec)
