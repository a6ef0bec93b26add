"""Lotelix without a GPU: the configuration and its refusals, the size that only a tensor's shape gives, tensor names of
the model description, the caches its layers ask for, and the plain float64 model (plain_lotelix.py) pinned by library
functions and hand-worked cases."""
import copy
import json
import math

import pytest
import torch

import plain_lotelix as plain

F = torch.float64


def routed(layer, experts=5, top=2, ff=24):
    return dict(layer, mlp=dict(kind="moe", expert=dict(ff=ff), router=dict(experts=experts, top=top)))


def gru(width=40):
    return routed(dict(type="mingru", mixer=dict(width=width)))


def attention(**kw):
    m = dict(heads=4, kv_heads=2, dim=16, vdim=8, scale=0.3, mask=dict(size=9), v_mix=True,
             rot=dict(base=1000.0, dims=12, scaling=dict(factor=4.0, low=1.0, high=3.0, original=64)))
    m.update(kw)
    return routed(dict(type="attention", mixer=m))


def parallel(rank=None):
    right = dict(heads=2, dim=16, vdim=24, tau=4.0)
    if rank is not None:
        right["decay_rank"] = rank
    return dict(type="parallel", mlp=None,
                mixer=dict(left=dict(heads=4, kv_heads=1, dim=16, vdim=8, scale=0.25, rot=dict(base=500.0, dims=4)), right=right))


def config(rank=6, **kw):
    cfg = dict(architecture="Lotelix", vocab=96, width=64, embedding=dict(scale=3.0), norm=dict(eps=1e-5, groups=4),
               layers=[gru(), parallel(rank), attention(), attention(heads=2, kv_heads=1, vdim=16)])
    cfg.update(kw)
    return cfg


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
    assert arch.name == "Lotelix" and cfg.vocab_size == 96 and cfg.hidden_size == 64 and cfg.first_mixing_layer == 2
    assert type(cfg).from_dict(json.loads(json.dumps(cfg.to_dict()))) == cfg
    plain_rot = parsed(config(layers=[attention(rot=dict(base=10.0, dims=16, scaling=None))]))[1]
    assert plain_rot.layers[0].mixer.rot.scaling is None
    assert parsed(config(norm=dict(eps=1e-5)))[1].norm_groups == 1
    bad = [dict(layers=[]), dict(norm=None), dict(norm=dict(eps=1e-5, groups=5)), dict(embedding=None),
           dict(layers=[dict(gru(), type="mamba")]), dict(layers=[dict(gru(), mlp=dict(kind="dense", ff=8))]),
           dict(layers=[changed(gru(), ["mlp", "router", "top"], 6)]), dict(layers=[changed(attention(), ["mixer", "kv_heads"], 3)]),
           dict(layers=[changed(attention(), ["mixer", "rot", "dims"], 18)]), dict(layers=[changed(attention(), ["mixer", "rot", "dims"], 7)]),
           dict(layers=[changed(attention(), ["mixer", "rot", "scaling", "high"], 1.0)]),
           dict(layers=[attention(), attention(vdim=12)])]              # mixed values of two sizes
    for change in bad:
        with pytest.raises(ConfigError):
            parsed(config(**change))
    with pytest.raises(ConfigError):                    # the decay projection's inner size is in no key and no tensor
        parsed(config(rank=None))
    parsed(config(layers=[attention(), attention(vdim=12, v_mix=False)]))      # a layer that does not mix may differ


def test_the_size_that_only_a_tensor_gives(tmp_path):
    from dinfer_amd.config import load_config
    from dinfer_amd.weights.safetensors_io import write_safetensors
    cfg = config(rank=None)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    write_safetensors(tmp_path / "model.safetensors", plain.random_weights(cfg, 3, low=11), metadata={"format": "pt"})
    assert load_config(tmp_path)[1].layers[1].mixer.right.decay_rank == 11
    cfg["layers"][1]["mixer"]["right"]["decay_rank"] = 4     # a file that names the size is taken at its word
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    assert load_config(tmp_path)[1].layers[1].mixer.right.decay_rank == 4


def test_tensor_names_and_caches():
    from dinfer_amd.parts import DecoderModel
    arch, cfg = parsed(config(rank=6))
    spec = arch.build_spec(cfg)
    assert spec.stream_dtype == "float32" and spec.embed_scale == 3.0 and not spec.tie_embeddings
    m = DecoderModel(spec)
    exp, optional = m.expected_tensors()
    assert not optional
    assert {n: tuple(s.shape) for n, s in exp.items()} == {n: tuple(s) for n, s in plain.tensor_shapes(config(rank=6)).items()}
    needs = m.cache_needs()
    assert needs[0].group_key() is None and needs[0].slot_bytes(torch.bfloat16) == 40 * 4
    assert needs[1].window is None and needs[1].slot_bytes(torch.bfloat16) == 2 * 16 * 24 * 4
    assert needs[2].window == 9 and needs[2].group_key() != needs[3].group_key()
    assert [b.mixer.value_mix for b in m.blocks if hasattr(b.mixer, "value_mix")] == ["keep", "mix"]


def test_only_layers_that_mix_take_part_in_it():
    from dinfer_amd.parts import DecoderModel
    arch, cfg = parsed(config(layers=[attention(v_mix=False), attention(), attention(), attention(v_mix=False)]))
    m = DecoderModel(arch.build_spec(cfg))
    assert [b.mixer.value_mix for b in m.blocks] == [None, "keep", "mix", None]
    exp, _ = m.expected_tensors()
    assert [f"l{i}.mix.vmix" in exp for i in range(4)] == [False, True, True, False]


def test_group_norm_by_hand():
    x = torch.tensor([[3.0, 4.0, 0.0, 2.0]], dtype=F)
    w = torch.tensor([1.0, 2.0, 3.0, 4.0], dtype=F)
    got = plain.group_norm(x, w, 0.0, 2)
    a, b = math.sqrt(12.5), math.sqrt(2.0)
    assert torch.allclose(got, torch.tensor([[3 / a, 8 / a, 0.0, 8 / b]], dtype=F))
    assert torch.allclose(plain.group_norm(x, w, 1e-3, 1), plain.rms_unit(x, 1e-3) * w)


def test_rotations_and_frequencies_by_hand():
    x = torch.tensor([[[1.0, 2.0, 3.0, 4.0, 5.0, 6.0]]], dtype=F).repeat(2, 1, 1)       # two positions, one head of 6
    rot = dict(base=100.0, dims=4)
    f = [1.0, 0.1]
    assert torch.allclose(plain.frequencies(rot), torch.tensor(f, dtype=F))
    for turn, pairs in ((plain.rotate_halves, [(0, 2), (1, 3)]), (plain.rotate_neighbours, [(0, 1), (2, 3)])):
        y = turn(x, rot)
        assert torch.equal(y[0], x[0]) and y[1, 0, 4:].tolist() == [5.0, 6.0]
        for i, (a, b) in enumerate(pairs):
            u, v = x[1, 0, a].item(), x[1, 0, b].item()
            assert abs(y[1, 0, a].item() - (u * math.cos(f[i]) - v * math.sin(f[i]))) < 1e-12
            assert abs(y[1, 0, b].item() - (v * math.cos(f[i]) + u * math.sin(f[i]))) < 1e-12
    # wavelengths 2 pi, 62.8, 628: kept (shorter than 60 / 3), in between (20 to 300), slowed (longer than 300)
    sc = dict(base=1000.0, dims=6, scaling=dict(factor=8.0, low=0.2, high=3.0, original=60.0))
    s = (60.0 * 0.1 / (2 * math.pi) - 0.2) / (3.0 - 0.2)
    assert torch.allclose(plain.frequencies(sc), torch.tensor([1.0, (1 - s) * 0.1 / 8 + s * 0.1, 0.01 / 8], dtype=F))


def test_the_engines_rotation_has_these_frequencies():
    from dinfer_amd.parts.position import Rotary
    for rot in (dict(base=1000.0, dims=12), dict(base=250.0, dims=16, scaling=dict(factor=5.0, low=0.5, high=4.0, original=96.0))):
        sc = dict(rot["scaling"], kind="wavelength_bands") if "scaling" in rot else None
        got, size = Rotary(16, rot["base"], 100, rotary_dim=rot["dims"], scaling=sc).frequencies()
        assert size == 1.0 and torch.allclose(got, plain.frequencies(rot))


def test_windows_sinks_and_sigmoid_weights():
    m = plain.visible(6, 3)
    assert m[5].tolist() == [False, False, False, True, True, True] and m[1].tolist() == [True, True, False, False, False, False]
    s = torch.randn(6, 6, dtype=F, generator=torch.Generator().manual_seed(1))
    sink = torch.tensor(0.7, dtype=F)
    p = plain.softmax_with_sink(s, m, sink)
    want = torch.softmax(torch.cat([s[5, 3:], sink[None]]), -1)      # the sink as one more score without a value
    assert torch.allclose(p[5, 3:], want[:3]) and p[5, :3].abs().max().item() == 0.0
    g = plain.sigmoid_weights(s, plain.visible(6), torch.tensor(-1.5, dtype=F))
    assert torch.allclose(g[4, :5], torch.sigmoid(s[4, :5] - 1.5)) and g[4, 5].item() == 0.0


def test_min_gru_by_hand():
    """One channel, two tokens: gates of 1/4 and 1/2, candidates above and below zero."""
    w = {"m.z": torch.tensor([[1.0, 0.0]], dtype=F), "m.z.b": torch.tensor([-math.log(3.0)], dtype=F),
         "m.x": torch.tensor([[0.0, 1.0]], dtype=F), "m.x.b": torch.tensor([0.0], dtype=F),
         "m.g": torch.tensor([[0.0, 0.0]], dtype=F) + 1.0, "m.o": torch.tensor([[1.0], [2.0]], dtype=F)}
    h = torch.tensor([[0.0, 2.0], [math.log(3.0), -1.0]], dtype=F)
    s0 = 0.25 * 2.5
    s1 = 0.5 * s0 + 0.5 / (1 + math.e)
    gate = plain.silu(h.sum(-1))
    want = torch.tensor([[s0, 2 * s0], [s1, 2 * s1]], dtype=F) * gate[:, None]
    assert torch.allclose(plain.min_gru(h, w, "m"), want)


def test_gated_linear_attention_by_hand():
    """One head of two channels whose decays are 1/4 and 1, two equal tokens."""
    eye, z = torch.eye(2, dtype=F), torch.zeros(2, 2, dtype=F)
    w = {"m.q": eye, "m.k": eye, "m.v": eye * 2, "m.g": eye, "m.o": eye, "m.norm": torch.ones(2, dtype=F),
         "m.a1": torch.zeros(1, 2, dtype=F), "m.a2": torch.zeros(2, 1, dtype=F),
         "m.a2.b": torch.tensor([-math.log(15.0), 60.0], dtype=F)}
    m = dict(heads=1, dim=2, vdim=2, tau=2.0)
    h = torch.tensor([[1.0, 1.0], [1.0, 1.0]], dtype=F)
    assert torch.allclose(plain.channel_decays(h, w, "m", m)[0, 0], torch.tensor([0.25, 1.0], dtype=F))
    # S after token 1: [[2, 2], [2, 2]], after token 2: [[0.5 + 2, ..], [4, 4]]; both entries of o are equal, so they norm to one
    out = plain.gated_linear_attention(h, w, "m", m, eps=0.0)
    assert torch.allclose(out, plain.silu(torch.ones(2, 2, dtype=F)))
    w["m.v"] = torch.tensor([[2.0, 0.0], [0.0, 2.0]], dtype=F)
    h = torch.tensor([[1.0, 0.0], [1.0, 1.0]], dtype=F)
    # token 1: S = [[2, 0], [0, 0]]; token 2: S = [[0.5 + 2, 2], [2, 2]], o ~ [4.5, 4]
    o = torch.tensor([4.5, 4.0], dtype=F)
    assert torch.allclose(plain.gated_linear_attention(h, w, "m", m, eps=0.0)[1], o / (o.pow(2).mean()).sqrt() * plain.silu(torch.ones((), dtype=F)))


def test_router_by_hand():
    """The score multiplies the expert's input: with the square of relu it counts twice in the output."""
    w = {"m.router": torch.tensor([[1.0, 0.0], [0.0, 1.0], [-1.0, 0.0]], dtype=F)}
    for e in range(3):
        w[f"m.e{e}.up"] = torch.eye(2, dtype=F) * (e + 1)
        w[f"m.e{e}.down"] = torch.eye(2, dtype=F)
    h = torch.tensor([[2.0, -1.0]], dtype=F)
    s = torch.sigmoid(torch.tensor([2.0, -1.0, -2.0], dtype=F))
    f = dict(router=dict(experts=3, top=2), expert=dict(ff=2))
    idx, share = plain.chosen_experts(h, w, "m", f)
    assert idx.tolist() == [[0, 1]] and torch.allclose(share, s[None, :2])
    want = torch.tensor([[(s[0] * 2) ** 2 + (s[1] * 2 * 2) ** 2, 0.0]], dtype=F)
    assert torch.allclose(plain.routed_ff(h, w, "m", f), want)


def test_values_mix_with_the_first_mixing_layers():
    cfg = config(layers=[attention(v_mix=False), attention(), gru(), attention()], rank=6)
    w = plain.as_float64(plain.random_weights(cfg, 5))
    ids = list(range(20))
    base = plain.forward(ids, w, cfg)
    for layer, matters in ((1, False), (3, True)):      # the first one's lambda is not used
        changed_w = dict(w, **{f"l{layer}.mix.vmix": w[f"l{layer}.mix.vmix"] + 0.3})
        assert (not torch.equal(plain.forward(ids, changed_w, cfg), base)) == matters
    kept = {}
    h = torch.randn(6, 64, dtype=F, generator=torch.Generator().manual_seed(1))
    plain.mixer(h, w, cfg, 0, kept)
    assert "v" not in kept
    plain.mixer(h, w, cfg, 1, kept)
    assert torch.equal(kept["v"], h @ w["l1.mix.v"].T)


def test_parts_refuse_what_they_do_not_do():
    from dinfer_amd.parts.registry import FEED_FORWARDS, MIXERS, NORMS
    from dinfer_amd.parts.spec import part
    att = MIXERS.get("attention")
    base = dict(hidden=32, heads=2, kv_heads=1, head_dim=8, position=part("none"))
    for kw in (dict(qk_row_eps=1e-5, qk_unit_eps=1e-5), dict(sigmoid_bias=True, sink=True), dict(value_mix="all"),
               dict(value_mix="mix", bias=True)):
        with pytest.raises(ValueError):
            att(**base, **kw)
    with pytest.raises(ValueError):
        NORMS.get("group_rmsnorm")(30, eps=1e-5, groups=4)
    with pytest.raises(ValueError):
        FEED_FORWARDS.get("moe")(32, experts=4, top=1, intermediate=8, weigh="input", scores="all", identity=1, gated=False)
    with pytest.raises(ValueError):
        MIXERS.get("gated_linear_attention")(32, heads=1, dim=512, vdim=8, low=4, tau=1.0, norm_eps=1e-5)
    members = [("left", part("attention", **{k: v for k, v in base.items() if k != "hidden"}), 0.5),
               ("right", part("gated_linear_attention", heads=1, dim=8, vdim=8, low=4, tau=1.0, norm_eps=1e-5), 0.25)]
    with pytest.raises(ValueError):
        MIXERS.get("joined")(32, members=members, out_norm_eps=1e-5)
    MIXERS.get("joined")(32, members=members)
