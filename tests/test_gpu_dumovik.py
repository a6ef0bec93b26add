"""Dumovik through the engine against the plain float64 implementation (plain_dumovik.py): every mechanism alone at the
level of its kernels or as a one-layer model, then whole models of made-up sizes in every way of cutting and batching,
32-bit and bfloat16, and greedy generation through the engine's own entry point."""
import copy
import json
import random

import pytest
import torch

import plain_dumovik as plain
from test_gpu_lotelix import unequal
from test_gpu_verorax import check_logits, cut, has_router, mixed_schedule, paged, replay, tokens_for

pytestmark = pytest.mark.gpu
F = torch.float64
DTYPES = ["float32", "bfloat16"]


def lightning(heads, dim, vdim, slow=0.99):
    """Decays from a short memory to a long one."""
    return dict(type="lightning", mixer=dict(heads=heads, dim=dim, vdim=vdim,
                                             decay=[0.3 + (slow - 0.3) * (h + 1) / heads for h in range(heads)]))


def latent(heads, dim, rot_dim, vdim, kv_rank, base=10000.0, scale=None, dims=None):
    return dict(type="latent_attention", mixer=dict(heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, kv_rank=kv_rank,
                                                    scale=scale or (dim + rot_dim) ** -0.5, rot=dict(base=base, dims=dims or rot_dim)))


def attention(heads, kv_heads, dim, vdim, size, softcap=5.0, scale=None, kv_from=None):
    m = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale or dim ** -0.5, softcap=softcap, mask=dict(size=size))
    return dict(type="attention", mixer=m if kv_from is None else dict(m, kv_from=kv_from))


def dense(layer, ff):
    return dict(layer, mlp=dict(kind="dense", ff=ff))


def routed(layer, experts, top, ff, limit=0.8):
    return dict(layer, mlp=dict(kind="moe", expert=dict(ff=ff, limit=limit), router=dict(experts=experts, top=top)))


def bare(layer):
    return dict(layer, mlp=None)


def model(vocab, width, layers, eps=1e-5):
    return dict(architecture="Dumovik", vocab=vocab, width=width, norm=dict(eps=eps), layers=layers)


CONFIGS = {
    # every mixer, both feed-forwards and none; a layer that reads another's keys with a longer chunk, and one with a shorter;
    # two layers of the same kind with other sizes; pages of 4
    "D1": (model(96, 64, [dense(lightning(3, 16, 24), 48), routed(attention(4, 2, 16, 8, 10), 6, 2, 24), routed(latent(3, 16, 8, 12, 20), 6, 2, 24),
                          bare(attention(4, 2, 16, 8, 27, kv_from=1, softcap=2.0, scale=0.5)), dense(lightning(2, 24, 8), 40),
                          bare(attention(4, 2, 16, 8, 4, kv_from=1)), dense(attention(6, 1, 24, 16, 33), 48)]), 4, 11),
    # sizes that are no multiples of 8, one choice, another eps, half of the shared key part rotated
    "D2": (model(131, 72, [routed(latent(3, 20, 12, 10, 28, base=300.0, dims=6), 5, 1, 41), dense(attention(3, 3, 20, 12, 13), 37),
                           routed(lightning(5, 20, 12), 5, 1, 40), bare(attention(3, 3, 20, 12, 13, kv_from=1)), dense(lightning(1, 7, 9), 20)],
                  eps=1e-3), 8, 12),
    # sizes the matrix-core kernels take; values narrower and wider than keys; all experts chosen; the model ends in a mixer
    "D3": (model(120, 128, [dense(lightning(2, 64, 64), 96), routed(latent(4, 32, 16, 32, 64), 8, 3, 64), dense(attention(4, 1, 64, 32, 40), 64),
                            routed(attention(4, 1, 64, 32, 24, kv_from=2), 2, 2, 48), bare(attention(4, 4, 32, 96, 18)), bare(lightning(3, 40, 72, 0.999))]),
           16, 13),
    # chunks of one token, one head, one expert; a cap that bites; chunks longer than the request
    "D4": (model(77, 40, [routed(attention(2, 1, 8, 16, 1), 1, 1, 16), bare(attention(2, 1, 8, 16, 500, kv_from=0, softcap=0.5)),
                          dense(lightning(1, 32, 16, 0.9), 24), routed(latent(1, 8, 2, 8, 16), 1, 1, 16)]), 4, 14),
}
ONE = {
    "lightning": (model(64, 32, [bare(lightning(4, 24, 16))]), 4, 21),
    "lightning_wide": (model(64, 48, [bare(lightning(2, 128, 64, 0.995))]), 8, 22),
    "latent": (model(64, 32, [bare(latent(4, 16, 8, 16, 24))]), 4, 23),
    "chunks": (model(64, 32, [bare(attention(4, 2, 16, 8, 6))]), 4, 24),
    "chunks_wide": (model(64, 48, [bare(attention(4, 2, 64, 64, 9))]), 8, 25),
    "borrowed": (model(64, 32, [bare(attention(4, 2, 16, 8, 6)), bare(attention(4, 2, 16, 8, 11, kv_from=0))]), 4, 26),
    "dense": (model(64, 32, [dense(lightning(1, 8, 8), 72)]), 4, 27),
    "routed": (model(64, 32, [routed(lightning(1, 8, 8), 7, 3, 24)]), 4, 28),
}
# scores so sharp that a key too many or too few, or a cap left out, shows: chunks of 6 and of 10 (on the same keys), pages of 4
SHARP = {
    "sharp": (model(80, 48, [bare(attention(2, 1, 16, 16, 6, softcap=20.0, scale=1.2)), bare(attention(2, 1, 16, 16, 10, softcap=3.0, scale=1.8, kv_from=0))]), 4, 31),
    "far": (model(80, 48, [bare(latent(2, 16, 8, 16, 24, scale=1.5))]), 4, 32),
}


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    from dinfer_amd.weights.safetensors_io import write_safetensors
    out = {}
    for name, (cfg, page, seed) in {**CONFIGS, **ONE, **SHARP}.items():
        d = tmp_path_factory.mktemp(f"dumovik_{name}")
        w = plain.random_weights(cfg, seed)
        (d / "config.json").write_text(json.dumps(cfg))
        write_safetensors(d / "model.safetensors", w, metadata={"format": "pt"})
        out[name] = (d, cfg, plain.as_float64(w), page)
    return out


def make_runner(models, name, dtype, max_tokens=512, num_blocks=160, max_seqs=4, max_len=512, graph=False):
    from dinfer_amd.config import EngineOptions
    from dinfer_amd.engine.runner import ModelRunner
    d, _, _, page = models[name]
    opt = EngineOptions(dtype=dtype, max_model_len=max_len, max_num_seqs=max_seqs, max_num_batched_tokens=max_tokens,
                        block_size=page, num_blocks=num_blocks, max_logits_rows=max_tokens,
                        decode_exempt_from_budget=False, hip_graph=graph)
    return ModelRunner.from_dir(d, opt)


def compare_rows(rows, cfg, w, toks, dtype, what, choices=None, sharp=False):
    """choices: what the engine's routers chose (replay). The plain model takes a choice over where the scores are so
    close that rounding the router's input may have turned it, and refuses any other; without them (steps replayed from
    graphs, another process) a model with routers is allowed some rows that differ by more."""
    assert rows
    for rid in {k[0] for k in rows}:
        want = plain.forward(toks[rid.split("#")[0]], w, cfg, choices=(choices or {}).get(rid))
        pos = sorted(p for (r, p) in rows if r == rid)
        check_logits(torch.stack([rows[(rid, p)] for p in pos]), want[pos], dtype, f"{what} request {rid}",
                     has_router(cfg) and choices is None, sharp)


def run_and_compare(runner, steps, cfg, w, toks, dtype, what):
    choices = {} if dtype == "bfloat16" and has_router(cfg) else None
    rows = replay(runner, steps, choices)
    compare_rows(rows, cfg, w, toks, dtype, what, choices)
    return rows


NAMES = list(CONFIGS)


# ---- one mechanism a model ------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(ONE))
def test_one_mechanism(models, name, dtype):
    """A model of one mechanism: a whole prompt, the same in portions of two and three, and token by token."""
    _, cfg, w, _ = models[name]
    ids = tokens_for(cfg, 45, 3)
    r = make_runner(models, name, dtype)
    for what, parts in (("whole", [ids]), ("portions", cut(ids, [2, 3])), ("longer portions", cut(ids, [9, 20])), ("single tokens", [[t] for t in ids])):
        steps = [([("x", p, list(range(len(p))))], []) for p in parts]
        steps[-1] = (steps[-1][0], ["x"])
        run_and_compare(r, steps, cfg, w, {"x": ids}, dtype, f"{name} alone, {what}")


# ---- kernels alone --------------------------------------------------------------------------------------------
@pytest.mark.parametrize("bdt,sdt,odt", [("float32", "float32", None), ("bfloat16", "float32", "bfloat16"), ("bfloat16", "float32", None),
                                         ("bfloat16", "bfloat16", None), (None, "float32", "bfloat16"), ("float32", "float32", "bfloat16")])
@pytest.mark.parametrize("width", [64, 72, 2048, 4096, 6144, 130, 35])
def test_norm_added_to_the_stream(width, bdt, sdt, odt):
    """A branch normed and added to the stream, and the copy that the next sublayer reads; a copy alone; rows beyond the
    step's left as they are."""
    from dinfer_amd.kernels import ops
    g = torch.Generator().manual_seed(width)
    T, n = 6, 5
    stream = torch.randn(T, width, generator=g).to(getattr(torch, sdt))
    branch = None if bdt is None else (3 * torch.randn(T, width, generator=g) + 1).to(getattr(torch, bdt))
    w, b = 1 + 0.3 * torch.randn(width, generator=g), torch.randn(width, generator=g)
    for bias in (b, None):
        st = stream.cuda()
        out = None if odt is None else torch.zeros(T, width, dtype=getattr(torch, odt), device="cuda")
        ops.layernorm_add(st, n, branch=None if branch is None else branch.cuda(), weight=w.cuda(),
                          bias=None if bias is None else bias.cuda(), eps=1e-3, out=out)
        want = stream.double()
        if branch is not None:
            want = want + plain.layer_norm(branch.double(), w.double(), 1e-3) + (0 if bias is None else bias.double())
        tol = 1e-5 if sdt == "float32" else 2e-2
        assert ((st[:n].double().cpu() - want[:n]).abs() / (1 + want[:n].abs())).max().item() < tol
        assert torch.equal(st[n:].cpu(), stream[n:])
        if out is not None:
            assert ((out[:n].double().cpu() - want[:n]).abs() / (1 + want[:n].abs())).max().item() < 1e-2 and not out[n:].any()


def recurrence(x, dec, lens, starts, slots, state, H, D, V, rounded):
    """(outputs, {slot: state}) of the rule token by token; rounded: the activated operands as bfloat16 holds them."""
    qk, wants, ends, at = H * D, [], {}, 0
    a = plain.silu(x.double())
    if rounded:
        a = a.to(torch.bfloat16).double()
    d = dec.double().view(H, 1, 1)
    for n, s, slot in zip(lens, starts, slots):
        S = state[slot].double().transpose(1, 2).clone() if s else torch.zeros(H, D, V, dtype=F)
        for t in range(at, at + n):
            S = d * S + a[t, qk:2 * qk].view(H, D, 1) * a[t, 2 * qk:2 * qk + H * V].view(H, 1, V)
            wants.append((S * a[t, :qk].view(H, D, 1)).sum(1).reshape(-1))
        ends[slot] = S
        at += n
    return torch.stack(wants), ends


@pytest.mark.parametrize("sizes", [(2, 16, 24), (1, 40, 8), (3, 64, 64), (2, 96, 40), (1, 128, 136), (1, 256, 16)])
@pytest.mark.parametrize("lens", [[1, 1, 1], [3, 40, 1], [63, 64, 65], [128, 129, 16], [300, 1, 260]])
def test_lightning_blocks_kernel(sizes, lens):
    """Unequal portions around the edges of blocks and chunks in one launch, one of them from a request's first token
    (whatever its slot held), with and without chunks side by side; the states afterwards, a slot of no request left alone."""
    from dinfer_amd.kernels import ops
    H, D, V = sizes
    g = torch.Generator().manual_seed(D + sum(lens))
    starts, slots = [4, 0, 7], [1, 3, 0]
    T, qk = sum(lens), H * D
    x = torch.randn(T, 2 * qk + H * V, generator=g).bfloat16()
    dec = torch.tensor([1.0, 0.2, 0.995][:H])
    state = torch.randn(4, H, V, D, generator=g)
    wants, ends = recurrence(x, dec, lens, starts, slots, state, H, D, V, True)
    y = x.cuda()
    assert ops.lightning_supports(D, V, y.shape[1])
    for cut_ in ([False, True] if max(lens) > 128 else [False]):
        st, out = state.cuda(), torch.full((T, H * V), 9.0, device="cuda")
        notes = torch.full((ops.lightning_places(T, 3), H * V * D), float("nan"), device="cuda")
        kw = unequal(lens, starts, slots)
        ops.lightning(y[:, :qk], y[:, qk:2 * qk], y[:, 2 * qk:], dec.cuda(), st, out, notes=notes, cut=cut_, heads=H, dim=D, vdim=V, **kw)
        # (the weighted scores are rounded once on their way into the product with the values)
        assert (out.double().cpu() - wants).abs().max().item() < 4e-3 * wants.abs().max().item(), f"cut {cut_}"
        assert ((out.double().cpu() - wants).pow(2).mean() / wants.pow(2).mean()).sqrt().item() < 2e-3
        for slot, S in ends.items():      # the state keeps 16 bits of what a product takes in
            err = (st[slot].double().cpu().transpose(1, 2) - S).abs().max().item()
            assert err < 1e-4 * max(1.0, S.abs().max().item()), f"cut {cut_}: state off by {err}"
        assert torch.equal(st[2].cpu(), state[2])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", [(2, 16, 24), (3, 20, 13), (1, 40, 8), (5, 64, 64), (2, 100, 33), (1, 128, 40), (1, 256, 16), (2, 7, 5)])
@pytest.mark.parametrize("lens", [[1, 1, 1], [3, 8, 1], [150, 2, 131]])
def test_lightning_token_by_token_kernels(sizes, lens, dtype):
    """The kernel for portions of a few rows, and the one that serves long ones in 32 bits (whole and in chunks)."""
    from dinfer_amd.kernels import ops
    H, D, V = sizes
    g = torch.Generator().manual_seed(D + sum(lens))
    starts, slots = [4, 0, 7], [1, 3, 0]
    T, qk = sum(lens), H * D
    x = torch.randn(T, 2 * qk + H * V + 3, generator=g).to(getattr(torch, dtype))
    dec = torch.tensor([0.9, 0.2, 0.995, 1.0, 0.6][:H])
    state = torch.randn(4, H, V, D, generator=g)
    wants, ends = recurrence(x, dec, lens, starts, slots, state, H, D, V, False)
    y = x.cuda()
    q, k, v = y[:, :qk], y[:, qk:2 * qk], y[:, 2 * qk:2 * qk + H * V]
    kw = unequal(lens, starts, slots)
    few = {n: a for n, a in kw.items() if n != "max_rows"}
    notes = torch.full((ops.gla_places(T, 3), H * V * D), float("nan"), device="cuda")
    products = torch.full((ops.gla_places(T, 3), qk), float("nan"), device="cuda")
    geo = dict(heads=H, dim=D, vdim=V)
    runs = [lambda st, out, c=c: ops.gla_recurrence(q, k, v, None, st, out, q_scale=1.0, notes=notes, products=products, cut=c,
                                                    fixed=dec.cuda(), act=True, **kw, **geo) for c in ([False, True] if max(lens) > 128 else [False])]
    if D % 4 == 0:
        runs.append(lambda st, out: ops.lightning_few(q, k, v, dec.cuda(), st, out, **few, **geo))
    for i, run in enumerate(runs):
        st, out = state.cuda(), torch.full((T, H * V), 9.0, device="cuda")
        run(st, out)
        assert (out.double().cpu() - wants).abs().max().item() < 2e-5 * max(1.0, wants.abs().max().item()), i
        for slot, S in ends.items():
            assert (st[slot].double().cpu().transpose(1, 2) - S).abs().max().item() < 2e-5 * max(1.0, S.abs().max().item()), i
        assert torch.equal(st[2].cpu(), state[2])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("groups,group", [(1, 40), (3, 24), (1, 256), (1, 320), (2, 1024), (1, 2048), (1, 4096), (1, 6144), (1, 300), (1, 9000)])
def test_norm_over_all_heads_with_a_sigmoid_gate(groups, group, dtype):
    from dinfer_amd.kernels import ops
    dt = getattr(torch, dtype)
    T, n = 5, groups * group
    g = torch.Generator().manual_seed(n)
    y, w = 2 * torch.randn(T, n, generator=g), 1 + 0.3 * torch.randn(n, generator=g)
    z = torch.randn(T, n + 8, generator=g).to(dt)
    want = plain.rms_norm(y.double().view(T, groups, group), 1.0, 1e-3).reshape(T, n) * w.double() * 0.6
    for gate, act in (("sigmoid", torch.sigmoid), ("silu", plain.silu)):
        out = torch.zeros(T, n + 16, dtype=dt, device="cuda")
        ops.gated_group_norm(y.cuda(), z.cuda(), 8, out, T, groups=groups, group=group, eps=1e-3, weight=w.cuda(), col_off=16, out_scale=0.6,
                             gate_first=False, gate=gate)
        full = want * act(z.double()[:, 8:])
        tol = 1e-5 if dtype == "float32" else 1e-2
        assert ((out[:, 16:].double().cpu() - full).abs() / (1 + full.abs())).max().item() < tol and not out[:, :16].any()


CHUNKED = [(4, 2, 16, 24, 4, 150, 20), (3, 3, 20, 12, 8, 200, 33), (4, 1, 64, 64, 16, 170, 64), (4, 2, 64, 32, 16, 140, 30), (8, 2, 32, 96, 8, 90, 7),
           (2, 2, 128, 128, 32, 300, 100), (2, 1, 96, 48, 64, 70, 1), (1, 1, 256, 256, 8, 60, 25), (2, 1, 48, 48, 24, 130, 41), (2, 1, 64, 64, 8, 500, 0)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("cap", [0.0, 6.0])
@pytest.mark.parametrize("case", CHUNKED)
def test_attention_in_chunks_with_capped_scores(case, cap, dtype):
    """A made-up cache in shuffled pages whose other places hold junk. Every query is some key of its request times a factor,
    so that one score stands out: its chunk's first key, the last key of the chunk before, its own, one in the middle. Whole
    prompts, the last rows, the last row alone; a chunk of 0 stands for none."""
    from dinfer_amd.kernels import ops
    H, G, D, V, page, n, chunk = case
    dt = getattr(torch, dtype)
    g = torch.Generator().manual_seed(n + D)
    k, v = torch.randn(G, n, D, generator=g).to(dt), torch.randn(G, n, V, generator=g).to(dt)
    q = torch.randn(n, H, D, generator=g) * 0.3
    start = lambda p: p // chunk * chunk if chunk else 0
    for p in range(n):
        target = max(0, [start(p), start(p) - 1, p, (start(p) + p) // 2, start(p)][p % 5])
        for h in range(H):
            key = k[h // (H // G), target].float()
            q[p, h] += 10.0 * key / key.norm()
    q = q.to(dt)
    order = list(range(-(-n // page) + 3))
    random.Random(n).shuffle(order)
    kp, table = paged(k, page, order)
    vp, _ = paged(v, page, order)
    k_cache, v_cache = ops.k_cache_pack(kp).cuda(), vp.permute(0, 1, 3, 2).contiguous().cuda()

    def attend(chunk, cap):
        out, mask = torch.zeros(n, H, V, dtype=F), plain.visible(n, chunk or None)
        for h in range(H):
            s = q[:, h].double() @ k[h // (H // G)].double().T * 0.4
            out[:, h] = 0.7 * plain.softmax(plain.soft_cap(s, cap) if cap else s, mask) @ v[h // (H // G)].double()
        return out.reshape(n, H * V)
    want = attend(chunk, cap)
    if chunk > 1:       # a chunk one key off, or another cap, is another result
        for other in (attend(chunk + 1, cap), attend(chunk - 1, cap), attend(chunk, 3.0)):
            assert ((other - want).abs().amax(-1) > 0.3).float().mean().item() > 0.1
    fast = dtype == "bfloat16" and ops.attn_flash_ext_supports(D, V, page, H, G)
    assert fast == (dtype == "bfloat16" and D in (32, 48, 64, 96, 128, 256) and page != 4)
    p = n - 1
    for first in (0, start(p), p - 20, p):
        m = n - first
        out = torch.zeros(m, H * V, dtype=dt, device="cuda")
        geo = dict(scale=0.4, window=0, heads=H, kv_heads=G, head_dim=D, page_size=page, v_dim=V, out_scale=0.7, softcap=cap, chunk=chunk)
        args = [q[first:].reshape(m, H * D).contiguous().cuda(), out, k_cache, v_cache, table.cuda(),
                torch.tensor([0, m], dtype=torch.int32, device="cuda"), torch.tensor([n], dtype=torch.int32, device="cuda"), 1, m]
        for kernel in ([ops.attn_paged_ext, ops.attn_flash_ext] if fast else [ops.attn_paged_ext]):
            out.zero_()
            kernel(*args, **geo)
            tol = 2e-5 if dtype == "float32" else 2e-2
            err = ((out.double().cpu() - want[first:]).abs() / (1 + want[first:].abs())).max().item()
            assert err < tol, f"{case} from row {first}, {kernel.__name__}: off by {err:.2e}"


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T", [3, 70, 600, 1100])
@pytest.mark.parametrize("H,D", [(4, 16), (3, 20), (16, 128), (40, 128)])
def test_queries_normed_alone(H, D, T, dtype):
    """A layer that reads another one's keys: the queries' norm over the whole projection, nothing else touched."""
    from dinfer_amd.kernels import ops
    dt = getattr(torch, dtype)
    g = torch.Generator().manual_seed(T + D)
    x = torch.randn(T, 8 + H * D + 8, generator=g).to(dt)
    w = 1 + 0.3 * torch.randn(H * D, generator=g)
    y = x.cuda()
    ops.qkv_post(y, T, heads=H, kv_heads=0, head_dim=D, q_off=8, k_off=8, v_off=8, q_gain=w.cuda(), k_gain=None, eps=1e-3, gain_offset=0.0,
                 positions=torch.zeros(T, dtype=torch.int32, device="cuda"), cos_sin=None, rotary_dim=0, rope_style=0, k_cache=None,
                 v_cache=None, slot_mapping=None, page_size=16, whole=True)
    want = plain.rms_norm(x[:, 8:8 + H * D].double(), w.double(), 1e-3)
    tol = 1e-5 if dtype == "float32" else 1e-2
    assert ((y[:, 8:8 + H * D].double().cpu() - want).abs() / (1 + want.abs())).max().item() < tol
    assert torch.equal(y[:, :8].cpu(), x[:, :8]) and torch.equal(y[:, 8 + H * D:].cpu(), x[:, 8 + H * D:])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", [(5, 16, 32, 40), (3, 12, 10, 37), (16, 64, 128, 200), (4, 64, 24, 3), (2, 40, 70, 140)])
def test_products_per_head_gated_entry_by_entry(sizes, dtype):
    from dinfer_amd.kernels import ops
    H, K, N, T = sizes
    dt = getattr(torch, dtype)
    g = torch.Generator().manual_seed(H)
    a, w = torch.randn(T, H * K, generator=g).to(dt), (torch.randn(H, N, K, generator=g) / K ** 0.5).to(dt)
    gate = torch.randn(T, H * N + 5, generator=g).to(dt)
    out = torch.zeros(T, H * N, dtype=dt, device="cuda")
    ops.heads_nt(a.cuda(), 0, K, w.cuda(), out, 0, N, T, gate=gate.cuda(), gate_off=5, gate_entries=True)
    want = torch.stack([a.double()[:, h * K:(h + 1) * K] @ w[h].double().T for h in range(H)], dim=1).reshape(T, H * N)
    want = want * torch.sigmoid(gate.double()[:, 5:])
    assert (out.double().cpu() - want).abs().max().item() < (1e-5 if dtype == "float32" else 0.02) * want.abs().max().item()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T", [5, 300])
def test_experts_with_clamps(T, dtype):
    """The gate cut from above, the value on both sides, at limits that many entries meet; sizes on the vector ALUs and both
    forms on the matrix cores."""
    from dinfer_amd.kernels import ops
    dt = getattr(torch, dtype)
    for E, top, W, I, limit in ((6, 2, 32, 24, 0.5), (5, 1, 41, 17, 1.0), (70, 4, 64, 16, 0.3), (2, 2, 128, 72, 7.0)):
        g = torch.Generator().manual_seed(E + T)
        x = torch.randn(T, W, generator=g).to(dt)
        gate_up = (1.5 * torch.randn(E, 2 * I, W, generator=g) / W ** 0.5).to(dt)
        n = T * top
        idx = torch.stack([torch.randperm(E, generator=g)[:top] for _ in range(T)]).to(torch.int32)
        i32 = dict(dtype=torch.int32, device="cuda")
        perm, offsets, tiles = torch.zeros(n, **i32), torch.zeros(E + 1, **i32), torch.zeros((ops.moe_max_tiles(n, E, 16), 2), **i32)
        rows = ops.moe_tile_rows(dt, n, E, W, I)
        ops.moe_scatter(idx.reshape(-1).cuda(), n, E, offsets, perm, tiles, rows)
        out = torch.zeros(n, I, dtype=dt, device="cuda")
        ops.experts_nt(x.cuda(), gate_up.cuda(), out, n, tiles, offsets, perm, gated=True, a_div=top, c_to_perm=True, tile_rows=rows,
                       clamp=(limit, 1.702))
        y = torch.stack([gate_up[e].double() @ x[t].double() for t in range(T) for e in idx[t].tolist()])
        gt, u = y[:, :I].clamp(max=limit), y[:, I:].clamp(-limit, limit)
        want = gt * torch.sigmoid(1.702 * gt) * (u + 1)
        err = ((out.double().cpu() - want).abs() / (1 + want.abs())).max().item()
        assert err < (1e-5 if dtype == "float32" else 1e-2), f"{E} experts, {top} chosen: {err}"


# ---- whole models ---------------------------------------------------------------------------------------------
def test_which_kernels_serve_which_model(models):
    """bfloat16 with sizes the matrix-core kernels take: those kernels; 32-bit and other sizes: the plain ones."""
    for name, dtype, mfma in (("D3", "bfloat16", True), ("D3", "float32", False), ("D2", "bfloat16", False)):
        r = make_runner(models, name, dtype)
        att = [b.mixer for b in r.model.blocks if hasattr(b.mixer, "mfma_ext")]
        assert att and all(m.mfma_ext == mfma for m in att)
        assert all(b.mixer.blocks == mfma for b in r.model.blocks if hasattr(b.mixer, "decay_vec"))
        assert not r.cache.prefix_caching       # state kept between steps cannot be found again in pages
    r = make_runner(models, "D1", "float32")
    assert [r.model.run[i].cache for i in (1, 3, 5)] == [1, 1, 1]
    assert r.model.head.weight.data_ptr() == r.model.embed.data_ptr()
    # one pool of pages for layer 1 and its readers, as long as the longest look back; one for layer 6; one for the latents
    assert sorted((s.window or 0) for s in r.group_specs) == [0, 27, 33]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
def test_whole_prompts(models, name, dtype):
    _, cfg, w, _ = models[name]
    r = make_runner(models, name, dtype)
    for n, seed in ((1, 1), (2, 2), (19, 3), (300, 4)):
        ids = tokens_for(cfg, n, seed)
        run_and_compare(r, [([("x", ids, list(range(n)))], ["x"])], cfg, w, {"x": ids}, dtype, f"{name} whole prompt of {n}")


@pytest.mark.parametrize("name", NAMES)
def test_residual_stream_after_every_layer(models, name):
    from dinfer_amd.engine.batch import Entry
    _, cfg, w, _ = models[name]
    r = make_runner(models, name, "float32")
    ids = tokens_for(cfg, 37, 9)
    want = []
    plain.forward(ids, w, cfg, want)
    seen = []
    for block in r.model.blocks:
        def spy(hidden, pending, batch, cache, _inner=block.forward, **kw):
            out = _inner(hidden, pending, batch, cache, **kw)
            x = hidden[:batch.num_tokens].double().cpu()      # the last branch is normed and added by the next block's kernel
            y = out.branch[:batch.num_tokens].double().cpu()
            seen.append(x + plain.layer_norm(y, out.norm.weight.double().cpu(), out.norm.eps))
            return out
        block.forward = spy
    assert r.reserve("x", 0, len(ids))
    r.step([Entry("x", ids, 0, [0])])
    assert len(seen) == len(want) == len(cfg["layers"])
    for i, (g, x) in enumerate(zip(seen, want)):
        assert (g - x).abs().max().item() < 2e-4 * max(1.0, x.abs().max().item()), f"{name}: the stream after layer {i} differs"


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
def test_prompt_then_long_decoding(models, name, dtype):
    """Decoding far beyond every chunk of the model, across many pages, from eager steps."""
    _, cfg, w, page = models[name]
    r = make_runner(models, name, dtype)
    ids = tokens_for(cfg, 3 * page + 120, 5)
    first = 3 * page - 1                      # the first decoded token opens a new page
    steps = [([("x", ids[:first], [first - 1])], [])]
    steps += [([("x", [ids[p]], [0])], []) for p in range(first, len(ids))]
    run_and_compare(r, steps, cfg, w, {"x": ids}, dtype, f"{name} decode after prompt")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
def test_token_by_token_from_the_first(models, name, dtype):
    _, cfg, w, _ = models[name]
    r = make_runner(models, name, dtype)
    ids = tokens_for(cfg, 60, 6)
    run_and_compare(r, [([("x", [t], [0])], []) for t in ids], cfg, w, {"x": ids}, dtype, f"{name} one token a step")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
@pytest.mark.parametrize("sizes", [[2], [7, 16, 2, 5, 3, 33, 2, 8, 1], [150, 3, 200]])
def test_portions(models, name, dtype, sizes):
    _, cfg, w, _ = models[name]
    r = make_runner(models, name, dtype)
    ids = tokens_for(cfg, {2: 48, 7: 131, 150: 420}[sizes[0]], 7)
    steps = [([("x", part, list(range(len(part))))], []) for part in cut(ids, sizes)]
    run_and_compare(r, steps, cfg, w, {"x": ids}, dtype, f"{name} portions of {sizes}")


def test_cuts_leave_the_same_logits_in_32bit(models):
    """32-bit: whole (where the recurrence runs in chunks), in portions and token by token, a position's logits are equal
    up to the last bits."""
    _, cfg, w, _ = models["D1"]
    ids = tokens_for(cfg, 180, 8)
    got = []
    for parts in ([ids], cut(ids, [5, 2, 11, 1]), cut(ids, [129, 40]), [[t] for t in ids]):
        r = make_runner(models, "D1", "float32")
        rows = replay(r, [([("x", p, list(range(len(p))))], []) for p in parts])
        got.append(torch.stack([rows[("x", p)] for p in range(len(ids))]))
    for other in got[1:]:
        assert (other - got[0]).abs().max().item() < 3e-5 * got[0].abs().max().item()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
def test_mixed_batches_with_reused_pages_and_slots(models, name, dtype):
    _, cfg, w, page = models[name]
    toks, steps = mixed_schedule(cfg, 3)
    # fewer pages than all requests together need, and as many state slots as live requests: both are used again
    r = make_runner(models, name, dtype, num_blocks=(90 + 70 + 57 + 33) // page + 12, max_len=96)
    rows = run_and_compare(r, steps, cfg, w, toks, dtype, f"{name} mixed")
    if dtype == "float32":      # each request alone gives the same rows
        alone = replay(make_runner(models, name, dtype), [([("b", toks["b"], list(range(33)))], ["b"])])
        for (rid, p), row in rows.items():
            if rid == "b":
                assert (row - alone[("b", p)]).abs().max().item() < 1e-4 * row.abs().max().item()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["D1", "D3"])
def test_a_long_portion_beside_single_tokens(models, name, dtype):
    """One portion of several chunks beside two decoding requests and a short portion: the recurrence runs in chunks for
    one request and whole for the others of the same launch."""
    _, cfg, w, page = models[name]
    ids = {"a": tokens_for(cfg, 420, 1), "b": tokens_for(cfg, 12, 2), "c": tokens_for(cfg, 40, 3), "d": tokens_for(cfg, 90, 4)}
    at = {"a": 20, "b": 9, "c": 3, "d": 0}
    steps = [([(k, ids[k][:n], [n - 1]) for k, n in at.items() if n], [])]
    steps.append(([("b", ids["b"][9:10], [0]), ("a", ids["a"][20:400], list(range(0, 380, 7))), ("c", ids["c"][3:4], [0]),
                   ("d", ids["d"][:60], list(range(60)))], []))
    steps.append(([("a", ids["a"][400:401], [0]), ("b", ids["b"][10:12], [0, 1]), ("c", ids["c"][4:40], list(range(36))),
                   ("d", ids["d"][60:61], [0])], []))
    steps.append(([("d", ids["d"][61:90], [28]), ("a", ids["a"][401:402], [0])], []))
    run_and_compare(make_runner(models, name, dtype, num_blocks=200), steps, cfg, w, ids, dtype, "a long portion among others")


# ---- edges that random weights would hide -------------------------------------------------------------------------
def with_masks(cfg, change=0, **also):
    out = copy.deepcopy(cfg)
    for l in out["layers"]:
        l["mixer"]["mask"]["size"] += change
        l["mixer"].update(also)
    return out


@pytest.mark.parametrize("dtype", DTYPES)
def test_keys_just_inside_and_outside_the_chunks(models, dtype):
    """Scores so sharp that single keys of a chunk often carry most of a row's weight. The engine agrees with the chunks as
    configured, in a prompt and in decoding, and the same model with chunks one key longer or shorter, or without its caps,
    gives rows that differ by far more than the tolerance."""
    _, cfg, w, page = models["sharp"]
    ids = tokens_for(cfg, 90, 2)
    want = plain.forward(ids, w, cfg)
    spread = want.std(dim=-1, keepdim=True)
    off = lambda other: ((other - want).abs() / spread).amax(dim=-1)[8:]
    for other in (with_masks(cfg, -1), with_masks(cfg, 1), with_masks(cfg, softcap=1000.0)):
        assert (off(plain.forward(ids, w, other)) > 0.6).float().mean().item() > 0.3, "a chunk one key off, or a cap left out, does not show"
    r = make_runner(models, "sharp", dtype)
    whole = replay(r, [([("x", ids, list(range(len(ids))))], ["x"])])
    compare_rows(whole, cfg, w, {"x": ids}, dtype, "sharp whole", sharp=True)
    steps = [([("y", ids[:11], list(range(11)))], [])] + [([("y", [t], [0])], []) for t in ids[11:]]
    compare_rows(replay(r, steps), cfg, w, {"y": ids}, dtype, "sharp decoded", sharp=True)
    compare_rows(replay(r, [([("z", p, list(range(len(p))))], []) for p in cut(ids, [3, 2, 7])]), cfg, w, {"z": ids}, dtype,
                 "sharp in portions across the chunks' edges", sharp=True)


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_key_far_back_among_hundreds(models, dtype):
    """The latent attention sees everything: many rows far into a long request take their output from single keys hundreds of
    tokens back; without the keys more than 64 back they would be others."""
    _, cfg, w, page = models["far"]
    ids = tokens_for(cfg, 420, 4)
    want = plain.forward(ids, w, cfg)

    def near_only(T, chunk=None):
        i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
        return (j <= i) & (i - j < 64)
    plain.visible, keep = near_only, plain.visible
    try:
        cut_off = plain.forward(ids, w, cfg)
    finally:
        plain.visible = keep
    off = ((cut_off - want).abs() / want.std(dim=-1, keepdim=True)).amax(dim=-1)
    assert (off[100:] > 0.6).float().mean().item() > 0.35, "the made-up weights do not show far keys"
    r = make_runner(models, "far", dtype)
    steps = [([("x", ids[:300], [0, 1, 70, 200, 299])], [])] + [([("x", [t], [0])], []) for t in ids[300:]]
    compare_rows(replay(r, steps), cfg, w, {"x": ids}, dtype, "far keys", sharp=True)


def test_pages_behind_the_chunks_are_given_back(models):
    _, cfg, w, page = models["sharp"]      # one cache for chunks of 6 and 10, pages of 4
    r = make_runner(models, "sharp", "float32", num_blocks=110, max_len=400)
    ids = tokens_for(cfg, 300, 4)
    rows = replay(r, [([("x", p, [len(p) - 1])], []) for p in cut(ids, [9, 1, 1, 30, 2])])
    compare_rows(rows, cfg, w, {"x": ids}, "float32", "a long request")
    assert [s.window for s in r.group_specs] == [10]
    held = [i for i, pg in enumerate(r.cache.block_table("x", 0)) if pg >= 0]
    assert held == list(range((len(ids) - 10 + 1) // page, (len(ids) - 1) // page + 1))


# ---- graphs and the engine's own entry point ----------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["D1", "D3"])
def test_decode_steps_from_graphs(models, name, dtype):
    """Steps of single rows replay captured graphs (batch sizes 1 to 3, requests of unequal length, padded rows that use
    the spare state slot)."""
    _, cfg, w, _ = models[name]
    r = make_runner(models, name, dtype, graph=True)
    assert r._graphs_allowed and r._portion_graphs_allowed
    ids = {k: tokens_for(cfg, n, s) for k, n, s in (("a", 60, 1), ("b", 45, 2), ("c", 70, 3))}
    steps = [([("a", ids["a"][:30], [29]), ("b", ids["b"][:5], [4])], []), ([("c", ids["c"][:41], [40])], [])]
    at = {"a": 30, "b": 5, "c": 41}
    while any(at[k] < len(ids[k]) for k in ids):
        es, ends = [], []
        for k in ids:
            if at[k] < len(ids[k]):
                es.append((k, [ids[k][at[k]]], [0]))
                at[k] += 1
                if at[k] == len(ids[k]):
                    ends.append(k)
        steps.append((es, ends))
    rows = replay(r, steps)
    assert r._graphs, "no decode graph was captured"
    # the same steps run eagerly agree with the plain model, and the replayed graphs with them
    eager = run_and_compare(make_runner(models, name, dtype), steps, cfg, w, ids, dtype, f"{name} eager decode")
    tol = 1e-5 if dtype == "float32" else 2e-2
    for key, row in rows.items():
        assert (row - eager[key]).abs().max().item() < tol * max(1.0, eager[key].abs().max().item()), f"{name} graph decode {key}"


@pytest.mark.parametrize("dtype", DTYPES)
def test_steps_with_portions_from_graphs(models, dtype):
    """Steps with the same counts come up again and again (a portion of several chunks beside a decoding request and a
    shorter portion) and are replayed from a graph, padded; every replay against the same step run eagerly."""
    _, cfg, w, _ = models["D3"]
    steps, toks = [], {}
    for i in range(6):
        for k, n, s in (("p", 160, 1), ("q", 20, 2), ("d", 12, 3)):
            toks[f"{k}{i}"] = tokens_for(cfg, n, 10 * s + i)
        steps.append(([(f"d{i}", toks[f"d{i}"][:11], [10])], []))
        steps.append(([(f"p{i}", toks[f"p{i}"], [0, 80, 159]), (f"d{i}", toks[f"d{i}"][11:], [0]), (f"q{i}", toks[f"q{i}"], [19])],
                      [f"p{i}", f"d{i}", f"q{i}"]))
    r = make_runner(models, "D3", dtype, graph=True)
    rows = replay(r, steps)
    assert r.portion_replays > 0, "no step with portions was replayed"
    eager = run_and_compare(make_runner(models, "D3", dtype), steps, cfg, w, toks, dtype, "eager portions")
    # (a padded step may take other kernels for its products: close, not equal)
    for key, row in rows.items():
        err = (row - eager[key]).abs().max().item() / max(1.0, eager[key].abs().max().item())
        assert err < (1e-5 if dtype == "float32" else 0.1), f"{key}: {err}"


@pytest.mark.parametrize("name", ["D1", "D2"])
def test_greedy_generation_through_the_engine(models, name):
    """Prompts of unequal length through the scheduler (portions of up to 64 beside decoding requests), from graphs."""
    from dinfer_amd import Engine, SamplingParams
    d, cfg, w, page = models[name]
    eng = Engine(str(d), dtype="float32", max_model_len=256, max_num_seqs=3, block_size=page, num_blocks=120,
                 max_num_batched_tokens=64)
    prompts = [tokens_for(cfg, n, s) for n, s in ((5, 1), (150, 2), (23, 3), (1, 4))]
    outs = eng.generate(prompts, SamplingParams(max_tokens=12, temperature=0.0))
    for prompt, out in zip(prompts, outs):
        assert len(out) == 12
        ids = list(prompt)
        for tok in out:
            logits = plain.forward(ids, w, cfg)[-1]
            top2 = logits.topk(2).values
            if (top2[0] - top2[1]).item() > 1e-3 * logits.std().item():     # a clear choice
                assert tok == int(logits.argmax()), f"{name}: greedy token differs after {len(ids)} tokens"
            ids.append(tok)


def test_bfloat16_generation_is_the_same_from_graphs(models):
    from dinfer_amd import Engine, SamplingParams
    d, cfg, _, page = models["D3"]
    prompts = [tokens_for(cfg, 40, s) for s in range(1, 9)] + [tokens_for(cfg, n, 20 + n) for n in (9, 3)]
    outs = []
    for graphs in (True, False):
        eng = Engine(str(d), dtype="bfloat16", max_model_len=128, max_num_seqs=2, block_size=page, num_blocks=96,
                     max_num_batched_tokens=16, hip_graph=graphs, gemm_tuning="heuristic")
        outs.append(eng.generate(prompts, SamplingParams(max_tokens=10, temperature=0.0)))
        if graphs:
            assert eng.runner._graphs
    assert outs[0] == outs[1]


@pytest.mark.parametrize("dtype", DTYPES)
def test_trace_replay_program(models, tmp_path, dtype):
    """bin/trace_run on a made-up model: two requests in mixed steps; its files hold the rows the plain model gives."""
    import subprocess
    import sys
    from pathlib import Path
    import numpy as np
    d, cfg, w, _ = models["D1" if dtype == "float32" else "borrowed"]     # (bfloat16: a model without routers, see compare_rows)
    ids = {"a": tokens_for(cfg, 40, 1), "b": tokens_for(cfg, 9, 2)}
    lines = [dict(step=0, entries=[dict(id="a", tokens=ids["a"][:25], want=[3, 24])], end=[]),
             dict(step=1, entries=[dict(id="a", tokens=ids["a"][25:26], want=[0]), dict(id="b", tokens=ids["b"], want=[8])], end=["b"]),
             dict(step=2, entries=[dict(id="a", tokens=ids["a"][26:], want=[13])], end=["a"])]
    prog = Path(__file__).resolve().parent.parent / "bin" / "trace_run"
    res = subprocess.run([sys.executable, str(prog), "--model", str(d), "--dtype", dtype, "--out", str(tmp_path),
                          "--max-tokens", "128", "--block-size", "4"], input="\n".join(map(json.dumps, lines)) + "\n",
                         capture_output=True, text=True, timeout=600)
    assert res.returncode == 0, res.stderr[-2000:]
    assert [l for l in res.stdout.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    full = {k: plain.forward(v, w, cfg) for k, v in ids.items()}
    for step, wanted in ((0, [("a", 3), ("a", 24)]), (1, [("a", 25), ("b", 8)]), (2, [("a", 39)])):
        got = torch.from_numpy(np.fromfile(tmp_path / f"{step}.f32", dtype="<f4").reshape(len(wanted), cfg["vocab"]))
        check_logits(got, torch.stack([full[k][p] for k, p in wanted]), dtype, f"trace step {step}")


def test_command_line_writes_random_weights_and_generates(models, tmp_path):
    """bin/dinfer random-weights from a configuration, then bin/dinfer generate on that folder and on a folder of the plain
    model's weights, where the greedy tokens are the plain model's wherever its choice is clear."""
    import subprocess
    import sys
    from pathlib import Path
    d, cfg, w, page = models["D1"]
    root = Path(__file__).resolve().parent.parent
    exe = [sys.executable, str(root / "bin" / "dinfer")]
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    p = subprocess.run(exe + ["random-weights", "--config", str(tmp_path / "config.json"), "--out", str(tmp_path / "m"), "--seed", "3"],
                       capture_output=True, text=True, timeout=300)
    assert p.returncode == 0, p.stderr[-2000:]
    common = ["--dtype", "float32", "--max-model-len", "128", "--max-num-seqs", "2", "--num-blocks", "64", "--block-size", str(page),
              "--max-num-batched-tokens", "64", "--max-tokens", "8", "--temperature", "0", "--prompt-ids", "5,9,2", "--prompt-ids", "7"]
    p = subprocess.run(exe + ["generate", "--model", str(tmp_path / "m")] + common, capture_output=True, text=True, timeout=300)
    assert p.returncode == 0, p.stderr[-2000:]
    recs = [json.loads(l) for l in p.stdout.splitlines() if l.startswith("{")]
    assert [r["prompt_ids"] for r in recs] == [[5, 9, 2], [7]] and all(len(r["output_ids"]) == 8 for r in recs)
    p = subprocess.run(exe + ["generate", "--model", str(d)] + common, capture_output=True, text=True, timeout=300)
    assert p.returncode == 0, p.stderr[-2000:]
    for r in (json.loads(l) for l in p.stdout.splitlines() if l.startswith("{")):
        ids = list(r["prompt_ids"])
        for tok in r["output_ids"]:
            logits = plain.forward(ids, w, cfg)[-1]
            top2 = logits.topk(2).values
            if (top2[0] - top2[1]).item() > 1e-3 * logits.std().item():
                assert tok == int(logits.argmax())
            ids.append(tok)
