"""Lotelix through the engine against the plain float64 implementation (plain_lotelix.py): every mechanism alone at the
level of its kernels or as a one-layer model, then whole models of made-up sizes in every way of cutting and batching,
32-bit and bfloat16, and greedy generation through the engine's own entry point."""
import copy
import json
import random

import pytest
import torch

import plain_lotelix as plain
from test_gpu_verorax import check_logits, cut, has_router, mixed_schedule, paged, replay, tokens_for

pytestmark = pytest.mark.gpu
F = torch.float64
DTYPES = ["float32", "bfloat16"]


def gru(width):
    return dict(type="mingru", mixer=dict(width=width))


def attention(heads, kv_heads, dim, vdim, size, dims, v_mix=True, base=10000.0, scale=None, scaling=None):
    rot = dict(base=base, dims=dims)
    if scaling:
        rot["scaling"] = dict(zip(("factor", "low", "high", "original"), scaling))
    return dict(type="attention", mixer=dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale or dim ** -0.5,
                                             mask=dict(size=size), v_mix=v_mix, rot=rot))


def parallel(lh, lg, ld, lv, dims, rh, rd, rv, tau, base=10000.0, scale=None):
    return dict(type="parallel", mixer=dict(
        left=dict(heads=lh, kv_heads=lg, dim=ld, vdim=lv, scale=scale or ld ** -0.5, rot=dict(base=base, dims=dims)),
        right=dict(heads=rh, dim=rd, vdim=rv, tau=tau)))


def routed(layer, experts, top, ff):
    return dict(layer, mlp=dict(kind="moe", expert=dict(ff=ff), router=dict(experts=experts, top=top)))


def bare(layer):
    return dict(layer, mlp=None)


def model(vocab, width, groups, layers, eps=1e-6, scale=1.0):
    return dict(architecture="Lotelix", vocab=vocab, width=width, embedding=dict(scale=scale), norm=dict(eps=eps, groups=groups),
                layers=layers)


BANDS = (4.0, 1.0, 3.0, 100)
P1 = parallel(4, 2, 16, 24, 8, 2, 16, 24, 4.0)                       # values wider than keys, half of a head rotated
A1 = attention(4, 2, 16, 8, 10, 16, scaling=BANDS)
A2 = attention(6, 1, 24, 16, 5, 10, base=300.0)                      # other heads, values of the same size in all
P2 = parallel(3, 1, 20, 10, 20, 3, 24, 40, 1.0)                      # sizes that are no multiples of 8
A3 = attention(3, 3, 20, 12, 33, 12)
P3 = parallel(4, 2, 64, 32, 32, 2, 64, 64, 16.0)                     # bfloat16: both attentions on the matrix cores
A4 = attention(4, 1, 32, 64, 18, 32, scaling=(8.0, 0.5, 2.0, 60))
P4 = parallel(4, 4, 48, 96, 48, 1, 40, 16, 8.0)                      # one recurrent head; the whole head rotated
CONFIGS = {
    # every mixer, two choices a token, a layer without a feed-forward, values mixed twice and once not; pages of 4
    "T1": (model(96, 64, 4, [routed(P1, 6, 2, 24), routed(gru(40), 6, 2, 24), routed(A1, 6, 2, 24), bare(gru(24)),
                             bare(attention(2, 2, 8, 16, 7, 4, v_mix=False)), routed(A2, 3, 1, 40)], scale=4.0), 4, 11),
    # odd sizes; one choice; another eps; three groups; the first layer is recurrent
    "T2": (model(131, 72, 3, [routed(gru(37), 5, 1, 40), routed(P2, 5, 1, 40), bare(A3)], eps=1e-3, scale=0.5), 8, 12),
    # sizes the matrix-core kernels take; a parallel layer behind one without a feed-forward; all experts chosen
    "T3": (model(120, 128, 2, [bare(A4), routed(P3, 8, 3, 64), bare(P4), bare(P3), routed(gru(96), 2, 2, 48), routed(A4, 8, 1, 64)]), 16, 13),
    # one group, one expert
    "T4": (model(77, 40, 1, [routed(A2, 1, 1, 16), routed(parallel(2, 2, 8, 4, 2, 4, 8, 8, 2.0), 1, 1, 16), routed(A2, 1, 1, 16)]), 4, 14),
}
ONE = {
    "gru": (model(64, 32, 2, [bare(gru(48))]), 4, 21),
    "window": (model(64, 32, 2, [bare(attention(4, 2, 16, 8, 6, 16, scaling=BANDS))]), 4, 22),
    "mix": (model(64, 32, 2, [bare(attention(4, 2, 16, 8, 6, 8)), bare(attention(2, 1, 8, 16, 9, 8))]), 4, 23),
    # bfloat16: heads of 64 of one size, rotated whole: the 16-byte kernels before the cache
    "whole": (model(64, 48, 2, [bare(attention(2, 1, 64, 64, 6, 64)), bare(attention(3, 1, 64, 64, 9, 64))]), 8, 24),
    "parallel": (model(64, 32, 2, [bare(parallel(4, 2, 16, 8, 8, 3, 24, 16, 4.0))]), 4, 25),
    "routed": (model(64, 32, 2, [routed(gru(8), 7, 3, 24)]), 4, 26),
}
# scores so sharp that one key too many or too few, or a sink left out, shows: windows of 6 and 4, pages of 4
SHARP = {
    "sharp": (model(80, 48, 2, [bare(attention(2, 1, 16, 16, 6, 8, scale=1.0)), bare(attention(2, 1, 16, 16, 4, 16, scale=1.0))]), 4, 31),
    "far": (model(80, 48, 2, [bare(parallel(2, 1, 16, 16, 8, 1, 8, 8, 1.0, scale=1.5))]), 4, 32),
}


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    from dinfer_amd.weights.safetensors_io import write_safetensors
    out = {}
    for name, (cfg, page, seed) in {**CONFIGS, **ONE, **SHARP}.items():
        d = tmp_path_factory.mktemp(f"lotelix_{name}")
        w = plain.random_weights(cfg, seed, low=5 + seed % 4)
        if name == "sharp":    # sinks that take a share beside scores of a spread of several units
            w = {k: (v + 3.0 if k.endswith(".sink") else v) for k, v in w.items()}
        if name == "far":      # few keys count, each with a weight near one: a key left out shows
            w["l0.mix.left.pb"] = torch.full((2,), -9.0).bfloat16()
            w["l0.mix.right.out"] = w["l0.mix.right.out"] * 0.1
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
    for what, parts in (("whole", [ids]), ("portions", cut(ids, [2, 3])), ("single tokens", [[t] for t in ids])):
        steps = [([("x", p, list(range(len(p))))], []) for p in parts]
        steps[-1] = (steps[-1][0], ["x"])
        run_and_compare(r, steps, cfg, w, {"x": ids}, dtype, f"{name} alone, {what}")


# ---- kernels alone --------------------------------------------------------------------------------------------
@pytest.mark.parametrize("xdt,sdt", [("float32", "float32"), ("bfloat16", "float32"), ("bfloat16", "bfloat16"), ("float32", None), ("bfloat16", None)])
@pytest.mark.parametrize("width,groups", [(64, 4), (72, 3), (2048, 4), (4096, 1), (6144, 16), (130, 2), (35, 7)])
def test_group_norm_kernels(width, groups, xdt, sdt):
    from dinfer_amd.kernels import ops
    g = torch.Generator().manual_seed(width)
    x = torch.randn(9, width, generator=g).to(getattr(torch, xdt))
    w = 1 + 0.3 * torch.randn(width, generator=g)
    rows = torch.tensor([3, 0, 8, 8, 5], dtype=torch.int32)
    for picked in (None, rows):
        st = None if sdt is None else torch.randn(9, width, generator=g).to(getattr(torch, sdt))
        n = 9 if picked is None else len(rows)
        if picked is not None and st is not None:
            continue
        out = torch.zeros(n, width, dtype=getattr(torch, "bfloat16" if xdt == "bfloat16" else "float32"), device="cuda")
        dst = None if st is None else st.cuda()
        ops.group_rmsnorm(x.cuda(), w.cuda(), out, 1e-3, n, groups, residual=dst, rows=None if picked is None else picked.cuda())
        v = x.double()
        if st is not None:
            v = (v + st.double()).to(st.dtype).double()
            assert (dst.double().cpu() - v).abs().max().item() < (1e-6 if sdt == "float32" else 2e-2)
        want = plain.group_norm(v, w.double(), 1e-3, groups)
        want = want if picked is None else want[rows.long()]
        tol = 2e-6 if out.dtype == torch.float32 else 1e-2
        assert ((out.double().cpu() - want).abs() / (1 + want.abs())).max().item() < tol


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width,groups,branches", [(64, 4, 2), (2048, 2, 2), (100, 5, 3), (36, 1, 1), (4096, 8, 2)])
def test_joined_norms_kernels(width, groups, branches, dtype):
    """Branches normed by themselves, biases added before the norms, summed; into a stream with the norm that reads it
    next, into a stream alone, and into a buffer of their own."""
    from dinfer_amd.kernels import ops
    dt = getattr(torch, dtype)
    g = torch.Generator().manual_seed(width)
    T, step = 7, -(-width // 8) * 8
    x = torch.randn(T, branches * step, generator=g).to(dt)
    bw, bias = 1 + 0.3 * torch.randn(branches, width, generator=g), torch.randn(branches, width, generator=g)
    w, stream = 1 + 0.3 * torch.randn(width, generator=g), torch.randn(T, width, generator=g)
    eps = [1e-3 * (m + 1) for m in range(branches)]
    for b in (bias, None):
        y = 0.5 * sum(plain.rms_unit(x[:, m * step:m * step + width].double() + (0 if b is None else b[m].double()), eps[m]) * bw[m].double()
                      for m in range(branches))
        kw = dict(eps=eps, scale=0.5, bias=None if b is None else b.cuda())
        out = torch.zeros(T, width, dtype=dt, device="cuda")
        tol = 5e-6 if dtype == "float32" else 2e-2
        ops.joined_norms(x.cuda(), bw.cuda(), T, out=out, **kw)
        assert ((out.double().cpu() - y).abs() / (1 + y.abs())).max().item() < tol
        for normed in (True, False):
            st = stream.cuda()
            out.zero_()
            ops.joined_norms(x.cuda(), bw.cuda(), T, stream=st, out=out if normed else None, weight=w.cuda(), norm_eps=1e-4,
                             groups=groups, **kw)
            s = stream.double() + y
            assert (st.double().cpu() - s).abs().max().item() < 1e-5
            want = plain.group_norm(s, w.double(), 1e-4, groups)
            if normed:
                assert ((out.double().cpu() - want).abs() / (1 + want.abs())).max().item() < tol
            else:
                assert not out.any()


def unequal(lens, starts, slots):
    cu = torch.tensor([0] + torch.tensor(lens).cumsum(0).tolist(), dtype=torch.int32, device="cuda")
    seq = torch.tensor([s + n for s, n in zip(starts, lens)], dtype=torch.int32, device="cuda")
    return dict(cu_seqlens=cu, seq_lens=seq, state_slots=torch.tensor(slots, dtype=torch.int32, device="cuda"), num_reqs=len(lens),
                tokens=sum(lens), max_rows=max(lens))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("lens", [[1, 1, 1, 1], [3, 1, 4, 2], [64, 1, 65, 9], [200, 7, 63, 128], [1, 500, 2, 8]])
@pytest.mark.parametrize("N", [40, 33, 200])
def test_min_gru_kernels(N, lens, dtype):
    """Portions of unequal length around the chunks' edges in one launch, some from a request's first token (whatever
    the slot holds), against the recurrence token by token; the states afterwards, a slot of no request left alone."""
    from dinfer_amd.kernels import ops
    dt = getattr(torch, dtype)
    g = torch.Generator().manual_seed(N + sum(lens))
    starts, slots = [5, 0, 9, 0], [2, 0, 3, 1]
    T, step = sum(lens), -(-N // 8) * 8
    proj = torch.randn(T, 3 * step, generator=g).to(dt)
    zb, xb = 2 * torch.randn(N, generator=g) - 3, torch.randn(N, generator=g)
    state = torch.randn(5, N, generator=g)
    st, out = state.cuda(), torch.zeros(T, step, dtype=dt, device="cuda")
    notes = torch.full((ops.min_gru_places(T, 4), 2 * N), float("nan"), device="cuda")
    ops.min_gru(proj.cuda(), out, z_off=0, x_off=step, g_off=2 * step, z_bias=zb.cuda(), x_bias=xb.cuda(), state=st, notes=notes,
                **unequal(lens, starts, slots))
    at, p = 0, proj.double()
    for n, s, slot in zip(lens, starts, slots):
        S = state[slot].double() if s else torch.zeros(N, dtype=F)
        for t in range(at, at + n):
            a = torch.sigmoid(p[t, :N] + zb.double())
            u = p[t, step:step + N] + xb.double()
            S = (1 - a) * S + a * torch.where(u >= 0, u + 0.5, torch.sigmoid(u))
            want = S * plain.silu(p[t, 2 * step:2 * step + N])
            err = ((out[t, :N].double().cpu() - want).abs() / (1 + want.abs())).max().item()
            assert err < (5e-6 if dtype == "float32" else 1e-2), f"token {t - at} of {n}: {err}"
        assert (st[slot].double().cpu() - S).abs().max().item() < 1e-5
        at += n
    assert torch.equal(st[4].cpu(), state[4])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", [(2, 16, 24), (1, 40, 8), (3, 20, 12), (2, 64, 64), (1, 128, 40), (1, 256, 16)])
@pytest.mark.parametrize("lens", [[1, 1, 1], [3, 40, 1], [128, 129, 16], [300, 1, 260]])
def test_gated_linear_attention_kernels(sizes, lens, dtype):
    """The decays and the recurrence on made-up projections: unequal portions in one launch, run whole and in chunks, one
    of them from a request's first token, states that hold junk; against the rule written out token by token."""
    from dinfer_amd.kernels import ops
    H, D, V = sizes
    dt = getattr(torch, dtype)
    g = torch.Generator().manual_seed(D + sum(lens))
    low, tau = 6, 2.0
    starts, slots = [4, 0, 7], [1, 3, 0]
    T, qk, v = sum(lens), H * D, H * V
    proj = torch.randn(T, -(-(2 * qk + v + low) // 8) * 8, generator=g).to(dt)
    w2, b = torch.randn(qk, low, generator=g), 2 * torch.randn(qk, generator=g) + 1
    state = torch.randn(4, H, V, D, generator=g)
    p = proj.double()
    alpha = torch.sigmoid(p[:, 2 * qk + v:2 * qk + v + low] @ w2.double().T + b.double()) ** (1 / tau)
    dec = torch.zeros(T, qk, device="cuda")
    ops.channel_decay(proj.cuda(), T, low_off=2 * qk + v, w2t=w2.t().contiguous().cuda(), bias=b.cuda(), tau=tau, out=dec)
    assert (dec.double().cpu() - alpha).abs().max().item() < 2e-6
    wants, ends, at = [], {}, 0
    for n, s, slot in zip(lens, starts, slots):
        S = state[slot].double().transpose(1, 2).clone() if s else torch.zeros(H, D, V, dtype=F)
        for t in range(at, at + n):
            S = alpha[t].view(H, D, 1) * S + p[t, qk:2 * qk].view(H, D, 1) * p[t, 2 * qk:2 * qk + v].view(H, 1, V)
            wants.append((S * (p[t, :qk].view(H, D, 1) * 0.3)).sum(1).reshape(-1))
        ends[slot] = S
        at += n
    wants = torch.stack(wants)
    kw = unequal(lens, starts, slots)
    for cut_ in ([False, True] if max(lens) > 128 else [False]):
        st, out = state.cuda(), torch.zeros(T, v, device="cuda")
        places = ops.gla_places(T, 3)
        notes = torch.full((places, H * V * D), float("nan"), device="cuda")
        products = torch.full((places, qk), float("nan"), device="cuda")
        x = proj.cuda()
        ops.gla_recurrence(x[:, :qk], x[:, qk:2 * qk], x[:, 2 * qk:2 * qk + v], dec, st, out, q_scale=0.3, notes=notes,
                           products=products, cut=cut_, heads=H, dim=D, vdim=V, **kw)
        scale = wants.abs().max().item()
        assert (out.double().cpu() - wants).abs().max().item() < 2e-5 * max(1.0, scale), f"cut {cut_}"
        for slot, S in ends.items():
            assert (st[slot].double().cpu().transpose(1, 2) - S).abs().max().item() < 2e-5 * max(1.0, S.abs().max().item())
        assert torch.equal(st[2].cpu(), state[2])


def test_decays_near_one_keep_what_sets_them_apart():
    """Very slow decays: what is lost a token must be right, not only the decay (it adds up over a long memory)."""
    from dinfer_amd.kernels import ops
    z = torch.linspace(-30, 30, 601)
    for tau in (1.0, 16.0):
        out = torch.zeros(1, 601, device="cuda")
        ops.channel_decay(torch.zeros(1, 8, device="cuda"), 1, low_off=0, w2t=torch.zeros(1, 601, device="cuda"), bias=z.cuda(), tau=tau, out=out)
        want = torch.sigmoid(z.double()) ** (1 / tau)
        err = (out[0].double().cpu() - want).abs() / want
        assert err.max().item() < 3e-6 and err[z > 0].max().item() < 1.3e-7


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("case", [(4, 2, 16, 24, 4, 150), (3, 3, 20, 12, 8, 200), (4, 1, 64, 64, 16, 170), (4, 2, 64, 32, 16, 140),
                                  (8, 2, 32, 96, 8, 90), (2, 2, 128, 128, 32, 300), (2, 1, 96, 48, 64, 70), (1, 1, 256, 256, 8, 60)])
def test_sigmoid_attention_kernels(case, dtype):
    """Sigmoid weights on a made-up cache in shuffled pages, whose other places hold junk. Each query is a key of its
    request times a factor so that one score stands out: the first key, far back, at a page's last and first place, the
    query's own; the bias keeps the others small. Whole prompts and the last row alone."""
    from dinfer_amd.kernels import ops
    H, G, D, V, page, n = case
    dt = getattr(torch, dtype)
    g = torch.Generator().manual_seed(n + D)
    k, v = torch.randn(G, n, D, generator=g).to(dt), torch.randn(G, n, V, generator=g).to(dt)
    bias = torch.randn(H, generator=g) - 7.0
    p = n - 1
    q = torch.randn(n, H, D, generator=g) * 0.3
    targets = {p - i: t for i, t in enumerate([0, 1, p, p - 1, (p // page) * page, max((p // page) * page - 1, 0), n // 2, 3])}
    for row, target in targets.items():
        for h in range(H):
            key = k[h // (H // G), min(target, row)].float()
            q[row, h] += 12.0 * key / key.norm()
    q = q.to(dt)
    order = list(range(-(-n // page) + 3))
    random.Random(n).shuffle(order)
    kp, table = paged(k, page, order)
    vp, _ = paged(v, page, order)
    k_cache, v_cache = ops.k_cache_pack(kp).cuda(), vp.permute(0, 1, 3, 2).contiguous().cuda()
    want = torch.zeros(n, H, V, dtype=F)
    for h in range(H):
        s = q[:, h].double() @ k[h // (H // G)].double().T * 0.8
        want[:, h] = 0.7 * plain.sigmoid_weights(s, plain.visible(n), bias[h].double()) @ v[h // (H // G)].double()
    assert want[list(targets)].abs().amax(dim=(1, 2)).min().item() > 0.5       # the key that stands out carries the row
    want = want.reshape(n, H * V)
    fast = dtype == "bfloat16" and ops.attn_flash_ext_supports(D, V, page, H, G, True)
    assert fast == (dtype == "bfloat16" and D in (32, 64, 96, 128, 256) and page != 4)
    for first in (0, p - 20, p):
        m = n - first
        out = torch.zeros(m, H * V, dtype=dt, device="cuda")
        geo = dict(scale=0.8, window=0, heads=H, kv_heads=G, head_dim=D, page_size=page, v_dim=V, out_scale=0.7,
                   sigmoid_bias=bias.cuda())
        args = [q[first:].reshape(m, H * D).contiguous().cuda(), out, k_cache, v_cache, table.cuda(),
                torch.tensor([0, m], dtype=torch.int32, device="cuda"), torch.tensor([n], dtype=torch.int32, device="cuda"), 1, m]
        for kernel in ([ops.attn_paged_ext, ops.attn_flash_ext] if fast else [ops.attn_paged_ext]):
            out.zero_()
            kernel(*args, **geo)
            tol = 2e-5 if dtype == "float32" else 2e-2
            err = ((out.double().cpu() - want[first:]).abs() / (1 + want[first:].abs())).max().item()
            assert err < tol, f"{case} from row {first}, {kernel.__name__}: off by {err:.2e}"


@pytest.mark.parametrize("case", [(4, 2, 64, 32, 16, 150, 20), (4, 1, 32, 128, 8, 200, 33), (2, 2, 128, 48, 32, 90, 7), (3, 1, 96, 64, 16, 70, 0),
                                  (2, 1, 48, 96, 8, 120, 64)])
def test_flash_kernel_with_values_of_another_size(case):
    """Softmax with sinks and a window over values narrower or wider than the keys, keys made to stand out at both sides
    of the window's edge; against the plain formula."""
    from dinfer_amd.kernels import ops
    H, G, D, V, page, n, window = case
    g = torch.Generator().manual_seed(n)
    k, v = torch.randn(G, n, D, generator=g).bfloat16(), torch.randn(G, n, V, generator=g).bfloat16()
    q, sinks = torch.randn(n, H, D, generator=g), torch.randn(H, generator=g) * 2
    for row in range(n):
        t = max(0, row - (window or row) + (row % 3) - 1)      # just outside, at and just inside the edge
        for h in range(H):
            key = k[h // (H // G), min(t, row)].float()
            q[row, h] += 8.0 * key / key.norm()
    q = q.bfloat16()
    order = list(range(-(-n // page) + 2))
    random.Random(n).shuffle(order)
    kp, table = paged(k, page, order)
    vp, _ = paged(v, page, order)
    out = torch.zeros(n, H * V, dtype=torch.bfloat16, device="cuda")
    ops.attn_flash_ext(q.reshape(n, H * D).cuda(), out, ops.k_cache_pack(kp).cuda(), vp.permute(0, 1, 3, 2).contiguous().cuda(), table.cuda(),
                       torch.tensor([0, n], dtype=torch.int32, device="cuda"), torch.tensor([n], dtype=torch.int32, device="cuda"), 1, n,
                       scale=0.5, window=window, heads=H, kv_heads=G, head_dim=D, page_size=page, v_dim=V, sinks=sinks.cuda())
    mask = plain.visible(n, window or None)
    want = torch.zeros(n, H, V, dtype=F)
    for h in range(H):
        s = q[:, h].double() @ k[h // (H // G)].double().T * 0.5
        want[:, h] = plain.softmax_with_sink(s, mask, sinks[h].double()) @ v[h // (H // G)].double()
    err = (out.double().cpu().view(n, H, V) - want).abs().max().item()
    assert err < 4e-2 * max(1.0, want.abs().max().item()), f"{case}: {err}"


ROWS = [(4, 2, 16, 24, 8, 1, 4), (3, 1, 20, 10, 20, 1, 8), (4, 2, 64, 64, 32, 1, 16), (4, 2, 64, 32, 64, 0, 16), (2, 2, 24, 12, 0, 0, 8),
        (40, 8, 128, 128, 128, 1, 16), (80, 8, 128, 64, 128, 0, 16)]      # heads, kv heads, key and value sizes, rotated, pairing, page


@pytest.mark.parametrize("case,T,dtype", [(c, T, dt) for c in ROWS[:6] for T in (3, 70) for dt in DTYPES]
                         + [(c, 1100, "bfloat16") for c in ROWS if c[0] >= 4])
def test_step_before_the_cache_with_whole_row_norms(case, T, dtype):
    """Norms over all heads at once, biases, both pairings, part of a head rotated, values mixed, keys and values in their
    pages (prompt portions that start anywhere, one row with no slot)."""
    from dinfer_amd.kernels import ops
    H, G, D, V, rot, style, page = case
    dt = getattr(torch, dtype)
    g = torch.Generator().manual_seed(T + D)
    nq, nk, nv = H * D, G * D, G * V
    off = 8
    qkv = torch.randn(T, off + nq + nk + nv + (-(nq + nk + nv)) % 8, generator=g).to(dt)
    wq, wk = 1 + 0.3 * torch.randn(nq, generator=g), 1 + 0.3 * torch.randn(nk, generator=g)
    bias = torch.randn(nq + nk + nv, generator=g)
    first = torch.randn(T, nv, generator=g).to(dt)
    pos = torch.arange(5, 5 + T, dtype=torch.int32)
    blocks = (T + 5) // page + 2
    slots = (pos.long() + page)                                # page 0 stays unused
    slots[T // 2] = -1
    table = None
    if rot:
        ang = torch.arange(T + 6, dtype=F)[:, None] * torch.tensor([50.0 ** (-2.0 * i / rot) for i in range(rot // 2)], dtype=F)
        table = torch.cat([ang.cos(), ang.sin()], -1).float()
    kc = torch.full(ops.k_cache_shape(blocks, G, page, D), 7.0, dtype=dt, device="cuda")
    vc = torch.full(ops.v_cache_shape(blocks, G, page, V), 7.0, dtype=dt, device="cuda")
    x = qkv.cuda()
    ops.qkv_post(x, T, heads=H, kv_heads=G, head_dim=D, q_off=off, k_off=off + nq, v_off=off + nq + nk, q_gain=wq.cuda(), k_gain=wk.cuda(),
                 eps=1e-3, gain_offset=0.0, positions=pos.cuda(), cos_sin=None if table is None else table.cuda(), rotary_dim=rot,
                 rope_style=style, k_cache=kc, v_cache=vc, slot_mapping=slots.cuda(), page_size=page, token_runs=T >= 8, v_dim=V,
                 bias=bias.cuda(), whole=True, v_first=first.cuda(), v_share=0.3)
    b = bias.double()
    d = qkv.double()[:, off:]
    q = plain.rms_unit(d[:, :nq] + b[:nq], 1e-3) * wq.double()
    k = plain.rms_unit(d[:, nq:nq + nk] + b[nq:nq + nk], 1e-3) * wk.double()
    v = 0.7 * (d[:, nq + nk:nq + nk + nv] + b[nq + nk:]) + 0.3 * first.double()
    q, k = q.view(T, H, D), k.view(T, G, D)
    if rot:
        turn = plain.rotate_neighbours if style else plain.rotate_halves
        pad = torch.zeros(5, 1, D, dtype=F)
        q, k = (torch.cat([pad.expand(5, t.shape[1], D), t]) for t in (q, k))
        q, k = turn(q, dict(base=50.0, dims=rot))[5:], turn(k, dict(base=50.0, dims=rot))[5:]
    tol = 2e-5 if dtype == "float32" else 2e-2
    close = lambda a, w: ((a.double().cpu() - w).abs() / (1 + w.abs())).max().item() < tol
    assert close(x[:, off:off + nq].view(T, H, D), q)
    assert torch.equal(x[:, :off].cpu(), qkv[:, :off])
    kr, vr = ops.k_cache_rows(kc).cpu(), vc.permute(0, 1, 3, 2).cpu()
    keep = slots >= 0
    s = slots[keep]
    assert close(kr[s // page, :, s % page, :D], k[keep]) and close(vr[s // page, :, s % page], v.view(T, G, V)[keep])
    gone = int(pos[T // 2]) + page
    assert (vr[gone // page, :, gone % page] == 7.0).all() and (vr[0] == 7.0).all()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("case", [(2, 1, 64, 64, 64), (4, 2, 128, 128, 128), (3, 1, 16, 8, 8), (2, 2, 256, 256, 256)])
@pytest.mark.parametrize("T", [5, 80])
def test_mixed_values_in_the_step_before_the_cache(case, T, dtype):
    from dinfer_amd.kernels import ops
    H, G, D, V, rot = case
    dt, page = getattr(torch, dtype), 16
    g = torch.Generator().manual_seed(D + T)
    n = H * D + G * D + G * V
    x, first = torch.randn(T, n, generator=g).to(dt), torch.randn(T, G * V, generator=g).to(dt)
    table = torch.randn(T, rot, generator=g)
    vc = torch.zeros(ops.v_cache_shape(T // page + 2, G, page, V), dtype=dt, device="cuda")
    kc = torch.zeros(ops.k_cache_shape(T // page + 2, G, page, D), dtype=dt, device="cuda")
    slots = torch.arange(T, dtype=torch.long) + 8
    ops.qkv_post(x.cuda(), T, heads=H, kv_heads=G, head_dim=D, q_off=0, k_off=H * D, v_off=(H + G) * D, q_gain=None, k_gain=None, eps=0.0,
                 gain_offset=0.0, positions=torch.arange(T, dtype=torch.int32, device="cuda"), cos_sin=table.cuda(), rotary_dim=rot, rope_style=0,
                 k_cache=kc, v_cache=vc, slot_mapping=slots.cuda(), page_size=page, token_runs=T >= 8, v_dim=V, v_first=first.cuda(), v_share=0.25)
    want = 0.75 * x.double()[:, (H + G) * D:] + 0.25 * first.double()
    got = vc.permute(0, 1, 3, 2).cpu()[slots // page, :, slots % page].double().reshape(T, -1)
    assert (got - want).abs().max().item() < (1e-6 if dtype == "float32" else 2e-2)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T", [5, 300])
def test_experts_weighted_at_their_input(T, dtype):
    """Sigmoid scores, the largest chosen and weighing as they are; the weight on the expert's input, the square of relu
    behind the first product, equal experts told apart by order."""
    from dinfer_amd.kernels import ops
    dt = getattr(torch, dtype)
    for E, top, W, I in ((6, 2, 32, 24), (5, 1, 40, 17), (70, 4, 64, 16)):
        g = torch.Generator().manual_seed(E + T)
        x = torch.randn(T, W, generator=g).to(dt)
        router = torch.randn(E, W, generator=g) * (2.0 / W ** 0.5)
        up, down = (torch.randn(E, I, W, generator=g) / W ** 0.5).to(dt), (torch.randn(E, W, I, generator=g) / I ** 0.5).to(dt)
        n, dev = T * top, "cuda"
        i32 = dict(dtype=torch.int32, device=dev)
        idx, perm, offsets = torch.zeros(n, **i32), torch.zeros(n, **i32), torch.zeros(E + 1, **i32)
        share, z = torch.zeros(n, device=dev), torch.zeros(T * (E + 1), device=dev)
        ops.moe_route(x.cuda(), router.cuda(), None, idx, share, None, T, top, z, all_scores=2)
        s = torch.sigmoid(x.double() @ router.double().T)
        got = idx.cpu().view(T, top).long()
        assert (share.cpu().view(T, top).double() - torch.gather(s, 1, got)).abs().max().item() < 1e-6
        assert (torch.gather(s, 1, got).min(-1).values >= torch.topk(s, top).values[:, -1] - 1e-6).all()
        rows = ops.moe_tile_rows(dt, n, E, W, I)
        tiles = torch.zeros((ops.moe_max_tiles(n, E, 16), 2), **i32)
        ops.moe_scatter(idx, n, E, offsets, perm, tiles, rows)
        act, y, out = (torch.zeros(n, I, dtype=dt, device=dev), torch.zeros(n, W, dtype=dt, device=dev), torch.zeros(T, W, dtype=dt, device=dev))
        ops.experts_nt(x.cuda(), up.cuda(), act, n, tiles, offsets, perm, gated=False, a_div=top, c_to_perm=False, tile_rows=rows,
                       act="relu2", row_scale=share)
        ops.experts_nt(act, down.cuda(), y, n, tiles, offsets, perm, gated=False, a_div=0, c_to_perm=True, tile_rows=rows)
        ops.moe_combine(y, None, top, None, None, out, T)
        want = torch.zeros(T, W, dtype=F)
        for t in range(T):
            for e in got[t].tolist():
                want[t] += torch.relu(up[e].double() @ (s[t, e] * x[t].double())) ** 2 @ down[e].double().T
        err = ((out.double().cpu() - want).abs() / (1 + want.abs())).max().item()
        assert err < (1e-5 if dtype == "float32" else 3e-2), f"{E} experts, {top} chosen: {err}"


def test_gated_experts_weighted_at_their_input():
    from dinfer_amd.kernels import ops
    g = torch.Generator().manual_seed(3)
    T, E, W, I = 21, 3, 24, 16
    for dt, tol in ((torch.float32, 1e-5), (torch.bfloat16, 3e-2)):
        x, w = torch.randn(T, W, generator=g).to(dt), (torch.randn(E, 2 * I, W, generator=g) / W ** 0.5).to(dt)
        idx = torch.randint(0, E, (T,), generator=g, dtype=torch.int32)
        share = torch.rand(T, generator=g)
        i32 = dict(dtype=torch.int32, device="cuda")
        perm, offsets, tiles = torch.zeros(T, **i32), torch.zeros(E + 1, **i32), torch.zeros((ops.moe_max_tiles(T, E, 16), 2), **i32)
        rows = ops.moe_tile_rows(dt, T, E, W, I)
        ops.moe_scatter(idx.cuda(), T, E, offsets, perm, tiles, rows)
        out = torch.zeros(T, I, dtype=dt, device="cuda")
        ops.experts_nt(x.cuda(), w.cuda(), out, T, tiles, offsets, perm, gated=True, a_div=1, c_to_perm=False, tile_rows=rows, row_scale=share.cuda())
        for place, t in enumerate(perm.cpu().tolist()):
            u = w[idx[t]].double() @ (share[t].double() * x[t].double())
            want = plain.silu(u[:I]) * u[I:]
            assert ((out[place].double().cpu() - want).abs() / (1 + want.abs())).max().item() < tol


# ---- whole models ---------------------------------------------------------------------------------------------
def test_which_kernels_serve_which_model(models):
    """bfloat16 with sizes the matrix-core kernels take: those kernels for both attentions; 32-bit and other sizes: the
    plain kernels. A layer's values are read by later layers from the buffer they were projected into."""
    for name, dtype, mfma in (("T3", "bfloat16", True), ("T3", "float32", False), ("T2", "bfloat16", False)):
        r = make_runner(models, name, dtype)
        found = []
        for b in r.model.blocks:
            found += [m for _, m, _, _ in b.mixer.members] if hasattr(b.mixer, "members") else [b.mixer]
        found = [m for m in found if hasattr(m, "mfma_ext")]
        assert found and all(m.mfma_ext == mfma for m in found)
        assert not r.cache.prefix_caching       # state kept between steps cannot be found again in pages
    r = make_runner(models, "T1", "float32")
    att = [b.mixer for b in r.model.blocks if getattr(b.mixer, "value_mix", None)]
    assert [m.value_mix for m in att] == ["keep", "mix"]
    keep, mix = att
    assert mix.kept_values.data_ptr() == keep.qkv_buf[:, keep.q_size + keep.kv_size:].data_ptr()
    assert all(b.mixer is keep or getattr(b.mixer, "qkv_buf", None) is None or b.mixer.qkv_buf.data_ptr() != keep.qkv_buf.data_ptr()
               for b in r.model.blocks)


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
    from dinfer_amd.parts.base import Carried
    _, cfg, w, _ = models[name]
    r = make_runner(models, name, "float32")
    ids = tokens_for(cfg, 37, 9)
    want = []
    plain.forward(ids, w, cfg, want)
    seen = []
    for block in r.model.blocks:
        def spy(hidden, pending, batch, cache, _inner=block.forward, **kw):
            out = _inner(hidden, pending, batch, cache, **kw)
            x = hidden[:batch.num_tokens].double().cpu()
            if out is not None and not isinstance(out, Carried):      # a branch that the next norm's kernel adds
                x = x + out[:batch.num_tokens].double().cpu()
            seen.append(x)
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
    """Decoding far beyond every window of the model, across many pages, from eager steps."""
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
    """32-bit: whole (where the recurrences run in chunks), in portions and token by token, a position's logits are equal
    up to the last bits."""
    _, cfg, w, _ = models["T1"]
    ids = tokens_for(cfg, 180, 8)
    got = []
    for parts in ([ids], cut(ids, [5, 2, 11, 1]), cut(ids, [129, 40]), [[t] for t in ids]):
        r = make_runner(models, "T1", "float32")
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
def test_a_long_portion_beside_single_tokens(models, dtype):
    """One portion of several chunks beside two decoding requests and a short portion: the recurrences run in chunks for
    one request and whole for the others of the same launch."""
    _, cfg, w, _ = models["T1"]
    ids = {"a": tokens_for(cfg, 420, 1), "b": tokens_for(cfg, 12, 2), "c": tokens_for(cfg, 40, 3), "d": tokens_for(cfg, 90, 4)}
    at = {"a": 20, "b": 9, "c": 3, "d": 0}
    steps = [([(k, ids[k][:n], [n - 1]) for k, n in at.items() if n], [])]
    steps.append(([("b", ids["b"][9:10], [0]), ("a", ids["a"][20:400], list(range(0, 380, 7))), ("c", ids["c"][3:4], [0]),
                   ("d", ids["d"][:60], list(range(60)))], []))
    steps.append(([("a", ids["a"][400:401], [0]), ("b", ids["b"][10:12], [0, 1]), ("c", ids["c"][4:40], list(range(36))),
                   ("d", ids["d"][60:61], [0])], []))
    steps.append(([("d", ids["d"][61:90], [28]), ("a", ids["a"][401:402], [0])], []))
    run_and_compare(make_runner(models, "T1", dtype, num_blocks=200), steps, cfg, w, ids, dtype, "a long portion among others")


# ---- edges that random weights would hide -------------------------------------------------------------------------
def with_windows(cfg, change):
    out = copy.deepcopy(cfg)
    for l in out["layers"]:
        if "mask" in l["mixer"]:
            l["mixer"]["mask"]["size"] += change
    return out


@pytest.mark.parametrize("dtype", DTYPES)
def test_keys_just_inside_and_outside_the_windows(models, dtype):
    """Scores so sharp that the oldest key a window holds often carries most of a row's weight. The engine agrees with the
    windows as configured, in a prompt and in decoding, and the same model with windows one key longer or shorter, or
    without its sinks, gives rows that differ by far more than the tolerance."""
    _, cfg, w, page = models["sharp"]
    ids = tokens_for(cfg, 90, 2)
    want = plain.forward(ids, w, cfg)
    spread = want.std(dim=-1, keepdim=True)
    off = lambda other: ((other - want).abs() / spread).amax(dim=-1)[8:]
    for change in (-1, 1):
        assert (off(plain.forward(ids, w, with_windows(cfg, change))) > 0.6).float().mean().item() > 0.4, "a window one key off does not show"
    no_sinks = {k: (v * 0 - 50.0 if k.endswith(".sink") else v) for k, v in w.items()}
    assert (off(plain.forward(ids, no_sinks, cfg)) > 0.6).float().mean().item() > 0.2, "a sink left out does not show"
    r = make_runner(models, "sharp", dtype)
    whole = replay(r, [([("x", ids, list(range(len(ids))))], ["x"])])
    compare_rows(whole, cfg, w, {"x": ids}, dtype, "sharp whole", sharp=True)
    steps = [([("y", ids[:11], list(range(11)))], [])] + [([("y", [t], [0])], []) for t in ids[11:]]
    compare_rows(replay(r, steps), cfg, w, {"y": ids}, dtype, "sharp decoded", sharp=True)
    compare_rows(replay(r, [([("z", p, list(range(len(p))))], []) for p in cut(ids, [3, 2, 7])]), cfg, w, {"z": ids}, dtype,
                 "sharp in portions across the windows' edges", sharp=True)


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_key_far_back_among_hundreds(models, dtype):
    """The sigmoid attention sees everything: many rows far into a long request take their output from single keys hundreds of
    tokens back; without the keys more than 64 back they would be others."""
    _, cfg, w, page = models["far"]
    ids = tokens_for(cfg, 420, 4)
    want = plain.forward(ids, w, cfg)

    def near_only(T, size=None, _v=plain.visible):
        return _v(T, 64 if size is None else size)
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


def test_pages_behind_the_window_are_given_back(models):
    _, cfg, w, page = models["sharp"]      # windows of 6 and 4, pages of 4
    r = make_runner(models, "sharp", "float32", num_blocks=110, max_len=400)
    ids = tokens_for(cfg, 300, 4)
    rows = replay(r, [([("x", p, [len(p) - 1])], []) for p in cut(ids, [9, 1, 1, 30, 2])])
    compare_rows(rows, cfg, w, {"x": ids}, "float32", "a long request")
    assert len(r.group_specs) == 2
    for g, spec in enumerate(r.group_specs):
        held = [i for i, pg in enumerate(r.cache.block_table("x", g)) if pg >= 0]
        assert held == list(range((len(ids) - spec.window + 1) // page, (len(ids) - 1) // page + 1))


# ---- graphs and the engine's own entry point ----------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["T1", "T3"])
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
    _, cfg, w, _ = models["T1"]
    steps, toks = [], {}
    for i in range(6):
        for k, n, s in (("p", 160, 1), ("q", 20, 2), ("d", 12, 3)):
            toks[f"{k}{i}"] = tokens_for(cfg, n, 10 * s + i)
        steps.append(([(f"d{i}", toks[f"d{i}"][:11], [10])], []))
        steps.append(([(f"p{i}", toks[f"p{i}"], [0, 80, 159]), (f"d{i}", toks[f"d{i}"][11:], [0]), (f"q{i}", toks[f"q{i}"], [19])],
                      [f"p{i}", f"d{i}", f"q{i}"]))
    r = make_runner(models, "T1", dtype, graph=True)
    rows = replay(r, steps)
    assert r.portion_replays > 0, "no step with portions was replayed"
    eager = run_and_compare(make_runner(models, "T1", dtype), steps, cfg, w, toks, dtype, "eager portions")
    # (a padded step may take other kernels for its products: close, not equal)
    for key, row in rows.items():
        err = (row - eager[key]).abs().max().item() / max(1.0, eager[key].abs().max().item())
        assert err < (1e-5 if dtype == "float32" else 0.1), f"{key}: {err}"


@pytest.mark.parametrize("name", ["T1", "T2"])
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
    d, cfg, _, page = models["T3"]
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
    d, cfg, w, _ = models["T1" if dtype == "float32" else "mix"]     # (bfloat16: a model without routers, see compare_rows)
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
    """bin/dinfer random-weights from a configuration that names the decay projection's inner size, then bin/dinfer
    generate on that folder and on a folder of the plain model's weights, where the greedy tokens are the plain model's
    wherever its choice is clear."""
    import subprocess
    import sys
    from pathlib import Path
    d, cfg, w, page = models["T1"]
    root = Path(__file__).resolve().parent.parent
    exe = [sys.executable, str(root / "bin" / "dinfer")]
    named = copy.deepcopy(cfg)
    for l in named["layers"]:
        if l["type"] == "parallel":
            l["mixer"]["right"]["decay_rank"] = 9
    (tmp_path / "config.json").write_text(json.dumps(named))
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
