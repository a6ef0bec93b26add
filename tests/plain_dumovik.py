"""A plain, slow Dumovik in float64 on the CPU: one function per mechanism, whole sequences at once, no cache.
It shares nothing with the engine; the tests compare the engine with it.

cfg is the parsed config.json (a dict), w a dict name -> float64 tensor.
"""
import math

import torch

F = torch.float64
EXPERT_SLOPE = 1.702      # of the sigmoid in an expert's gate


def layer_norm(x, weight, eps):
    """Mean off, divided by the root of the mean squared deviation, times a gain; no bias."""
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * weight


def rms_norm(x, weight, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * weight


def silu(z):
    return z * torch.sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))


def rotate_halves(x, rot):
    """x [T, heads, dim]: entry i of the first rot['dims'] turns with entry i + dims/2, row p by p * base^(-2i/dims)."""
    half = rot["dims"] // 2
    p = torch.arange(x.shape[0], dtype=F)
    y = x.clone()
    for i in range(half):
        a = (p * rot["base"] ** (-2.0 * i / rot["dims"]))[:, None]
        u, v = x[..., i], x[..., i + half]
        y[..., i], y[..., i + half] = u * a.cos() - v * a.sin(), v * a.cos() + u * a.sin()
    return y


def visible(T, chunk=None):
    """[T, T] bool: row i sees column j <= i, and with chunks only one of its own chunk (counted from position 0)."""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    m = j <= i
    return m if chunk is None else m & (i // chunk == j // chunk)


def softmax(scores, mask):
    return torch.softmax(scores.masked_fill(~mask, float("-inf")), dim=-1)


def soft_cap(scores, cap):
    return cap * torch.tanh(scores / cap)


def latent_attention(h, w, p, m, eps):
    """Keys and values of all heads are made from one normed latent a token; one rotated key part serves all heads."""
    T = h.shape[0]
    H, D, R, V, K = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    q = (h @ w[p + ".q"].T).view(T, H, D + R)
    down = h @ w[p + ".dkv"].T
    c = rms_norm(down[:, :K], w[p + ".dkv.norm"], eps)
    kr = rotate_halves(down[:, None, K:], m["rot"])[:, 0]
    qr = rotate_halves(q[..., D:], m["rot"])
    k, v = (c @ w[p + ".uk"].T).view(T, H, D), (c @ w[p + ".uv"].T).view(T, H, V)
    mask, out = visible(T), torch.zeros(T, H, V, dtype=F)
    for hd in range(H):
        s = (q[:, hd, :D] @ k[:, hd].T + qr[:, hd] @ kr.T) * m["scale"]
        out[:, hd] = softmax(s, mask) @ v[:, hd]
    return (out.reshape(T, H * V) * torch.sigmoid(h @ w[p + ".g"].T)) @ w[p + ".o"].T


def keys_values(h, w, p, m, eps):
    """What an attention layer caches: keys normed over the whole projection, and values."""
    T, G = h.shape[0], m["kv_heads"]
    k = rms_norm(h @ w[p + ".k"].T, w[p + ".k.norm"], eps).view(T, G, m["dim"])
    return k, (h @ w[p + ".v"].T).view(T, G, m["vdim"])


def chunked_attention(h, w, p, m, eps, k, v):
    """Softmax attention inside chunks of positions, scores capped by a tanh; queries normed over the whole projection."""
    T, H, G, D, V = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms_norm(h @ w[p + ".q"].T, w[p + ".q.norm"], eps).view(T, H, D)
    mask, out = visible(T, m["mask"]["size"]), torch.zeros(T, H, V, dtype=F)
    for hd in range(H):
        g = hd // (H // G)
        s = soft_cap(q[:, hd] @ k[:, g].T * m["scale"], m["softcap"])
        out[:, hd] = softmax(s, mask) @ v[:, g]
    return out.reshape(T, H * V) @ w[p + ".o"].T


def lightning(h, w, p, m, eps):
    """A state S [dim, vdim] a head with a fixed decay: S <- decay S + k v^T, o = S^T q; one norm over all heads."""
    T, H, D, V = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q, k = silu(h @ w[p + ".q"].T).view(T, H, D), silu(h @ w[p + ".k"].T).view(T, H, D)
    v = silu(h @ w[p + ".v"].T).view(T, H, V)
    decay = torch.tensor(m["decay"], dtype=F)[:, None, None]
    S, o = torch.zeros(H, D, V, dtype=F), torch.zeros(T, H, V, dtype=F)
    for t in range(T):
        S = decay * S + k[t][:, :, None] * v[t][:, None, :]
        o[t] = (S * q[t][:, :, None]).sum(1)
    o = rms_norm(o.reshape(T, H * V), w[p + ".norm"], eps)
    return (o * torch.sigmoid(h @ w[p + ".g"].T)) @ w[p + ".o"].T


def dense_ff(h, w, p):
    return (gelu_tanh(h @ w[p + ".gate"].T) * (h @ w[p + ".up"].T)) @ w[p + ".down"].T


def expert(h, w, p, limit):
    g = torch.clamp(h @ w[p + ".gate"].T, max=limit)
    u = torch.clamp(h @ w[p + ".up"].T, min=-limit, max=limit)
    return (g * torch.sigmoid(EXPERT_SLOPE * g) * (u + 1)) @ w[p + ".down"].T


CLOSE_CALL = 0.1      # logits nearer than this may fall either way once the router's input is rounded


def chosen_experts(h, w, p, f, given=None):
    """(indices [T, top], weights [T, top]): the largest logits, weighted by the softmax over the chosen ones.
    given {row: [experts]}: the choice somebody else made for some rows (an engine whose router read rounded rows). It
    is taken over where it could be right: every expert it names scores within CLOSE_CALL of the last one chosen here,
    and every expert chosen here that it leaves out is within CLOSE_CALL of the best one it could have left out."""
    top = f["router"]["top"]
    z = h @ w[p + ".router"].T
    idx = torch.topk(z, top, dim=-1).indices
    for t, other in (given or {}).items():
        assert len(other) == top == len(set(other)), f"{p} row {t}: {other} are not {top} experts"
        line = z[t, idx[t]].min().item()
        assert all(z[t, e].item() > line - CLOSE_CALL for e in other), f"{p} row {t}: {other} chosen, {idx[t].tolist()} score best"
        assert all(z[t, e].item() < line + CLOSE_CALL for e in idx[t].tolist() if e not in other), \
            f"{p} row {t}: {other} chosen, {idx[t].tolist()} score best"
        idx[t] = torch.tensor(other)
    return idx, torch.softmax(torch.gather(z, 1, idx), dim=-1)


def routed_ff(h, w, p, f, given=None):
    idx, share = chosen_experts(h, w, p, f, given)
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, s in zip(idx[t].tolist(), share[t]):
            out[t] += s * expert(h[t], w, f"{p}.e{e}", f["expert"]["limit"])
    return out


def mixer(h, w, cfg, i, kept):
    """kept: a dict layer -> (keys, values), what the attention layers before this one cached."""
    l, p, eps = cfg["layers"][i], f"l{i}.mix", cfg["norm"]["eps"]
    m = l["mixer"]
    if l["type"] == "lightning":
        return lightning(h, w, p, m, eps)
    if l["type"] == "latent_attention":
        return latent_attention(h, w, p, m, eps)
    source = m.get("kv_from")
    if source is None:
        kept[i] = keys_values(h, w, p, m, eps)
    return chunked_attention(h, w, p, m, eps, *kept[i if source is None else source])


def layer(x, w, cfg, i, kept, given=None):
    """One layer on the stream x [T, width]: each sublayer reads the stream, its output is normed and added."""
    l, p, eps = cfg["layers"][i], f"l{i}", cfg["norm"]["eps"]
    x = x + layer_norm(mixer(x, w, cfg, i, kept), w[p + ".norm1"], eps)
    f = l.get("mlp")
    if f is not None:
        y = dense_ff(x, w, p + ".mlp") if f["kind"] == "dense" else routed_ff(x, w, p + ".mlp", f, given)
        x = x + layer_norm(y, w[p + ".norm2"], eps)
    return x


def forward(tokens, w, cfg, streams=None, choices=None):
    """Logits [T, vocab] of a whole sequence; `streams`, a list, receives the stream after every layer.
    choices {(layer, row): [experts]}: routing choices to take over where they could be right (chosen_experts)."""
    x = w["embed"][torch.as_tensor(tokens)]
    kept = {}
    for i in range(len(cfg["layers"])):
        x = layer(x, w, cfg, i, kept, {t: e for (l, t), e in (choices or {}).items() if l == i})
        if streams is not None:
            streams.append(x)
    return layer_norm(x, w["final.norm"], cfg["norm"]["eps"]) @ w["embed"].T


# ---- made-up weights for the tests -------------------------------------------------------------------------------
def tensor_shapes(cfg):
    """name -> shape of every tensor a configuration asks for."""
    W, out = cfg["width"], {"embed": (cfg["vocab"], cfg["width"]), "final.norm": (cfg["width"],)}
    for i, l in enumerate(cfg["layers"]):
        p, m = f"l{i}", l["mixer"]
        q = p + ".mix"
        out[f"{p}.norm1"] = (W,)
        H, D, V = m["heads"], m["dim"], m["vdim"]
        if l["type"] == "lightning":
            out.update({f"{q}.q": (H * D, W), f"{q}.k": (H * D, W), f"{q}.v": (H * V, W), f"{q}.g": (H * V, W),
                        f"{q}.o": (W, H * V), f"{q}.norm": (H * V,)})
        elif l["type"] == "latent_attention":
            R, K = m["rot_dim"], m["kv_rank"]
            out.update({f"{q}.q": (H * (D + R), W), f"{q}.dkv": (K + R, W), f"{q}.dkv.norm": (K,), f"{q}.uk": (H * D, K),
                        f"{q}.uv": (H * V, K), f"{q}.g": (H * V, W), f"{q}.o": (W, H * V)})
        else:
            G = m["kv_heads"]
            out.update({f"{q}.q": (H * D, W), f"{q}.q.norm": (H * D,), f"{q}.o": (W, H * V)})
            if m.get("kv_from") is None:
                out.update({f"{q}.k": (G * D, W), f"{q}.v": (G * V, W), f"{q}.k.norm": (G * D,)})
        f = l.get("mlp")
        if f is None:
            continue
        out[f"{p}.norm2"] = (W,)
        if f["kind"] == "dense":
            parts = [(f"{p}.mlp", f["ff"])]
        else:
            out[f"{p}.mlp.router"] = (f["router"]["experts"], W)
            parts = [(f"{p}.mlp.e{e}", f["expert"]["ff"]) for e in range(f["router"]["experts"])]
        for n, ff in parts:
            out.update({f"{n}.gate": (ff, W), f"{n}.up": (ff, W), f"{n}.down": (W, ff)})
    return out


def random_weights(cfg, seed):
    """bfloat16 tensors of sizes that keep every mechanism awake: the stream grows by about one a sublayer, so the
    projections of later layers are made smaller; gains around one."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        x = torch.randn(shape, generator=g)
        last = name.split(".")[-1]
        if name == "embed":
            t = x
        elif last in ("norm1", "norm2", "norm"):
            t = 1.0 + x * 0.2
        else:
            depth = 1 + 2 * int(name[1:name.index(".")]) if name[0] == "l" else 1      # sublayers added before
            reads_stream = shape[-1] == cfg["width"] and last not in ("o", "down", "uk", "uv")
            t = x * (1.5 / shape[-1] ** 0.5) / (depth ** 0.5 if reads_stream else 1.0)
        out[name] = t.to(torch.bfloat16)
    return out


def as_float64(w):
    return {k: v.to(F) for k, v in w.items()}
