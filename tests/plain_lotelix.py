"""A plain, slow Lotelix in float64 on the CPU: one function per mechanism, whole sequences at once, no cache.
It shares nothing with the engine; the tests compare the engine with it.

cfg is the parsed config.json (a dict), w a dict name -> float64 tensor.
"""
import math

import torch

F = torch.float64


def rms_unit(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last dimension."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def group_norm(x, weight, eps, groups):
    """Each of `groups` equal consecutive parts of a row is brought to unit root mean square by itself."""
    parts = x.reshape(*x.shape[:-1], groups, x.shape[-1] // groups)
    return rms_unit(parts, eps).reshape(x.shape) * weight


def silu(z):
    return z * torch.sigmoid(z)


def frequencies(rot):
    """One frequency a pair; with `scaling`, slow pairs are slowed by the factor and those between the two wavelengths
    in part."""
    dims, out = rot["dims"], []
    for i in range(dims // 2):
        f = rot["base"] ** (-2.0 * i / dims)
        sc = rot.get("scaling")
        if sc is not None:
            turn = 2 * math.pi / f
            if turn > sc["original"] / sc["low"]:
                f = f / sc["factor"]
            elif turn >= sc["original"] / sc["high"]:
                s = (sc["original"] / turn - sc["low"]) / (sc["high"] - sc["low"])
                f = (1 - s) * f / sc["factor"] + s * f
        out.append(f)
    return torch.tensor(out, dtype=F)


def angles(rot, T):
    return torch.arange(T, dtype=F)[:, None] * frequencies(rot)[None, :]


def rotate_halves(x, rot):
    """x [T, heads, dim]: entry i of the first rot['dims'] turns with entry i + dims/2; the others stay."""
    half = rot["dims"] // 2
    a = angles(rot, x.shape[0])
    y = x.clone()
    for i in range(half):
        c, s = a[:, i, None].cos(), a[:, i, None].sin()
        u, v = x[..., i], x[..., i + half]
        y[..., i], y[..., i + half] = u * c - v * s, v * c + u * s
    return y


def rotate_neighbours(x, rot):
    """The same with entry 2i turning with entry 2i + 1."""
    a = angles(rot, x.shape[0])
    y = x.clone()
    for i in range(rot["dims"] // 2):
        c, s = a[:, i, None].cos(), a[:, i, None].sin()
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        y[..., 2 * i], y[..., 2 * i + 1] = u * c - v * s, v * c + u * s
    return y


def visible(T, size=None):
    """[T, T] bool: row i sees column j (j <= i, and with a window i - j < size)."""
    i = torch.arange(T)[:, None]
    j = torch.arange(T)[None, :]
    m = j <= i
    if size is not None:
        m = m & (i - j < size)
    return m


def softmax_with_sink(scores, mask, sink):
    """Softmax over the visible keys with exp(sink) as one more term of the denominator."""
    s = scores.masked_fill(~mask, float("-inf"))
    top = torch.clamp(s.max(-1, keepdim=True).values, min=float(sink))
    e = torch.exp(s - top)
    return e / (e.sum(-1, keepdim=True) + torch.exp(sink - top))


def sigmoid_weights(scores, mask, bias):
    return torch.sigmoid(scores + bias) * mask.to(F)


def window_attention(h, w, p, m, v_first):
    """Windowed softmax attention with a sink a head and a gate an output entry. v_first: the values of the first layer
    that mixes values (None where this is it, or the layer does not mix). Returns (output, this layer's own values)."""
    T = h.shape[0]
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rotate_halves((h @ w[p + ".q"].T).view(T, H, D), m["rot"])
    k = rotate_halves((h @ w[p + ".k"].T).view(T, G, D), m["rot"])
    own = h @ w[p + ".v"].T
    v = own
    if v_first is not None:
        lam = w[p + ".vmix"]
        v = (1 - lam) * own + lam * v_first
    v = v.view(T, G, V)
    mask = visible(T, m["mask"]["size"])
    out = torch.zeros(T, H, V, dtype=F)
    for hd in range(H):
        g = hd // (H // G)
        out[:, hd] = softmax_with_sink(q[:, hd] @ k[:, g].T * m["scale"], mask, w[p + ".sink"][hd]) @ v[:, g]
    gated = out.reshape(T, H * V) * torch.sigmoid(h @ w[p + ".g"].T)
    return gated @ w[p + ".o"].T, own


def sigmoid_attention(h, w, p, m, eps):
    """Causal attention whose weights are sigmoids of the scores: nothing is normalised over the keys. q and k are
    normed over all heads at once before they are rotated."""
    T = h.shape[0]
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms_unit(h @ w[p + ".q"].T + w[p + ".q.b"], eps) * w[p + ".q.norm"]
    k = rms_unit(h @ w[p + ".k"].T + w[p + ".k.b"], eps) * w[p + ".k.norm"]
    v = (h @ w[p + ".v"].T + w[p + ".v.b"]).view(T, G, V)
    q, k = rotate_neighbours(q.view(T, H, D), m["rot"]), rotate_neighbours(k.view(T, G, D), m["rot"])
    mask = visible(T)
    out = torch.zeros(T, H, V, dtype=F)
    for hd in range(H):
        g = hd // (H // G)
        out[:, hd] = sigmoid_weights(q[:, hd] @ k[:, g].T * m["scale"], mask, w[p + ".pb"][hd]) @ v[:, g]
    return out.reshape(T, H * V) @ w[p + ".o"].T + w[p + ".o.b"]


def channel_decays(h, w, p, m):
    """alpha [T, heads, dim]: sigmoid(z)^(1/tau), z from the input through a small inner size."""
    z = h @ w[p + ".a1"].T @ w[p + ".a2"].T + w[p + ".a2.b"]
    return (torch.sigmoid(z) ** (1.0 / m["tau"])).view(h.shape[0], m["heads"], m["dim"])


def gated_linear_attention(h, w, p, m, eps):
    """A state S [dim, vdim] a head: every key channel decays by its own factor, then k v^T is added; o = S^T q."""
    T = h.shape[0]
    H, D, V = m["heads"], m["dim"], m["vdim"]
    q = (h @ w[p + ".q"].T).view(T, H, D) * D ** -0.5
    k = (h @ w[p + ".k"].T).view(T, H, D)
    v = (h @ w[p + ".v"].T).view(T, H, V)
    alpha = channel_decays(h, w, p, m)
    o = torch.zeros(T, H, V, dtype=F)
    S = torch.zeros(H, D, V, dtype=F)
    for t in range(T):
        S = alpha[t][:, :, None] * S + k[t][:, :, None] * v[t][:, None, :]
        o[t] = (S * q[t][:, :, None]).sum(1)
    o = rms_unit(o, eps) * w[p + ".norm"]
    return (o.reshape(T, H * V) * silu(h @ w[p + ".g"].T)) @ w[p + ".o"].T


def parallel(h, w, p, m, eps):
    left = sigmoid_attention(h, w, p + ".left", m["left"], eps)
    right = gated_linear_attention(h, w, p + ".right", m["right"], eps)
    return 0.5 * (rms_unit(left, eps) * w[p + ".left.out"] + rms_unit(right, eps) * w[p + ".right.out"])


def min_gru(h, w, p):
    z = torch.sigmoid(h @ w[p + ".z"].T + w[p + ".z.b"])
    u = h @ w[p + ".x"].T + w[p + ".x.b"]
    candidate = torch.where(u >= 0, u + 0.5, torch.sigmoid(u))
    S, out = torch.zeros_like(z[0]), torch.zeros_like(z)
    for t in range(h.shape[0]):
        S = (1 - z[t]) * S + z[t] * candidate[t]
        out[t] = S
    return (out * silu(h @ w[p + ".g"].T)) @ w[p + ".o"].T


CLOSE_CALL = 0.05     # choice scores nearer than this may fall either way once the router's input is rounded


def chosen_experts(h, w, p, f, given=None):
    """(indices [T, top], weights [T, top]): scores are sigmoids of the logits, the largest are chosen and weigh as they are.
    given {row: [experts]}: the choice somebody else made for some rows (an engine whose router read rounded rows). It
    is taken over where it could be right: every expert it names scores within CLOSE_CALL of the last one chosen here,
    and every expert chosen here that it leaves out is within CLOSE_CALL of the best one it could have left out."""
    top = f["router"]["top"]
    s = torch.sigmoid(h @ w[p + ".router"].T)
    idx = torch.topk(s, top, dim=-1).indices
    for t, other in (given or {}).items():
        assert len(other) == top == len(set(other)), f"{p} row {t}: {other} are not {top} experts"
        line = s[t, idx[t]].min().item()
        assert all(s[t, e].item() > line - CLOSE_CALL for e in other), f"{p} row {t}: {other} chosen, {idx[t].tolist()} score best"
        assert all(s[t, e].item() < line + CLOSE_CALL for e in idx[t].tolist() if e not in other), \
            f"{p} row {t}: {other} chosen, {idx[t].tolist()} score best"
        idx[t] = torch.tensor(other)
    return idx, torch.gather(s, 1, idx)


def routed_ff(h, w, p, f, given=None):
    """The weight of an expert multiplies what goes into it."""
    idx, share = chosen_experts(h, w, p, f, given)
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, s in zip(idx[t].tolist(), share[t]):
            out[t] += torch.relu(w[f"{p}.e{e}.up"] @ (s * h[t])) ** 2 @ w[f"{p}.e{e}.down"].T
    return out


def first_that_mixes(cfg):
    for i, l in enumerate(cfg["layers"]):
        if l["type"] == "attention" and l["mixer"].get("v_mix"):
            return i
    return None


def mixer(h, w, cfg, i, kept):
    """kept: a dict that carries the first mixing layer's values from layer to layer."""
    l, p, eps = cfg["layers"][i], f"l{i}.mix", cfg["norm"]["eps"]
    if l["type"] == "mingru":
        return min_gru(h, w, p)
    if l["type"] == "parallel":
        return parallel(h, w, p, l["mixer"], eps)
    mixes = bool(l["mixer"].get("v_mix"))
    out, own = window_attention(h, w, p, l["mixer"], kept.get("v") if mixes else None)
    if mixes:
        kept.setdefault("v", own)
    return out


def layer(x, w, cfg, i, kept, given=None):
    """One layer on the stream x [T, width]. given: see chosen_experts."""
    l, p = cfg["layers"][i], f"l{i}"
    eps, groups = cfg["norm"]["eps"], cfg["norm"].get("groups", 1)
    x = x + mixer(group_norm(x, w[p + ".norm1"], eps, groups), w, cfg, i, kept)
    if l.get("mlp") is not None:
        x = x + routed_ff(group_norm(x, w[p + ".norm2"], eps, groups), w, p + ".mlp", l["mlp"], given)
    return x


def forward(tokens, w, cfg, streams=None, choices=None):
    """Logits [T, vocab] of a whole sequence; `streams`, a list, receives the stream after every layer.
    choices {(layer, row): [experts]}: routing choices to take over where they could be right (chosen_experts)."""
    x = w["embed"][torch.as_tensor(tokens)] * cfg["embedding"]["scale"]
    kept = {}
    for i in range(len(cfg["layers"])):
        x = layer(x, w, cfg, i, kept, {t: e for (l, t), e in (choices or {}).items() if l == i})
        if streams is not None:
            streams.append(x)
    return group_norm(x, w["final.norm"], cfg["norm"]["eps"], cfg["norm"].get("groups", 1)) @ w["head"].T


# ---- made-up weights for the tests -------------------------------------------------------------------------------
def tensor_shapes(cfg, low=6):
    """name -> shape of every tensor a configuration asks for; `low`: the inner size of the decay projections (the
    configuration does not hold it: the engine reads it off the tensor)."""
    W, out = cfg["width"], {"embed": (cfg["vocab"], cfg["width"]), "final.norm": (cfg["width"],), "head": (cfg["vocab"], cfg["width"])}
    for i, l in enumerate(cfg["layers"]):
        p, m = f"l{i}", l["mixer"]
        out[f"{p}.norm1"] = (W,)
        if l["type"] == "mingru":
            N = m["width"]
            out.update({f"{p}.mix.z": (N, W), f"{p}.mix.z.b": (N,), f"{p}.mix.x": (N, W), f"{p}.mix.x.b": (N,),
                        f"{p}.mix.g": (N, W), f"{p}.mix.o": (W, N)})
        elif l["type"] == "attention":
            H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            out.update({f"{p}.mix.q": (H * D, W), f"{p}.mix.k": (G * D, W), f"{p}.mix.v": (G * V, W), f"{p}.mix.sink": (H,),
                        f"{p}.mix.g": (H * V, W), f"{p}.mix.o": (W, H * V)})
            if m.get("v_mix"):
                out[f"{p}.mix.vmix"] = ()
        else:
            a, r = m["left"], m["right"]
            H, G, D, V = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
            q = f"{p}.mix.left"
            for n, s in (("q", H * D), ("k", G * D), ("v", G * V)):
                out[f"{q}.{n}"], out[f"{q}.{n}.b"] = (s, W), (s,)
            out.update({f"{q}.q.norm": (H * D,), f"{q}.k.norm": (G * D,), f"{q}.pb": (H,), f"{q}.o": (W, H * V),
                        f"{q}.o.b": (W,), f"{q}.out": (W,)})
            H, D, V = r["heads"], r["dim"], r["vdim"]
            q = f"{p}.mix.right"
            rank = r.get("decay_rank", low)
            out.update({f"{q}.q": (H * D, W), f"{q}.k": (H * D, W), f"{q}.v": (H * V, W), f"{q}.g": (H * V, W),
                        f"{q}.o": (W, H * V), f"{q}.norm": (V,), f"{q}.a1": (rank, W), f"{q}.a2": (H * D, rank),
                        f"{q}.a2.b": (H * D,), f"{q}.out": (W,)})
        f = l.get("mlp")
        if f is not None:
            out[f"{p}.norm2"] = (W,)
            out[f"{p}.mlp.router"] = (f["router"]["experts"], W)
            for e in range(f["router"]["experts"]):
                out.update({f"{p}.mlp.e{e}.up": (f["expert"]["ff"], W), f"{p}.mlp.e{e}.down": (W, f["expert"]["ff"])})
    return out


def random_weights(cfg, seed, low=6):
    """bfloat16 tensors of sizes that keep every mechanism awake: products of about unit spread, gains around one,
    sinks and sigmoid biases that matter beside the scores, decays and update gates from short to long memory."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg, low).items():
        x = torch.randn(shape, generator=g)
        last = name.split(".")[-1]
        if name == "embed":
            t = x / cfg["embedding"]["scale"]
        elif name.endswith(".vmix"):
            t = 0.3 + 0.4 * torch.rand(shape, generator=g)
        elif last in ("norm1", "norm2", "norm", "out"):
            t = 1.0 + x * 0.2
        elif last == "sink":
            t = 1.0 + x
        elif last == "pb":
            t = x - 1.5
        elif name.endswith(".z.b"):
            t = 2.0 * x - 2.0
        elif name.endswith(".a2.b"):
            t = 2.0 * x + 1.0
        elif last == "b":
            t = x * 0.5
        elif last == "router":
            t = x * (2.0 / shape[-1] ** 0.5)
        else:
            t = x * (1.5 / shape[-1] ** 0.5)
        out[name] = t.to(torch.bfloat16)
    return out


def as_float64(w):
    return {k: v.to(F) for k, v in w.items()}
