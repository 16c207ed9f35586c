"""Reverax, the slow way: every mechanism of the design as one plain function over a whole sequence.

Double precision on the CPU, full score matrices, recurrences walked token by token, experts row by row.  Shares
nothing with the package: it is what the package's parts and kernels are held against.

A model is ``(config, weights)``: the config.json mapping and name -> tensor.  A layer's tensors start with
``l<i>.`` (``l<j>.`` for a layer that takes layer j's weights); a mixer's with ``l<i>.mix.``, a feed-forward's with
``l<i>.mlp.``; linear weights are ``[out, in]``.
"""
import torch

F = torch.float64


def unit_rms(x, eps):
    """x over its root mean square along the last axis, eps inside the root."""
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def grouped_norm(x, w, eps, groups):
    """Every one of ``groups`` equal consecutive parts of a row over its own root mean square, the whole row times w."""
    steps, width = x.shape
    return unit_rms(x.reshape(steps, groups, width // groups), eps).reshape(steps, width) * w


def silu(z):
    return z * torch.sigmoid(z)


def angles(positions, dims, base):
    freq = torch.tensor([base ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=F)
    return torch.tensor(positions, dtype=F)[:, None] * freq[None, :]


def rotate_halves(x, positions, dims, base):
    """x [steps, heads, size]: element i turns together with element i + dims/2; what lies beyond ``dims`` stays."""
    a = angles(positions, dims, base)
    cos, sin = torch.cos(a)[:, None, :], torch.sin(a)[:, None, :]
    u, v = x[..., :dims // 2], x[..., dims // 2:dims]
    return torch.cat([u * cos - v * sin, v * cos + u * sin, x[..., dims:]], dim=-1)


def rotate_neighbours(x, positions, dims, base):
    """x [steps, heads, size]: element 2i turns together with element 2i + 1; what lies beyond ``dims`` stays."""
    a = angles(positions, dims, base)
    cos, sin = torch.cos(a)[:, None, :], torch.sin(a)[:, None, :]
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    turned = torch.stack([u * cos - v * sin, v * cos + u * sin], dim=-1).reshape(*x.shape[:-1], dims)
    return torch.cat([turned, x[..., dims:]], dim=-1)


def visible(steps, window=None):
    """[i, j] true where position i sees position j: j <= i, and with a window i - j < window."""
    i, j = torch.arange(steps)[:, None], torch.arange(steps)[None, :]
    see = j <= i
    return see & (i - j < window) if window else see


def cap_scores(score, cap):
    return cap * torch.tanh(score / cap)


def softmax_with_sink(score, see, sink):
    """Weights of the visible keys; the denominator also holds exp(sink), which weighs no value."""
    score = score.masked_fill(~see, float("-inf"))
    top = torch.maximum(score.max(dim=-1, keepdim=True).values, sink)
    e = torch.exp(score - top)
    return e / (e.sum(dim=-1, keepdim=True) + torch.exp(sink - top))


def heads_of(h, w, p, name, heads, size):
    return (h @ w[p + name].T + w[p + name + ".b"]).view(h.shape[0], heads, size)


def turned_value_attention(h, m, w, p, eps):
    """The left branch: projections with biases, q and k normed per head, half pairs rotated on the first ``rot.dims``
    elements, values that turn with their position and are turned back where they are read, capped scores, a sink a
    head in the denominator, a window."""
    steps = h.shape[0]
    heads, kv_heads, dim, vdim = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    positions = list(range(steps))
    dims, base = int(m["rot"]["dims"]), float(m["rot"]["base"])
    q, k, v = (heads_of(h, w, p, n, c, d) for n, c, d in (("q", heads, dim), ("k", kv_heads, dim), ("v", kv_heads, vdim)))
    q = rotate_halves(unit_rms(q, eps) * w[p + "q.norm"], positions, dims, base)
    k = rotate_halves(unit_rms(k, eps) * w[p + "k.norm"], positions, dims, base)
    v = rotate_halves(v, positions, vdim, base)
    see = visible(steps, int(m["mask"]["size"]) if m.get("mask") else None)
    out = torch.zeros(steps, heads, vdim, dtype=F)
    for head in range(heads):
        g = head // (heads // kv_heads)
        score = (q[:, head] @ k[:, g].T) * float(m["scale"])
        if m.get("softcap"):
            score = cap_scores(score, float(m["softcap"]))
        out[:, head] = softmax_with_sink(score, see, w[p + "sink"][head]) @ v[:, g]
    out = rotate_halves(out, [-i for i in positions], vdim, base)
    return out.reshape(steps, heads * vdim) @ w[p + "o"].T


def token_mix(h, mu):
    """h + (h' - h) * mu with h' the token before (zeros before the first)."""
    before = torch.cat([torch.zeros_like(h[:1]), h[:-1]])
    return h + (before - h) * mu


def time_mixing(h, m, w, p, eps):
    """The right branch (RWKV): per head o_t = (S + diag(u) k v^T)^T r, then S <- diag(w_t) S + k v^T, from S = 0, with
    a decay w_t = exp(-exp(.)) that the token makes per key channel."""
    steps = h.shape[0]
    heads, dim = int(m["heads"]), int(m["dim"])
    mixed = {n: token_mix(h, w[p + "mu." + n]) for n in ("r", "k", "v", "g", "w")}
    r, k, v = ((mixed[n] @ w[p + n].T).view(steps, heads, dim) for n in ("r", "k", "v"))
    gate = silu(mixed["g"] @ w[p + "g"].T)
    decay = torch.exp(-torch.exp(torch.tanh(mixed["w"] @ w[p + "w1"].T) @ w[p + "w2"].T + w[p + "w0"])).view(steps, heads, dim)
    u = w[p + "u"]
    out = torch.zeros(steps, heads, dim, dtype=F)
    S = torch.zeros(heads, dim, dim, dtype=F)
    for t in range(steps):
        for head in range(heads):
            write = torch.outer(k[t, head], v[t, head])
            out[t, head] = (S[head] + u[head][:, None] * write).T @ r[t, head]
            S[head] = decay[t, head][:, None] * S[head] + write
    out = unit_rms(out, eps).reshape(steps, heads * dim) * w[p + "norm"] * gate
    return out @ w[p + "o"].T


def side_by_side(h, m, w, p, eps):
    return float(m["left_scale"]) * turned_value_attention(h, m["left"], w, p + "left.", eps) + \
        float(m["right_scale"]) * time_mixing(h, m["right"], w, p + "right.", eps)


def talking_attention(h, m, w, p):
    """The 'attention' mixer: neighbouring pairs rotated, the heads' scaled scores mixed by a matrix before the softmax."""
    steps = h.shape[0]
    heads, kv_heads, dim, vdim = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    positions = list(range(steps))
    dims, base = int(m["rot"]["dims"]), float(m["rot"]["base"])
    q, k, v = (heads_of(h, w, p, n, c, d) for n, c, d in (("q", heads, dim), ("k", kv_heads, dim), ("v", kv_heads, vdim)))
    q, k = rotate_neighbours(q, positions, dims, base), rotate_neighbours(k, positions, dims, base)
    per_kv = heads // kv_heads
    score = torch.stack([(q[:, g] @ k[:, g // per_kv].T) * float(m["scale"]) for g in range(heads)])
    mixed = torch.zeros_like(score)
    for head in range(heads):
        for g in range(heads):
            mixed[head] += w[p + "talk"][head, g] * score[g]
    see = visible(steps)
    out = torch.zeros(steps, heads, vdim, dtype=F)
    for head in range(heads):
        out[:, head] = torch.softmax(mixed[head].masked_fill(~see, float("-inf")), dim=-1) @ v[:, head // per_kv]
    return out.reshape(steps, heads * vdim) @ w[p + "o"].T


def dense_feed_forward(h, w, p):
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def expert(h, w, p):
    return torch.relu(h @ w[p + "up"].T) ** 2 @ w[p + "down"].T


def route(h, router, top):
    """For every row the experts with the largest sigmoid scores, and these scores as they are."""
    best = torch.topk(torch.sigmoid(h @ router.T), top, dim=-1)
    return best.indices, best.values


def mixture(h, mlp, w, p):
    """Every chosen expert reads the row times its score."""
    chosen, weight = route(h, w[p + "router"], int(mlp["router"]["top"]))
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, a in zip(chosen[t].tolist(), weight[t]):
            out[t] += expert(a * h[t:t + 1], w, f"{p}e{e}.")[0]
    return out


def mixer(kind, h, m, w, p, eps):
    if kind == "attention":
        return talking_attention(h, m, w, p)
    if kind == "parallel":
        return side_by_side(h, m, w, p, eps)
    raise ValueError(f"unknown layer type {kind!r}")


def forward(config, weights, tokens, layers_out=None):
    """Logits [steps, vocab] of one sequence from position 0; ``layers_out`` (a list) receives the stream after
    every layer."""
    w = {k: v.to(F) for k, v in weights.items()}
    eps, groups = float(config["norm"]["eps"]), int(config["norm"]["groups"])
    x = w["embed"][torch.tensor(tokens)]
    for i, layer in enumerate(config["layers"]):
        p = f"l{layer.get('weights_of', i)}."
        delta = mixer(layer["type"], grouped_norm(x, w[p + "norm1"], eps, groups), layer["mixer"], w, p + "mix.", eps) * w[p + "ls1"]
        mlp = layer.get("mlp")
        if mlp:
            h = grouped_norm(x, w[p + "norm2"], eps, groups)
            delta = delta + (mixture(h, mlp, w, p + "mlp.") if mlp["kind"] == "moe" else dense_feed_forward(h, w, p + "mlp.")) * w[p + "ls2"]
        x = x + delta
        if layers_out is not None:
            layers_out.append(x.clone())
    return grouped_norm(x, w["final.norm"], eps, groups) @ w["embed"].T * float(config["logit_scale"])
