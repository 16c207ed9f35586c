"""Sonulorn, the slow way: every mechanism of the design as one plain function over a whole sequence.

Double precision on the CPU, full score matrices, recurrences walked token by token.  Shares nothing with the package:
it is what the package's parts and kernels are held against.

A model is ``(config, weights)``: the config.json mapping and name -> tensor.  A layer's tensors start with ``l<i>.``, a
mixer's with ``l<i>.mix.``, a feed-forward's with ``l<i>.mlp.``; linear weights are ``[out, in]``.
"""
import torch

F = torch.float64


def unit_rms(x, eps):
    """x over its root mean square along the last axis, eps inside the root."""
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def silu(z):
    return z * torch.sigmoid(z)


def softplus(z):
    return torch.logaddexp(z, torch.zeros_like(z))


def unit_vector(x, small=1e-6):
    """x over its length along the last axis, ``small`` under the root."""
    return x / torch.sqrt((x * x).sum(dim=-1, keepdim=True) + small)


def rotate_halves(x, positions, dims, base):
    """x [steps, heads, size]: element i turns together with element i + dims/2; what lies beyond ``dims`` stays."""
    freq = torch.tensor([base ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=F)
    a = torch.tensor(positions, dtype=F)[:, None] * freq[None, :]
    cos, sin = torch.cos(a)[:, None, :], torch.sin(a)[:, None, :]
    u, v = x[..., :dims // 2], x[..., dims // 2:dims]
    return torch.cat([u * cos - v * sin, v * cos + u * sin, x[..., dims:]], dim=-1)


def short_convolution(x, w):
    """x [steps, channels], w [channels, taps]: every channel's last ``taps`` values weighed, the newest by the last tap,
    zeros ahead of the sequence."""
    taps = w.shape[1]
    padded = torch.cat([torch.zeros(taps - 1, x.shape[1], dtype=x.dtype), x])
    out = torch.zeros_like(x)
    for j in range(taps):
        out += w[:, j] * padded[j:j + x.shape[0]]
    return out


def visible(steps, chunk=None):
    """[i, j] true where position i sees position j: j <= i, and with chunks only inside the same chunk of positions."""
    i, j = torch.arange(steps)[:, None], torch.arange(steps)[None, :]
    see = j <= i
    return see & (i // chunk == j // chunk) if chunk else see


def softmax_with_sink(score, see, sink):
    """Weights of the visible keys; the denominator also holds exp(sink), which weighs no value."""
    score = score.masked_fill(~see, float("-inf"))
    top = torch.maximum(score.max(dim=-1, keepdim=True).values, sink)
    e = torch.exp(score - top)
    return e / (e.sum(dim=-1, keepdim=True) + torch.exp(sink - top))


def sink_attention(h, m, w, p, chunk=None, conv=False, gate_each=False):
    """Grouped-query attention with half pairs rotated, a sink a head and an output gate (one a head, or one an element);
    q, k and v through short convolutions ahead of the rotation with ``conv``; only keys of the same chunk with ``chunk``."""
    steps = h.shape[0]
    heads, kv_heads, dim, vdim = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    positions, dims, base = list(range(steps)), int(m["rot"]["dims"]), float(m["rot"]["base"])

    def project(name, count, size):
        x = h @ w[p + name].T
        if conv:
            x = short_convolution(x, w[p + name + ".conv"])
        return x.view(steps, count, size)
    q = rotate_halves(project("q", heads, dim), positions, dims, base)
    k = rotate_halves(project("k", kv_heads, dim), positions, dims, base)
    v = project("v", kv_heads, vdim)
    see = visible(steps, chunk)
    out = torch.zeros(steps, heads, vdim, dtype=F)
    for head in range(heads):
        g = head // (heads // kv_heads)
        score = (q[:, head] @ k[:, g].T) * float(m["scale"])
        out[:, head] = softmax_with_sink(score, see, w[p + "sink"][head]) @ v[:, g]
    gate = torch.sigmoid(h @ w[p + "g"].T)
    out = out * (gate.view(steps, heads, vdim) if gate_each else gate[:, :, None])
    return out.reshape(steps, heads * vdim) @ w[p + "o"].T


def head_decay_delta(h, m, w, p, eps):
    """The gated delta rule with one decay a head: S <- g S, u = beta (v - S^T k), S <- S + k u^T, o = S^T q."""
    steps = h.shape[0]
    heads, kv_heads, dim, vdim = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    q, k, v = (silu(short_convolution(h @ w[p + n].T, w[p + n + ".conv"])) for n in ("q", "k", "v"))
    q = unit_vector(q.view(steps, kv_heads, dim)) * dim ** -0.5
    k = unit_vector(k.view(steps, kv_heads, dim))
    v = v.view(steps, heads, vdim)
    beta = torch.sigmoid(h @ w[p + "b"].T)
    decay = torch.exp(-torch.exp(w[p + "A_log"]) * softplus(h @ w[p + "a"].T + w[p + "dt_bias"]))
    out = torch.zeros(steps, heads, vdim, dtype=F)
    S = torch.zeros(heads, dim, vdim, dtype=F)
    for t in range(steps):
        for head in range(heads):
            g = head // (heads // kv_heads)
            kept = decay[t, head] * S[head]
            u = beta[t, head] * (v[t, head] - kept.T @ k[t, g])
            S[head] = kept + torch.outer(k[t, g], u)
            out[t, head] = S[head].T @ q[t, g]
    out = unit_rms(out, eps) * w[p + "norm"] * silu(h @ w[p + "g"].T).view(steps, heads, vdim)
    return out.reshape(steps, heads * vdim) @ w[p + "o"].T


def side_by_side(h, m, w, p, eps):
    return float(m["left_scale"]) * sink_attention(h, m["left"], w, p + "left.", conv=True) + \
        float(m["right_scale"]) * head_decay_delta(h, m["right"], w, p + "right.", eps)


def fixed_decay_memory(h, m, w, p, eps):
    """Lightning attention: silu on q, k and v, S <- decay S + k v^T, o = S^T q; the heads normed together."""
    steps = h.shape[0]
    heads, dim, vdim = int(m["heads"]), int(m["dim"]), int(m["vdim"])
    q, k = (silu(h @ w[p + n].T).view(steps, heads, dim) for n in ("q", "k"))
    v = silu(h @ w[p + "v"].T).view(steps, heads, vdim)
    decay = torch.tensor([float(d) for d in m["decay"]], dtype=F)[:, None, None]
    out = torch.zeros(steps, heads, vdim, dtype=F)
    S = torch.zeros(heads, dim, vdim, dtype=F)
    for t in range(steps):
        S = decay * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(dim=1)
    out = unit_rms(out.reshape(steps, heads * vdim), eps) * w[p + "norm"] * torch.sigmoid(h @ w[p + "g"].T)
    return out @ w[p + "o"].T


def clamped_feed_forward(h, w, p, limit):
    g = torch.clamp(h @ w[p + "gate"].T, max=limit)
    u = torch.clamp(h @ w[p + "up"].T, min=-limit, max=limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1.0)) @ w[p + "down"].T


def mixer(kind, h, m, w, p, eps):
    if kind == "attention":
        return sink_attention(h, m, w, p, chunk=int(m["mask"]["size"]), gate_each=True)
    if kind == "parallel":
        return side_by_side(h, m, w, p, eps)
    if kind == "lightning":
        return fixed_decay_memory(h, m, w, p, eps)
    raise ValueError(f"unknown layer type {kind!r}")


def layer_order(config):
    """The layers as they run: (layer, pass number if a pass of the loop begins here, else None)."""
    n = len(config["layers"])
    loop = config.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    start, stop, times = int(loop["start"]), int(loop["stop"]), int(loop["times"])
    order = [(i, None) for i in range(start)]
    for t in range(times):
        order += [(i, t if i == start else None) for i in range(start, stop)]
    return order + [(i, None) for i in range(stop, n)]


def join_pass(x, x0, w_in, step):
    """What a pass of the loop starts from: the stream and the embedding's output side by side through one matrix, and a
    vector of the pass added."""
    return torch.cat([x, x0], dim=-1) @ w_in.T + step


def forward(config, weights, tokens, layers_out=None):
    """Logits [steps, vocab] of one sequence from position 0; ``layers_out`` (a list) receives the stream after every
    layer run."""
    w = {k: v.to(F) for k, v in weights.items()}
    eps = float(config["norm"]["eps"])
    x = w["embed"][torch.tensor(tokens)] * float(config["embedding"]["scale"])
    x0 = x
    for i, begins in layer_order(config):
        if begins is not None:
            x = join_pass(x, x0, w["loop.in"], w["loop.step"][begins])
        layer, p = config["layers"][i], f"l{i}."
        h = unit_rms(x, eps) * w[p + "norm1"]
        delta = mixer(layer["type"], h, layer["mixer"], w, p + "mix.", eps)
        mlp = layer.get("mlp")
        if mlp:
            delta = delta + clamped_feed_forward(h, w, p + "mlp.", float(mlp["limit"]))
        x = x + delta
        if layers_out is not None:
            layers_out.append(x.clone())
    return unit_rms(x, eps) * w["final.norm"] @ w["head"].T
