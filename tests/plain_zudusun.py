"""A plain, slow rendition of the Zudusun design on one whole sequence: no cache, no batch, one function per
mechanism, written from the design's equations with torch tensor arithmetic only. It shares no code with the
package and is what the package's parts, kernels and engine are tested against.

A model is `(cfg, w)`: `cfg` the dictionary of its config.json, `w` a dictionary of tensors by checkpoint name.
Everything is computed in the dtype of `w`'s tensors after `widen` (float64 by default).

Notation: T tokens, D the model's width, H heads, G key/value heads, n the query/key size of a head, v its value
size, E the experts.
"""
import torch


def widen(w, dtype=torch.float64):
    return {k: (x.to(dtype) if x.is_floating_point() else x) for k, x in w.items()}


# ---------------------------------------------------------------- norms and activations

def unit_rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def centred_norm(x, weight, eps):
    """The model's norm: mean taken off, unit variance (mean of the squared deviations, eps inside the root), times
    weight."""
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * weight


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def log_sigmoid(z):
    """-ln(1 + e^-z)."""
    return -torch.logaddexp(-z, torch.zeros_like(z))


def silu(z):
    return z * sigmoid(z)


def squared_relu(z):
    return torch.clamp(z, min=0.0) ** 2


# ---------------------------------------------------------------- positions

def frequencies(base, dims, dtype=torch.float64):
    return torch.tensor([base ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=torch.float64).to(dtype)


def turn_neighbours(x, positions, base, dims):
    """x `[T, heads, n]`: elements 2i and 2i + 1 of the first `dims` turned by position * base^(-2i/dims)."""
    out = x.clone()
    f = frequencies(base, dims, x.dtype)
    for i in range(dims // 2):
        a = (positions.to(x.dtype) * f[i])[:, None]
        u, v = x[:, :, 2 * i], x[:, :, 2 * i + 1]
        out[:, :, 2 * i] = u * torch.cos(a) - v * torch.sin(a)
        out[:, :, 2 * i + 1] = v * torch.cos(a) + u * torch.sin(a)
    return out


def turn_halves(x, positions, base, dims):
    """The same with element i paired with i + dims / 2."""
    out = x.clone()
    f = frequencies(base, dims, x.dtype)
    half = dims // 2
    for i in range(half):
        a = (positions.to(x.dtype) * f[i])[:, None]
        u, v = x[:, :, i], x[:, :, i + half]
        out[:, :, i] = u * torch.cos(a) - v * torch.sin(a)
        out[:, :, i + half] = v * torch.cos(a) + u * torch.sin(a)
    return out


# ---------------------------------------------------------------- mechanisms over time

def attend(q, k, v, scale, window=None, one_more=False):
    """q `[T, H, n]`, k `[T, G, n]`, v `[T, G, v]`, query by query: softmax over the keys j <= i (and i - j < window);
    with `one_more` the denominator also holds a 1, a term of score 0 that stands for no token."""
    t, heads, _ = q.shape
    per = heads // k.shape[1]
    out = torch.zeros(t, heads, v.shape[2], dtype=q.dtype)
    for i in range(t):
        first = 0 if window is None else max(0, i - window + 1)
        for h in range(heads):
            s = (k[first:i + 1, h // per] @ q[i, h]) * scale
            top = s.max()
            if one_more:
                top = torch.clamp(top, min=0.0)
            e = torch.exp(s - top)
            total = e.sum() + (torch.exp(-top) if one_more else 0.0)
            out[i, h] = (e / total) @ v[first:i + 1, h // per]
    return out


def decaying_memory(q, k, v, log_decay):
    """q, k and log_decay `[T, H, n]`, v `[T, H, v]`: S `[n, v]` a head from zero, S_t = diag(e^log_decay_t) S_(t-1) +
    k_t v_t^T, o_t = S_t^T q_t. (A decay a head: the same number in all n places.)"""
    t, heads, n = q.shape
    s = torch.zeros(heads, n, v.shape[2], dtype=q.dtype)
    out = torch.zeros_like(v)
    for i in range(t):
        s = torch.exp(log_decay[i])[:, :, None] * s + k[i][:, :, None] * v[i][:, None, :]
        out[i] = (s * q[i][:, :, None]).sum(1)
    return out


# ---------------------------------------------------------------- the mixers

def softmax_side(m, w, p, h):
    """Attention without positions, norms, biases or window."""
    t = h.shape[0]
    heads, groups, n, v = m["heads"], m.get("kv_heads", m["heads"]), m["dim"], m["vdim"]
    q = (h @ w[p + "q"].T).view(t, heads, n)
    k = (h @ w[p + "k"].T).view(t, groups, n)
    val = (h @ w[p + "v"].T).view(t, groups, v)
    return attend(q, k, val, m["scale"]).reshape(t, heads * v) @ w[p + "o"].T


def gated_linear_side(m, w, p, h, eps):
    """Gated linear attention: a decay a key channel, sigmoid(z)^(1/tau) with z through a bottleneck."""
    t = h.shape[0]
    heads, n, v = m["heads"], m["dim"], m["vdim"]
    q = (h @ w[p + "q"].T).view(t, heads, n) * n ** -0.5
    k = (h @ w[p + "k"].T).view(t, heads, n)
    val = (h @ w[p + "v"].T).view(t, heads, v)
    z = (h @ w[p + "a1"].T) @ w[p + "a2"].T + w[p + "a2.b"]
    o = decaying_memory(q, k, val, (log_sigmoid(z) / m["tau"]).view(t, heads, n))
    o = (unit_rms(o, eps) * w[p + "norm"]).reshape(t, heads * v)
    return (o * silu(h @ w[p + "g"].T)) @ w[p + "o"].T


def parallel(m, w, p, h, eps):
    return (m["left_scale"] * softmax_side(m["left"], w, p + "left.", h)
            + m["right_scale"] * gated_linear_side(m["right"], w, p + "right.", h, eps))


def attention(m, w, p, h, eps):
    t = h.shape[0]
    heads, groups, n, v = m["heads"], m.get("kv_heads", m["heads"]), m["dim"], m["vdim"]
    q = (h @ w[p + "q"].T + w[p + "q.b"]).view(t, heads, n)
    k = (h @ w[p + "k"].T + w[p + "k.b"]).view(t, groups, n)
    val = (h @ w[p + "v"].T + w[p + "v.b"]).view(t, groups, v)
    at = torch.arange(t)
    q = turn_neighbours(unit_rms(q, eps) * w[p + "q.norm"], at, m["rot"]["base"], m["rot"]["dims"])
    k = turn_neighbours(unit_rms(k, eps) * w[p + "k.norm"], at, m["rot"]["base"], m["rot"]["dims"])
    o = attend(q, k, val, m["scale"], m["mask"]["size"], one_more=True)
    return o.reshape(t, heads * v) @ w[p + "o"].T + w[p + "o.b"]


def retention(m, w, p, h, eps):
    t = h.shape[0]
    heads, n, v = m["heads"], m["dim"], m["vdim"]
    at = torch.arange(t)
    q = turn_halves((h @ w[p + "q"].T).view(t, heads, n), at, m["rot"]["base"], m["rot"]["dims"])
    k = turn_halves((h @ w[p + "k"].T).view(t, heads, n), at, m["rot"]["base"], m["rot"]["dims"]) * n ** -0.5
    val = (h @ w[p + "v"].T).view(t, heads, v)
    decay = torch.log(torch.tensor(m["decay"], dtype=torch.float64)).to(h.dtype)
    o = decaying_memory(q, k, val, decay[None, :, None].expand(t, heads, n))
    return (unit_rms(o, eps).reshape(t, heads * v) * silu(h @ w[p + "g"].T)) @ w[p + "o"].T


# ---------------------------------------------------------------- feed-forward

def expert(w, p, h):
    return squared_relu(h @ w[p + "up"].T) @ w[p + "down"].T


def route(z, top):
    """z `[T, E]` router logits -> (chosen `[T, top]`, weights): the largest logits (the lower number where two are
    equal), weighted by the softmax over the chosen ones alone."""
    chosen = torch.tensor([sorted(range(z.shape[1]), key=lambda e: (-float(row[e]), e))[:top] for row in z])
    picked = torch.gather(z, 1, chosen)
    e = torch.exp(picked - picked.max(-1, keepdim=True).values)
    return chosen, e / e.sum(-1, keepdim=True)


def mixture(mlp, w, p, h):
    chosen, weights = route(h @ w[p + "router"].T + w[p + "router.b"], mlp["router"]["top"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for c in range(chosen.shape[1]):
            out[t] += weights[t, c] * expert(w, f"{p}e{int(chosen[t, c])}.", h[t:t + 1])[0]
    if mlp.get("shared") is not None:
        out = out + sigmoid(h @ w[p + "shared.sg"].T) * expert(w, p + "shared.", h)
    return out


# ---------------------------------------------------------------- the model

def mix(kind, m, w, p, h, eps):
    return dict(parallel=parallel, attention=attention, retention=retention)[kind](m, w, p, h, eps)


def forward(cfg, w, tokens, return_layers=False):
    """Logits `[T, vocab]` of one sequence; with `return_layers` also the stream after every layer."""
    eps = cfg["norm"]["eps"]
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    after = []
    for i, layer in enumerate(cfg["layers"]):
        owner = i
        while cfg["layers"][owner].get("weights_of") is not None:
            owner = cfg["layers"][owner]["weights_of"]
        p = f"l{owner}."
        h = centred_norm(x, w[p + "norm1"], eps)
        y = mix(layer["type"], layer["mixer"], w, p + "mix.", h, eps)
        if layer.get("mlp") is not None:
            y = y + mixture(layer["mlp"], w, p + "mlp.", h)
        x = x + y
        after.append(x)
    logits = centred_norm(x, w["final.norm"], eps) @ w["embed"].T
    return (logits, after) if return_layers else logits
