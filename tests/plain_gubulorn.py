"""A plain, slow rendition of the Gubulorn design on one whole sequence: no cache, no batch, one function per
mechanism, written from the design's equations with torch tensor arithmetic only. It shares no code with the
package and is what the package's parts, kernels and engine are tested against.

A model is `(cfg, w)`: `cfg` the dictionary of its config.json, `w` a dictionary of tensors by checkpoint name.
Everything is computed in the dtype of `w`'s tensors after `widen` (float64 by default).

Notation: T tokens, D the model's width, H heads, G key/value heads (or groups), n the query/key size of a head, v
its value size, N the state size of the state-space mixer, E the experts that have tensors, I the ones that do not.
"""
import math

import torch


def widen(w, dtype=torch.float64):
    return {k: (x.to(dtype) if x.is_floating_point() else x) for k, x in w.items()}


# ---------------------------------------------------------------- norms and activations

def unit_rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def offset_norm(x, weight, eps):
    """The model's norm: unit root mean square, then times 1 + weight (stored around zero)."""
    return unit_rms(x, eps) * (1.0 + weight)


def unit_vector(x):
    """x / sqrt(sum(x^2) + 1e-6) over the last axis."""
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    """ln(1 + e^z)."""
    return torch.logaddexp(z, torch.zeros_like(z))


# ---------------------------------------------------------------- mechanisms over time

def short_conv(x, weight, bias=None):
    """x `[T, C]`, weight `[C, taps]`: y_t = bias + sum_j weight[:, j] x_(t - taps + 1 + j), zeros before the start (the
    last column meets the current token)."""
    taps = weight.shape[1]
    y = torch.zeros_like(x)
    for t in range(x.shape[0]):
        for j in range(taps):
            at = t - taps + 1 + j
            if at >= 0:
                y[t] += weight[:, j] * x[at]
    return y if bias is None else y + bias


def delta_rule(q, k, v, log_decay, beta):
    """q, k `[T, H, n]`, v `[T, H, v]`, log_decay and beta `[T, H]`: with S `[n, v]` a head, from zero,
    S_t = S' + k_t w_t^T where S' = e^log_decay_t S_(t-1) and w_t = beta_t (v_t - S'^T k_t); o_t = S_t^T q_t."""
    t, heads, n = q.shape
    s = torch.zeros(heads, n, v.shape[2], dtype=q.dtype)
    out = torch.zeros_like(v)
    for i in range(t):
        s = s * torch.exp(log_decay[i])[:, None, None]
        u = beta[i][:, None] * (v[i] - torch.einsum("hnv,hn->hv", s, k[i]))
        s = s + torch.einsum("hn,hv->hnv", k[i], u)
        out[i] = torch.einsum("hnv,hn->hv", s, q[i])
    return out


def state_space(x, b, c, log_decay, dt):
    """x `[T, H, v]`, b and c `[T, H, N]`, log_decay and dt `[T, H]`: S <- e^log_decay S + dt b x^T, y = S^T c."""
    t, heads, n = b.shape
    s = torch.zeros(heads, n, x.shape[2], dtype=x.dtype)
    out = torch.zeros_like(x)
    for i in range(t):
        s = s * torch.exp(log_decay[i])[:, None, None] + dt[i][:, None, None] * b[i][:, :, None] * x[i][:, None, :]
        out[i] = torch.einsum("hnv,hn->hv", s, c[i])
    return out


def sink_weights(scores, sink):
    """scores `[H, T, T]` (query i, key j): the weights over j <= i, query by query; the denominator also holds
    exp(sink) of the head, once: a term that stands for no token."""
    out = torch.zeros_like(scores)
    for i in range(scores.shape[1]):
        s = scores[:, i, :i + 1]
        top = torch.maximum(s.max(-1, keepdim=True).values, sink[:, None])
        e = torch.exp(s - top)
        out[:, i, :i + 1] = e / (e.sum(-1, keepdim=True) + torch.exp(sink[:, None] - top))
    return out


def query_temperature(positions, coef, every):
    """1 + coef ln(floor((p + 1) / every) + 1)."""
    return torch.tensor([1.0 + coef * math.log((int(p) + 1) // every + 1.0) for p in positions], dtype=torch.float64)


# ---------------------------------------------------------------- the mixers

def delta(m, w, p, h, eps):
    """The gated delta rule: `m` the mixer's entry of the configuration, `w` the tensors, `p` the prefix, `h` `[T, D]`."""
    t = h.shape[0]
    heads, groups, n, v = m["heads"], m.get("kv_heads", m["heads"]), m["dim"], m["vdim"]
    q = silu(short_conv(h @ w[p + "q"].T, w[p + "q.conv"])).view(t, groups, n)
    k = silu(short_conv(h @ w[p + "k"].T, w[p + "k.conv"])).view(t, groups, n)
    val = silu(short_conv(h @ w[p + "v"].T, w[p + "v.conv"])).view(t, heads, v)
    q, k = unit_vector(q) * n ** -0.5, unit_vector(k)
    share = [head // (heads // groups) for head in range(heads)]
    q, k = q[:, share], k[:, share]
    beta = sigmoid(h @ w[p + "b"].T)
    log_decay = -torch.exp(w[p + "A_log"]) * softplus(h @ w[p + "a"].T + w[p + "dt_bias"])
    o = delta_rule(q, k, val, log_decay, beta)
    o = unit_rms(o, eps) * w[p + "norm"] * silu(h @ w[p + "g"].T).view(t, heads, v)
    return o.reshape(t, heads * v) @ w[p + "o"].T


def attention(m, w, p, h, eps):
    """Softmax attention with a norm a head, a temperature on the queries, a sink and one gate number a head."""
    t = h.shape[0]
    heads, groups, n, v = m["heads"], m.get("kv_heads", m["heads"]), m["dim"], m["vdim"]
    q = unit_rms((h @ w[p + "q"].T).view(t, heads, n), eps) * w[p + "q.norm"]
    k = unit_rms((h @ w[p + "k"].T).view(t, groups, n), eps) * w[p + "k.norm"]
    val = (h @ w[p + "v"].T).view(t, groups, v)
    if m.get("q_temp"):
        q = q * query_temperature(range(t), m["q_temp"]["coef"], m["q_temp"]["every"]).to(q.dtype)[:, None, None]
    out = torch.zeros(t, heads, v, dtype=h.dtype)
    for head in range(heads):
        g = head // (heads // groups)
        weights = sink_weights(((q[:, head] @ k[:, g].T) * m["scale"])[None], w[p + "sink"][head:head + 1])[0]
        out[:, head] = weights @ val[:, g]
    out = out * sigmoid(h @ w[p + "g"].T)[:, :, None]
    return out.reshape(t, heads * v) @ w[p + "o"].T


def mamba2(m, w, p, h, eps):
    """The state-space mixer: one projection [z | x | B | C | dt], a convolution over x, B and C together, the
    recurrence, the gate and then the norm in `norm_groups` parts."""
    t = h.shape[0]
    heads, v, n, groups = m["heads"], m["vdim"], m["state"], m["groups"]
    inner, gn = heads * v, groups * n
    proj = h @ w[p + "in"].T
    z, xbc, dt = proj[:, :inner], proj[:, inner:2 * inner + 2 * gn], proj[:, 2 * inner + 2 * gn:]
    xbc = silu(short_conv(xbc, w[p + "conv"], w[p + "conv.b"]))
    x = xbc[:, :inner].view(t, heads, v)
    b = xbc[:, inner:inner + gn].view(t, groups, n)
    c = xbc[:, inner + gn:].view(t, groups, n)
    share = [head // (heads // groups) for head in range(heads)]
    dt = softplus(dt + w[p + "dt_bias"])
    y = state_space(x, b[:, share], c[:, share], -torch.exp(w[p + "A_log"]) * dt, dt) + w[p + "D"][:, None] * x
    y = y.reshape(t, inner) * silu(z)
    y = unit_rms(y.view(t, m["norm_groups"], -1), eps).reshape(t, inner) * w[p + "norm"]
    return y @ w[p + "o"].T


def parallel(m, w, p, h, eps):
    """Attention and the state-space mixer on the same input: half the sum of the two results, each normed."""
    left = unit_rms(attention(m["left"], w, p + "left.", h, eps), eps) * w[p + "left.out"]
    right = unit_rms(mamba2(m["right"], w, p + "right.", h, eps), eps) * w[p + "right.out"]
    return 0.5 * (left + right)


# ---------------------------------------------------------------- feed-forward

def dense(mlp, w, p, h):
    """With a = W_gate h kept below `limit` and b = W_up h kept inside +-`limit`: W_down (a sigmoid(1.702 a) (b + 1))."""
    g = torch.clamp(h @ w[p + "gate"].T, max=mlp["limit"])
    u = torch.clamp(h @ w[p + "up"].T, min=-mlp["limit"], max=mlp["limit"])
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ w[p + "down"].T


def expert(w, p, h):
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def route(z, correction, top, count, keep):
    """z `[T, E + I]` router logits -> (chosen `[T, top]`, weights): scores softmax(z), choice scores with the
    correction, the `keep` best of `count` groups of neighbours (by their largest choice score), within them the
    `top` largest choice scores; weights are the scores without the correction. Lower numbers where two are equal."""
    s = torch.softmax(z, dim=-1)
    choice = s + correction
    per = z.shape[1] // count
    chosen = torch.zeros(z.shape[0], top, dtype=torch.long)
    for t in range(z.shape[0]):
        best = [float(choice[t, g * per:(g + 1) * per].max()) for g in range(count)]
        kept = sorted(range(count), key=lambda g: (-best[g], g))[:keep]
        allowed = [e for g in sorted(kept) for e in range(g * per, (g + 1) * per)]
        chosen[t] = torch.tensor(sorted(allowed, key=lambda e: (-float(choice[t, e]), e))[:top])
    return chosen, torch.gather(s, 1, chosen)


def mixture(mlp, w, p, h):
    r = mlp["router"]
    groups = r.get("groups") or dict(count=1, keep=1)
    chosen, weights = route(h @ w[p + "router"].T, w[p + "correction"], r["top"], groups["count"], groups["keep"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for c in range(r["top"]):
            e = int(chosen[t, c])
            out[t] += weights[t, c] * (expert(w, f"{p}e{e}.", h[t:t + 1])[0] if e < r["experts"] else h[t])
    return out


# ---------------------------------------------------------------- the model

MIXERS = dict(delta=delta, parallel=parallel)


def forward(cfg, w, tokens, return_layers=False):
    """Logits `[T, vocab]` of one sequence; with `return_layers` also the stream after every layer."""
    eps, alpha = cfg["norm"]["eps"], cfg["postln_alpha"]
    x = offset_norm(w["embed"][torch.as_tensor(tokens, dtype=torch.long)], w["embed.norm"], eps)
    after = []
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        x = offset_norm(alpha * x + MIXERS[layer["type"]](layer["mixer"], w, p + "mix.", x, eps), w[p + "norm1"], eps)
        mlp = layer.get("mlp")
        if mlp is not None:
            ff = dense(mlp, w, p + "mlp.", x) if mlp["kind"] == "dense" else mixture(mlp, w, p + "mlp.", x)
            x = offset_norm(alpha * x + ff, w[p + "norm2"], eps)
        after.append(x)
    logits = (offset_norm(x, w["final.norm"], eps) @ w["head"].T) * cfg.get("logit_scale", 1.0)
    if cfg.get("logit_softcap"):
        logits = cfg["logit_softcap"] * torch.tanh(logits / cfg["logit_softcap"])
    return (logits, after) if return_layers else logits
