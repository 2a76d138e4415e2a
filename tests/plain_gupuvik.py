"""Plain, slow evaluation of the Gupuvik design: the oracle of its tests.

One function per mechanism, written from the equations, in float64 by default, one sequence at a
time and token by token where there is a state. It takes a parsed config.json (a dict) and a dict of
named tensors, and shares no code with the package.
"""
import math

import torch


def rms(x, eps):
    """x over its root mean square, eps inside the root."""
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def scalar_norm(x, g, eps):
    """RMS norm whose weight is one number."""
    return rms(x, eps) * g


def gelu(z):
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))


def silu(z):
    return z * torch.sigmoid(z)


# ------------------------------------------------------------------------------ attention
def visible(n, size, keep_first):
    """[n, n]: does row i see key j: the last ``size`` keys up to itself, and the first ones."""
    i, j = torch.arange(n)[:, None], torch.arange(n)[None, :]
    return (j <= i) & ((i - j < size) | (j < keep_first))


def capped(s, cap):
    return cap * torch.tanh(s / cap)


def keys_values(h, w, m):
    """[n, kv_heads, dim] keys and [n, kv_heads, vdim] values of a layer with projections of its own."""
    k = h @ w["k"].T + w["k.b"]
    v = h @ w["v"].T + w["v.b"]
    return k.view(-1, m["kv_heads"], m["dim"]), v.view(-1, m["kv_heads"], m["vdim"])


def attention(h, kv, w, m):
    """The mixer on one sequence h [n, width] over keys and values ``kv`` (its own or another layer's)."""
    n, H = h.shape[0], m["heads"]
    q = (h @ w["q"].T + w["q.b"]).view(n, H, m["dim"])
    k, v = kv
    see = visible(n, m["mask"]["size"], m["mask"]["keep_first"])
    gate = head_gate(h, w)
    out = torch.empty(n, H, m["vdim"], dtype=h.dtype)
    for a in range(H):
        b = a // (H // m["kv_heads"])
        s = (q[:, a] @ k[:, b].T) * m["scale"] * w["temp"][a]
        s = capped(s, m["softcap"]).masked_fill(~see, -math.inf)
        out[:, a] = (torch.softmax(s, -1) @ v[:, b]) * gate[:, a:a + 1]
    return out.reshape(n, -1) @ w["o"].T


def head_gate(h, w):
    return torch.sigmoid(h @ w["g"].T)


# ------------------------------------------------------------------------------ gated delta rule
def short_conv(x, taps):
    """Causal convolution over time per channel: x [n, c], taps [c, t], the last column on the current token."""
    t = taps.shape[1]
    out = torch.zeros_like(x)
    for j in range(t):
        back = t - 1 - j  # how far back this column looks
        if back < x.shape[0]:
            out[back:] += x[:x.shape[0] - back] * taps[:, j]
    return out


def unit_eps(x, eps):
    """x over its length, eps inside the root."""
    return x / torch.sqrt((x * x).sum(dim=-1, keepdim=True) + eps)


def unit(x):
    return unit_eps(x, 1e-6)


def log_decay(h, w, m):
    """Logarithm of the decay of every head's key channels, [n, heads, dim]."""
    z = (h @ w["a1"].T) @ w["a2"].T + w["dt_bias"]
    soft = torch.clamp(z, min=0) + torch.log1p(torch.exp(-z.abs()))
    return -torch.exp(w["A_log"])[None, :, None] * soft.view(-1, m["heads"], m["dim"])


def delta_rule(q, k, v, decay, beta, state=None):
    """One head: q, k [n, dim], v [n, vdim], decay [n, dim], beta [n] -> (outputs [n, vdim], state)."""
    S = torch.zeros(k.shape[1], v.shape[1], dtype=k.dtype) if state is None else state.clone()
    out = torch.empty(k.shape[0], v.shape[1], dtype=k.dtype)
    for t in range(k.shape[0]):
        S = decay[t][:, None] * S
        u = beta[t] * (v[t] - S.T @ k[t])
        S = S + k[t][:, None] * u[None, :]
        out[t] = S.T @ q[t]
    return out, S


def channel_delta(h, w, m, eps):
    """The whole mixer on one sequence h [n, width]."""
    n, H, G = h.shape[0], m["heads"], m["kv_heads"]
    q = silu(short_conv(h @ w["q"].T, w["q.conv"])).view(n, G, m["dim"])
    k = silu(short_conv(h @ w["k"].T, w["k.conv"])).view(n, G, m["dim"])
    v = silu(short_conv(h @ w["v"].T, w["v.conv"])).view(n, H, m["vdim"])
    q, k = unit(q) * m["dim"] ** -0.5, unit(k)
    decay, beta = torch.exp(log_decay(h, w, m)), torch.sigmoid(h @ w["b"].T)
    gate = torch.sigmoid((h @ w["g1"].T) @ w["g2"].T).view(n, H, m["vdim"])
    out = torch.empty(n, H, m["vdim"], dtype=h.dtype)
    for a in range(H):
        b = a // (H // G)
        o, _ = delta_rule(q[:, b], k[:, b], v[:, a], decay[:, a], beta[:, a])
        out[:, a] = rms(o, eps) * w["norm"] * gate[:, a]
    return out.reshape(n, -1) @ w["o"].T


# ------------------------------------------------------------------------------ feed-forward
def dense(h, w):
    return gelu(h @ w["up"].T) @ w["down"].T


def route(z, top):
    """Router logits [n, experts] -> (chosen experts, their weights) [n, top]."""
    best, at = z.sort(dim=-1, descending=True)
    return at[:, :top], torch.softmax(best[:, :top], -1)


def experts(h, w, m):
    at, weight = route(h @ w["router"].T, m["router"]["top"])
    out = torch.zeros_like(h)
    for i in range(h.shape[0]):
        for e, g in zip(at[i].tolist(), weight[i]):
            a = silu(w[f"e{e}.gate"] @ h[i]) * (w[f"e{e}.up"] @ h[i])
            out[i] += g * (w[f"e{e}.down"] @ a)
    return out


def feed_forward(h, w, m):
    return dense(h, w) if m["kind"] == "dense" else experts(h, w, m)


# ------------------------------------------------------------------------------ the model
def residual_gate(h, w, b):
    return torch.sigmoid(h @ w.T + b)


def run(cfg, tensors, ids, dtype=torch.float64, trail=None):
    """Logits [n, vocab] of one whole sequence; ``trail`` collects the stream after every layer."""
    t = {k: v.to(dtype) for k, v in tensors.items()}
    eps = cfg["norm"]["eps"]
    x = t["embed"][torch.as_tensor(ids).long()] * cfg["embedding"]["scale"]
    kv = {}
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        sub = {k[len(p):]: v for k, v in t.items() if k.startswith(p)}
        mix = {k[4:]: v for k, v in sub.items() if k.startswith("mix.")}
        mlp = {k[4:]: v for k, v in sub.items() if k.startswith("mlp.")}
        m = layer["mixer"]
        h = scalar_norm(x, sub["norm1"], eps)
        if layer["type"] == "attention":
            kv[i] = keys_values(h, mix, m) if m.get("kv_from") is None else kv[m["kv_from"]]
            y = attention(h, kv[i], mix, m)
        else:
            y = channel_delta(h, mix, m, eps)
        y = y * residual_gate(h, sub["rg1"], sub["rg1.b"])
        if layer.get("mlp") is not None:
            y = y + feed_forward(h, mlp, layer["mlp"]) * residual_gate(h, sub["rg2"], sub["rg2.b"])
        x = x + y
        if trail is not None:
            trail.append(x.clone())
    return scalar_norm(x, t["final.norm"], eps) @ t["head"].T


def greedy(cfg, tensors, ids, n_new, dtype=torch.float64):
    """Greedy continuation by recomputing the whole sequence: (tokens, gap between the best and the
    second logit at each)."""
    ids, out, gaps = list(ids), [], []
    for _ in range(n_new):
        top = run(cfg, tensors, ids, dtype)[-1].topk(2)
        out.append(int(top.indices[0]))
        gaps.append(float(top.values[0] - top.values[1]))
        ids.append(out[-1])
    return out, gaps
