"""Plain, slow evaluation of the Runidra design: the oracle of its tests.

One function per mechanism, written from the equations, in float64 by default, one sequence at a
time and token by token where there is a state. It takes a parsed config.json (a dict) and a dict of
named tensors, and shares no code with the package.
"""
import math

import torch


def rms(x, eps):
    """x over its root mean square, eps inside the root."""
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def norm(x, w, eps):
    return rms(x, eps) * w


def silu(z):
    return z * torch.sigmoid(z)


def gelu(z):
    """The tanh form."""
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))


def capped(z, cap):
    return cap * torch.tanh(z / cap)


def linear(h, w, name):
    y = h @ w[name].T
    return y + w[name + ".b"] if name + ".b" in w else y


def heads(x, n):
    return x.view(x.shape[0], n, -1)


# ------------------------------------------------------------------------------ streams
def gather(xs, w):
    """What a sublayer reads: the streams [n, s, width] summed with weights."""
    return torch.einsum("nsw,s->nw", xs, w)


def scatter(xs, mix, out, y):
    """Every stream anew from all old ones (mix is [from, to]) and the sublayer's result."""
    return torch.einsum("nsw,st->ntw", xs, mix) + out[None, :, None] * y[:, None]


def leave(xs):
    return xs.sum(1)


# ------------------------------------------------------------------------------ matrix memory
def denominator(nq, m):
    return torch.maximum(nq.abs(), torch.exp(-m)) + 1e-6


def memory(q, k, v, i, f, state=None):
    """One head: q, k [n, dim], v [n, vdim], log gates i and f [n] -> (outputs [n, vdim], state (S, n, m))."""
    if state is None:
        state = (torch.zeros(k.shape[1], v.shape[1], dtype=k.dtype), torch.zeros(k.shape[1], dtype=k.dtype),
                 torch.zeros((), dtype=k.dtype))
    S, z, m = state
    out = torch.empty(k.shape[0], v.shape[1], dtype=k.dtype)
    for t in range(k.shape[0]):
        top = torch.maximum(f[t] + m, i[t])
        keep, add = torch.exp(f[t] + m - top), torch.exp(i[t] - top)
        S = keep * S + add * k[t][:, None] * v[t][None, :]
        z, m = keep * z + add * k[t], top
        out[t] = (S.T @ q[t]) / denominator(z @ q[t], m)
    return out, (S, z, m)


def mlstm(h, w, m, eps):
    n, H = h.shape[0], m["heads"]
    q, k, v = (heads(h @ w[x].T, H) for x in "qkv")
    q = q * m["dim"] ** -0.5
    i = capped(h @ w["i"].T + w["i.b"], m["gate_cap"])
    f = torch.nn.functional.logsigmoid(capped(h @ w["f"].T + w["f.b"], m["gate_cap"]))
    out = torch.stack([rms(memory(q[:, a], k[:, a], v[:, a], i[:, a], f[:, a])[0], eps) for a in range(H)], 1)
    return (out.reshape(n, -1) * w["norm"] * torch.sigmoid(h @ w["g"].T)) @ w["o"].T


# ------------------------------------------------------------------------------ latent attention
def rotate(x, rot):
    """x [n, heads, d] at positions 0..n-1: pairs (2i, 2i + 1) of the first dims turn."""
    n, dims = x.shape[0], rot["dims"]
    rate = torch.tensor([rot["base"] ** (-2 * i / dims) for i in range(dims // 2)], dtype=x.dtype)
    a = torch.arange(n, dtype=x.dtype)[:, None, None] * rate
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    out = x.clone()
    out[..., 0:dims:2] = u * torch.cos(a) - v * torch.sin(a)
    out[..., 1:dims:2] = v * torch.cos(a) + u * torch.sin(a)
    return out


def window(n, size):
    """[n, n]: row i sees key j of the last ``size`` up to itself."""
    i, j = torch.arange(n)[:, None], torch.arange(n)[None, :]
    return (j <= i) & (i - j < size)


def sink_softmax(s, sink):
    """Softmax with exp(sink) in the denominator."""
    top = torch.clamp(s.max(-1, keepdim=True).values, min=float(sink))
    e = torch.exp(s - top)
    return e / (torch.exp(sink - top) + e.sum(-1, keepdim=True))


def latent_attention(h, w, m, eps):
    n, H, D, R, C = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["kv_rank"]
    q = heads(norm(h @ w["dq"].T, w["dq.norm"], eps) @ w["uq"].T, H)
    kv = h @ w["dkv"].T
    c, turned = norm(kv[:, :C], w["dkv.norm"], eps), rotate(kv[:, None, C:], m["rot"])[:, 0]
    k, v = heads(c @ w["uk"].T, H), heads(c @ w["uv"].T, H)
    qr = rotate(q[..., D:], m["rot"])
    see = window(n, m["mask"]["size"])
    out = torch.empty(n, H, m["vdim"], dtype=h.dtype)
    for a in range(H):
        s = (q[:, a, :D] @ k[:, a].T + qr[:, a] @ turned.T) * m["scale"]
        out[:, a] = sink_softmax(s.masked_fill(~see, -math.inf), w["sink"][a]) @ v[:, a]
    return out.reshape(n, -1) @ w["o"].T


def mixer(kind, h, w, m, eps):
    return mlstm(h, w, m, eps) if kind == "mlstm" else latent_attention(h, w, m, eps)


# ------------------------------------------------------------------------------ feed-forward
def unit(h, w, act):
    """W_down (act(W_gate h) * (W_up h))."""
    return linear(act(linear(h, w, "gate")) * linear(h, w, "up"), w, "down")


def route(z, top):
    """Router logits -> (chosen experts, their weights) [n, top]."""
    best = z.sort(-1, descending=True)
    return best.indices[:, :top], torch.softmax(best.values[:, :top], -1)


def _sub(w, p):
    return {k[len(p):]: v for k, v in w.items() if k.startswith(p)}


def experts(h, w, m):
    at, g = route(linear(h, w, "router"), m["router"]["top"])
    out = torch.sigmoid(h @ w["shared.sg"].T) * unit(h, _sub(w, "shared."), silu)
    for e in range(m["router"]["experts"]):
        row, k = (at == e).nonzero(as_tuple=True)
        if row.numel():
            out[row] = out[row] + g[row, k, None] * unit(h[row], _sub(w, f"e{e}."), silu)
    return out


def feed_forward(h, w, m):
    return unit(h, w, gelu) if m["kind"] == "dense" else experts(h, w, m)


# ------------------------------------------------------------------------------ the model
def order(cfg):
    """Layers as they run."""
    n, lp = len(cfg["layers"]), cfg.get("loop")
    if not lp:
        return list(range(n))
    a, b = lp["start"], lp["stop"]
    return list(range(a)) + list(range(a, b)) * lp["times"] + list(range(b, n))


def run(cfg, tensors, ids, dtype=torch.float64, trail=None):
    """Logits [n, vocab] of one whole sequence; ``trail`` collects the sum of the streams after every layer run."""
    t = {k: v.to(dtype) for k, v in tensors.items()}
    eps = cfg["norm"]["eps"]
    xs = t["embed"][torch.as_tensor(ids).long()][:, None].repeat(1, cfg["streams"], 1)
    for i in order(cfg):
        layer, sub = cfg["layers"][i], _sub(t, f"l{i}.")
        y = mixer(layer["type"], norm(gather(xs, sub["hc1.in"]), sub["norm1"], eps), _sub(sub, "mix."), layer["mixer"], eps)
        xs = scatter(xs, sub["hc1.mix"], sub["hc1.out"], y)
        if layer.get("mlp") is not None:
            y = feed_forward(norm(gather(xs, sub["hc2.in"]), sub["norm2"], eps), _sub(sub, "mlp."), layer["mlp"])
            xs = scatter(xs, sub["hc2.mix"], sub["hc2.out"], y)
        if trail is not None:
            trail.append(leave(xs))
    return capped(norm(leave(xs), t["final.norm"], eps) @ t["head"].T * cfg["logit_scale"], cfg["logit_softcap"])


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
