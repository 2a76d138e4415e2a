"""Plain, slow evaluation of the Deretar design: the oracle of its tests.

One function per mechanism, written from the equations, in float64 by default, one sequence at a
time and without a cache. It takes a parsed config.json (a dict) and a dict of named tensors, and
shares no code with the package.
"""
import math

import torch


def rms(x, eps):
    """x over its root mean square, eps inside the root."""
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def gain_norm(x, w, eps):
    """RMS norm with a plain weight."""
    return rms(x, eps) * w


def centred_norm(x, w, eps):
    """RMS norm whose weight is stored around zero."""
    return rms(x, eps) * (1 + w)


def rotate(x, pos, base, dims):
    """Turn the first ``dims`` entries of x [n, ..., d] by the angles of positions ``pos`` [n];
    entry i goes with entry i + dims / 2."""
    half = dims // 2
    out = x.clone()
    for i in range(half):
        a = pos.to(torch.float64) * base ** (-2.0 * i / dims)
        c, s = torch.cos(a).to(x.dtype), torch.sin(a).to(x.dtype)
        while c.dim() < x.dim() - 1:
            c, s = c.unsqueeze(-1), s.unsqueeze(-1)
        u, v = x[..., i], x[..., i + half]
        out[..., i] = u * c - v * s
        out[..., i + half] = v * c + u * s
    return out


def latents(h, pos, w, m, eps):
    """(c, shared rotated key) of every token: what a cache would hold."""
    d = h @ w["dkv"].T
    c = gain_norm(d[:, :m["kv_rank"]], w["dkv.norm"], eps)
    kr = rotate(d[:, m["kv_rank"]:], pos, m["rot"]["base"], m["rot"]["dims"])
    return c, kr


def queries(h, pos, w, m, eps):
    """(unrotated, rotated) query parts, [n, heads, dim] and [n, heads, rot_dim]."""
    cq = gain_norm(h @ w["dq"].T, w["dq.norm"], eps)
    q = (cq @ w["uq"].T).view(h.shape[0], m["heads"], m["dim"] + m["rot_dim"])
    return q[..., :m["dim"]], rotate(q[..., m["dim"]:], pos, m["rot"]["base"], m["rot"]["dims"])


def softmax_heads(qn, qr, kn, kr, v, scale):
    """Causal softmax attention of every head: qn, kn [n, H, dim], qr [n, H, r], kr [n, r] (one key
    part for all heads), v [n, H, vdim] -> [n, H, vdim]."""
    n, H = qn.shape[:2]
    out = torch.empty(n, H, v.shape[-1], dtype=v.dtype)
    for t in range(H):
        s = (qn[:, t] @ kn[:, t].T + qr[:, t] @ kr.T) * scale
        s = s.masked_fill(torch.ones(n, n, dtype=torch.bool).triu(1), -math.inf)
        out[:, t] = torch.softmax(s, -1) @ v[:, t]
    return out


def latent_attention(h, w, m, eps):
    """The whole mixer on one sequence h [n, width]."""
    n, H = h.shape[0], m["heads"]
    pos = torch.arange(n)
    c, kr = latents(h, pos, w, m, eps)
    qn, qr = queries(h, pos, w, m, eps)
    kn = (c @ w["uk"].T).view(n, H, m["dim"])
    v = (c @ w["uv"].T).view(n, H, m["vdim"])
    o = softmax_heads(qn, qr, kn, kr, v, m["scale"]).reshape(n, H * m["vdim"])
    return (o * torch.sigmoid(h @ w["g"].T)) @ w["o"].T


def clipped_glu(a, b, limit):
    """The gate's and the up projection's outputs -> the down projection's input."""
    g = torch.clamp(a, max=limit)
    u = torch.clamp(b, min=-limit, max=limit)
    return g * torch.sigmoid(1.702 * g) * (u + 1)


def feed_forward(h, w, limit):
    return clipped_glu(h @ w["gate"].T, h @ w["up"].T, limit) @ w["down"].T


def add_normed(x, y, w, ls, eps):
    """A sublayer's result, normed and scaled per element, joins the stream."""
    return x + centred_norm(y, w, eps) * ls


def owner(layers, i):
    """The layer whose tensors layer i uses."""
    while layers[i].get("weights_of") is not None:
        i = layers[i]["weights_of"]
    return i


def run(cfg, tensors, ids, dtype=torch.float64, trail=None):
    """Logits [n, vocab] of one whole sequence; ``trail`` collects the stream after every layer."""
    t = {k: v.to(dtype) for k, v in tensors.items()}
    eps = cfg["norm"]["eps"]
    x = t["embed"][torch.as_tensor(ids).long()] * cfg["embedding"]["scale"]
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{owner(cfg['layers'], i)}."
        sub = {k[len(p):]: v for k, v in t.items() if k.startswith(p)}
        mix = {k[4:]: v for k, v in sub.items() if k.startswith("mix.")}
        x = add_normed(x, latent_attention(x, mix, layer["mixer"], eps), sub["norm1"], sub["ls1"], eps)
        if layer.get("mlp") is not None:
            mlp = {k[4:]: v for k, v in sub.items() if k.startswith("mlp.")}
            x = add_normed(x, feed_forward(x, mlp, layer["mlp"]["limit"]), sub["norm2"], sub["ls2"], eps)
        if trail is not None:
            trail.append(x.clone())
    return centred_norm(x, t["final.norm"], eps) @ t["embed"].T


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
