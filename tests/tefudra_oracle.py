"""Plain float64 definition of the Tefudra design: one function per mechanism, whole sequences, no cache, no batching.

It takes the config as the dictionary a ``config.json`` holds and the weights as a dictionary of checkpoint names, and
shares no code with the framework's model path. Slow on purpose: every function is the equation it stands for.
"""
import functools
import math

import torch

F64 = torch.float64


def rms(x, eps):
    return x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps)


def group_norm(x, w, groups, eps):
    """The row in ``groups`` equal consecutive parts, each divided by its own root mean square; then times w."""
    n = x.shape[-1] // groups
    return torch.cat([rms(x[..., g * n:(g + 1) * n], eps) for g in range(groups)], -1) * w


def gelu_erf(z):
    return 0.5 * z * (1.0 + torch.erf(z / math.sqrt(2.0)))


def relu2(z):
    return torch.clamp(z, min=0.0) ** 2


def rotate_half(x, positions, dims, base, sign=1.0):
    """x [T, heads, n]: dimension i < dims / 2 paired with i + dims / 2, turned by sign * position * base^(-2i/dims)."""
    out = x.clone()
    half = dims // 2
    for i in range(half):
        a = sign * positions.to(F64) * base ** (-2.0 * i / dims)
        c, s = torch.cos(a)[:, None], torch.sin(a)[:, None]
        u, v = x[..., i], x[..., i + half]
        out[..., i] = u * c - v * s
        out[..., i + half] = v * c + u * s
    return out


def causal_conv(u, w):
    """u [T, C], w [C, taps]: y_t = sum_j w[:, j] u_(t - taps + 1 + j), zeros before the start."""
    T, taps = u.shape[0], w.shape[1]
    full = torch.cat([torch.zeros(taps - 1, u.shape[1], dtype=F64), u])
    return sum(w[:, j] * full[j:j + T] for j in range(taps))


def visible(i, j, size, keep_first):
    return j <= i and ((not size) or i - j < size or j < keep_first)


@functools.lru_cache(maxsize=64)
def visibility(T, size, keep_first):
    return torch.tensor([[visible(i, j, size, keep_first) for j in range(T)] for i in range(T)])


def softmax_attention(q, k, v, scale, size, keep_first=0, softcap=0.0, sink=None):
    """q [T, H, dim], k [T, G, dim], v [T, G, vdim]. Position i sees j <= i with i - j < size (size 0: all) or j <
    keep_first; scores q . k * scale, soft-capped; the softmax's denominator also holds exp(sink[h])."""
    T, H, _ = q.shape
    G = k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=F64)
    seen = visibility(T, size, keep_first)
    for h in range(H):
        g = h // (H // G)
        s = (q[:, h] @ k[:, g].T) * scale
        if softcap:
            s = softcap * torch.tanh(s / softcap)
        s = torch.where(seen, s, torch.tensor(-math.inf, dtype=F64))
        if sink is not None:  # one more entry in the denominator, without a value
            s = torch.cat([s, sink[h].expand(T, 1)], 1)
        out[:, h] = torch.softmax(s, 1)[:, :T] @ v[:, g]
    return out


def mlstm(q, k, v, i_gate, f_gate):
    """q, k [T, H, dim] (q scaled), v [T, H, vdim], log input gate and log forget gate [T, H] -> o [T, H, vdim]."""
    T, H, dim = q.shape
    S = torch.zeros(H, dim, v.shape[2], dtype=F64)
    n = torch.zeros(H, dim, dtype=F64)
    m = torch.zeros(H, dtype=F64)
    out = torch.zeros(T, H, v.shape[2], dtype=F64)
    for t in range(T):
        mt = torch.maximum(f_gate[t] + m, i_gate[t])
        a, b = torch.exp(f_gate[t] + m - mt), torch.exp(i_gate[t] - mt)
        S = a[:, None, None] * S + b[:, None, None] * k[t][:, :, None] * v[t][:, None, :]
        n = a[:, None] * n + b[:, None] * k[t]
        m = mt
        den = torch.maximum((n * q[t]).sum(-1).abs(), torch.exp(-m)) + 1e-6
        out[t] = (S * q[t][:, :, None]).sum(1) / den[:, None]
    return out


def log_gates(zi, zf, cap):
    """(log input gate, log forget gate) from the gates' projections with their biases added."""
    i = cap * torch.tanh(zi / cap)
    return i, torch.nn.functional.logsigmoid(cap * torch.tanh(zf / cap))


def route(z, correction, top):
    """Scores softmax(z); the ``top`` largest of score + correction chosen (ties: the lower index); weights = chosen
    scores over their sum (+ 1e-20). Returns (indices [T, top], weights [T, top])."""
    s = torch.softmax(z, -1)
    order = torch.sort(s + correction, dim=-1, descending=True, stable=True).indices[:, :top]
    w = torch.gather(s, 1, order)
    return order, w / (w.sum(-1, keepdim=True) + 1e-20)


class Weights:
    def __init__(self, sd):
        self.sd = sd

    def __call__(self, name):
        return self.sd[name].to(F64)

    def has(self, name):
        return name in self.sd


def attention_mixer(W, p, m, h, eps):
    T = h.shape[0]
    H, G, dim = m["heads"], m["kv_heads"], m["dim"]
    pos = torch.arange(T)
    q = (h @ W(p + "q").T).view(T, H, dim)
    k = (h @ W(p + "k").T).view(T, G, dim)
    v = k  # the values are the keys as projected
    q, k = rms(q, eps) * W(p + "q.norm"), rms(k, eps) * W(p + "k.norm")
    rot = m.get("rot")
    if rot:
        q, k = (rotate_half(x, pos, rot["dims"], rot["base"]) for x in (q, k))
    mask = m.get("mask") or {}
    o = softmax_attention(q, k, v, m["scale"], mask.get("size", 0), mask.get("keep_first", 0), sink=W(p + "sink"))
    return o.reshape(T, -1) @ W(p + "o").T


def parallel_left(W, p, a, h, eps):
    T = h.shape[0]
    H, G, dim, vdim = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
    pos = torch.arange(T)

    def proj(n):
        return causal_conv(h @ W(p + n).T + W(p + n + ".b"), W(p + n + ".conv"))
    q, k, v = proj("q").view(T, H, dim), proj("k").view(T, G, dim), proj("v").view(T, G, vdim)
    rot = a["rot"]
    q, k = (rotate_half(x, pos, rot["dims"], rot["base"]) for x in (q, k))
    v = rotate_half(rms(v, eps), pos, vdim, rot["base"])
    o = softmax_attention(q, k, v, a["scale"], (a.get("mask") or {}).get("size", 0), softcap=a.get("softcap", 0.0))
    o = rotate_half(o, pos, vdim, rot["base"], sign=-1.0)
    return o.reshape(T, -1) @ W(p + "o").T + W(p + "o.b")


def parallel_right(W, p, r, h, eps):
    T = h.shape[0]
    H, dim, vdim = r["heads"], r["dim"], r["vdim"]
    q = (h @ W(p + "q").T).view(T, H, dim) * dim ** -0.5
    k, v = (h @ W(p + "k").T).view(T, H, dim), (h @ W(p + "v").T).view(T, H, vdim)
    i, f = log_gates(h @ W(p + "i").T + W(p + "i.b"), h @ W(p + "f").T + W(p + "f.b"), r["gate_cap"])
    o = rms(mlstm(q, k, v, i, f), eps).reshape(T, -1) * W(p + "norm")
    return (o * torch.sigmoid(h @ W(p + "g").T)) @ W(p + "o").T


def parallel_mixer(W, p, m, h, eps):
    left = rms(parallel_left(W, p + "left.", m["left"], h, eps), eps) * W(p + "left.out")
    right = rms(parallel_right(W, p + "right.", m["right"], h, eps), eps) * W(p + "right.out")
    return 0.5 * (left + right)


def expert(W, p, h):
    return gelu_erf(h @ W(p + "up").T) @ W(p + "down").T


def feed_forward(W, p, f, h):
    if f["kind"] == "dense":
        return relu2(h @ W(p + "up").T) @ W(p + "down").T
    r = f["router"]
    idx, w = route(h @ W(p + "router").T, W(p + "correction"), r["top"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for j in range(r["top"]):
            e = int(idx[t, j])
            out[t] += w[t, j] * (expert(W, f"{p}e{e}.", h[t]) if e < r["experts"] else h[t])
    if f.get("shared"):
        out = out + expert(W, p + "shared.", h)
    return out


def owner(layers, i):
    """The layer whose tensors layer i uses."""
    while layers[i].get("weights_of") is not None:
        i = layers[i]["weights_of"]
    return i


def forward(cfg, sd, tokens, layers_out=None):
    """Logits [T, vocab] of a token list; ``layers_out`` (a list) receives the residual after every layer."""
    W = Weights(sd)
    eps, groups = cfg["norm"]["eps"], cfg["norm"].get("groups", 1)
    x = W("embed")[torch.tensor(tokens)]
    for i, L in enumerate(cfg["layers"]):
        p = f"l{owner(cfg['layers'], i)}."

        def norm(n, y):
            return group_norm(y, W(p + n), groups, eps)
        mix = attention_mixer if L["type"] == "attention" else parallel_mixer
        x = x + norm("norm1b", mix(W, p + "mix.", L["mixer"], norm("norm1", x), eps))
        if L.get("mlp"):
            x = x + norm("norm2b", feed_forward(W, p + "mlp.", L["mlp"], norm("norm2", x)))
        if layers_out is not None:
            layers_out.append(x.clone())
    return group_norm(x, W("final.norm"), groups, eps) @ W("embed").T


def greedy(cfg, sd, prompt, n):
    out = list(prompt)
    for _ in range(n):
        out.append(int(forward(cfg, sd, out)[-1].argmax()))
    return out[len(prompt):]
