"""Plain float64 definition of the Nolavik design: one function per mechanism, whole sequences, no cache, no batching.

It takes the config as the dictionary a ``config.json`` holds and the weights as a dictionary of checkpoint names, and
shares no code with the framework's model path. Slow on purpose: every function is the equation it stands for.
"""
import math

import torch

F64 = torch.float64


def rms(x, eps):
    return x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps)


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return torch.clamp(z, min=0.0) + torch.log1p(torch.exp(-z.abs()))


def step_angles(dims, base, scaling=None):
    """Angle per position of every pair. ``scaling`` {factor, low, high, original}: pairs whose wavelength is beyond
    original / low turn ``factor`` times slower, those below original / high keep their pace, in between a blend."""
    out = []
    for i in range(dims // 2):
        f = base ** (-2.0 * i / dims)
        if scaling:
            wave = 2.0 * math.pi / f
            turns = scaling["original"] / wave
            if wave > scaling["original"] / scaling["low"]:
                f = f / scaling["factor"]
            elif wave >= scaling["original"] / scaling["high"]:
                s = (turns - scaling["low"]) / (scaling["high"] - scaling["low"])
                f = (1.0 - s) * f / scaling["factor"] + s * f
        out.append(f)
    return out


def rotate_half(x, positions, angles):
    """x [T, heads, n]: number i < len(angles) paired with i + len(angles), turned by position * angles[i]."""
    out = x.clone()
    half = len(angles)
    for i, f in enumerate(angles):
        a = positions.to(F64) * f
        c, s = torch.cos(a)[:, None], torch.sin(a)[:, None]
        u, v = x[..., i], x[..., i + half]
        out[..., i] = u * c - v * s
        out[..., i + half] = v * c + u * s
    return out


def causal_conv(u, w, b=None):
    """u [T, C], w [C, taps]: y_t = sum_j w[:, j] u_(t - taps + 1 + j) (+ b), zeros before the start."""
    T, taps = u.shape[0], w.shape[1]
    full = torch.cat([torch.zeros(taps - 1, u.shape[1], dtype=F64), u])
    y = sum(w[:, j] * full[j:j + T] for j in range(taps))
    return y if b is None else y + b


def causal_attention(q, k, v, scale, sink=False):
    """q [T, H, dim], k [T, G, dim], v [T, G, vdim] -> [T, H, vdim]; ``sink``: one is added to every denominator."""
    T, H, _ = q.shape
    G = k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=F64)
    later = torch.arange(T)[None, :] > torch.arange(T)[:, None]
    for h in range(H):
        g = h // (H // G)
        s = ((q[:, h] @ k[:, g].T) * scale).masked_fill(later, -math.inf)
        m = s.max(-1, keepdim=True).values
        m = m.clamp(min=0.0) if sink else m
        e = torch.exp(s - m)
        out[:, h] = (e @ v[:, g]) / (e.sum(-1, keepdim=True) + (torch.exp(-m) if sink else 0.0))
    return out


def selective_scan(x, dt, A, B, C, D):
    """x, dt [T, inner], A [inner, state], B, C [T, state], D [inner]."""
    S = torch.zeros_like(A)
    out = torch.zeros_like(x)
    for t in range(x.shape[0]):
        S = torch.exp(dt[t][:, None] * A) * S + (dt[t] * x[t])[:, None] * B[t][None, :]
        out[t] = S @ C[t] + D * x[t]
    return out


def delta_rule(q, k, v, beta, g):
    """q, k [T, H, dim], v [T, H, vdim], beta, g [T, H] -> [T, H, vdim]."""
    T, H, dim = q.shape
    S = torch.zeros(H, dim, v.shape[2], dtype=F64)
    out = torch.zeros(T, H, v.shape[2], dtype=F64)
    for t in range(T):
        S = S * g[t, :, None, None]
        u = beta[t, :, None] * (v[t] - (S * k[t, :, :, None]).sum(1))
        S = S + k[t, :, :, None] * u[:, None, :]
        out[t] = (S * q[t, :, :, None]).sum(1)
    return out


def unit(x):
    return x / torch.sqrt(x.pow(2).sum(-1, keepdim=True) + 1e-6)


def route(z, top):
    """The ``top`` largest logits (ties: the lower index), weighted by a softmax over them alone."""
    order = torch.sort(z, dim=-1, descending=True, stable=True).indices[:, :top]
    return order, torch.softmax(torch.gather(z, 1, order), -1)


def expert(W, p, h):
    return (silu(h @ W(p + "gate").T) * (h @ W(p + "up").T)) @ W(p + "down").T


class Weights:
    def __init__(self, sd):
        self.sd = sd

    def __call__(self, name):
        return self.sd[name].to(F64)


def delta_mixer(W, p, m, h, eps):
    T, H, G, dim, vd = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (silu(causal_conv(h @ W(p + n).T, W(p + n + ".conv"))) for n in "qkv")
    rep = H // G
    q = (unit(q.view(T, G, dim)) * dim ** -0.5).repeat_interleave(rep, 1)
    k = unit(k.view(T, G, dim)).repeat_interleave(rep, 1)
    beta = sigmoid(h @ W(p + "b").T)
    g = torch.exp(-torch.exp(W(p + "A_log")) * softplus(h @ W(p + "a").T + W(p + "dt_bias")))
    o = rms(delta_rule(q, k, v.view(T, H, vd), beta, g), eps) * W(p + "norm")
    return (o.reshape(T, H * vd) * silu(h @ W(p + "g").T)) @ W(p + "o").T


def attention_branch(W, p, m, h, eps):
    T, H, G, dim, vd = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    pos = torch.arange(T)
    q, k = (h @ W(p + "q").T).view(T, H, dim), (h @ W(p + "k").T).view(T, G, dim)
    v = (h @ W(p + "v").T).view(T, G, vd)
    r = m.get("rot")
    if r:
        ang = step_angles(r["dims"], r["base"], r.get("scaling"))
        q, k = rotate_half(q, pos, ang), rotate_half(k, pos, ang)
    o = causal_attention(rms(q, eps), rms(k, eps), v, m["scale"], sink=True)
    return o.reshape(T, H * vd) @ W(p + "o").T


def mamba_branch(W, p, m, h):
    inner, N, R = m["inner"], m["state"], m["dt_rank"]
    xz = h @ W(p + "in").T
    x, z = xz[:, :inner], xz[:, inner:]
    x = silu(causal_conv(x, W(p + "conv"), W(p + "conv.b")))
    dbc = x @ W(p + "x").T
    dt = softplus(dbc[:, :R] @ W(p + "dt").T + W(p + "dt.b"))
    y = selective_scan(x, dt, -torch.exp(W(p + "A_log")), dbc[:, R:R + N], dbc[:, R + N:], W(p + "D"))
    return (y * silu(z)) @ W(p + "o").T


def parallel_mixer(W, p, m, h, eps):
    return m["left_scale"] * attention_branch(W, p + "left.", m["left"], h, eps) + \
        m["right_scale"] * mamba_branch(W, p + "right.", m["right"], h)


def latent_mixer(W, p, m, h, eps):
    T, H, dim, rd, vd, R = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    pos = torch.arange(T)
    cq = rms(h @ W(p + "dq").T, eps) * W(p + "dq.norm")
    q = (cq @ W(p + "uq").T).view(T, H, dim + rd)
    down = h @ W(p + "dkv").T
    c = rms(down[:, :R], eps) * W(p + "dkv.norm")
    ang = step_angles(rd, m["rot"]["base"])
    kr = rotate_half(down[:, R:].view(T, 1, rd), pos, ang).expand(T, H, rd)
    k = torch.cat([(c @ W(p + "uk").T).view(T, H, dim), kr], -1)
    q = torch.cat([q[..., :dim], rotate_half(q[..., dim:], pos, ang)], -1)
    o = causal_attention(q, k, (c @ W(p + "uv").T).view(T, H, vd), m["scale"])
    return o.reshape(T, H * vd) @ W(p + "o").T


def moe(W, p, f, h):
    idx, w = route(h @ W(p + "router").T + W(p + "router.b"), f["router"]["top"])
    out = torch.zeros_like(h)
    for e in range(f["router"]["experts"]):
        share = torch.where(idx == e, w, torch.zeros_like(w)).sum(-1, keepdim=True)
        out = out + share * expert(W, f"{p}e{e}.", h)
    if f.get("shared"):
        out = out + sigmoid(h @ W(p + "shared.sg").T) * expert(W, p + "shared.", h)
    return out


def mixer(W, p, L, h, eps):
    m = L["mixer"]
    if L["type"] == "delta":
        return delta_mixer(W, p, m, h, eps)
    if L["type"] == "parallel":
        return parallel_mixer(W, p, m, h, eps)
    return latent_mixer(W, p, m, h, eps)


def layer_order(cfg):
    """(layer, pass) of every layer run; pass is None outside the repeated stretch."""
    n, lp = len(cfg["layers"]), cfg.get("loop")
    if not lp:
        return [(i, None) for i in range(n)]
    a, b = lp["start"], lp["stop"]
    return [(i, None) for i in range(a)] + [(i, t) for t in range(lp["times"]) for i in range(a, b)] + \
        [(i, None) for i in range(b, n)]


def forward(cfg, sd, tokens, tap=None):
    """Logits [T, vocab] of the token list; ``tap(run, x)`` sees the residual after every layer run."""
    W, eps = Weights(sd), cfg["norm"]["eps"]
    x = W("embed")[torch.as_tensor(tokens)]
    for r, (i, t) in enumerate(layer_order(cfg)):
        p, L = f"l{i}.", cfg["layers"][i]
        if t is not None and i == cfg["loop"]["start"]:
            x = x + W("loop.step")[t]
        x = x + rms(mixer(W, p + "mix.", L, rms(x, eps) * W(p + "norm1"), eps), eps) * W(p + "norm1b")
        if L.get("mlp"):
            x = x + rms(moe(W, p + "mlp.", L["mlp"], rms(x, eps) * W(p + "norm2")), eps) * W(p + "norm2b")
        if tap is not None:
            tap(r, x)
    return (rms(x, eps) * W("final.norm")) @ W("head").T


def greedy(cfg, sd, prompt, n):
    t = list(prompt)
    for _ in range(n):
        t.append(int(forward(cfg, sd, t)[-1].argmax()))
    return t[len(prompt):]
