"""Each mechanism of the Tefudra design alone: the framework's op (CPU definition, and on a GPU box the HIP kernel in fp32
and bf16 storage) against the plain float64 function in tefudra_oracle.py, over scattered pages, state slots that held
something else before, portions cut at awkward places, and inputs built so that a fault shows: a key whose score stands out
placed at page borders, just inside and just outside the window, among and just behind the kept first positions; a sink
that takes most of a row's weight; an expert nobody chooses and tokens that choose identity experts only."""
import math

import pytest
import torch

import tefudra_oracle as oracle
from llmss_amd import ops
from test_fizelix_ops import RUNS, Pages, close, i32, meta, rnd, steps_of

F64 = torch.float64
BF = torch.bfloat16


def to(t, device, dtype=torch.float32):
    return None if t is None else t.to(device=device, dtype=dtype).contiguous()


# ------------------------------------------------------------------------------------------- the block's closing ops
@pytest.mark.parametrize("device,dtype", RUNS)
@pytest.mark.parametrize("W,groups", [(48, 1), (48, 3), (56, 8), (54, 2), (45, 5), (520, 4), (1032, 1)])
def test_closing_op_with_norms_in_parts(device, dtype, W, groups):
    T, eps = 6, 1e-5
    x, y = rnd(T, W, seed=1, mul=2.0), rnd(T, W, seed=2, dtype=dtype)
    y[:, : W // groups] *= 4.0  # parts of different size: a norm over the whole row would differ
    y = y.to(dtype).double()
    post, nxt = 1 + 0.2 * rnd(W, seed=3), 1 + 0.2 * rnd(W, seed=4)
    want = x + oracle.group_norm(y, post, groups, eps)
    xs = to(x, device)
    got = ops.sandwich_add_norm(xs, to(y, device, dtype), None, None, to(post, device), eps, None, to(nxt, device), dtype,
                                groups)
    close(xs, want, torch.float32, "residual")
    close(got, oracle.group_norm(want, nxt, groups, eps), dtype, "next input")
    got = ops.sandwich_add_norm(to(x, device), None, None, None, None, eps, None, to(nxt, device), dtype, groups)
    close(got, oracle.group_norm(x, nxt, groups, eps), dtype, "norm alone")
    if groups > 1:
        assert float((oracle.group_norm(y, post, groups, eps) - oracle.group_norm(y, post, 1, eps)).abs().max()) > 0.1


@pytest.mark.parametrize("device,dtype", RUNS)
@pytest.mark.parametrize("W,groups", [(48, 1), (54, 3), (520, 2)])
def test_closing_op_joins_two_mixers(device, dtype, W, groups):
    T, eps = 5, 1e-5
    x, l, r = rnd(T, W, seed=1), rnd(T, W, seed=2, dtype=dtype, mul=5.0), rnd(T, W, seed=3, dtype=dtype, mul=0.2)
    wl, wr, post, nxt = (1 + 0.3 * rnd(W, seed=s) for s in (4, 5, 6, 7))
    joined = 0.5 * (oracle.rms(l, eps) * wl + oracle.rms(r, eps) * wr)
    want = x + oracle.group_norm(joined, post, groups, eps)
    xs = to(x, device)
    # the two results are columns of wider rows
    wide = torch.zeros(T, 2 * W + 8, dtype=dtype, device=device)
    wide[:, :W], wide[:, W + 8:] = to(l, device, dtype), to(r, device, dtype)
    pair = ops.PairPending(wide[:, :W], wide[:, W + 8:], to(wl, device), to(wr, device))
    got = ops.sandwich_add_norm(xs, pair, None, None, to(post, device), eps, None, to(nxt, device), dtype, groups)
    close(xs, want, torch.float32, "residual")
    close(got, oracle.group_norm(want, nxt, groups, eps), dtype, "next input")


# ------------------------------------------------------------------------------------------------- projections
@pytest.mark.parametrize("device,dtype", RUNS)
@pytest.mark.parametrize("M,N,K", [(3, 24, 32), (70, 40, 48), (5, 12, 20), (600, 136, 64)])
@pytest.mark.parametrize("act", ["none", "gelu", "relu2"])
def test_projection_with_bias_and_activation(device, dtype, M, N, K, act):
    x, w, b = rnd(M, K, seed=1, dtype=dtype), rnd(N, K, seed=2, dtype=dtype, mul=K ** -0.5), rnd(N, seed=3, dtype=dtype)
    f = {"none": lambda z: z, "gelu": oracle.gelu_erf, "relu2": oracle.relu2}[act]
    for bias in (None, b):
        got = ops.linear_f(to(x, device, dtype), to(w, device, dtype), dtype, bias=to(bias, device, dtype), act=act)
        close(got, f(x @ w.T + (0 if bias is None else bias)), dtype, f"{act} bias {bias is not None}")


# ------------------------------------------------------------------------------------------------- experts
@pytest.mark.parametrize("device,dtype", RUNS)
@pytest.mark.parametrize("E,ident,top", [(4, 2, 2), (3, 1, 4), (6, 0, 1), (9, 5, 3), (2, 30, 2)])
def test_softmax_router_chooses_over_experts_and_identity_experts(device, dtype, E, ident, top):
    T, W = 13, 40
    h, rw = rnd(T, W, seed=1, dtype=dtype), rnd(E + ident, W, seed=2, dtype=dtype, mul=2 * W ** -0.5)
    corr = rnd(E + ident, seed=3, mul=0.3)
    idx, w = oracle.route(h @ rw.T, corr, top)
    gi, gw = ops.moe_router(to(h, device, dtype), to(rw, device, dtype), to(corr, device), top, True, "softmax")
    assert gi.cpu().tolist() == idx.tolist()
    close(gw, w, torch.float32, "weights", slack=5.0)
    z = (h @ rw.T).float()
    gi2, gw2 = ops.moe_route(to(z, device), to(corr, device), top, True, "softmax")  # the form a long prompt takes
    assert gi2.cpu().tolist() == idx.tolist()
    close(gw2, w, torch.float32, "weights", slack=5.0)
    plain = oracle.route(h @ rw.T, torch.zeros(E + ident, dtype=F64), top)[0]
    assert plain.tolist() != idx.tolist()  # the correction decides some choice here


@pytest.mark.parametrize("device,dtype", RUNS)
@pytest.mark.parametrize("E,ident,top,W,F,T", [(4, 2, 2, 48, 24, 11), (3, 3, 3, 50, 17, 9), (2, 1, 1, 64, 160, 700), (2, 1, 2, 264, 328, 1500),
                                                (5, 0, 2, 40, 8, 6)])
@pytest.mark.parametrize("shared", [False, True])
def test_ungated_experts_and_identity_experts(device, dtype, E, ident, top, W, F, T, shared):
    h = rnd(T, W, seed=1, dtype=dtype)
    up, down = rnd(E, F, W, seed=2, dtype=dtype, mul=W ** -0.5), rnd(E, W, F, seed=3, dtype=dtype, mul=F ** -0.5)
    g = torch.Generator().manual_seed(4)
    idx = torch.stack([torch.randperm(E + ident, generator=g)[:top] for _ in range(T)])
    if E > 2:
        idx[idx == 1] = E + ident - 1  # nobody chooses expert 1; some tokens choose the last output more than once
    if ident:
        idx[2] = E  # a token that has identity experts only
    w = torch.rand(T, top, generator=g).double() + 0.1
    sh = rnd(T, W, seed=5, dtype=dtype) if shared else None
    want = torch.zeros(T, W, dtype=F64)
    for t in range(T):
        for j in range(top):
            e = int(idx[t, j])
            want[t] += w[t, j] * (oracle.gelu_erf(h[t] @ up[e].T) @ down[e].T if e < E else h[t])
    want = want + (sh if shared else 0)
    args = (to(h, device, dtype), i32(idx.tolist(), device), to(w, device), None, to(up, device, dtype),
            to(down, device, dtype), 0.0, 0.0)
    kw = dict(shared=to(sh, device, dtype), act="gelu", identity=ident > 0)
    close(ops.moe_experts(*args, **kw), want, dtype, "combined")
    # pending: the sum is formed inside the closing op (the CPU definition hands the finished rows on)
    eps, groups = 1e-5, 2
    post, nxt, x = 1 + 0.1 * rnd(W, seed=6), 1 + 0.1 * rnd(W, seed=7), rnd(T, W, seed=8)
    xs = to(x, device)
    got = ops.sandwich_add_norm(xs, ops.moe_experts(*args, combine=False, **kw), None, None, to(post, device), eps, None,
                                to(nxt, device), dtype, groups)
    xw = x + oracle.group_norm(want, post, groups, eps)
    close(xs, xw, dtype, "residual")
    close(got, oracle.group_norm(xw, nxt, groups, eps), dtype, "next input")


# ------------------------------------------------------------------- heads on their way into the cache, and attention
class Attn:
    """A layer's attention over scattered pages, fed in portions through head_prep_cache and window_attn."""

    def __init__(self, device, dtype, H, G, dim, vdim, scale, window, keep=0, cap=0.0, sink=False, qk_norm=False,
                 shared_kv=False, conv=0, v_norm=False, rot=0, base=100.0, rotv=False, bs=16, seed=0, q_storage=True):
        self.__dict__.update(locals())
        n = H * dim + G * dim + (0 if shared_kv else G * vdim)
        self.cols = n
        self.qw = 1 + 0.3 * rnd(dim, seed=seed + 1) if qk_norm else None
        self.kw = 1 + 0.3 * rnd(dim, seed=seed + 2) if qk_norm else None
        self.sinks = rnd(H, seed=seed + 3, mul=1.5) if sink else None
        self.w = rnd(n, conv, seed=seed + 4, dtype=dtype, mul=conv ** -0.5) if conv else None
        self.eps = 1e-5

    def want(self, proj):
        """[T, H * vdim] of a whole sequence's projection rows."""
        T, H, G, dim, vdim = proj.shape[0], self.H, self.G, self.dim, self.vdim
        pos = torch.arange(T)
        u = oracle.causal_conv(proj, self.w) if self.conv else proj
        q, k = u[:, :H * dim].reshape(T, H, dim), u[:, H * dim:(H + G) * dim].reshape(T, G, dim)
        v = k if self.shared_kv else u[:, (H + G) * dim:].reshape(T, G, vdim)
        if self.qk_norm:
            q, k = oracle.rms(q, self.eps) * self.qw, oracle.rms(k, self.eps) * self.kw
        if self.v_norm:
            v = oracle.rms(v, self.eps)
        if self.rot:
            q, k = (oracle.rotate_half(x, pos, self.rot, self.base) for x in (q, k))
        if self.rotv:
            v = oracle.rotate_half(v, pos, vdim, self.base)
        k, v = k.to(self.dtype).double(), v.to(self.dtype).double()  # as the cache holds them
        o = oracle.softmax_attention(q, k, v, self.scale, self.window, self.keep, self.cap, self.sinks)
        if self.rotv:
            o = oracle.rotate_half(o, pos, vdim, self.base, sign=-1.0)
        return o.reshape(T, -1)

    def run(self, seqs, cuts, split=True, num_decode=True, slots=None):
        """Feed the sequences' rows in portions; returns the results per sequence."""
        dev, dt, H, G, dim, vdim = self.device, self.dtype, self.H, self.G, self.dim, self.vdim
        pg = Pages([len(s) for s in seqs], self.bs, dev, seed=5)
        kc = torch.full((pg.blocks, self.bs, G * dim), 7.0, dtype=dt, device=dev)
        vc = torch.full((pg.blocks, self.bs, G * vdim), 7.0, dtype=dt, device=dev)
        slots = slots or list(range(len(seqs)))
        tail = torch.full((max(slots) + 1, max(self.conv - 1, 0), self.cols), 3.0, device=dev)
        f = lambda d: torch.tensor([self.base ** (-2.0 * i / d) for i in range(d // 2)], dtype=torch.float32, device=dev)
        got = [[] for _ in seqs]
        for step in steps_of(cuts):
            step = sorted(step, key=lambda e: not (e[2] == 1 and e[1] > 0))  # single rows first
            nd = sum(1 for e in step if e[2] == 1 and e[1] > 0) if num_decode else 0
            cu, ctx, ss = meta(step, slots, dev)
            ql = max(n for _, _, n in step)
            rows = torch.cat([seqs[s][p0:p0 + n] for s, p0, n in step])
            # the columns sit in a wider projection
            proj = torch.zeros(rows.shape[0], self.cols + 16, dtype=dt, device=dev)
            proj[:, 8:8 + self.cols] = rows.to(dev, dt)
            pos = torch.cat([torch.arange(p0, p0 + n) for _, p0, n in step]).to(dev)
            sl = torch.tensor([x for s, p0, n in step for x in pg.slots(s, p0, n)], dtype=torch.int64, device=dev)
            cs = ops.rope_angles(pos, f(self.rot)) if self.rot else None
            vcs = ops.rope_angles(pos, f(vdim)) if self.rotv else None
            ok = 8 + H * dim
            q = ops.head_prep_cache(proj, 8, ok, ok if self.shared_kv else ok + G * dim,
                                    to(self.w.t(), dev, dt) if self.conv else None, tail if self.conv > 1 else None,
                                    to(self.qw, dev), to(self.kw, dev), self.v_norm, self.eps, cs, vcs, kc, vc, sl, H, G,
                                    dim, vdim, cu, ctx, ss, single=ql == 1,
                                    q_dtype=ops.window_q_dtype(kc, dim, vdim) if self.q_storage else torch.float32)
            y = ops.window_attn(q, kc, vc, pg.bt([s for s, _, _ in step]), cu, ctx, H, G, dim, vdim, self.scale, self.cap,
                                self.window, self.keep, to(self.sinks, dev), vcs, dt, max_qlen=ql,
                                num_decode=nd if nd < len(step) else 0,
                                max_ctx=max(len(s) for s in seqs) if split else 0)
            at = 0
            for s, _, n in step:
                got[s].append(y[at:at + n])
                at += n
        return [torch.cat(g) for g in got]

    def rows(self, T, seed):
        return rnd(T, self.cols, seed=seed, dtype=self.dtype)


SHAPES = {
    # the attention mixer: shared keys and values, query / key norm, partial rotation, kept positions, sinks
    "kept": dict(H=4, G=2, dim=12, vdim=12, scale=0.4, window=9, keep=3, sink=True, qk_norm=True, shared_kv=True, rot=8),
    "kept_mfma": dict(H=6, G=2, dim=40, vdim=40, scale=0.25, window=21, keep=5, sink=True, qk_norm=True, shared_kv=True,
                      rot=40),
    "kept_wide": dict(H=4, G=1, dim=128, vdim=128, scale=0.15, window=70, keep=17, sink=True, qk_norm=True,
                      shared_kv=True, rot=32),
    # the pair's left side: bias-free here, convolution, value norm, rotated values, soft cap
    "turned": dict(H=4, G=2, dim=8, vdim=12, scale=0.5, window=7, cap=3.0, conv=4, v_norm=True, rot=6, rotv=True),
    "turned_mfma": dict(H=4, G=4, dim=32, vdim=64, scale=0.3, window=33, cap=5.0, conv=2, v_norm=True, rot=32, rotv=True),
    "turned_wide": dict(H=8, G=2, dim=64, vdim=128, scale=0.2, window=50, cap=8.0, conv=3, v_norm=True, rot=16, rotv=True),
    "turned_odd": dict(H=3, G=3, dim=10, vdim=6, scale=0.5, window=5, cap=2.0, conv=6, v_norm=True, rot=10, rotv=True, bs=4),
    # nothing optional: no window, no rotation, one tap
    "bare": dict(H=2, G=1, dim=16, vdim=24, scale=0.3, window=0, conv=1),
    "window_of_one": dict(H=2, G=2, dim=8, vdim=8, scale=0.3, window=1, keep=1, sink=True, qk_norm=True, shared_kv=True),
}


@pytest.mark.parametrize("device,dtype", RUNS)
@pytest.mark.parametrize("name", list(SHAPES))
def test_attention_over_portions_and_single_rows(device, dtype, name):
    a = Attn(device, dtype, **SHAPES[name])
    T = 75
    x = a.rows(T, 11)
    want = a.want(x)
    for cuts in ([T], [2, 2, 3, 16, 15, 17, 2, 1, 1, 16], [1] * 6 + [40] + [1] * 29):
        close(a.run([x], [cuts], slots=[2])[0], want, dtype, f"cuts {cuts}")
    close(a.run([x], [[60] + [1] * 15], split=False)[0], want, dtype, "single rows without the key split")
    a.q_storage = False  # fp32 queries, split into two numbers on the matrix cores
    close(a.run([x], [[60] + [1] * 15])[0], want, dtype, "fp32 queries")


@pytest.mark.parametrize("device,dtype", RUNS)
@pytest.mark.parametrize("name", ["kept_mfma", "turned", "turned_wide"])
def test_attention_over_unequal_sequences_in_one_step(device, dtype, name):
    a = Attn(device, dtype, **SHAPES[name])
    xs = [a.rows(n, 20 + n) for n in (50, 23, 9, 64)]
    cuts = [[17, 1, 1, 31], [2, 5, 16], [9], [1, 60, 1, 1, 1]]
    got = a.run(xs, cuts, slots=[3, 0, 2, 1])
    for i, x in enumerate(xs):
        close(got[i], a.want(x), dtype, f"sequence {i}")


@pytest.mark.parametrize("device,dtype", RUNS)
@pytest.mark.parametrize("dim,bs", [(16, 16), (12, 16), (64, 8)])
def test_one_key_that_stands_out_at_every_edge(device, dtype, dim, bs):
    """A single key answers the query: its value must come back whole where it is seen (inside the window, among the kept
    positions) and not at all where it is not (just outside the window, just behind the kept positions)."""
    window, keep, T = 33, 5, 150
    a = Attn(device, dtype, H=2, G=1, dim=dim, vdim=dim, scale=1.0, window=window, keep=keep, sink=True, bs=bs)
    a.sinks = torch.tensor([0.0, -2.0], dtype=F64)
    row = 140
    for pos in (0, 4, 5, 6, 15, 16, 17, row - window - 1, row - window, row - window + 1, row - window + 2, 127, 128, 139, 140):
        x = torch.zeros(T, a.cols, dtype=F64)
        x[row, :2 * dim] = 6.0  # the queries of both heads at the asking row
        x[pos, 2 * dim:3 * dim] = 5.0  # the key
        x[pos, 3 * dim:] = 2.0  # its value
        x = x.to(dtype).double()
        want = a.want(x)
        seen = row - pos < window or pos < keep
        assert bool(want[row].min() > 1.99) == seen and (seen or float(want[row].abs().max()) == 0.0)
        for cuts in ([T], [row] + [1] * (T - row), [row - 1, 2, T - row - 1]):
            got = a.run([x], [cuts])[0]
            close(got[row], want[row], dtype, f"key at {pos}, cuts {cuts[:3]}", scale=2.0)
            close(got, want, dtype, f"key at {pos}", scale=2.0)


@pytest.mark.parametrize("device,dtype", RUNS)
def test_sinks_take_their_share(device, dtype):
    """Sinks from hardly there to dominant; without them the first row would return its value whole."""
    a = Attn(device, dtype, H=4, G=2, dim=16, vdim=16, scale=0.3, window=12, sink=True)
    a.sinks = torch.tensor([-20.0, 0.0, 3.0, 8.0], dtype=F64)
    x = a.rows(40, 3)
    want = a.want(x)
    close(a.run([x], [[25] + [1] * 15])[0], want, dtype, "sinks")
    v0 = x[0, 6 * 16:].view(2, 16)
    assert float((want[0].view(4, 16)[0] - v0[0]).abs().max()) < 1e-6 and float(want[0].view(4, 16)[3].abs().max()) < 0.02


@pytest.mark.parametrize("device,dtype", RUNS)
def test_rows_without_a_page_slot_are_not_cached(device, dtype):
    a = Attn(device, dtype, H=2, G=1, dim=8, vdim=8, scale=0.3, window=0, conv=2, v_norm=True, rot=4, rotv=True)
    x = to(a.rows(3, 1), device, dtype)
    kc = torch.full((2, 4, 8), 7.0, dtype=dtype, device=device)
    vc, tail = kc.clone(), torch.zeros(3, 1, a.cols, device=device)
    cs = ops.rope_angles(torch.arange(3, device=device), torch.ones(2, device=device))
    vcs = ops.rope_angles(torch.arange(3, device=device), torch.ones(4, device=device))
    ops.head_prep_cache(x, 0, 16, 24, to(a.w.t(), device, dtype), tail, None, None, True, 1e-5, cs, vcs, kc, vc,
                        torch.tensor([5, -1, 2], device=device), 2, 1, 8, 8, i32([0, 3], device), i32([3], device),
                        i32([1], device))
    untouched = [i for i in range(8) if i not in (5, 2)]
    assert bool((kc.view(8, 8)[untouched] == 7).all()) and bool((vc.view(8, 8)[untouched] == 7).all())
    assert bool((kc.view(8, 8)[[5, 2]] != 7).any(1).all())


# ------------------------------------------------------------------------------- matrix memory with exponential gates
class Memory:
    def __init__(self, device, dtype, H, dim, vdim, cap=8.0, seed=0, fb=2.0):
        self.__dict__.update(locals())
        self.w = 1 + 0.2 * rnd(H * vdim, seed=seed + 1, dtype=dtype)
        self.w = self.w.to(dtype).double()
        self.bi, self.bf = rnd(H, seed=seed + 2), fb + rnd(H, seed=seed + 3)
        self.n = 2 * H * dim + 2 * H * vdim + 2 * H
        self.eps = 1e-5

    def rows(self, T, seed):
        return rnd(T, self.n, seed=seed, dtype=self.dtype)

    def parts(self, x):
        H, dim, vdim = self.H, self.dim, self.vdim
        return torch.split(x, [H * dim, H * dim, H * vdim, H * vdim, H, H], -1)

    def want(self, x):
        q, k, v, g, zi, zf = self.parts(x)
        T, H = x.shape[0], self.H
        i, f = oracle.log_gates(zi + self.bi, zf + self.bf, self.cap)
        o = oracle.mlstm(q.view(T, H, -1) * self.dim ** -0.5, k.view(T, H, -1), v.view(T, H, -1), i, f)
        return oracle.rms(o, self.eps).reshape(T, -1) * self.w * torch.sigmoid(g)

    def run(self, seqs, cuts, slots=None):
        dev, dt, H, dim, vdim = self.device, self.dtype, self.H, self.dim, self.vdim
        slots = slots or list(range(len(seqs)))
        ns = max(slots) + 1
        S, n, m = (torch.full(s, 2.0, device=dev) for s in ((ns, H, dim, vdim), (ns, H, dim), (ns, H)))  # leftovers
        got = [[] for _ in seqs]
        for step in steps_of(cuts):
            step = sorted(step, key=lambda e: not (e[2] == 1 and e[1] > 0))
            cu, ctx, ss = meta(step, slots, dev)
            rows = torch.cat([seqs[s][p0:p0 + c] for s, p0, c in step]).to(dev, dt)
            wide = torch.zeros(rows.shape[0], -(-self.n // 8) * 8 + 8, dtype=dt, device=dev)
            wide[:, 8:8 + self.n] = rows
            q, k, v, g, zi, zf = self.parts(wide[:, 8:8 + self.n])
            y = ops.mlstm_mix(q, k, v, zi, zf, to(self.bi, dev), to(self.bf, dev), self.cap, S, n, m, cu, ctx, ss, H, dim,
                              vdim, g, to(self.w, dev, dt), self.eps, dt, max_qlen=max(c for _, _, c in step),
                              num_decode=sum(1 for e in step if e[2] == 1 and e[1] > 0))
            at = 0
            for s, _, c in step:
                got[s].append(y[at:at + c])
                at += c
        return [torch.cat(g) for g in got]


@pytest.mark.parametrize("device,dtype", RUNS)
@pytest.mark.parametrize("H,dim,vdim", [(2, 8, 12), (3, 5, 7), (1, 40, 16), (4, 32, 32), (2, 64, 128), (2, 128, 64), (1, 96, 80),
                                        (1, 200, 24)])
def test_exponential_gate_memory(device, dtype, H, dim, vdim):
    a = Memory(device, dtype, H, dim, vdim)
    T = 150
    x = a.rows(T, 5)
    want = a.want(x)
    for cuts in ([T], [2, 3, 64, 1, 63, 2, 1, 1, 13], [100] + [1] * 50, [65, 65, 20]):
        close(a.run([x], [cuts], slots=[1])[0], want, dtype, f"cuts {cuts[:4]}")


@pytest.mark.parametrize("device,dtype", RUNS)
def test_memory_of_unequal_sequences_and_reused_slots(device, dtype):
    a = Memory(device, dtype, 4, 32, 64)
    xs = [a.rows(n, 40 + n) for n in (130, 70, 9, 1)]
    cuts = [[60, 1, 1, 68], [2, 5, 63], [9], [1]]
    got = a.run(xs, cuts, slots=[3, 0, 2, 1])
    for i, x in enumerate(xs):
        close(got[i], a.want(x), dtype, f"sequence {i}")


@pytest.mark.parametrize("device,dtype", RUNS)
@pytest.mark.parametrize("dim,vdim", [(16, 8), (64, 64)])
def test_memory_gates_at_their_ends(device, dtype, dim, vdim):
    """Input gates that jump to the cap and back (the running maximum jumps, later tokens weigh next to nothing), forget gates
    from fully open to fully shut, and a first token whose gate is far below the starting maximum 0."""
    H, T, cap = 2, 140, 6.0
    a = Memory(device, dtype, H, dim, vdim, cap=cap)
    a.bi, a.bf = torch.zeros(H, dtype=F64), torch.zeros(H, dtype=F64)
    x = a.rows(T, 8)
    zi, zf = x[:, -2 * H:-H], x[:, -H:]
    zf[:] = 12.0  # sigmoid(cap tanh(2)): keeps nearly everything
    zi[0] = -30.0
    zi[33], zi[64], zi[100:110] = 40.0, 40.0, -40.0
    zf[20], zf[65, 0], zf[90:92] = -40.0, -40.0, -40.0
    x = x.to(dtype).double()
    want = a.want(x)
    assert math.isfinite(float(want.abs().max()))
    for cuts in ([T], [33, 1, 31, 2, 73], [60] + [1] * 80):
        close(a.run([x], [cuts])[0], want, dtype, f"cuts {cuts[:4]}")


@pytest.mark.parametrize("device,dtype", RUNS)
def test_memory_stays_exact_over_a_long_sequence(device, dtype):
    """A token written early, kept by open forget gates over hundreds of tokens whose own gates are shut."""
    H, dim, vdim, T = 1, 32, 32, 600
    a = Memory(device, dtype, H, dim, vdim, cap=15.0)
    a.bi, a.bf = torch.zeros(H, dtype=F64), torch.zeros(H, dtype=F64)
    x = a.rows(T, 9)
    x[:, -2], x[:, -1] = -6.0, 14.0
    x[3, -2] = 4.0
    x = x.to(dtype).double()
    want = a.want(x)
    gone = x.clone()
    gone[3, -2] = -6.0
    assert float((a.want(gone)[-1] - want[-1]).abs().max()) > 0.05  # the early token still decides the last row
    # (m' = f + m rounds a forget gate of almost 0 against a maximum of 4 at every token, in any 32-bit form)
    for cuts in ([T], [300, 2, 200] + [1] * 98):
        close(a.run([x], [cuts])[0], want, dtype, f"cuts {cuts[:3]}", slack=10.0 if dtype == torch.float32 else 1.0)
