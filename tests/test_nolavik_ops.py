"""Each mechanism of the Nolavik design alone: the framework's op (CPU definition, and on a GPU box the HIP kernel in fp32 and
bf16 storage) against the plain float64 function in nolavik_oracle.py, over scattered pages, state slots that held something
else before, portions cut at awkward places (chunks of 64, pages of 16, two tokens), and inputs built so that a fault shows: a
key whose score stands out placed far back and at page borders, an early token that a state keeps over hundreds, decays and
step sizes at both ends of their range, a sink beside weak and strong keys, router logits decided by the bias."""
import math

import pytest
import torch

import nolavik_oracle as oracle
from llmss_amd import ops
from llmss_amd.models.config import RotarySpec
from llmss_amd.models.weights import _pair_rows
from test_fizelix_ops import RUNS, Pages, close, i32, meta, rnd, steps_of

F64 = torch.float64
BF = torch.bfloat16


def to(t, device, dtype=torch.float32):
    return None if t is None else t.to(device=device, dtype=dtype).contiguous()


# ------------------------------------------------------------------------------------------- the block's closing op
@pytest.mark.parametrize("device,dtype", RUNS)
@pytest.mark.parametrize("W", [48, 50, 264])
def test_closing_op_sums_two_mixers_with_scales(device, dtype, W):
    T, eps = 5, 1e-5
    x, l, r = rnd(T, W, seed=1), rnd(T, W, seed=2, dtype=dtype, mul=5.0), rnd(T, W, seed=3, dtype=dtype, mul=0.7)
    post, nxt, step = 1 + 0.3 * rnd(W, seed=4), 1 + 0.3 * rnd(W, seed=5), rnd(3, W, seed=6)
    want = x + oracle.rms(0.3 * l - 1.7 * r, eps) * post
    wide = torch.zeros(T, 2 * W + 8, dtype=dtype, device=device)  # the two results are columns of wider rows
    wide[:, :W], wide[:, W + 8:] = to(l, device, dtype), to(r, device, dtype)
    pair = ops.PairPending(wide[:, :W], wide[:, W + 8:], None, None, (0.3, -1.7))
    xs = to(x, device)
    got = ops.sandwich_add_norm(xs, pair, None, None, to(post, device), eps, None, to(nxt, device), dtype)
    close(xs, want, torch.float32, "residual")
    close(got, oracle.rms(want, eps) * nxt, dtype, "next input")
    # one vector for every row comes on top (a pass of the repeated stretch begins)
    steps = to(step, device)
    xs = to(x, device)
    got = ops.sandwich_add_norm(xs, pair, None, None, to(post, device), eps, steps[2], to(nxt, device), dtype)
    close(xs, want + step[2], torch.float32, "residual with the pass's vector")
    close(got, oracle.rms(want + step[2], eps) * nxt, dtype, "next input with the pass's vector")
    xs = to(x, device)
    got = ops.sandwich_add_norm(xs, None, None, None, None, eps, steps[1], to(nxt, device), dtype)
    close(xs, x + step[1], torch.float32, "the vector alone")
    close(got, oracle.rms(x + step[1], eps) * nxt, dtype, "norm after the vector alone")


# ------------------------------------------------------------------------------------------------- experts
@pytest.mark.parametrize("device,dtype", RUNS)
@pytest.mark.parametrize("W,T", [(40, 13), (64, 300), (288, 259)])  # (many rows of whole 32s: the matrix cores take bf16)
@pytest.mark.parametrize("E,top,gate", [(4, 2, True), (3, 3, True), (6, 1, False), (70, 5, True), (1, 1, True), (20, 7, False),
                                        (128, 9, False), (127, 70, True)])
def test_router_weighs_the_chosen_logits_alone(device, dtype, E, top, gate, W, T):
    h, rw = rnd(T, W, seed=1, dtype=dtype), rnd(E + gate, W, seed=2, dtype=dtype, mul=2 * W ** -0.5)
    bias = rnd(E, seed=3, mul=2.0)
    bias[0] += 100.0  # a logit far above the others: weights of the rest vanish, and its own logit alone must not overflow
    z = h @ rw.T
    idx, w = oracle.route(z[:, :E] + bias, top)
    want = [w] + ([oracle.sigmoid(z[:, E])] if gate else [])
    for got in (ops.moe_router(to(h, device, dtype), to(rw, device, dtype), None, top, True, "chosen", bias=to(bias, device),
                               gate=gate),
                ops.moe_route(to(z, device), None, top, True, "chosen", bias=to(bias, device), gate=gate)):  # a long prompt's
        assert len(got) == 2 + gate and got[0].cpu().tolist() == idx.tolist()
        for g, x in zip(got[1:], want):
            close(g, x, torch.float32, "weights", slack=5.0)
    if 1 < top < E:
        assert oracle.route(z[:, :E], top)[0].tolist() != idx.tolist()  # the bias decides some choice here
    # logits so low that a softmax over all experts would lose the chosen ones' order
    far = torch.linspace(0, -3000, E).double().repeat(T, 1)
    far[:, 0] = -2950.0
    idx, w = oracle.route(far, top)
    got = ops.moe_route(to(far, device), None, top, True, "chosen")
    assert got[0].cpu().tolist() == idx.tolist()
    close(got[1], w, torch.float32, "far apart")


@pytest.mark.parametrize("device,dtype", RUNS)
@pytest.mark.parametrize("E,top,W,F,T", [(4, 2, 48, 24, 11), (3, 3, 50, 17, 9), (2, 1, 64, 160, 700)])
def test_shared_expert_behind_a_gate(device, dtype, E, top, W, F, T):
    h = rnd(T, W, seed=1, dtype=dtype)
    gate, up = (rnd(E, F, W, seed=s, dtype=dtype, mul=W ** -0.5) for s in (2, 3))
    down = rnd(E, W, F, seed=4, dtype=dtype, mul=F ** -0.5)
    g = torch.Generator().manual_seed(5)
    idx = torch.stack([torch.randperm(E, generator=g)[:top] for _ in range(T)])
    if E > top:
        idx[idx == 1] = 0 if top == 1 else idx[idx == 1]
    w, sg, sh = torch.rand(T, top, generator=g).double(), torch.rand(T, generator=g).double() * 2, rnd(T, W, seed=6, dtype=dtype)
    want = sg[:, None] * sh
    for t in range(T):
        for j in range(top):
            e = int(idx[t, j])
            want[t] += w[t, j] * ((oracle.silu(h[t] @ gate[e].T) * (h[t] @ up[e].T)) @ down[e].T)
    args = (to(h, device, dtype), i32(idx.tolist(), device), to(w, device), to(gate, device, dtype), to(up, device, dtype),
            to(down, device, dtype), 0.0, 0.0)
    kw = dict(shared=to(sh, device, dtype), act="silu", shared_w=to(sg, device))
    close(ops.moe_experts(*args, **kw), want, dtype, "combined")
    eps, post, nxt, x = 1e-5, 1 + 0.1 * rnd(W, seed=7), 1 + 0.1 * rnd(W, seed=8), rnd(T, W, seed=9)
    xs = to(x, device)
    got = ops.sandwich_add_norm(xs, ops.moe_experts(*args, combine=False, **kw), None, None, to(post, device), eps, None,
                                to(nxt, device), dtype)
    xw = x + oracle.rms(want, eps) * post
    close(xs, xw, dtype, "residual")
    close(got, oracle.rms(xw, eps) * nxt, dtype, "next input")


@pytest.mark.parametrize("device,dtype", [RUNS[0], RUNS[2]])
@pytest.mark.parametrize("E,top,W,F,T", [(4, 2, 48, 32, 11), (3, 1, 64, 16, 700), (2, 2, 264, 272, 900), (3, 2, 256, 320, 1500)])
def test_experts_with_interleaved_gate_and_up_rows(device, dtype, E, top, W, F, T):
    """The layout whose epilogue applies the gated SiLU, from single rows to hundreds per expert (the larger cases run the
    256-row products), one expert nobody chooses."""
    h = rnd(T, W, seed=1, dtype=dtype)
    gate, up = (rnd(E, F, W, seed=s, dtype=dtype, mul=W ** -0.5) for s in (2, 3))
    down = rnd(E, W, F, seed=4, dtype=dtype, mul=F ** -0.5)
    g = torch.Generator().manual_seed(5)
    idx = torch.stack([torch.randperm(E, generator=g)[:top] for _ in range(T)])
    if top == 1:
        idx[idx == 1] = 0
    w = torch.rand(T, top, generator=g).double()
    want = torch.zeros(T, W, dtype=F64)
    for e in range(E):
        share = torch.where(idx == e, w, torch.zeros_like(w)).sum(-1, keepdim=True)
        want += share * ((oracle.silu(h @ gate[e].T) * (h @ up[e].T)) @ down[e].T)
    gu = ops.glu_interleave(gate, up, 1)
    assert torch.equal(gu[:, :16], gate[:, :16]) and torch.equal(gu[:, 16:32], up[:, :16])
    got = ops.moe_experts(to(h, device, dtype), i32(idx.tolist(), device), to(w, device), None, to(gu, device, dtype),
                          to(down, device, dtype), 0.0, 0.0, act="silu", interleaved=True)
    close(got, want, dtype, "experts")


@pytest.mark.parametrize("device,dtype", [RUNS[0], RUNS[2]])
@pytest.mark.parametrize("M,N,K", [(2048, 160, 1024), (2100, 1000, 192), (4096, 136, 2064), (2048, 512, 64), (3000, 96, 128)])
def test_narrow_products_of_long_prompts(device, dtype, M, N, K):
    x, w = rnd(M, K, seed=1, dtype=dtype), rnd(N, K, seed=2, dtype=dtype, mul=K ** -0.5)
    for out in (dtype, torch.float32):
        close(ops.linear_f(to(x, device, dtype), to(w, device, dtype), out), x @ w.T, dtype, f"product to {out}")


# ------------------------------------------------------------------------------------------------- convolution
@pytest.mark.parametrize("device,dtype", RUNS)
@pytest.mark.parametrize("C,taps", [(40, 4), (7, 1), (264, 2), (1032, 6)])
def test_convolution_of_single_rows_renews_its_tail(device, dtype, C, taps):
    """Decode steps, where one launch forms the rows and renews the tails, against the portions' form; a slot that held
    something else; a padded row."""
    x, w, b = rnd(30, C, seed=1, dtype=dtype), rnd(C, taps, seed=2, dtype=dtype, mul=taps ** -0.5), rnd(C, seed=3, dtype=dtype)
    want = oracle.silu(oracle.causal_conv(x, w, b))
    for first in (0, 1, 17):
        tail = torch.full((3, taps - 1, C), 9.0, device=device)
        got = []
        for p0, n in ([(0, first)] if first else []) + [(p, 1) for p in range(first, 30)]:
            one = n == 1
            rows = to(x[p0:p0 + n], device, dtype)
            cu, ctx, ss = [0, n], [p0 + n], [1]
            if one:  # a padded row rides along
                rows = torch.cat([rows, rows])
                cu, ctx, ss = [0, 1, 2], [p0 + 1, 0], [1, -1]
            y = ops.causal_conv(rows, to(w, device, dtype), tail, i32(cu, device), i32(ctx, device), i32(ss, device), False, True,
                                dtype, bias=to(b, device, dtype), single=one)
            got.append(y[:n])
        close(torch.cat(got), want, dtype, f"after {first} rows")
        assert bool((tail[0] == 9.0).all()) and bool((tail[2] == 9.0).all())


# ------------------------------------------------------------------------------------------------- rotation
@pytest.mark.parametrize("dims,base,scaling", [(8, 1000.0, None), (32, 1e6, dict(factor=8.0, low=1.0, high=4.0, original=256)),
                                               (64, 500.0, dict(factor=3.0, low=2.0, high=2.5, original=90)),
                                               (16, 40.0, dict(factor=16.0, low=0.5, high=8.0, original=70))])
def test_scaled_angular_steps(dims, base, scaling):
    want = oracle.step_angles(dims, base, scaling)
    rot = RotarySpec(dims, base, llama3=None if scaling is None else tuple(
        float(scaling[n]) for n in ("factor", "low", "high", "original")))
    assert len(rot.steps()) == dims // 2
    assert max(abs(a - b) / b for a, b in zip(rot.steps(), want)) < 1e-12
    plain = oracle.step_angles(dims, base)
    kinds = {"kept" if a == b else "slowed" if abs(a * (scaling or {"factor": 1})["factor"] / b - 1) < 1e-12 else "blended"
             for a, b in zip(want, plain)}
    assert kinds == ({"kept"} if scaling is None else {"kept", "slowed", "blended"})  # every branch is met


def test_partners_become_neighbours_and_scores_stay():
    H, plain, rot, dims, W = 3, 5, 10, 6, 7
    w = rnd(H * (plain + rot), W, seed=1)
    x = rnd(4, W, seed=2)
    a, b = (x @ w.T).view(4, H, -1), (x @ _pair_rows(w, H, plain, rot, dims).T).view(4, H, -1)
    assert torch.equal(a[..., :plain], b[..., :plain]) and torch.equal(a[..., plain + dims:], b[..., plain + dims:])
    for i in range(dims // 2):
        assert torch.equal(b[..., plain + 2 * i], a[..., plain + i])
        assert torch.equal(b[..., plain + 2 * i + 1], a[..., plain + i + dims // 2])


# ------------------------------------------------------------------------------- attention with unit queries and keys
class Attn:
    """The attention branch between its projections, over scattered pages, fed in portions."""

    def __init__(self, device, dtype, H, G, dim, vdim, scale, rot=0, base=100.0, scaling=None, bs=16):
        self.__dict__.update(locals())
        self.cols, self.eps = (H + G) * dim + G * vdim, 1e-5
        self.ang = oracle.step_angles(rot, base, scaling)

    def want(self, proj):
        T, H, G, dim, vdim = proj.shape[0], self.H, self.G, self.dim, self.vdim
        pos = torch.arange(T)
        q, k = proj[:, :H * dim].reshape(T, H, dim), proj[:, H * dim:(H + G) * dim].reshape(T, G, dim)
        q, k = (oracle.rms(oracle.rotate_half(x, pos, self.ang), self.eps) for x in (q, k))  # the rotation first
        v = proj[:, (H + G) * dim:].reshape(T, G, vdim)
        k = k.to(self.dtype).double()  # as the cache holds them
        return oracle.causal_attention(q, k, v, self.scale, sink=True).reshape(T, -1)

    def run(self, seqs, cuts, slots=None, split=True):
        dev, dt, H, G, dim, vdim = self.device, self.dtype, self.H, self.G, self.dim, self.vdim
        pg = Pages([len(s) for s in seqs], self.bs, dev, seed=5)
        kc = torch.full((pg.blocks, self.bs, G * dim), 7.0, dtype=dt, device=dev)
        vc = torch.full((pg.blocks, self.bs, G * vdim), 7.0, dtype=dt, device=dev)
        ones, zero = torch.ones(dim, device=dev), torch.zeros(H, device=dev)
        f = torch.tensor(self.ang, dtype=torch.float32, device=dev)
        got = [[] for _ in seqs]
        for step in steps_of(cuts):
            step = sorted(step, key=lambda e: not (e[2] == 1 and e[1] > 0))  # single rows first
            nd = sum(1 for e in step if e[2] == 1 and e[1] > 0)
            cu, ctx, ss = meta(step, list(range(len(seqs))), dev)
            ql = max(n for _, _, n in step)
            proj = torch.cat([seqs[s][p0:p0 + n] for s, p0, n in step]).to(dev, dt)
            pos = torch.cat([torch.arange(p0, p0 + n) for _, p0, n in step]).to(dev)
            sl = torch.tensor([x for s, p0, n in step for x in pg.slots(s, p0, n)], dtype=torch.int64, device=dev)
            cs = ops.rope_angles(pos, f) if self.rot else None
            q = ops.head_prep_cache(proj, 0, H * dim, (H + G) * dim, None, None, ones, ones, False, self.eps, cs, None, kc, vc,
                                    sl, H, G, dim, vdim, cu, ctx, ss, single=ql == 1, q_dtype=ops.window_q_dtype(kc, dim, vdim))
            y = ops.window_attn(q, kc, vc, pg.bt([s for s, _, _ in step]), cu, ctx, H, G, dim, vdim, self.scale, 0.0, 0, 0,
                                zero, None, dt, max_qlen=ql, num_decode=nd if nd < len(step) else 0,
                                max_ctx=max(len(s) for s in seqs) if split else 0)
            at = 0
            for s, _, n in step:
                got[s].append(y[at:at + n])
                at += n
        return [torch.cat(g) for g in got]


ATTN = {"small": dict(H=4, G=2, dim=8, vdim=12, scale=3.0, rot=6, scaling=dict(factor=4.0, low=1.0, high=3.0, original=64)),
        "mfma": dict(H=6, G=2, dim=48, vdim=56, scale=1.5, rot=24, base=3000.0,
                     scaling=dict(factor=2.0, low=1.0, high=8.0, original=512)),
        "wide": dict(H=4, G=1, dim=128, vdim=64, scale=0.5, rot=128), "one": dict(H=1, G=1, dim=64, vdim=128, scale=0.125),
        "odd": dict(H=3, G=3, dim=10, vdim=7, scale=0.7, rot=10, bs=4)}


@pytest.mark.parametrize("device,dtype", RUNS)
@pytest.mark.parametrize("name", list(ATTN))
def test_unit_query_attention_over_portions_single_rows_and_batches(device, dtype, name):
    a = Attn(device, dtype, **ATTN[name])
    xs = [rnd(n, a.cols, seed=n, dtype=dtype, mul=2.0) for n in (75, 23, 9, 64)]
    want = [a.want(x) for x in xs]
    for cuts in ([75], [2, 2, 3, 16, 15, 17, 2, 1, 1, 16], [1] * 6 + [40] + [1] * 29):
        close(a.run([xs[0]], [cuts])[0], want[0], dtype, f"cuts {cuts}")
    close(a.run([xs[0]], [[60] + [1] * 15], split=False)[0], want[0], dtype, "single rows without the key split")
    got = a.run(xs, [[17, 1, 1, 56], [2, 5, 16], [9], [1, 60, 1, 1, 1]])
    for i in range(4):
        close(got[i], want[i], dtype, f"sequence {i}")


@pytest.mark.parametrize("device,dtype", RUNS)
@pytest.mark.parametrize("dim", [16, 12])
@pytest.mark.parametrize("far", [0, 15, 16, 17, 63, 64, 150, 299])
def test_a_far_key_among_hundreds_and_the_sink(device, dtype, dim, far):
    """Queries point along one key: nearly all of the weight sits there. A head whose scores are far below zero leaves its
    weight to the sink and returns next to nothing."""
    T = 301
    a = Attn(device, dtype, H=2, G=1, dim=dim, vdim=8, scale=1.0, rot=0)
    x = rnd(T, a.cols, seed=far, dtype=dtype)
    key = torch.ones(dim).double()
    x[:, 2 * dim:3 * dim] = torch.tensor([1.0, -1.0] * (dim // 2)).double()  # every other key is orthogonal to the query
    x[far, 2 * dim:3 * dim] = key
    x[-1, :dim], x[-1, dim:2 * dim] = key, -key  # head 0 finds it (score dim), head 1 sees it at -dim
    want = a.want(x)
    v = x[far, 3 * dim:]
    w0 = math.exp(dim) / (math.exp(dim) + T)
    assert float((want[-1, :8] - v).abs().max()) < 3 * (1 - w0) * float(x[:, 3 * dim:].abs().max()) + 1e-3
    for cuts in ([T], [T - 1, 1], [T - 2, 2]):
        close(a.run([x], [cuts])[0], want, dtype, f"cuts {cuts}")
    a.scale = -30.0  # orthogonal keys score 0; with every key along the query, all scores are -30 dim
    y = x.clone()
    y[:, 2 * dim:3 * dim] = key
    y[:, :2 * dim] = key.repeat(2)
    got = a.run([y], [[T - 1, 1]])[0]
    assert float(got.abs().max()) < 1e-6 and float(a.want(y).abs().max()) < 1e-6  # the sink has it all


# ------------------------------------------------------------------------------- latent attention with a query latent
def latent(device, dtype, H, d, r, dv, R, Q, lens, cuts, scale, base=1000.0, bs=16, seed=0, far=None):
    eps = 1e-5
    pg = Pages(lens, bs, device, seed)
    cache = torch.full((pg.blocks, bs, R + r), 5.0, dtype=dtype, device=device)
    uk, uv = (rnd(H * n, R, seed=seed + s, dtype=dtype, mul=R ** -0.5) for n, s in ((d, 50), (dv, 51)))
    uq = rnd(H * (d + r), Q, seed=seed + 52, dtype=dtype, mul=Q ** -0.5)
    nq, nc = ((1 + 0.1 * rnd(n, seed=seed + s)).to(dtype).double() for n, s in ((Q, 53), (R, 54)))
    downs = [rnd(n, Q + R + r, seed=seed + i, dtype=dtype) for i, n in enumerate(lens)]
    ang = oracle.step_angles(r, base)
    f = torch.tensor(ang, dtype=torch.float32, device=device)
    order = _pair_rows(torch.arange(r).double()[:, None], 1, 0, r, r)[:, 0].long()
    uq_p = _pair_rows(uq, H, d, r, r).to(dtype).to(device)
    uk_t = uk.view(H, d, R).transpose(1, 2).contiguous().to(dtype).to(device)
    want = []
    for x in downs:
        T = len(x)
        pos = torch.arange(T)
        cq = oracle.rms(x[:, :Q], eps) * nq
        if far is not None:  # the last rows' queries point along one key
            c = oracle.rms(x[far:far + 1, Q:Q + R], eps) * nc
            x[far, Q + R:] *= 4.0
        c = oracle.rms(x[:, Q:Q + R], eps) * nc
        q = (cq @ uq.T).view(T, H, d + r)
        kr = oracle.rotate_half(x[:, Q + R:].view(T, 1, r), pos, ang).expand(T, H, r)
        k = torch.cat([(c @ uk.T).view(T, H, d), kr], -1)
        q = torch.cat([q[..., :d], oracle.rotate_half(q[..., d:], pos, ang)], -1)
        want.append(oracle.causal_attention(q, k, (c @ uv.T).view(T, H, dv), scale).reshape(T, -1))
    got = [[] for _ in lens]
    for step in steps_of(cuts):
        step = sorted(step, key=lambda e: not (e[2] == 1 and e[1] > 0))
        cu, ctx, _ = meta(step, [0] * len(lens), device)
        rows = torch.cat([downs[s][p0:p0 + n] for s, p0, n in step])
        src = torch.cat([rows[:, :Q + R], rows[:, Q + R:][:, order]], 1).to(dtype).to(device)
        pos = torch.cat([torch.arange(p0, p0 + n) for _, p0, n in step]).to(device)
        sl = torch.tensor([x for s, p0, n in step for x in pg.slots(s, p0, n)], dtype=torch.int64, device=device)
        cq = ops.rms_cols(src, 0, Q, nq.to(dtype).to(device), eps, dtype)
        qs = ops.linear_f(cq, uq_p, dtype)
        qa = ops.head_absorb(qs, uk_t, ops.latent_qa_dtype(cache), extra=r)
        ops.latent_norm_cache(src, Q, R, nc.to(dtype).to(device), eps, cache, sl, r, ops.rope_angles(pos, f), qa, 0, d, q_src=qs)
        single = all(n == 1 for _, _, n in step)
        o = ops.latent_attn(qa, cache, pg.bt([s for s, _, _ in step]), cu, ctx, 0, scale,
                            max_qlen=max(n for _, _, n in step), max_ctx=max(lens) if single else 0)
        y = ops.head_expand(o, uv.to(dtype).to(device), torch.float32)
        at = 0
        for s, _, n in step:
            got[s].append(y[at:at + n])
            at += n
    return [torch.cat(g) for g in got], want


@pytest.mark.parametrize("device,dtype", RUNS)
@pytest.mark.parametrize("H,d,r,dv,R,Q", [(3, 8, 4, 12, 20, 17), (1, 16, 2, 8, 8, 8), (2, 32, 16, 32, 48, 24), (2, 24, 64, 16, 192, 80),
                                          (5, 6, 6, 7, 10, 9)])
def test_latent_attention_with_a_query_latent(device, dtype, H, d, r, dv, R, Q):
    # cached rows of 64 / 256 numbers: in bf16 on a GPU the matrix-core kernel runs
    slack = 1.0 if dtype == torch.float32 else 2.0
    for lens, cuts, seed in (([70, 1, 33], [[16, 1, 15, 2, 1, 1, 30, 3, 1], [1], [2, 31]], 0), ([150], [[65, 64, 1, 20]], 7)):
        got, want = latent(device, dtype, H, d, r, dv, R, Q, lens, cuts, 0.3, seed=seed)
        for g, w in zip(got, want):
            close(g, w, dtype, "latent attention", slack=slack)


# ------------------------------------------------------------------------------------------------- gated delta rule
class Delta:
    """The delta mixer between its projections: convolution, recurrence, per-head norm, gate."""

    def __init__(self, device, dtype, H, G, dim, vdim, taps=3, scale=1.0, seed=0, conv=None):
        self.__dict__.update(locals())
        self.nqk, self.nv = G * dim, H * vdim
        self.c = 2 * self.nqk + self.nv
        self.n = self.c + self.nv + 2 * H
        self.w = rnd(self.c, taps, seed=seed + 1, dtype=dtype, mul=taps ** -0.5)
        self.norm = (1 + 0.2 * rnd(vdim, seed=seed + 2)).to(dtype).double()
        self.A_log, self.dtb = rnd(H, seed=seed + 3) * 0.5 - 1, rnd(H, seed=seed + 4) * 0.3
        self.conv_dtype = dtype if conv is None else conv
        self.eps = 1e-5

    def rows(self, T, seed):
        return rnd(T, self.n, seed=seed, dtype=self.dtype)

    def want(self, x):
        T, H, G, dim, vdim, rep = x.shape[0], self.H, self.G, self.dim, self.vdim, self.H // self.G
        # the convolved rows are rounded to the type they are handed on in
        u = oracle.silu(oracle.causal_conv(x[:, :self.c], self.w)).to(self.conv_dtype).double()
        q, k, v = u[:, :self.nqk], u[:, self.nqk:2 * self.nqk], u[:, 2 * self.nqk:]
        q = (oracle.unit(q.reshape(T, G, dim)) * dim ** -0.5).repeat_interleave(rep, 1)
        k = oracle.unit(k.reshape(T, G, dim)).repeat_interleave(rep, 1)
        gate, b, a = x[:, self.c:self.c + self.nv], x[:, self.c + self.nv:self.c + self.nv + H], x[:, -H:]
        g = torch.exp(-torch.exp(self.A_log) * oracle.softplus(a + self.dtb))
        o = oracle.rms(oracle.delta_rule(q, k, v.reshape(T, H, vdim), oracle.sigmoid(b), g), self.eps) * self.norm
        return o.reshape(T, -1) * oracle.silu(gate) * self.scale

    def run(self, seqs, cuts, slots=None):
        dev, dt, H, G, dim, vdim = self.device, self.dtype, self.H, self.G, self.dim, self.vdim
        slots = slots or list(range(len(seqs)))
        S = torch.full((max(slots) + 1, H, dim, vdim), 3.0, device=dev)  # leftovers
        tail = torch.full((max(slots) + 1, self.taps - 1, self.c), -2.0, device=dev)
        got = [[] for _ in seqs]
        for step in steps_of(cuts):
            step = sorted(step, key=lambda e: not (e[2] == 1 and e[1] > 0))
            nd = sum(1 for e in step if e[2] == 1 and e[1] > 0)
            cu, ctx, ss = meta(step, slots, dev)
            rows = torch.cat([seqs[s][p0:p0 + n] for s, p0, n in step]).to(dev, dt)
            proj = torch.zeros(rows.shape[0], -(-self.n // 8) * 8 + 8, dtype=dt, device=dev)
            proj[:, 8:8 + self.n] = rows
            p = proj[:, 8:8 + self.n]
            u = ops.causal_conv(p[:, :self.c], to(self.w, dev, dt), tail, cu, ctx, ss, False, True, self.conv_dtype)
            out = torch.full((rows.shape[0], self.nv + 8), 9.0, dtype=dt, device=dev)
            ops.delta_mix(u[:, :self.nqk], u[:, self.nqk:2 * self.nqk], u[:, 2 * self.nqk:], p[:, -H:],
                          p[:, self.c + self.nv:self.c + self.nv + H], to(self.A_log, dev), to(self.dtb, dev), S, cu, ctx, ss,
                          H, G, dim, vdim, p[:, self.c:self.c + self.nv], to(self.norm, dev, dt), self.eps, self.scale,
                          out[:, :self.nv], max_qlen=max(n for _, _, n in step), num_decode=nd)
            assert bool((out[:, self.nv:] == 9.0).all())
            at = 0
            for s, _, n in step:
                got[s].append(out[at:at + n, :self.nv].clone())
                at += n
        return [torch.cat(g) for g in got]


DELTA = [(2, 1, 8, 12, 3, 1.0), (3, 3, 5, 7, 1, 0.5), (4, 2, 32, 24, 4, 1.0), (2, 2, 64, 128, 2, -0.7), (2, 1, 128, 64, 3, 1.0),
         (1, 1, 96, 80, 5, 2.0), (6, 2, 16, 256, 2, 1.0), (1, 1, 200, 40, 2, 1.0), (2, 1, 256, 16, 3, 1.0)]


@pytest.mark.parametrize("device,dtype", RUNS)
@pytest.mark.parametrize("H,G,dim,vdim,taps,scale", DELTA)
def test_delta_rule_over_portions_and_single_rows(device, dtype, H, G, dim, vdim, taps, scale):
    a = Delta(device, dtype, H, G, dim, vdim, taps, scale)
    T = 150
    x = a.rows(T, 5)
    want = a.want(x)
    # (a row whose numbers nearly cancel in the per-head norm magnifies the rounding of the convolved rows)
    slack = 1.0 if dtype == torch.float32 else 2.0
    for cuts in ([T], [2, 3, 64, 1, 63, 2, 1, 1, 13], [100] + [1] * 50, [65, 65, 20], [1] * 4 + [128, 18]):
        close(a.run([x], [cuts], slots=[1])[0], want, dtype, f"cuts {cuts[:4]}", slack=slack)


@pytest.mark.parametrize("device,dtype", RUNS)
def test_delta_rule_of_unequal_sequences_and_reused_slots(device, dtype):
    a = Delta(device, dtype, 4, 2, 32, 64)
    xs = [a.rows(n, 40 + n) for n in (130, 70, 9, 1)]
    got = a.run(xs, [[60, 1, 1, 68], [2, 5, 63], [9], [1]], slots=[3, 0, 2, 1])
    for i, x in enumerate(xs):
        close(got[i], a.want(x), dtype, f"sequence {i}", slack=1.0 if dtype == torch.float32 else 2.0)


@pytest.mark.parametrize("device,dtype", RUNS)
def test_delta_rule_on_rows_in_32_bit(device, dtype):
    """q, k and v handed on in fp32 beside gates in the storage type: the token-by-token walk at every size."""
    a = Delta(device, dtype, 2, 1, 32, 32, conv=torch.float32)
    xs = [a.rows(n, 60 + n) for n in (90, 5)]
    got = a.run(xs, [[70, 1, 19], [1, 4]])
    for i, x in enumerate(xs):
        close(got[i], a.want(x), dtype, f"sequence {i}")


@pytest.mark.parametrize("device,dtype", RUNS)
@pytest.mark.parametrize("dim,vdim", [(16, 8), (64, 64)])
def test_delta_rule_gates_at_their_ends(device, dtype, dim, vdim):
    """Decays from none to total (inside a chunk and at its edges), write strengths from 0 to 1, a key written again and again
    (each write must first take out what the key already holds), and a token kept over hundreds."""
    H, T = 2, 330
    a = Delta(device, dtype, H, 1, dim, vdim, taps=1)
    a.A_log, a.dtb = torch.zeros(H, dtype=F64), torch.zeros(H, dtype=F64)
    x = a.rows(T, 8)
    b, g = x[:, -2 * H:-H], x[:, -H:]
    g[:], b[:] = -12.0, 2.0  # nearly no decay
    g[40], g[64], g[127, 0], g[200:203] = 30.0, 30.0, 30.0, 6.0
    b[10:20], b[90] = -30.0, 30.0
    x[140:180, a.nqk:2 * a.nqk] = x[140, a.nqk:2 * a.nqk]  # one key, forty writes
    b[140:180] = 30.0
    x = x.to(dtype).double()
    want = a.want(x)
    slack = 2.0 if dtype == torch.float32 else 3.0
    for cuts in ([T], [40, 1, 23, 1, 62, 1, 2, 200], [250] + [1] * 80):
        close(a.run([x], [cuts])[0], want, dtype, f"cuts {cuts[:4]}", slack=slack)


@pytest.mark.parametrize("device,dtype", RUNS)
def test_delta_rule_keeps_an_early_token(device, dtype):
    """A write long ago under open gates decides a late row; without it the row is another one."""
    H, dim, vdim, T = 1, 32, 32, 600
    a = Delta(device, dtype, H, 1, dim, vdim, taps=1)
    a.A_log, a.dtb = torch.zeros(H, dtype=F64), torch.zeros(H, dtype=F64)
    x = a.rows(T, 9)
    x[:, -2], x[:, -1] = -40.0, -14.0  # nothing written, nothing forgotten
    x[3, -2], x[500:, -2] = 30.0, -7.0
    x = x.to(dtype).double()
    want = a.want(x)
    gone = x.clone()
    gone[3, -2] = -40.0
    assert float((a.want(gone)[-1] - want[-1]).abs().max()) > 0.05
    for cuts in ([T], [300, 2, 200] + [1] * 98):
        close(a.run([x], [cuts])[0], want, dtype, f"cuts {cuts[:3]}", slack=2.0)


@pytest.mark.parametrize("device,dtype", RUNS)
def test_padded_sequences_leave_zero_rows(device, dtype):
    """A decode step's padding: no slot, no context. Its rows are zero and no state changes."""
    H, G, dim, vdim = 2, 1, 16, 8
    q, k, v = (to(rnd(3, n, seed=i, dtype=dtype), device, dtype) for i, n in enumerate((G * dim, G * dim, H * vdim)))
    ab, gate = (to(rnd(3, n, seed=9 + n, dtype=dtype), device, dtype) for n in (2 * H, H * vdim))
    S = torch.full((2, H, dim, vdim), 3.0, device=device)
    out = torch.full((3, H * vdim), 5.0, dtype=dtype, device=device)
    z = torch.zeros(H, device=device)
    one = torch.ones(vdim, dtype=dtype, device=device)
    ops.delta_mix(q, k, v, ab[:, :H], ab[:, H:], z, z, S, i32([0, 1, 2, 3], device), i32([4, 0, 0], device),
                  i32([1, -1, -1], device), H, G, dim, vdim, gate, one, 1e-5, 1.0, out, max_qlen=1)
    assert bool((out[1:] == 0).all()) and bool((out[0] != 0).any()) and bool((S[0] == 3.0).all()) and bool((S[1] != 3.0).any())
    x, dtl = to(rnd(3, 24, seed=1, dtype=dtype), device, dtype), to(rnd(3, 24, seed=2), device)
    bc, st = to(rnd(3, 10, seed=3, dtype=dtype), device, dtype), torch.full((2, 24, 5), 3.0, device=device)
    y = ops.selective_scan(x, dtl, torch.zeros(24, device=device), bc[:, :5], bc[:, 5:], -torch.ones(24, 5, device=device),
                           torch.ones(24, device=device), x, st, i32([0, 1, 2, 3], device), i32([4, 0, 0], device),
                           i32([1, -1, -1], device), dtype)
    assert bool((y[1:] == 0).all()) and bool((y[0] != 0).any()) and bool((st[0] == 3.0).all()) and bool((st[1] != 3.0).any())


# ------------------------------------------------------------------------------------------------- selective scan
class Scan:
    def __init__(self, device, dtype, inner, N, seed=0):
        self.__dict__.update(locals())
        self.A, self.D = -torch.exp(rnd(inner, N, seed=seed + 1) * 0.7), 1 + 0.3 * rnd(inner, seed=seed + 2)
        self.dtb = rnd(inner, seed=seed + 3) - 1.0

    def rows(self, T, seed):
        """x, z, B, C in the storage type and the step inputs in fp32, for T tokens."""
        return tuple(rnd(T, n, seed=seed * 10 + i, dtype=self.dtype if i < 4 else torch.float32)
                     for i, n in enumerate((self.inner, self.inner, self.N, self.N, self.inner)))

    def want(self, x, z, Bm, Cm, dt):
        return oracle.selective_scan(x, oracle.softplus(dt + self.dtb), self.A, Bm, Cm, self.D) * oracle.silu(z)

    def run(self, seqs, cuts, slots=None):
        dev, dt = self.device, self.dtype
        slots = slots or list(range(len(seqs)))
        S = torch.full((max(slots) + 1, self.inner, self.N), 4.0, device=dev)  # leftovers
        got = [[] for _ in seqs]
        for step in steps_of(cuts):
            cu, ctx, ss = meta(step, slots, dev)
            x, z, Bm, Cm, d = (torch.cat([seqs[s][j][p0:p0 + n] for s, p0, n in step]) for j in range(5))
            wide = torch.zeros(x.shape[0], 2 * self.inner + 3, dtype=dt, device=dev)  # x | z are columns of wider rows
            wide[:, 1:1 + self.inner], wide[:, 3 + self.inner:] = x.to(dev, dt), z.to(dev, dt)
            bc = torch.cat([x[:, :2], Bm, Cm], 1).to(dev, dt)
            y = ops.selective_scan(wide[:, 1:1 + self.inner], to(d, dev), to(self.dtb, dev), bc[:, 2:2 + self.N],
                                   bc[:, 2 + self.N:], to(self.A, dev), to(self.D, dev), wide[:, 3 + self.inner:], S, cu, ctx,
                                   ss, dt)
            at = 0
            for s, _, n in step:
                got[s].append(y[at:at + n])
                at += n
        return [torch.cat(g) for g in got]


@pytest.mark.parametrize("device,dtype", RUNS)
@pytest.mark.parametrize("inner,N", [(40, 6), (64, 16), (130, 4), (7, 24), (192, 1), (33, 40), (16, 100), (70, 200), (96, 65)])
def test_selective_scan_over_portions_and_single_rows(device, dtype, inner, N):
    a = Scan(device, dtype, inner, N)
    x = a.rows(75, 5)
    want = a.want(*x)
    for cuts in ([75], [2, 3, 16, 1, 15, 17, 2, 1, 1, 17], [1] * 5 + [40] + [1] * 30):
        close(a.run([x], [cuts], slots=[1])[0], want, dtype, f"cuts {cuts[:4]}")
    xs = [a.rows(n, 20 + n) for n in (50, 23, 9, 1)]
    got = a.run(xs, [[17, 1, 1, 31], [2, 5, 16], [9], [1]], slots=[3, 0, 2, 1])
    for i, x in enumerate(xs):
        close(got[i], a.want(*x), dtype, f"sequence {i}")


@pytest.mark.parametrize("device,dtype", RUNS)
def test_selective_scan_step_sizes_at_their_ends(device, dtype):
    """Steps of nearly nothing (the state stays: an early token decides a late row) and steps so long that the state is gone."""
    a = Scan(device, dtype, 24, 8)
    a.dtb = torch.zeros(24, dtype=F64)
    T = 400
    x, z, Bm, Cm, dt = a.rows(T, 3)
    dt[:] = -15.0
    dt[4], dt[5] = 3.0, -9.0
    want = a.want(x, z, Bm, Cm, dt)
    gone = dt.clone()
    gone[4] = -15.0
    # a.D x is the same either way: the difference is what the state kept
    assert float((a.want(x, z, Bm, Cm, gone)[-1] - want[-1]).abs().max()) > 0.1
    for cuts in ([T], [300, 2] + [1] * 98):
        close(a.run([(x, z, Bm, Cm, dt)], [cuts])[0], want, dtype, f"cuts {cuts[:3]}", slack=2.0)
    dt[200], dt[390] = 60.0, 25.0  # softplus beyond its linear end; the state before is forgotten
    want = a.want(x, z, Bm, Cm, dt)
    for cuts in ([T], [200, 1, 189] + [1] * 10):
        close(a.run([(x, z, Bm, Cm, dt)], [cuts])[0], want, dtype, f"cuts {cuts[:3]}", slack=2.0)
