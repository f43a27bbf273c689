"""Per-kernel rates of the Tefudra design beside the like kernel of the Llama family, at layer shapes of
bench/tefudra_compare.py, each at a prompt step (sequences of --seq tokens, --tokens in all) and a decode step
(--batch single tokens after --ctx cached ones). "of roofline" = the time the kernel's own roofline allows (the
larger of flops / 2.5 PFLOP/s and bytes / 8 TB/s) over the time measured. Prints one JSON object.

    python bench/tefudra_kernels.py [--size w2048] [--tokens 8192] [--seq 1024] [--batch 64] [--ctx 1024]
"""
import argparse
import json
import os
import sys

import torch

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
sys.path.insert(0, ROOT)
sys.path.insert(0, os.path.join(ROOT, "bench"))

from babotar_kernels import PEAK_TBS, PEAK_TFLOPS  # noqa: E402
from babotar_kernels import timed as timed_graph  # noqa: E402


def main():
    ap = argparse.ArgumentParser()
    ap.add_argument("--size", default="w2048")
    ap.add_argument("--tokens", type=int, default=8192)
    ap.add_argument("--seq", type=int, default=1024)
    ap.add_argument("--batch", type=int, default=64)
    ap.add_argument("--ctx", type=int, default=1000)
    a = ap.parse_args()
    from tefudra_compare import SIZES, dense_ff

    from llmss_amd import ops
    from llmss_amd.ops import hip as Hp

    s = SIZES[a.size]
    dev = torch.device("cuda", 0)
    bf = torch.bfloat16
    W = s["width"]
    H, G, D, win, keep, lwin = s["heads"], s["kv"], s["dim"], s["window"], s["keep"], s["lwindow"]
    MH, MD, MV = s["mheads"], s["mdim"], s["mvdim"]
    E, ident, top, EF, SF, F = s["experts"], s["ident"], s["top"], s["eff"], s["sff"], s["ff"]
    # columns of the pair's input projection
    s = dict(s, pcols=-(-((H + 2 * G) * D + 2 * MH * MD + 2 * MH * MV + 2 * MH) // 8) * 8)
    gen = torch.Generator(device=dev).manual_seed(0)

    def rn(*shape, dt=bf, std=1.0):
        return (torch.randn(*shape, device=dev, generator=gen) * std).to(dt)

    def i32(x):
        return torch.tensor(x, dtype=torch.int32, device=dev)

    Hp.reserve_workspace(dev, 64 << 20)
    rows = []

    def add(name, phase, sec, flops=0.0, bytes_=0.0, like=None):
        ideal = max(flops / (PEAK_TFLOPS * 1e12), bytes_ / (PEAK_TBS * 1e12))
        rows.append(dict(kernel=name, phase=phase, us=round(sec * 1e6, 1), tflops=round(flops / sec / 1e12, 1),
                         tbs=round(bytes_ / sec / 1e12, 2), of_roofline=round(ideal / sec, 3), like=like))
        print(f"[kernels] {name} {phase}: {sec * 1e6:.1f} us, {ideal / sec:.3f} of roofline", file=sys.stderr, flush=True)

    bs = 16
    for phase in ("prompt", "decode"):
        def timed(fn, iters=10, warm=2, reps=8 if phase == "decode" else 1):
            return timed_graph(fn, iters=iters, warm=warm, reps=reps)

        if phase == "prompt":
            B, q, ctx = a.tokens // a.seq, a.seq, a.seq
        else:
            B, q, ctx = a.batch, 1, a.ctx + 1
        T = B * q
        cu = i32([i * q for i in range(B + 1)])
        cl = i32([ctx] * B)
        ss = i32(list(range(B)))
        nblk = -(-ctx // bs)
        bt = torch.arange(B * nblk, dtype=torch.int32, device=dev).view(B, nblk).contiguous()
        pos = (torch.arange(q, device=dev) + (ctx - q)).repeat(B)
        slots = (bt.long()[:, :, None] * bs + torch.arange(bs, device=dev)).view(B, -1)[:, ctx - q:ctx].reshape(-1).contiguous()
        full = B * (q * (q + 1) // 2 + q * (ctx - q))

        # ---- the block's closing ops (Llama: residual add + RMS norm)
        x, y = rn(T, W, dt=torch.float32), rn(T, W)
        f32 = lambda *sh: rn(*sh, dt=torch.float32)
        wpost, wnext, wl, wr = f32(W), f32(W), f32(W), f32(W)
        t = timed(lambda: ops.sandwich_add_norm(x, y, None, None, wpost, 1e-6, None, wnext, bf, 4))
        add("sandwich_add_norm (norms in 4 parts, add)", phase, t, bytes_=T * W * (2 + 4 + 4 + 2))
        y2 = rn(T, W)
        t = timed(lambda: ops.sandwich_add_norm(x, ops.PairPending(y, y2, wl, wr), None, None, wpost, 1e-6, None, wnext, bf, 4))
        add("sandwich_add_norm joining two mixers", phase, t, bytes_=T * W * (2 + 2 + 4 + 4 + 2))
        xb, wb, rr = rn(T, W), rn(W), rn(T, W)
        t = timed(lambda: ops.add_norm(xb, wb, None, 1e-6, True, residual=rr))
        add("add_norm", phase, t, bytes_=T * W * 2 * 4, like="sandwich_add_norm")
        # ---- attention: heads into the cache, window attention
        nq, nk = H * D, G * D
        kc, vc = rn(B * nblk, bs, nk), rn(B * nblk, bs, nk)
        fr = lambda dims: torch.tensor([10000.0 ** (-2.0 * i / dims) for i in range(dims // 2)], device=dev)
        cs_h, cs = ops.rope_angles(pos, fr(D // 2)), ops.rope_angles(pos, fr(D))
        qw, kw, sinks = f32(D), f32(D), f32(H)
        pa = rn(T, nq + nk)
        single = phase == "decode"
        f_att = lambda: ops.head_prep_cache(pa, 0, nq, nq, None, None, qw, kw, False, 1e-6, cs_h, None, kc, vc, slots, H, G, D,
                                            D, cu, cl, ss, single=single, q_dtype=bf)
        t = timed(f_att)
        add("head_prep (q / k norm, rotation, cache)", phase, t, bytes_=T * ((nq + nk) * 2 + nq * 2 + 2 * nk * 2))
        qf = f_att()
        proj = rn(T, s["pcols"])
        conv, tail = rn(4, nq + 2 * nk, std=0.5), torch.zeros(B, 3, nq + 2 * nk, device=dev)
        f_par = lambda: ops.head_prep_cache(proj, 0, nq, nq + nk, conv, tail, None, None, True, 1e-6, cs, cs, kc, vc, slots, H,
                                            G, D, D, cu, cl, ss, single=single, q_dtype=bf)
        t = timed(f_par)
        add("head_prep (4-tap convolution, value norm, rotations, cache)", phase, t,
            bytes_=T * ((nq + 2 * nk) * 2 + nq * 2 + 2 * nk * 2))
        for nm, wnd, kp, cap, sk, vcs in (("window_attn (kept positions, sinks)", win, keep, 0.0, sinks, None),
                                          ("window_attn (soft cap, turned back)", lwin, 0, 30.0, None, cs)):
            vis = lambda p: min(p + 1, wnd) + min(kp, max(0, p + 1 - wnd))
            pairs = B * sum(vis(p) for p in range(ctx - q, ctx))
            fa = lambda: ops.window_attn(qf, kc, vc, bt, cu, cl, H, G, D, D, D ** -0.5, cap, wnd, kp, sk, vcs, bf, max_qlen=q,
                                         max_ctx=ctx if single else 0)
            t = timed(fa, iters=3, warm=1)
            add(nm, phase, t, flops=pairs * H * 4 * D,
                bytes_=(T * nq * 2 + B * 2 * nk * min(ctx, wnd + kp) * 2 + T * nq * 2) if single else 0)
        kc2, vc2 = rn(B * nblk, G, bs, D), rn(B * nblk, G, bs, D)
        qkv = rn(T, (H + 2 * G) * D)
        if phase == "prompt":
            t = timed(lambda: ops.attn_prefill(qkv, cu, q, H, G, D, D ** -0.5))
            add("attn_prefill (flash, full causal)", phase, t, flops=full * H * 4 * D, like="window_attn")
        else:
            t = timed(lambda: ops.attn_decode(qkv, kc2, vc2, bt, cl, H, G, D, D ** -0.5, ctx))
            add("attn_decode (split-K, all keys)", phase, t, bytes_=B * ctx * 2 * G * D * 2, like="window_attn")
        # ---- matrix memory (gates, recurrence, norm and gate: one op)
        c0 = nq + 2 * nk
        nqk, nv = MH * MD, MH * MV
        cut = lambda o, n: proj[:, o:o + n]
        S, n_, m_ = (torch.zeros(B, MH, *sh, device=dev) for sh in ((MD, MV), (MD,), ()))
        bi, bff, nw = f32(MH), f32(MH) + 3.0, rn(nv)
        f_mem = lambda: ops.mlstm_mix(cut(c0, nqk), cut(c0 + nqk, nqk), cut(c0 + 2 * nqk, nv), cut(c0 + 2 * nqk + 2 * nv, MH),
                                      cut(c0 + 2 * nqk + 2 * nv + MH, MH), bi, bff, 15.0, S, n_, m_, cu, cl, ss, MH, MD, MV,
                                      cut(c0 + 2 * nqk + nv, nv), nw, 1e-6, bf, max_qlen=q)
        t = timed(f_mem, iters=3, warm=1)
        add("mlstm_mix (gates, recurrence, norm, gate)", phase, t, flops=T * MH * MD * MV * 4,
            bytes_=B * MH * MD * MV * 8 + T * (2 * nqk + 3 * nv) * 2)
        # ---- experts
        h = rn(T, W)
        rw, corr = rn(E + ident, W, std=W ** -0.5), f32(E + ident) * 0.01
        t = timed(lambda: ops.moe_router(h, rw, corr, top, True, "softmax"))
        add("moe_router (softmax)", phase, t, flops=T * W * (E + ident) * 2, bytes_=T * W * 2)
        idx, wts = ops.moe_router(h, rw, corr, top, True, "softmax")
        eu, ed = rn(E, EF, W, std=W ** -0.5), rn(E, W, EF, std=EF ** -0.5)
        real = int((idx < E).sum())
        t = timed(lambda: ops.moe_experts(h, idx, wts, None, eu, ed, 0.0, 0.0, combine=False, act="gelu", identity=True),
                  iters=5)
        touched = len(idx[idx < E].unique())
        add("experts (group + grouped up, gelu + down)", phase, t, flops=real * W * EF * 4, bytes_=touched * 2 * W * EF * 2)
        # ---- dense feed-forward; Llama's gated one
        up_w, dn_w = rn(F, W, std=W ** -0.5), rn(W, F, std=F ** -0.5)
        t = timed(lambda: ops.linear_f(ops.linear_f(h, up_w, bf, act="relu2"), dn_w, bf))
        add("feed-forward (up GEMM with relu^2, down GEMM)", phase, t, flops=T * W * F * 4, bytes_=2 * F * W * 2)
        LF = dense_ff(s)
        gu_i = ops.glu_interleave(rn(LF, W, std=W ** -0.5), rn(LF, W, std=W ** -0.5)).contiguous()
        d_w = rn(W, LF, std=LF ** -0.5)
        t = timed(lambda: ops.linear(ops.linear(h, gu_i, None, "none", True), d_w))
        add("gated MLP (fused epilogue)", phase, t, flops=T * W * LF * 6, bytes_=3 * W * LF * 2, like="feed-forward, experts")
        # ---- the pair's input GEMM
        pw, pb = rn(s["pcols"], W, std=W ** -0.5), rn(s["pcols"])
        t = timed(lambda: ops.linear_f(h, pw, bf, bias=pb))
        add("pair input GEMM (attention q | k | v, memory q | k | v | g | i | f, bias)", phase, t,
            flops=T * W * s["pcols"] * 2, bytes_=W * s["pcols"] * 2)
    print(json.dumps(dict(size=a.size, shape=s, tokens=a.tokens, seq=a.seq, batch=a.batch, ctx=a.ctx, kernels=rows)))


if __name__ == "__main__":
    main()
