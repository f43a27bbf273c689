"""Per-kernel rates of the Nolavik design beside the like kernel of the Llama family, at layer shapes of
bench/nolavik_compare.py, each at a prompt step (sequences of --seq tokens, --tokens in all) and a decode step
(--batch single tokens after --ctx cached ones). "of roofline" = the time the kernel's own roofline allows (the
largest of flops / 2.5 PFLOP/s, bytes / 8 TB/s and, for the selective scan, exponentials at a quarter of the vector rate)
over the time measured. Prints one JSON object.

    python bench/nolavik_kernels.py [--size w2048] [--tokens 8192] [--seq 1024] [--batch 64] [--ctx 1024]
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

EXP_PER_S = 256 * 4 * 4 * 2.4e9  # CUs x SIMDs x lanes per cycle of a transcendental instruction x clock


def main():
    ap = argparse.ArgumentParser()
    ap.add_argument("--size", default="w2048")
    ap.add_argument("--tokens", type=int, default=8192)
    ap.add_argument("--seq", type=int, default=1024)
    ap.add_argument("--batch", type=int, default=64)
    ap.add_argument("--ctx", type=int, default=1000)
    ap.add_argument("--only", default="", help="kernels whose name contains this")
    a = ap.parse_args()
    from nolavik_compare import SIZES, dense_ff

    from llmss_amd import ops
    from llmss_amd.ops import hip as Hp

    s = SIZES[a.size]
    dev = torch.device("cuda", 0)
    bf = torch.bfloat16
    W = s["width"]
    H, G, D, N_in, N_st, R_dt = s["heads"], s["kv"], s["dim"], s["inner"], s["state"], s["dtr"]
    DH, DG, DD, DV = s["dheads"], s["dkv"], s["ddim"], s["dvdim"]
    rot, Q, R = s["rot"], s["qrank"], s["krank"]
    E, top, EF, SF = s["experts"], s["top"], s["eff"], s["sff"]
    gen = torch.Generator(device=dev).manual_seed(0)

    def rn(*shape, dt=bf, std=1.0):
        return (torch.randn(*shape, device=dev, generator=gen) * std).to(dt)

    def i32(x):
        return torch.tensor(x, dtype=torch.int32, device=dev)

    Hp.reserve_workspace(dev, 64 << 20)
    rows = []
    phase = ""

    def bench(name, fn, flops=0.0, bytes_=0.0, exps=0.0, like=None, iters=10, warm=2):
        if a.only and a.only not in name:
            return
        sec = timed_graph(fn, iters=iters, warm=warm, reps=8 if phase == "decode" else 1)
        ideal = max(flops / (PEAK_TFLOPS * 1e12), bytes_ / (PEAK_TBS * 1e12), exps / EXP_PER_S)
        rows.append(dict(kernel=name, phase=phase, us=round(sec * 1e6, 1), tflops=round(flops / sec / 1e12, 1),
                         tbs=round(bytes_ / sec / 1e12, 2), of_roofline=round(ideal / sec, 3), like=like))
        print(f"[kernels] {name} {phase}: {sec * 1e6:.1f} us, {ideal / sec:.3f} of roofline", file=sys.stderr, flush=True)

    bs = 16
    f32 = lambda *sh: rn(*sh, dt=torch.float32)
    for phase in ("prompt", "decode"):
        if phase == "prompt":
            B, q, ctx = a.tokens // a.seq, a.seq, a.seq
        else:
            B, q, ctx = a.batch, 1, a.ctx + 1
        T = B * q
        single = phase == "decode"
        cu, cl, ss = i32([i * q for i in range(B + 1)]), i32([ctx] * B), i32(list(range(B)))
        nblk = -(-ctx // bs)
        bt = torch.arange(B * nblk, dtype=torch.int32, device=dev).view(B, nblk).contiguous()
        pos = (torch.arange(q, device=dev) + (ctx - q)).repeat(B)
        slots = (bt.long()[:, :, None] * bs + torch.arange(bs, device=dev)).view(B, -1)[:, ctx - q:ctx].reshape(-1).contiguous()
        full = B * (q * (q + 1) // 2 + q * (ctx - q))

        # ---- the block's closing ops (Llama: residual add + RMS norm)
        x, y, y2 = rn(T, W, dt=torch.float32), rn(T, W), rn(T, W)
        wpost, wnext = f32(W), f32(W)
        bench("sandwich_add_norm", lambda: ops.sandwich_add_norm(x, y, None, None, wpost, 1e-6, None, wnext, bf),
              bytes_=T * W * (2 + 4 + 4 + 2))
        bench("sandwich_add_norm summing two mixers",
              lambda: ops.sandwich_add_norm(x, ops.PairPending(y, y2, None, None, (0.7, 0.6)), None, None, wpost, 1e-6, wnext,
                                            wnext, bf), bytes_=T * W * (2 + 2 + 4 + 4 + 2))
        wb = rn(W)
        bench("add_norm", lambda: ops.add_norm(y, wb, None, 1e-6, True, residual=y2), bytes_=T * W * 2 * 4,
              like="sandwich_add_norm")
        # ---- gated delta rule
        nqk, nv = DG * DD, DH * DV
        C = 2 * nqk + nv
        pc = -(-(C + nv + 2 * DH) // 8) * 8
        proj = rn(T, pc)
        conv, tail = rn(C, 4, std=0.5), torch.zeros(B, 3, C, device=dev)
        f_conv = lambda: ops.causal_conv(proj[:, :C], conv, tail, cu, cl, ss, False, True, bf, single=single)
        bench("causal_conv + SiLU + tail (delta)", f_conv, bytes_=T * C * 4)
        u = f_conv()
        S = torch.zeros(B, DH, DD, DV, device=dev)
        A_log, dtb, nw = f32(DH) * 0.5 - 1, f32(DH) * 0.3, rn(DV)
        out = torch.empty(T, nv, dtype=bf, device=dev)
        bench("delta_mix (recurrence, norm, gate)",
              lambda: ops.delta_mix(u[:, :nqk], u[:, nqk:2 * nqk], u[:, 2 * nqk:], proj[:, C + nv + DH:C + nv + 2 * DH],
                                    proj[:, C + nv:C + nv + DH], A_log, dtb, S, cu, cl, ss, DH, DG, DD, DV, proj[:, C:C + nv], nw,
                                    1e-6, 1.0, out, max_qlen=q), flops=T * DH * DD * DV * 6,
              bytes_=B * DH * DD * DV * 8 + T * (2 * nqk + 3 * nv) * 2, iters=3, warm=1)
        # ---- attention branch: heads into the cache, attention with the sink
        nq, nk = H * D, G * D
        kc, vc = rn(B * nblk, bs, nk), rn(B * nblk, bs, nk)
        cs = ops.rope_angles(pos, torch.tensor([10000.0 ** (-2.0 * i / D) for i in range(D // 2)], device=dev))
        ones, zero = torch.ones(D, device=dev), torch.zeros(H, device=dev)
        pa = rn(T, nq + 2 * nk + 2 * N_in)
        f_prep = lambda: ops.head_prep_cache(pa, 0, nq, nq + nk, None, None, ones, ones, False, 1e-6, cs, None, kc, vc, slots, H,
                                             G, D, D, cu, cl, ss, single=single, q_dtype=bf)
        bench("head_prep (unit q / k, rotation, cache)", f_prep, bytes_=T * ((nq + 2 * nk) * 2 + nq * 2 + 2 * nk * 2))
        qf = f_prep()
        bench("window_attn (unit queries, constant sink)",
              lambda: ops.window_attn(qf, kc, vc, bt, cu, cl, H, G, D, D, D ** -0.5, 0.0, 0, 0, zero, None, bf, max_qlen=q,
                                      max_ctx=ctx if single else 0), flops=full * H * 4 * D,
              bytes_=(T * nq * 2 + B * 2 * nk * ctx * 2 + T * nq * 2) if single else 0, iters=3, warm=1)
        kc2, vc2 = rn(B * nblk, G, bs, D), rn(B * nblk, G, bs, D)
        qkv = rn(T, (H + 2 * G) * D)
        if phase == "prompt":
            bench("attn_prefill (flash, full causal)", lambda: ops.attn_prefill(qkv, cu, q, H, G, D, D ** -0.5),
                  flops=full * H * 4 * D, like="window_attn, latent_attn")
        else:
            bench("attn_decode (split-K)", lambda: ops.attn_decode(qkv, kc2, vc2, bt, cl, H, G, D, D ** -0.5, ctx),
                  bytes_=B * ctx * 2 * G * D * 2, like="window_attn, latent_attn")
        # ---- selective scan
        cx, cb, ct = rn(N_in, 4, std=0.5), rn(N_in), torch.zeros(B, 3, N_in, device=dev)
        x0 = nq + 2 * nk
        f_cx = lambda: ops.causal_conv(pa[:, x0:x0 + N_in], cx, ct, cu, cl, ss, False, True, bf, bias=cb, single=single)
        bench("causal_conv + bias + SiLU + tail (scan)", f_cx, bytes_=T * N_in * 4)
        xs = f_cx()
        xw, dw = rn(-(-(R_dt + 2 * N_st) // 8) * 8, N_in, std=N_in ** -0.5), rn(N_in, R_dt, std=R_dt ** -0.5)
        bench("step | B | C product", lambda: ops.linear_f(xs, xw, bf), flops=T * N_in * xw.shape[0] * 2,
              bytes_=T * N_in * 2 + xw.numel() * 2)
        dbc = ops.linear_f(xs, xw, bf)
        bench("step size product (fp32 out)", lambda: ops.linear_f(dbc[:, :R_dt], dw, torch.float32),
              flops=T * N_in * R_dt * 2, bytes_=T * N_in * 4 + dw.numel() * 2)
        st = ops.linear_f(dbc[:, :R_dt], dw, torch.float32)
        SS = torch.zeros(B, N_in, N_st, device=dev)
        A, Dk, sb = -torch.exp(f32(N_in, N_st) * 0.5), f32(N_in), f32(N_in) - 2
        bench("selective_scan",
              lambda: ops.selective_scan(xs, st, sb, dbc[:, R_dt:R_dt + N_st], dbc[:, R_dt + N_st:R_dt + 2 * N_st], A, Dk,
                                         pa[:, x0 + N_in:x0 + 2 * N_in], SS, cu, cl, ss, bf),
              bytes_=T * N_in * (2 + 4 + 2 + 2) + B * N_in * N_st * 8, exps=T * N_in * (N_st + 3), iters=3, warm=1)
        # ---- latent attention
        down = rn(T, Q + R + rot)
        qn, kn = rn(Q), rn(R)
        bench("rms_cols (query latent)", lambda: ops.rms_cols(down, 0, Q, qn, 1e-6, bf), bytes_=T * Q * 4)
        qs = rn(T, H * (D + rot))
        cache = rn(B * nblk, bs, R + rot)
        uk, uv = rn(H, R, D, std=D ** -0.5), rn(H * D, R, std=R ** -0.5)
        f_abs = lambda: ops.head_absorb(qs, uk, ops.latent_qa_dtype(cache), extra=rot)
        bench("head_absorb", f_abs, flops=T * H * D * R * 2, bytes_=T * H * (D + R) * 2)
        qa = f_abs()
        ca = ops.rope_angles(pos, torch.tensor([10000.0 ** (-2.0 * i / rot) for i in range(rot // 2)], device=dev))
        bench("latent_norm_cache (norm, rotations, cache)",
              lambda: ops.latent_norm_cache(down, Q, R, kn, 1e-6, cache, slots, rot, ca, qa, 0, D, q_src=qs),
              bytes_=T * (2 * (R + rot) + 2 * H * rot) * 2)
        bench("latent_attn",
              lambda: ops.latent_attn(qa, cache, bt, cu, cl, 0, (D + rot) ** -0.5, max_qlen=q, max_ctx=ctx if single else 0),
              flops=full * H * 2 * (R + rot + R), bytes_=B * ctx * (R + rot) * 2 + T * H * (R + rot) * 4 if single else 0, iters=3,
              warm=1)
        o = rn(T, H, R + rot)
        bench("head_expand", lambda: ops.head_expand(o, uv, bf), flops=T * H * D * R * 2, bytes_=T * H * (D + R) * 2)
        # ---- experts
        h = rn(T, W)
        rw, rb = rn(E + 1, W, std=W ** -0.5), f32(E) * 0.01
        bench("moe_router (logits, choice, shared gate)",
              lambda: ops.moe_router(h, rw, None, top, True, "chosen", bias=rb, gate=True), flops=T * W * (E + 1) * 2,
              bytes_=T * W * 2)
        idx, wts, sg = ops.moe_router(h, rw, None, top, True, "chosen", bias=rb, gate=True)
        egu, ed = rn(E, 2 * EF, W, std=W ** -0.5), rn(E, W, EF, std=EF ** -0.5)  # gate and up rows interleaved
        f_exp = lambda **kw: ops.moe_experts(h, idx, wts, None, egu, ed, 0.0, 0.0, combine=False, act="silu", interleaved=True,
                                             **kw)
        touched = len(idx.unique())
        bench("experts (group + grouped gate / up + down)",
              f_exp, flops=T * top * W * EF * 6, bytes_=touched * 3 * W * EF * 2, iters=5)
        pend = f_exp(shared=y, shared_w=sg)
        bench("sandwich_add_norm combining experts",
              lambda: ops.sandwich_add_norm(x, pend, None, None, wpost, 1e-6, None, wnext, bf),
              bytes_=T * W * (4 * top + 2 + 4 + 4 + 2))
        sgu, sd = rn(2 * SF, W, std=W ** -0.5), rn(W, SF, std=SF ** -0.5)
        bench("shared expert (gate | up GEMM with the activation, down GEMM)",
              lambda: ops.linear_f(ops.linear(h, sgu, None, "none", True), sd, bf), flops=T * W * SF * 6,
              bytes_=3 * W * SF * 2)
        LF = dense_ff(s)
        gu_i = ops.glu_interleave(rn(LF, W, std=W ** -0.5), rn(LF, W, std=W ** -0.5)).contiguous()
        d_w = rn(W, LF, std=LF ** -0.5)
        bench("gated MLP (fused epilogue)", lambda: ops.linear(ops.linear(h, gu_i, None, "none", True), d_w),
              flops=T * W * LF * 6, bytes_=3 * W * LF * 2, like="experts, shared expert")
        # ---- input GEMMs
        for nm, n in (("delta input GEMM", pc), ("pair input GEMM", pa.shape[1]), ("latent down GEMM", Q + R + rot)):
            pw = rn(n, W, std=W ** -0.5)
            bench(nm, lambda: ops.linear_f(h, pw, bf), flops=T * W * n * 2, bytes_=W * n * 2)
        qw = rn(H * (D + rot), Q, std=Q ** -0.5)
        cq = rn(T, Q)
        bench("query up GEMM", lambda: ops.linear_f(cq, qw, bf), flops=T * Q * qw.shape[0] * 2, bytes_=qw.numel() * 2)
        dq = rn((H + 2 * G) * D, W, std=W ** -0.5)
        bench("dense qkv GEMM", lambda: ops.linear(h, dq), flops=T * W * dq.shape[0] * 2, bytes_=dq.numel() * 2,
              like="input GEMMs")
    print(json.dumps(dict(size=a.size, shape=s, tokens=a.tokens, seq=a.seq, batch=a.batch, ctx=a.ctx, kernels=rows)))


if __name__ == "__main__":
    main()
