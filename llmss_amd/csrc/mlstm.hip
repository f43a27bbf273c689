// The exponential-gate matrix memory (mlstm) in the two forms that carry a serving step, beside the token-by-token walk of
// recurrent.hip (which also holds the gates' kernel):
//
//   mlstm_step:   steps of single rows. One workgroup per (sequence, head) does everything: the gates and the running maximum,
//                 S <- g S + e k v^T and n likewise in one pass over the state (16-byte accesses, columns over lanes, state
//                 rows over groups of threads), o = S^T q / (max(|n . q|, exp(-m)) + 1e-6), the per-head norm, the gate.
//   mlstm_chunk:  portions of bf16 rows on the matrix cores, 64 tokens at a time. With F_t the sum of the log forget gates
//                 from the chunk's start to t, A_t = F_t - m_t and B_s = i_s - F_s, the token-by-token recurrence is
//                   num_t = sum_{s <= t} exp(A_t + B_s) (q_t . k_s) v_s + exp(A_t + m_0) S_0^T q_t
//                   S_C   = exp(A_C + m_0) S_0 + sum_s exp(A_C + B_s) k_s v_s^T
//                 (m_0, S_0 before the chunk, C its last token; every exponent is <= 0 because m_t is the running
//                 maximum): four matrix products per chunk, only the state sequential from chunk to chunk. q, k and v are
//                 exact in bf16; the fp32 factors - the weighted scores, the state, the weighted values - enter as value +
//                 remainder (two bf16 numbers, two matrix instructions), sums and the state itself stay fp32.
#include "anytype.h"

// ------------------------------------------------------------------------------------------------ single rows
struct MlstmStepArgs {
  const void* q;
  const void* k;
  const void* v;
  int64_t ldq, ldk, ldv;
  const void* zi;
  const void* zf;
  int64_t ldz;
  const float* bi;
  const float* bf;
  float cap;
  float* S;  // [slots, H, dim, vdim]
  float* n;  // [slots, H, dim]
  float* m;  // [slots, H]
  const int* cu;
  const int* ctx;
  const int* sslots;
  const void* gate;
  int64_t ldg;
  const void* w;  // [H * vdim]
  float eps, qs;
  void* y;
  int64_t ldy;
  int H, dim, vdim;
};

template <typename T>
__global__ __launch_bounds__(256) void mlstm_step_kernel(MlstmStepArgs A) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  __shared__ float red[32];
  const int h = blockIdx.x, b = blockIdx.y, tid = threadIdx.x;
  const int dim = A.dim, vdim = A.vdim, H = A.H;
  const int t = A.cu[b], slot = A.sslots[b], pos = A.ctx[b] - 1;
  T* yr = (T*)A.y + (int64_t)t * A.ldy + (int64_t)h * vdim;
  if (slot < 0 || pos < 0) {
    for (int c = tid; c < vdim; c += 256) El<T>::st(yr + c, 0.f);
    return;
  }
  float* qs = sm;             // [dim]
  float* ks = qs + dim;       // [dim], times the input gate's weight
  float* part = ks + ((dim + 3) & ~3) + ((4 - (dim & 3)) & 3);  // [row groups][vdim]
  const float icap = 1.0f / A.cap;
  const float m0 = pos > 0 ? A.m[(int64_t)slot * H + h] : 0.f;
  const float gi = A.cap * tanhf((El<T>::ld((const T*)A.zi + (int64_t)t * A.ldz + h) + A.bi[h]) * icap);
  const float zf = A.cap * tanhf((El<T>::ld((const T*)A.zf + (int64_t)t * A.ldz + h) + A.bf[h]) * icap);
  const float gf = fminf(zf, 0.f) - log1pf(expf(-fabsf(zf)));
  const float mt = fmaxf(gf + m0, gi);
  const float a = expf(gf + m0 - mt), e = expf(gi - mt);
  const T* qr = (const T*)A.q + (int64_t)t * A.ldq + (int64_t)h * dim;
  const T* kr = (const T*)A.k + (int64_t)t * A.ldk + (int64_t)h * dim;
  float* np = A.n + ((int64_t)slot * H + h) * dim;
  float dot = 0.f;
  for (int d = tid; d < dim; d += 256) {
    const float qd = El<T>::ld(qr + d), kd = El<T>::ld(kr + d) * e;
    qs[d] = qd;
    ks[d] = kd;
    const float nv = fmaf(a, pos > 0 ? np[d] : 0.f, kd);
    np[d] = nv;
    dot = fmaf(nv, qd, dot);
  }
  dot = block_sum(dot, red);  // (its barriers also make qs, ks visible and follow every thread's read of m)
  if (tid == 0) A.m[(int64_t)slot * H + h] = mt;
  // thread (rg, cg): columns 4 cg .. 4 cg + 3 of the state rows rg, rg + RG, ...
  const int ncg = vdim >> 2, RG = 256 / ncg, cg = tid % ncg, rg = tid / ncg;
  if (rg < RG) {
    f32x4 v4;
    const T* vr = (const T*)A.v + (int64_t)t * A.ldv + (int64_t)h * vdim + 4 * cg;
#pragma unroll
    for (int i = 0; i < 4; ++i) v4[i] = El<T>::ld(vr + i);
    float* sp = A.S + (((int64_t)slot * H + h) * dim) * (int64_t)vdim + 4 * cg;
    f32x4 o = {0.f, 0.f, 0.f, 0.f};
    constexpr int U = 8;
    for (int r0 = rg; r0 < dim; r0 += RG * U) {
      f32x4 s[U];
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const int r = min(r0 + u * RG, dim - 1);
        s[u] = pos > 0 ? *reinterpret_cast<const f32x4*>(sp + (int64_t)r * vdim) : f32x4{0.f, 0.f, 0.f, 0.f};
      }
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const int r = r0 + u * RG;
        if (r < dim) {
          const float kd = ks[r], qd = qs[r];
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            s[u][i] = fmaf(a, s[u][i], kd * v4[i]);
            o[i] = fmaf(s[u][i], qd, o[i]);
          }
          *reinterpret_cast<f32x4*>(sp + (int64_t)r * vdim) = s[u];
        }
      }
    }
    *reinterpret_cast<f32x4*>(part + (int64_t)rg * vdim + 4 * cg) = o;
  }
  __syncthreads();
  const float mul = A.qs / (fmaxf(fabsf(A.qs * dot), expf(-mt)) + 1e-6f);
  float ss = 0.f;
  for (int c = tid; c < vdim; c += 256) {
    float o = 0.f;
    for (int r = 0; r < RG; ++r) o += part[r * vdim + c];
    o *= mul;
    part[c] = o;  // (row 0 of the parts at this column: read by this thread alone)
    ss = fmaf(o, o, ss);
  }
  ss = block_sum(ss, red);
  const float inv = 1.0f / sqrtf(ss / (float)vdim + A.eps);
  const T* gr = (const T*)A.gate + (int64_t)t * A.ldg + (int64_t)h * vdim;
  const T* wr = (const T*)A.w + (int64_t)h * vdim;
  for (int c = tid; c < vdim; c += 256)
    El<T>::st(yr + c, part[c] * inv * El<T>::ld(wr + c) / (1.0f + expf(-El<T>::ld(gr + c))));
}

bool mlstm_step_ok(int dim, int vdim) { return vdim % 4 == 0 && vdim >= 4 && vdim <= 1024 && dim >= 1 && dim <= 2048; }

// B sequences of one row each
void launch_mlstm_step(const void* q, const void* k, const void* v, int64_t ldq, int64_t ldk, int64_t ldv, const void* zi,
                       const void* zf, int64_t ldz, const void* bi, const void* bf, float cap, void* S, void* n, void* m,
                       const void* cu, const void* ctx, const void* sslots, const void* gate, int64_t ldg, const void* w,
                       float eps, float qs, void* y, int64_t ldy, int B, int H, int dim, int vdim, int dt,
                       hipStream_t st) {
  if (B == 0) return;
  if (!mlstm_step_ok(dim, vdim) || B > 65535) throw std::runtime_error("mlstm_step: shape");
  MlstmStepArgs A{q, k, v, ldq, ldk, ldv, zi, zf, ldz, (const float*)bi, (const float*)bf, cap, (float*)S, (float*)n,
                  (float*)m, (const int*)cu, (const int*)ctx, (const int*)sslots, gate, ldg, w, eps, qs, y, ldy, H, dim,
                  vdim};
  const int RG = 256 / (vdim / 4);
  const size_t lds = ((size_t)2 * dim + 8 + (size_t)RG * vdim) * 4;
  dim3 g(H, B);
  DISPATCH_T(dt, T, (mlstm_step_kernel<T><<<g, 256, lds, st>>>(A)));
  HIP_CHECK_LAUNCH();
}

// ------------------------------------------------------------------------------------------------ portions
struct MlstmChunkArgs {
  const bf16_t* q;
  const bf16_t* k;
  const bf16_t* v;
  int64_t ldq, ldk, ldv;
  const f32x4* gates;  // [T, H] (f, i, m, m before)
  float* S;
  float* n;
  const int* cu;
  const int* ctx;
  const int* sslots;
  float* num;  // [T, H * vdim]
  float* den;  // [T, H]
  int H, dim, vdim;
};

// Workgroup (head, block of 64 value columns or the normaliser, sequence), 4 waves. KT: 16-row tiles of the state (dim padded
// with zeros to 16 KT, an even number of tiles). A wave owns 16 value columns: its part of the state lives in registers in the
// accumulator layout (lane (li, g): column li, rows 16 tile + 4 g + i), whose rows are, without any exchange, the k-slots
// (8 g + j -> row 4 g + j of tile 2 ks, j < 4, or 4 g + j - 4 of tile 2 ks + 1) of the B operand of Q S; the transposing LDS
// reads of K and V deliver the same slot order over tokens. The next chunk's rows are fetched into registers while this one
// is computed.
template <int KT>
__global__ __launch_bounds__(256, KT <= 8 ? 2 : 1) void mlstm_chunk_kernel(MlstmChunkArgs A) {
  constexpr int C = 64, DKP = 16 * KT, LDK = DKP + 8, LDV = 64 + 8, LDP = 64 + 8;
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
  bf16_t* Qs = reinterpret_cast<bf16_t*>(smem);
  bf16_t* Ks = Qs + C * LDK;
  bf16_t* Vs = Ks + C * LDK;
  bf16_t* Ph = Vs + C * LDV;
  bf16_t* Pl = Ph + C * LDP;
  float* At = reinterpret_cast<float*>(Pl + C * LDP);  // [64] F_t - m_t
  float* Bs = At + C;                                  // [64] i_s - F_s
  float* gt = Bs + C;                                  // [64] exp(A_t + m_0)
  float* ws = gt + C;                                  // [64] exp(A_C + B_s)
  float* ac = ws + C;                                  // [4] exp(A_C + m_0)
  float* nst = ac + 4;                                 // [DKP] the normaliser's state
  float* nred = nst + DKP;                             // [2][DKP]
  const int h = blockIdx.x, b = gridDim.z - 1 - blockIdx.z;
  const bool ncol = blockIdx.y == gridDim.y - 1;
  const int c0 = blockIdx.y * 64;
  const int dim = A.dim, vdim = A.vdim, H = A.H;
  const int t0 = A.cu[b], qlen = A.cu[b + 1] - t0, slot = A.sslots[b], ctx = A.ctx[b];
  if (qlen <= 0) return;
  const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6, li = lane & 15, g = lane >> 4;
  const int col = c0 + 16 * w + li;
  if (slot < 0 || ctx <= 0) {
    for (int j = 0; j < qlen; ++j) {
      if (ncol) {
        if (tid == 0) A.den[(int64_t)(t0 + j) * H + h] = 0.f;
      } else if (g == 0 && col < vdim) {
        A.num[(int64_t)(t0 + j) * H * vdim + (int64_t)h * vdim + col] = 0.f;
      }
    }
    return;
  }
  const bool cont = ctx > qlen;  // continues an earlier portion
  f32x4 S[KT];
  float* sp = A.S + (((int64_t)slot * H + h) * dim) * (int64_t)vdim;
  float* np = A.n + ((int64_t)slot * H + h) * dim;
#pragma unroll
  for (int kt = 0; kt < KT; ++kt)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int r = 16 * kt + 4 * g + i;
      S[kt][i] = (!ncol && cont && r < dim && col < vdim) ? sp[(int64_t)r * vdim + col] : 0.f;
    }
  if (ncol)
    for (int d = tid; d < DKP; d += 256) nst[d] = cont && d < dim ? np[d] : 0.f;
  constexpr int CHK = DKP / 8, NK = C * CHK / 256, NV = 2;
  static_assert((C * CHK) % 256 == 0, "whole 16-byte pieces per thread");
  u16x8 rq[NK], rk[NK], rv[NV];
  f32x4 rg = {0.f, 0.f, 0.f, 0.f};
  const u16x8 zero8 = {0, 0, 0, 0, 0, 0, 0, 0};
  auto fetch = [&](int j0) {
#pragma unroll
    for (int j = 0; j < NK; ++j) {
      const int c = tid + 256 * j, r = c / CHK, d = (c % CHK) * 8;
      const bool in = j0 + r < qlen && d < dim;
      const int64_t tt = t0 + j0 + r;
      rq[j] = in ? *reinterpret_cast<const u16x8*>(A.q + tt * A.ldq + (int64_t)h * dim + d) : zero8;
      rk[j] = in ? *reinterpret_cast<const u16x8*>(A.k + tt * A.ldk + (int64_t)h * dim + d) : zero8;
    }
    if (!ncol) {
#pragma unroll
      for (int j = 0; j < NV; ++j) {
        const int c = tid + 256 * j, r = c >> 3, d = c0 + (c & 7) * 8;
        rv[j] = (j0 + r < qlen && d < vdim)
                    ? *reinterpret_cast<const u16x8*>(A.v + (int64_t)(t0 + j0 + r) * A.ldv + (int64_t)h * vdim + d) : zero8;
      }
    }
    if (w == 0) rg = A.gates[(int64_t)(t0 + min(j0 + lane, qlen - 1)) * H + h];
  };
  fetch(0);
  for (int j0 = 0; j0 < qlen; j0 += C) {
    const int nt = min(C, qlen - j0);
    __syncthreads();  // the previous chunk's readers are done
#pragma unroll
    for (int j = 0; j < NK; ++j) {
      const int c = tid + 256 * j, r = c / CHK, d = (c % CHK) * 8;
      *reinterpret_cast<u16x8*>(&Qs[r * LDK + d]) = rq[j];
      *reinterpret_cast<u16x8*>(&Ks[r * LDK + d]) = rk[j];
    }
    if (!ncol) {
#pragma unroll
      for (int j = 0; j < NV; ++j) {
        const int c = tid + 256 * j;
        *reinterpret_cast<u16x8*>(&Vs[(c >> 3) * LDV + (c & 7) * 8]) = rv[j];
      }
    }
    if (w == 0) {
      const bool in = lane < nt;
      float F = in ? rg[0] : 0.f;
#pragma unroll
      for (int o = 1; o < 64; o <<= 1) {
        const float x = __shfl_up(F, o, 64);
        if (lane >= o) F += x;
      }
      const float m0 = __shfl(rg[3], 0, 64);
      const float a = in ? F - rg[2] : -INFINITY, bb = in ? rg[1] - F : -INFINITY;
      const float aC = __shfl(a, nt - 1, 64);
      At[lane] = a;
      Bs[lane] = bb;
      gt[lane] = expf(a + m0);
      ws[lane] = expf(aC + bb);
      if (lane == 0) ac[0] = expf(aC + m0);
    }
    __syncthreads();
    if (j0 + C < qlen) fetch(j0 + C);
    // weighted scores: wave w owns the tokens 16 w .. 16 w + 15 (rows), all 64 keys (columns)
    {
      f32x4 p[4];
#pragma unroll
      for (int ct = 0; ct < 4; ++ct) p[ct] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int ks = 0; ks < KT / 2; ++ks) {
        const s16x8 qa = *reinterpret_cast<const s16x8*>(&Qs[(16 * w + li) * LDK + 32 * ks + 8 * g]);
#pragma unroll
        for (int ct = 0; ct < 4; ++ct) {
          if (ct > w) continue;  // keys after every token of the wave
          const s16x8 kb = *reinterpret_cast<const s16x8*>(&Ks[(16 * ct + li) * LDK + 32 * ks + 8 * g]);
          p[ct] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qa, kb, p[ct], 0, 0, 0);
        }
      }
      const f32x4 a4 = *reinterpret_cast<const f32x4*>(&At[16 * w + 4 * g]);
      float rs[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int ct = 0; ct < 4; ++ct) {
        const float bb = Bs[16 * ct + li];
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int t = 16 * w + 4 * g + i, s = 16 * ct + li;
          const float x = s <= t ? p[ct][i] * __expf(a4[i] + bb) : 0.f;
          if (ncol) {
            rs[i] += x;
          } else {
            const bf16_t hi = f2bf(x);
            Ph[t * LDP + s] = hi;
            Pl[t * LDP + s] = f2bf(x - bf2f(hi));
          }
        }
      }
      if (ncol) {
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          float x = rs[i];
          x += __shfl_xor(x, 1, 64);
          x += __shfl_xor(x, 2, 64);
          x += __shfl_xor(x, 4, 64);
          x += __shfl_xor(x, 8, 64);
          // n_0 . q_t: the 16 lanes of a row share the state's rows
          const int t = 16 * w + 4 * g + i;
          float y = 0.f;
          for (int d = li; d < DKP; d += 16) y = fmaf(bf2f(Qs[t * LDK + d]), nst[d], y);
          y += __shfl_xor(y, 1, 64);
          y += __shfl_xor(y, 2, 64);
          y += __shfl_xor(y, 4, 64);
          y += __shfl_xor(y, 8, 64);
          if (li == 0 && t < nt) A.den[(int64_t)(t0 + j0 + t) * H + h] = fmaf(gt[t], y, x);
        }
        // n <- exp(A_C + m_0) n + sum_s w_s k_s: two groups of 32 tokens, DKP columns each
        for (int e = tid; e < 2 * DKP; e += 256) {
          const int d = e % DKP, half = e / DKP;
          float x = 0.f;
          for (int s = 32 * half; s < 32 * half + 32; ++s) x = fmaf(ws[s], bf2f(Ks[s * LDK + d]), x);
          nred[e] = x;
        }
        __syncthreads();  // (the whole workgroup takes this branch)
        for (int d = tid; d < DKP; d += 256) nst[d] = fmaf(ac[0], nst[d], nred[d] + nred[DKP + d]);
        continue;
      }
    }
    // Q S for this wave's columns while the other waves finish their scores
    f32x4 o[4];
#pragma unroll
    for (int rt = 0; rt < 4; ++rt) o[rt] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int ks = 0; ks < KT / 2; ++ks) {
      s16x8 sh, sl;
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        const float x = S[2 * ks + (j >> 2)][j & 3];
        const bf16_t hi = f2bf(x);
        sh[j] = (short)hi;
        sl[j] = (short)f2bf(x - bf2f(hi));
      }
#pragma unroll
      for (int rt = 0; rt < 4; ++rt) {
        const bf16_t* qp = &Qs[(16 * rt + li) * LDK + 32 * ks + 4 * g];
        const s16x4 q0 = *reinterpret_cast<const s16x4*>(qp), q1 = *reinterpret_cast<const s16x4*>(qp + 16);
        const s16x8 qa = {q0[0], q0[1], q0[2], q0[3], q1[0], q1[1], q1[2], q1[3]};
        o[rt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qa, sh, o[rt], 0, 0, 0);
        o[rt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qa, sl, o[rt], 0, 0, 0);
      }
    }
#pragma unroll
    for (int rt = 0; rt < 4; ++rt) {
      const f32x4 g4 = *reinterpret_cast<const f32x4*>(&gt[16 * rt + 4 * g]);
#pragma unroll
      for (int i = 0; i < 4; ++i) o[rt][i] *= g4[i];
    }
    __syncthreads();  // every wave's weighted scores are in LDS
    const float a_all = ac[0];
#pragma unroll
    for (int kt = 0; kt < KT; ++kt)
#pragma unroll
      for (int i = 0; i < 4; ++i) S[kt][i] *= a_all;
    const int tq = li >> 2, tp = li & 3;
#pragma unroll
    for (int ks = 0; ks < 2; ++ks) {
      const bf16_t* v0 = &Vs[(32 * ks + 4 * g + tq) * LDV + 16 * w + 4 * tp];
      const s16x4 x0 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((LDS_AS s16x4*)(v0));
      const s16x4 x1 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((LDS_AS s16x4*)(v0 + 16 * LDV));
      const s16x8 vb = {x0[0], x0[1], x0[2], x0[3], x1[0], x1[1], x1[2], x1[3]};
#pragma unroll
      for (int rt = 0; rt < 4; ++rt) {
        if (16 * rt + 15 < 32 * ks) continue;  // tokens before every key of this half
        const bf16_t* pp = &Ph[(16 * rt + li) * LDP + 32 * ks + 4 * g];
        const s16x4 h0 = *reinterpret_cast<const s16x4*>(pp), h1 = *reinterpret_cast<const s16x4*>(pp + 16);
        const bf16_t* pq = &Pl[(16 * rt + li) * LDP + 32 * ks + 4 * g];
        const s16x4 l0 = *reinterpret_cast<const s16x4*>(pq), l1 = *reinterpret_cast<const s16x4*>(pq + 16);
        const s16x8 ph = {h0[0], h0[1], h0[2], h0[3], h1[0], h1[1], h1[2], h1[3]};
        const s16x8 pl = {l0[0], l0[1], l0[2], l0[3], l1[0], l1[1], l1[2], l1[3]};
        o[rt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ph, vb, o[rt], 0, 0, 0);
        o[rt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(pl, vb, o[rt], 0, 0, 0);
      }
      // the state: K^T (w v)
      const f32x4 w0 = *reinterpret_cast<const f32x4*>(&ws[32 * ks + 4 * g]);
      const f32x4 w1 = *reinterpret_cast<const f32x4*>(&ws[32 * ks + 16 + 4 * g]);
      s16x8 vh, vl;
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        const float x = bf2f((bf16_t)vb[j]) * (j < 4 ? w0[j & 3] : w1[j & 3]);
        const bf16_t hi = f2bf(x);
        vh[j] = (short)hi;
        vl[j] = (short)f2bf(x - bf2f(hi));
      }
#pragma unroll
      for (int kt = 0; kt < KT; ++kt) {
        const bf16_t* k0 = &Ks[(32 * ks + 4 * g + tq) * LDK + 16 * kt + 4 * tp];
        const s16x4 y0 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((LDS_AS s16x4*)(k0));
        const s16x4 y1 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((LDS_AS s16x4*)(k0 + 16 * LDK));
        const s16x8 ka = {y0[0], y0[1], y0[2], y0[3], y1[0], y1[1], y1[2], y1[3]};
        S[kt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ka, vh, S[kt], 0, 0, 0);
        S[kt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ka, vl, S[kt], 0, 0, 0);
      }
    }
    if (col < vdim) {
#pragma unroll
      for (int rt = 0; rt < 4; ++rt)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int t = 16 * rt + 4 * g + i;
          if (t < nt) A.num[(int64_t)(t0 + j0 + t) * H * vdim + (int64_t)h * vdim + col] = o[rt][i];
        }
    }
  }
  if (ncol) {
    __syncthreads();
    for (int d = tid; d < dim; d += 256) np[d] = nst[d];
  } else if (col < vdim) {
#pragma unroll
    for (int kt = 0; kt < KT; ++kt)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int r = 16 * kt + 4 * g + i;
        if (r < dim) sp[(int64_t)r * vdim + col] = S[kt][i];
      }
  }
}

bool mlstm_chunk_ok(int dim, int vdim) { return dim % 8 == 0 && dim >= 8 && dim <= 256 && vdim % 8 == 0 && vdim >= 8; }

void launch_mlstm_chunk(const void* q, const void* k, const void* v, int64_t ldq, int64_t ldk, int64_t ldv,
                        const void* gates, void* S, void* n, const void* cu, const void* ctx, const void* sslots,
                        void* num, void* den, int B, int H, int dim, int vdim, hipStream_t st) {
  if (B == 0) return;
  if (!mlstm_chunk_ok(dim, vdim) || B > 65535) throw std::runtime_error("mlstm_chunk: shape");
  if (((uintptr_t)q | (uintptr_t)k | (uintptr_t)v) & 15 || (ldq | ldk | ldv) & 7)
    throw std::runtime_error("mlstm_chunk: rows must be 16-byte aligned");
  MlstmChunkArgs A{(const bf16_t*)q, (const bf16_t*)k, (const bf16_t*)v, ldq, ldk, ldv, (const f32x4*)gates, (float*)S,
                   (float*)n, (const int*)cu, (const int*)ctx, (const int*)sslots, (float*)num, (float*)den, H, dim, vdim};
  dim3 g(H, (vdim + 63) / 64 + 1, B);
  auto lds = [](int kt) {
    return (size_t)2 * (2 * 64 * (16 * kt + 8) + 3 * 64 * 72) + (size_t)4 * (4 * 64 + 4 + 3 * 16 * kt);
  };
#define LAUNCH_MC(KT_)                                                                                         \
  do {                                                                                                         \
    static bool once = [] {                                                                                    \
      (void)hipFuncSetAttribute((const void*)mlstm_chunk_kernel<KT_>, hipFuncAttributeMaxDynamicSharedMemorySize, \
                                160 * 1024);                                                                   \
      return true;                                                                                             \
    }();                                                                                                       \
    (void)once;                                                                                                \
    mlstm_chunk_kernel<KT_><<<g, 256, lds(KT_), st>>>(A);                                                      \
  } while (0)
  if (dim <= 32) LAUNCH_MC(2);
  else if (dim <= 64) LAUNCH_MC(4);
  else if (dim <= 128) LAUNCH_MC(8);
  else LAUNCH_MC(16);
#undef LAUNCH_MC
  HIP_CHECK_LAUNCH();
}
