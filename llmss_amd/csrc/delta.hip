// The gated delta rule in the two forms that carry a serving step, beside the token-by-token walk of recurrent.hip. Per head,
// with unit vectors k, q (q also times dim^-1/2), write strength beta = sigmoid(b) and decay g = exp(-exp(A_log) softplus(a +
// dt_bias)):   S <- g S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q
//
//   delta_step:   steps of single rows. One workgroup per (sequence, head): the state is read once into registers and written
//                 once; S^T k and S^T q come from the same pass (o = g S^T q + (k . q) u), then the update, the per-head norm
//                 and the output gate.
//   delta_chunk:  portions of bf16 rows on the matrix cores, 64 tokens at a time. With b_t the sum of the log decays from the
//                 chunk's start to t and S_0 the state before it, the u of a chunk solve a unit lower triangular system,
//                   (I + L) U = beta (V - e^b K S_0),   L_ts = beta_t e^(b_t - b_s) k_t . k_s  (s < t)
//                   O = e^b Q S_0 + P U,                P_ts = e^(b_t - b_s) q_t . k_s         (s <= t)
//                   S_C = e^(b_C) S_0 + sum_s e^(b_C - b_s) k_s u_s^T
//                 What does not depend on the state - X = (I + L)^-1 diag(beta), P and the tokens' factors - is formed for all
//                 chunks side by side (delta_prep); the walk over the chunks is matrix products alone. The projections' q, k, v
//                 are exact in bf16 and enter unnormed, the norms being factors of rows and columns; every fp32 factor (S, U,
//                 X, P) enters as value + remainder, two bf16 numbers, and sums and the state itself stay fp32. The inverse is
//                 taken in fp32: 16 x 16 diagonal blocks by substitution, the blocks below by fp32 matrix instructions.
#include "anytype.h"

// ------------------------------------------------------------------------------------------------ single rows
struct DeltaStepArgs {
  const void* q;  // [T, ldq]: head group's query at q + (h / rep) * dim
  const void* k;
  const void* v;
  int64_t ldq, ldk, ldv;
  const void* a;
  const void* b;
  int64_t ldab;
  const float* A_log;
  const float* dt_bias;
  float* S;  // [slots, H, dim, vdim]
  const int* cu;
  const int* ctx;
  const int* sslots;
  const void* gate;
  int64_t ldg;
  const void* w;  // [vdim]
  float eps, scale;
  void* y;
  int64_t ldy;
  int H, G, dim, vdim;
};

// U: state rows per thread; a thread holds U rows x 4 columns of the state
template <typename T, int U>
__global__ __launch_bounds__(512) void delta_step_kernel(DeltaStepArgs A) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  __shared__ float red[32];
  const int h = blockIdx.x, bq = blockIdx.y, tid = threadIdx.x, nthr = blockDim.x;
  const int dim = A.dim, vdim = A.vdim, H = A.H, gq = h / (H / A.G);
  const int t = A.cu[bq], slot = A.sslots[bq], pos = A.ctx[bq] - 1;
  T* yr = (T*)A.y + (int64_t)t * A.ldy + (int64_t)h * vdim;
  if (slot < 0 || pos < 0) {
    for (int c = tid; c < vdim; c += nthr) El<T>::st(yr + c, 0.f);
    return;
  }
  float* qs = sm;                       // [dim]
  float* ks = qs + dim;                 // [dim]
  float* us = sm + ((2 * dim + 3) & ~3);  // [vdim] u
  float* pk = us + vdim;                // [row groups][vdim] parts of S^T k, then o in row 0
  const int ncg = vdim >> 2, RG = nthr / ncg, cg = tid % ncg, rg = tid / ncg;
  float* pq = pk + (int64_t)RG * vdim;
  // thread (rg, cg): columns 4 cg .. 4 cg + 3 of the state rows rg, rg + RG, ...
  float* sp = A.S + (((int64_t)slot * H + h) * dim) * (int64_t)vdim + 4 * cg;
  f32x4 s[U];
#pragma unroll
  for (int u = 0; u < U; ++u) {
    const int r = rg + u * RG;
    s[u] = (pos > 0 && rg < RG && r < dim) ? *reinterpret_cast<const f32x4*>(sp + (int64_t)r * vdim) : f32x4{0.f, 0.f, 0.f, 0.f};
  }
  const float zb = El<T>::ld((const T*)A.b + (int64_t)t * A.ldab + h);
  const float za = El<T>::ld((const T*)A.a + (int64_t)t * A.ldab + h) + A.dt_bias[h];
  const float beta = 1.0f / (1.0f + expf(-zb));
  const float g = expf(-expf(A.A_log[h]) * (za > 20.f ? za : log1pf(expf(za))));
  const T* qr = (const T*)A.q + (int64_t)t * A.ldq + (int64_t)gq * dim;
  const T* kr = (const T*)A.k + (int64_t)t * A.ldk + (int64_t)gq * dim;
  float qq = 0.f, kk = 0.f, kq = 0.f;
  for (int d = tid; d < dim; d += nthr) {
    const float qd = El<T>::ld(qr + d), kd = El<T>::ld(kr + d);
    qs[d] = qd;
    ks[d] = kd;
    qq = fmaf(qd, qd, qq);
    kk = fmaf(kd, kd, kk);
    kq = fmaf(kd, qd, kq);
  }
  const f32x2 s2 = block_sum2(qq, kk, red);
  kq = block_sum(kq, red);  // (the barriers also make qs, ks visible)
  const float qn = 1.0f / (sqrtf(s2[0] + 1e-6f) * sqrtf((float)dim)), kn = 1.0f / sqrtf(s2[1] + 1e-6f);
  if (rg < RG) {
    f32x4 ak = {0.f, 0.f, 0.f, 0.f}, aq = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int r = min(rg + u * RG, dim - 1);  // (rows past the state hold zeros)
      const float kd = ks[r], qd = qs[r];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        ak[i] = fmaf(s[u][i], kd, ak[i]);
        aq[i] = fmaf(s[u][i], qd, aq[i]);
      }
    }
    *reinterpret_cast<f32x4*>(pk + (int64_t)rg * vdim + 4 * cg) = ak;
    *reinterpret_cast<f32x4*>(pq + (int64_t)rg * vdim + 4 * cg) = aq;
  }
  __syncthreads();
  float ss = 0.f;
  for (int c = tid; c < vdim; c += nthr) {
    float a = 0.f, o = 0.f;
    for (int r = 0; r < RG; ++r) {
      a += pk[r * vdim + c];
      o += pq[r * vdim + c];
    }
    const float v = El<T>::ld((const T*)A.v + (int64_t)t * A.ldv + (int64_t)h * vdim + c);
    const float u = beta * (v - g * kn * a);
    us[c] = u;
    o = g * qn * o + kq * kn * qn * u;
    pk[c] = o;  // (row 0 of the parts at this column: read by this thread alone)
    ss = fmaf(o, o, ss);
  }
  ss = block_sum(ss, red);  // (its barriers make us visible)
  if (rg < RG) {
    const f32x4 u4 = *reinterpret_cast<const f32x4*>(us + 4 * cg);
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int r = rg + u * RG;
      if (r < dim) {
        const float kd = ks[r] * kn;
        f32x4 x;
#pragma unroll
        for (int i = 0; i < 4; ++i) x[i] = fmaf(g, s[u][i], kd * u4[i]);
        *reinterpret_cast<f32x4*>(sp + (int64_t)r * vdim) = x;
      }
    }
  }
  const float inv = A.scale / sqrtf(ss / (float)vdim + A.eps);
  const T* gr = (const T*)A.gate + (int64_t)t * A.ldg + (int64_t)h * vdim;
  for (int c = tid; c < vdim; c += nthr) {
    const float z = El<T>::ld(gr + c);
    El<T>::st(yr + c, pk[c] * inv * El<T>::ld((const T*)A.w + c) * (z / (1.0f + expf(-z))));
  }
}

static int delta_step_threads(int dim, int vdim) {
  if (vdim % 4 || vdim < 4 || vdim > 1024 || dim < 1 || dim > 512) return 0;
  for (int th = 256; th <= 512; th *= 2)
    if (th >= vdim / 4 && (dim + th / (vdim / 4) - 1) / (th / (vdim / 4)) <= 16) return th;
  return 0;
}
bool delta_step_ok(int dim, int vdim) { return delta_step_threads(dim, vdim) > 0; }

// B sequences of one row each
void launch_delta_step(const void* q, const void* k, const void* v, int64_t ldq, int64_t ldk, int64_t ldv, const void* a,
                       const void* b, int64_t ldab, const void* A_log, const void* dt_bias, void* S, const void* cu,
                       const void* ctx, const void* sslots, const void* gate, int64_t ldg, const void* w, float eps,
                       float scale, void* y, int64_t ldy, int B, int H, int G, int dim, int vdim, int dt, hipStream_t st) {
  if (B == 0) return;
  const int th = delta_step_threads(dim, vdim);
  if (!th || B > 65535 || G < 1 || H % G) throw std::runtime_error("delta_step: shape");
  if ((uintptr_t)S & 15) throw std::runtime_error("delta_step: the state must be 16-byte aligned");
  DeltaStepArgs A{q, k, v, ldq, ldk, ldv, a, b, ldab, (const float*)A_log, (const float*)dt_bias, (float*)S, (const int*)cu,
                  (const int*)ctx, (const int*)sslots, gate, ldg, w, eps, scale, y, ldy, H, G, dim, vdim};
  const int RG = th / (vdim / 4), U = (dim + RG - 1) / RG;
  const size_t lds = ((size_t)2 * dim + 4 + vdim + (size_t)2 * RG * vdim) * 4;
  dim3 g(H, B);
  DISPATCH_T(dt, T, {
    if (U <= 4) delta_step_kernel<T, 4><<<g, th, lds, st>>>(A);
    else if (U <= 8) delta_step_kernel<T, 8><<<g, th, lds, st>>>(A);
    else delta_step_kernel<T, 16><<<g, th, lds, st>>>(A);
  });
  HIP_CHECK_LAUNCH();
}

// ------------------------------------------------------------------------------------------------ portions
struct DeltaChunkArgs {
  const bf16_t* q;
  const bf16_t* k;
  const bf16_t* v;
  int64_t ldq, ldk, ldv;
  const bf16_t* a;
  const bf16_t* b;
  int64_t ldab;
  const float* A_log;
  const float* dt_bias;
  float* S;
  const int* cu;
  const int* ctx;
  const int* sslots;
  float* out;  // [T, H * vdim]
  bf16_t* X;   // [4][T, H, 64]: X value, X remainder, P value, P remainder; row t of its chunk
  int64_t mat;  // numbers per matrix
  f32x4* aux;  // [T, H] (e^b |k|^-1, e^b |q|^-1 dim^-1/2, e^(b_C - b) |k|^-1, e^(b_C))
  int H, G, dim, vdim;
};

__device__ __forceinline__ void split2(float x, bf16_t& hi, bf16_t& lo) {
  hi = f2bf(x);
  lo = f2bf(x - bf2f(hi));
}

constexpr int prep_kq_bytes(int kt) {  // K and Q rows, or P (value, remainder) and the fp32 inverse
  return 2 * 64 * (16 * kt + 8) * 2 > 2 * 64 * 72 * 2 + 64 * 68 * 4 ? 2 * 64 * (16 * kt + 8) * 2 : 2 * 64 * 72 * 2 + 64 * 68 * 4;
}

// Workgroup (chunk of a portion, head, sequence), 4 waves
template <int KT>
__global__ __launch_bounds__(256) void delta_prep_kernel(DeltaChunkArgs A) {
  constexpr int C = 64, DKP = 16 * KT, LDK = DKP + 8, LDP = 64 + 8, LDL = 64 + 4;
  constexpr int KQ = prep_kq_bytes(KT);  // the rows' region; once their products are taken P and the inverse lie there
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
  bf16_t* Ks = reinterpret_cast<bf16_t*>(smem);
  bf16_t* Qs = Ks + C * LDK;
  bf16_t* Ph = reinterpret_cast<bf16_t*>(smem);
  bf16_t* Pl = Ph + C * LDP;
  float* Xs = reinterpret_cast<float*>(Pl + C * LDP);     // [64][LDL]
  float* Ls = reinterpret_cast<float*>(smem + KQ);        // [64][LDL]
  float* bs = Ls + C * LDL;                               // [64] sum of the log decays
  float* be = bs + C;                                  // [64] write strength
  float* nk = be + C;                                  // [64] 1 / |k|
  float* nq = nk + C;                                  // [64] dim^-1/2 / |q|
  const int b = blockIdx.z, h = blockIdx.y, tid = threadIdx.x, lane = tid & 63, w = tid >> 6, li = lane & 15, g = lane >> 4;
  const int t0 = A.cu[b], qlen = A.cu[b + 1] - t0, j0 = blockIdx.x * C;
  if (j0 >= qlen || A.sslots[b] < 0 || A.ctx[b] <= 0) return;
  const int nt = min(C, qlen - j0), dim = A.dim, H = A.H, gq = h / (H / A.G);
  constexpr int CHK = DKP / 8, NK = C * CHK / 256;
  static_assert((C * CHK) % 256 == 0, "whole 16-byte pieces per thread");
  const u16x8 zero8 = {0, 0, 0, 0, 0, 0, 0, 0};
#pragma unroll
  for (int j = 0; j < NK; ++j) {
    const int c = tid + 256 * j, r = c / CHK, d = (c % CHK) * 8;
    const bool in = r < nt && d < dim;
    const int64_t tt = t0 + j0 + r;
    *reinterpret_cast<u16x8*>(&Ks[r * LDK + d]) = in ? *reinterpret_cast<const u16x8*>(A.k + tt * A.ldk + (int64_t)gq * dim + d) : zero8;
    *reinterpret_cast<u16x8*>(&Qs[r * LDK + d]) = in ? *reinterpret_cast<const u16x8*>(A.q + tt * A.ldq + (int64_t)gq * dim + d) : zero8;
  }
  if (w == 0) {  // the tokens' decays and write strengths
    const bool in = lane < nt;
    const int64_t tt = (int64_t)(t0 + j0 + min(lane, nt - 1)) * A.ldab + h;
    const float z = bf2f(A.a[tt]) + A.dt_bias[h];
    float F = in ? -expf(A.A_log[h]) * (z > 20.f ? z : log1pf(expf(z))) : 0.f;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const float x = __shfl_up(F, o, 64);
      if (lane >= o) F += x;
    }
    bs[lane] = F;
    be[lane] = in ? 1.0f / (1.0f + expf(-bf2f(A.b[tt]))) : 0.f;
  }
  __syncthreads();
  {  // norms: four neighbouring lanes per row
    const int r = tid >> 2, part = tid & 3;
    float kk = 0.f, qq = 0.f;
    for (int d = part * 8; d < DKP; d += 32) {
      const u16x8 x = *reinterpret_cast<const u16x8*>(&Ks[r * LDK + d]), y = *reinterpret_cast<const u16x8*>(&Qs[r * LDK + d]);
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        kk = fmaf(bf2f(x[i]), bf2f(x[i]), kk);
        qq = fmaf(bf2f(y[i]), bf2f(y[i]), qq);
      }
    }
    kk += __shfl_xor(kk, 1, 64);
    kk += __shfl_xor(kk, 2, 64);
    qq += __shfl_xor(qq, 1, 64);
    qq += __shfl_xor(qq, 2, 64);
    if (part == 0) {
      nk[r] = 1.0f / sqrtf(kk + 1e-6f);
      nq[r] = 1.0f / (sqrtf(qq + 1e-6f) * sqrtf((float)dim));
    }
  }
  __syncthreads();
  // wave w: the products of its 16 tokens (rows) with the keys of the blocks up to its own (columns)
  {
    f32x4 pk[4], pq[4];
#pragma unroll
    for (int ct = 0; ct < 4; ++ct) pk[ct] = pq[ct] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int ks = 0; ks < KT / 2; ++ks) {
      const s16x8 ka = *reinterpret_cast<const s16x8*>(&Ks[(16 * w + li) * LDK + 32 * ks + 8 * g]);
      const s16x8 qa = *reinterpret_cast<const s16x8*>(&Qs[(16 * w + li) * LDK + 32 * ks + 8 * g]);
#pragma unroll
      for (int ct = 0; ct < 4; ++ct) {
        if (ct > w) continue;
        const s16x8 kb = *reinterpret_cast<const s16x8*>(&Ks[(16 * ct + li) * LDK + 32 * ks + 8 * g]);
        pk[ct] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ka, kb, pk[ct], 0, 0, 0);
        pq[ct] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qa, kb, pq[ct], 0, 0, 0);
      }
    }
    __syncthreads();  // every wave has read its rows
#pragma unroll
    for (int ct = 0; ct < 4; ++ct) {
      const int s = 16 * ct + li;
      const float bsv = bs[s], nks = nk[s];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int t = 16 * w + 4 * g + i;
        const float e = s <= t ? expf(bs[t] - bsv) * nks : 0.f;
        Ls[t * LDL + s] = s < t ? e * be[t] * nk[t] * pk[ct][i] : 0.f;
        split2(s <= t ? e * nq[t] * pq[ct][i] : 0.f, Ph[t * LDP + s], Pl[t * LDP + s]);
        if (ct > w) Xs[t * LDL + s] = 0.f;  // the blocks of the inverse above the diagonal
      }
    }
  }
  __syncthreads();
  // (I + L)^-1: wave w its 16 x 16 diagonal block by substitution, a column per lane (four copies of each)
  {
    float x[16];
#pragma unroll
    for (int t = 0; t < 16; ++t) x[t] = t == li ? 1.0f : 0.f;
#pragma unroll
    for (int t = 1; t < 16; ++t) {
      const float* lr = &Ls[(16 * w + t) * LDL + 16 * w];
      float acc = 0.f, acc2 = 0.f;
#pragma unroll
      for (int s = 0; s < t; ++s) {
        if (s & 1) acc2 = fmaf(lr[s], x[s], acc2);
        else acc = fmaf(lr[s], x[s], acc);
      }
      x[t] -= acc + acc2;
    }
#pragma unroll
    for (int t = 0; t < 16; ++t)
      if ((t >> 2) == g) Xs[(16 * w + t) * LDL + 16 * w + li] = x[t];
  }
  // the blocks below, a diagonal at a time: X_ij = -X_ii sum_{j <= m < i} L_im X_mj
#pragma unroll
  for (int lev = 1; lev < 4; ++lev) {
    __syncthreads();
    const int bi = w + lev, bj = w;
    if (bi < 4) {
      f32x4 z = {0.f, 0.f, 0.f, 0.f}, o = {0.f, 0.f, 0.f, 0.f};
      for (int m = bj; m < bi; ++m) {
#pragma unroll
        for (int i = 0; i < 4; ++i)
          z = __builtin_amdgcn_mfma_f32_16x16x4f32(Ls[(16 * bi + li) * LDL + 16 * m + 4 * g + i],
                                                   Xs[(16 * m + 4 * g + i) * LDL + 16 * bj + li], z, 0, 0, 0);
      }
#pragma unroll
      for (int i = 0; i < 4; ++i)  // (the accumulator's rows 4 g + i are the second operand as they stand)
        o = __builtin_amdgcn_mfma_f32_16x16x4f32(Xs[(16 * bi + li) * LDL + 16 * bi + 4 * g + i], z[i], o, 0, 0, 0);
#pragma unroll
      for (int i = 0; i < 4; ++i) Xs[(16 * bi + 4 * g + i) * LDL + 16 * bj + li] = -o[i];
    }
  }
  __syncthreads();
  const int64_t row = (int64_t)(t0 + j0) * H + h;
  for (int e = tid; e < C * 8; e += 256) {
    const int r = e >> 3, s0 = (e & 7) * 8;
    if (r >= nt) continue;
    u16x8 xh, xl;
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      bf16_t hi, lo;
      split2(Xs[r * LDL + s0 + i] * be[s0 + i], hi, lo);
      xh[i] = hi;
      xl[i] = lo;
    }
    bf16_t* dst = A.X + (row + (int64_t)r * H) * 64 + s0;
    *reinterpret_cast<u16x8*>(dst) = xh;
    *reinterpret_cast<u16x8*>(dst + A.mat) = xl;
    *reinterpret_cast<u16x8*>(dst + 2 * A.mat) = *reinterpret_cast<const u16x8*>(&Ph[r * LDP + s0]);
    *reinterpret_cast<u16x8*>(dst + 3 * A.mat) = *reinterpret_cast<const u16x8*>(&Pl[r * LDP + s0]);
  }
  if (tid < nt) {
    const float e = expf(bs[tid]), bc = bs[C - 1];
    A.aux[row + (int64_t)tid * H] = f32x4{e * nk[tid], e * nq[tid], expf(bc - bs[tid]) * nk[tid], expf(bc)};
  }
}

// Workgroup (head, block of 64 value columns, sequence), 4 waves, the portion's chunks in order. A wave owns 16 value columns:
// its part of the state lives in registers in the accumulator layout (lane (li, g): column li, rows 16 tile + 4 g + i), whose
// rows are, without any exchange, the k-slots (8 g + j -> row 4 g + j of tile 2 ks, j < 4, or 4 g + j - 4 of tile 2 ks + 1) of
// the second operand of the next product - and so are V - e^b K S_0 and U over the tokens. The next chunk's rows and
// matrices are fetched into registers while this one is computed; nothing inside a chunk waits for another wave.
template <int KT>
__global__ __launch_bounds__(256) void delta_chunk_kernel(DeltaChunkArgs A) {
  constexpr int C = 64, DKP = 16 * KT, LDK = DKP + 8, LDP = 64 + 8;
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
  bf16_t* Qs = reinterpret_cast<bf16_t*>(smem);
  bf16_t* Ks = Qs + C * LDK;
  bf16_t* Ms = Ks + C * LDK;                          // [4][64][LDP]
  f32x4* ax = reinterpret_cast<f32x4*>(Ms + 4 * C * LDP);  // [64]
  const int h = blockIdx.x, b = gridDim.z - 1 - blockIdx.z;
  const int dim = A.dim, vdim = A.vdim, H = A.H, gq = h / (H / A.G);
  const int t0 = A.cu[b], qlen = A.cu[b + 1] - t0, slot = A.sslots[b], ctx = A.ctx[b];
  if (qlen <= 0) return;
  const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6, li = lane & 15, g = lane >> 4;
  const int col = blockIdx.y * 64 + 16 * w + li, colc = min(col, vdim - 1);
  float* outp = A.out + (int64_t)t0 * H * vdim + (int64_t)h * vdim + col;
  if (slot < 0 || ctx <= 0) {
    if (g == 0 && col < vdim)
      for (int j = 0; j < qlen; ++j) outp[(int64_t)j * H * vdim] = 0.f;
    return;
  }
  const bool cont = ctx > qlen;  // continues an earlier portion
  f32x4 S[KT];
  float* sp = A.S + (((int64_t)slot * H + h) * dim) * (int64_t)vdim;
#pragma unroll
  for (int kt = 0; kt < KT; ++kt)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int r = 16 * kt + 4 * g + i;
      S[kt][i] = (cont && r < dim && col < vdim) ? sp[(int64_t)r * vdim + col] : 0.f;
    }
  constexpr int CHK = DKP / 8, NK = C * CHK / 256;
  u16x8 rq[NK], rk[NK], rm[8];
  bf16_t rv[16];
  f32x4 ra = {0.f, 0.f, 0.f, 0.f};
  const u16x8 zero8 = {0, 0, 0, 0, 0, 0, 0, 0};
  auto fetch = [&](int j0) {
#pragma unroll
    for (int j = 0; j < NK; ++j) {
      const int c = tid + 256 * j, r = c / CHK, d = (c % CHK) * 8;
      const bool in = j0 + r < qlen && d < dim;
      const int64_t tt = t0 + j0 + r;
      rq[j] = in ? *reinterpret_cast<const u16x8*>(A.q + tt * A.ldq + (int64_t)gq * dim + d) : zero8;
      rk[j] = in ? *reinterpret_cast<const u16x8*>(A.k + tt * A.ldk + (int64_t)gq * dim + d) : zero8;
    }
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      const int c = tid + 256 * (j & 1), r = c >> 3, s0 = (c & 7) * 8;
      rm[j] = j0 + r < qlen ? *reinterpret_cast<const u16x8*>(A.X + (j >> 1) * A.mat + ((int64_t)(t0 + j0 + r) * H + h) * 64 + s0)
                            : zero8;
    }
#pragma unroll
    for (int j = 0; j < 16; ++j) {  // token 16 (j / 4) + 4 g + j % 4 at this lane's column
      const int r = j0 + 16 * (j >> 2) + 4 * g + (j & 3);
      rv[j] = A.v[(int64_t)(t0 + min(r, qlen - 1)) * A.ldv + (int64_t)h * vdim + colc];
    }
    if (w == 0) ra = A.aux[(int64_t)(t0 + min(j0 + lane, qlen - 1)) * H + h];
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
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      const int c = tid + 256 * (j & 1);
      *reinterpret_cast<u16x8*>(&Ms[(j >> 1) * C * LDP + (c >> 3) * LDP + (c & 7) * 8]) = rm[j];
    }
    if (w == 0) ax[lane] = ra;
    f32x4 u[4];  // first V, then V - e^b K S_0
#pragma unroll
    for (int j = 0; j < 16; ++j) u[j >> 2][j & 3] = bf2f(rv[j]);
    __syncthreads();
    if (j0 + C < qlen) fetch(j0 + C);
    // K S_0 and Q S_0 for this wave's columns
    f32x4 o[4], ksv[4];
#pragma unroll
    for (int rt = 0; rt < 4; ++rt) o[rt] = ksv[rt] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int ks = 0; ks < KT / 2; ++ks) {
      s16x8 sh, sl;
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        bf16_t hi, lo;
        split2(S[2 * ks + (j >> 2)][j & 3], hi, lo);
        sh[j] = (short)hi;
        sl[j] = (short)lo;
      }
#pragma unroll
      for (int rt = 0; rt < 4; ++rt) {
        const bf16_t* kp = &Ks[(16 * rt + li) * LDK + 32 * ks + 4 * g];
        const s16x4 k0 = *reinterpret_cast<const s16x4*>(kp), k1 = *reinterpret_cast<const s16x4*>(kp + 16);
        const s16x8 ka = {k0[0], k0[1], k0[2], k0[3], k1[0], k1[1], k1[2], k1[3]};
        ksv[rt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ka, sh, ksv[rt], 0, 0, 0);
        ksv[rt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ka, sl, ksv[rt], 0, 0, 0);
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
    f32x4 wgt[4];  // e^(b_C - b) |k|^-1 of this lane's tokens
#pragma unroll
    for (int rt = 0; rt < 4; ++rt)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const f32x4 x = ax[16 * rt + 4 * g + i];
        u[rt][i] = fmaf(-x[0], ksv[rt][i], u[rt][i]);
        o[rt][i] *= x[1];
        wgt[rt][i] = x[2];
      }
    const float a_all = ax[0][3];
    // the products with X and then P: operand rows 16 rt + li, the second operand in registers
    auto lower = [&](const bf16_t* m, const f32x4* x, f32x4* acc) {
#pragma unroll
      for (int ks = 0; ks < 2; ++ks) {
        s16x8 xh, xl;
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          bf16_t hi, lo;
          split2(x[2 * ks + (j >> 2)][j & 3], hi, lo);
          xh[j] = (short)hi;
          xl[j] = (short)lo;
        }
#pragma unroll
        for (int rt = 0; rt < 4; ++rt) {
          if (16 * rt + 15 < 32 * ks) continue;  // tokens before every token of this half
          const bf16_t* p = &m[(16 * rt + li) * LDP + 32 * ks + 4 * g];
          const s16x4 h0 = *reinterpret_cast<const s16x4*>(p), h1 = *reinterpret_cast<const s16x4*>(p + 16);
          const s16x4 l0 = *reinterpret_cast<const s16x4*>(p + C * LDP), l1 = *reinterpret_cast<const s16x4*>(p + C * LDP + 16);
          const s16x8 mh = {h0[0], h0[1], h0[2], h0[3], h1[0], h1[1], h1[2], h1[3]};
          const s16x8 ml = {l0[0], l0[1], l0[2], l0[3], l1[0], l1[1], l1[2], l1[3]};
          acc[rt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(mh, xh, acc[rt], 0, 0, 0);
          acc[rt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(mh, xl, acc[rt], 0, 0, 0);
          acc[rt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ml, xh, acc[rt], 0, 0, 0);
        }
      }
    };
    f32x4 U[4];
#pragma unroll
    for (int rt = 0; rt < 4; ++rt) U[rt] = f32x4{0.f, 0.f, 0.f, 0.f};
    lower(Ms, u, U);
    lower(Ms + 2 * C * LDP, U, o);
    // the state: K^T (w U)
#pragma unroll
    for (int kt = 0; kt < KT; ++kt)
#pragma unroll
      for (int i = 0; i < 4; ++i) S[kt][i] *= a_all;
    const int tq = li >> 2, tp = li & 3;
#pragma unroll
    for (int ks = 0; ks < 2; ++ks) {
      s16x8 vh, vl;
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        bf16_t hi, lo;
        split2(U[2 * ks + (j >> 2)][j & 3] * wgt[2 * ks + (j >> 2)][j & 3], hi, lo);
        vh[j] = (short)hi;
        vl[j] = (short)lo;
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
          if (t < nt) outp[(int64_t)(j0 + t) * H * vdim] = o[rt][i];
        }
    }
  }
  if (col < vdim) {
#pragma unroll
    for (int kt = 0; kt < KT; ++kt)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int r = 16 * kt + 4 * g + i;
        if (r < dim) sp[(int64_t)r * vdim + col] = S[kt][i];
      }
  }
}

bool delta_chunk_ok(int dim, int vdim) { return dim % 8 == 0 && dim >= 8 && dim <= 256 && vdim >= 1; }

// max_qlen: rows of the longest portion; work: bf16 [4][T, H, 64]; aux: fp32 [T, H, 4]
void launch_delta_chunk(const void* q, const void* k, const void* v, int64_t ldq, int64_t ldk, int64_t ldv, const void* a,
                        const void* b, int64_t ldab, const void* A_log, const void* dt_bias, void* S, const void* cu,
                        const void* ctx, const void* sslots, void* out, void* work, void* aux, int T_, int B, int max_qlen,
                        int H, int G, int dim, int vdim, hipStream_t st) {
  if (B == 0 || max_qlen <= 0) return;
  if (!delta_chunk_ok(dim, vdim) || B > 65535 || H > 65535 || G < 1 || H % G) throw std::runtime_error("delta_chunk: shape");
  if (((uintptr_t)q | (uintptr_t)k | (uintptr_t)work | (uintptr_t)aux) & 15 || (ldq | ldk) & 7)
    throw std::runtime_error("delta_chunk: rows must be 16-byte aligned");
  DeltaChunkArgs A{(const bf16_t*)q, (const bf16_t*)k, (const bf16_t*)v, ldq, ldk, ldv, (const bf16_t*)a, (const bf16_t*)b,
                   ldab, (const float*)A_log, (const float*)dt_bias, (float*)S, (const int*)cu, (const int*)ctx,
                   (const int*)sslots, (float*)out, (bf16_t*)work, (int64_t)T_ * H * 64, (f32x4*)aux, H, G, dim, vdim};
  dim3 g1((max_qlen + 63) / 64, H, B), g2(H, (vdim + 63) / 64, B);
  auto lds1 = [](int kt) {
    return (size_t)prep_kq_bytes(kt) + (size_t)4 * (64 * 68 + 4 * 64);
  };
  auto lds2 = [](int kt) { return (size_t)2 * (2 * 64 * (16 * kt + 8) + 4 * 64 * 72) + (size_t)16 * 64; };
#define LAUNCH_DC(KT_)                                                                                           \
  do {                                                                                                           \
    static bool once = [] {                                                                                      \
      (void)hipFuncSetAttribute((const void*)delta_prep_kernel<KT_>, hipFuncAttributeMaxDynamicSharedMemorySize, \
                                160 * 1024);                                                                     \
      (void)hipFuncSetAttribute((const void*)delta_chunk_kernel<KT_>, hipFuncAttributeMaxDynamicSharedMemorySize, \
                                160 * 1024);                                                                     \
      return true;                                                                                               \
    }();                                                                                                         \
    (void)once;                                                                                                  \
    delta_prep_kernel<KT_><<<g1, 256, lds1(KT_), st>>>(A);                                                       \
    delta_chunk_kernel<KT_><<<g2, 256, lds2(KT_), st>>>(A);                                                      \
  } while (0)
  if (dim <= 32) LAUNCH_DC(2);
  else if (dim <= 64) LAUNCH_DC(4);
  else if (dim <= 128) LAUNCH_DC(8);
  else LAUNCH_DC(16);
#undef LAUNCH_DC
  HIP_CHECK_LAUNCH();
}
