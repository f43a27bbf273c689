// Selective scan: a diagonal state-space recurrence whose step size, input and output vectors depend on the token.
//
// Every channel c keeps a state S[c, :] of N fp32 numbers. Per token, with the channel's input x_c, step input dt_c and the
// token's vectors B and C (shared by all channels):
//
//   d = softplus(dt_c + dt_bias_c);  S[c, n] <- exp(d A[c, n]) S[c, n] + d x_c B_n;  y_c = sum_n S[c, n] C_n + D_c x_c
//   out = y_c * silu(z_c)
//
// A workgroup owns (64 channels, sequence): four neighbouring lanes share a channel and hold R = ceil(N / 4) of its state
// numbers each in registers, with the matching decay rates; a channel's sum over n is two lane swaps. Tokens are walked in
// order, CT of them staged in LDS at a time (step size, step size * input, skip term and gate per channel, computed once
// while staging; B and C once per workgroup), the next CT tokens' numbers in flight in registers behind the arithmetic. The
// decay is exp2 of the fp32 product with A log2(e). The state is read from the sequence's slot unless the portion starts at
// position 0 (then it is zero, whatever the slot held) and written back at the end. Rows of a padded sequence are zeroed.
// Tokens past a portion's end are staged with step size 0, which leaves the state as it is.
#include "anytype.h"

#define SS_CH 64
#define SS_LDY 80  // row stride of the sums: the four lanes of a channel write four rows, 16 banks apart

struct ScanArgs {
  const void* x;  // [T, ldx]
  int64_t ldx;
  const float* dt;  // [T, ldt]
  int64_t ldt;
  const float* dt_bias;  // [inner]
  const void* Bm;        // [T, ldb]
  const void* Cm;
  int64_t ldb;
  const float* A;  // [inner, N]
  const float* D;  // [inner]
  const void* z;   // [T, ldz]
  int64_t ldz;
  float* state;  // [slots, inner, N]
  const int* cu;
  const int* ctx;
  const int* sslots;
  void* out;  // [T, ldo]
  int64_t ldo;
  int inner, N;
};

template <int CTRL>
__device__ __forceinline__ float ss_swap(float v) {
  return __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), CTRL, 0xF, 0xF, false));
}

// softplus and silu: bf16 rows take the hardware's exponential, logarithm and reciprocal (a few units in the last place of
// fp32; log(1 + e) corrected for the rounding of 1 + e), fp32 rows the library's functions
template <typename T>
__device__ __forceinline__ float ss_softplus(float q) {
  if constexpr (sizeof(T) == 4) {
    return q > 20.f ? q : log1pf(expf(q));
  } else {
    const float e = __builtin_amdgcn_exp2f(1.4426950408889634f * q), u = 1.0f + e, d = u - 1.0f;
    const float l = 0.6931471805599453f * __builtin_amdgcn_logf(u) * e * __builtin_amdgcn_rcpf(d);
    return q > 20.f ? q : (d == 0.f ? e : l);
  }
}
template <typename T>
__device__ __forceinline__ float ss_silu(float z) {
  if constexpr (sizeof(T) == 4) return z / (1.0f + expf(-z));
  else return z * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-1.4426950408889634f * z));
}

// CT: tokens staged at a time (16 in portions, 4 where every sequence has one row)
template <typename T, int R, int CT>
__global__ __launch_bounds__(256) void selective_scan_kernel(ScanArgs p) {
  constexpr int NP = 4 * R, NI = CT / 4, NB = (CT * 2 * NP + 255) / 256;
  __shared__ __attribute__((aligned(16))) float sdx[CT * SS_CH * 2];  // (step size, step size * input)
  __shared__ __attribute__((aligned(16))) float sy[CT * SS_LDY], sg[CT * SS_CH];
  __shared__ __attribute__((aligned(16))) float sbc[CT * 2 * NP];  // per token: B padded to NP, C padded to NP
  // sequences in reverse step order: the step's long portions come last and are dispatched first
  const int b = gridDim.y - 1 - blockIdx.y, tid = threadIdx.x;
  const int t0 = p.cu[b], qlen = p.cu[b + 1] - t0, n = p.ctx[b], slot = p.sslots[b];
  if (qlen <= 0) return;
  const int c0 = blockIdx.x * SS_CH, N = p.N;
  // staging: this thread's channel and its tokens it, it + 4, ... of every CT
  const int ic = tid & 63, it = tid >> 6, cs = min(c0 + ic, p.inner - 1);
  const bool live_s = c0 + ic < p.inner;
  T* outp = (T*)p.out + (int64_t)t0 * p.ldo + c0 + ic;
  if (slot < 0 || n <= 0) {
    if (live_s)
      for (int j = it; j < qlen; j += 4) El<T>::st(outp + (int64_t)j * p.ldo, 0.f);
    return;
  }
  // recurrence: this lane's channel and its part of the state
  const int ch = tid >> 2, part = tid & 3, d0 = part * R;
  const int c = min(c0 + ch, p.inner - 1);
  const bool live = c0 + ch < p.inner;
  float* sp = p.state + ((int64_t)slot * p.inner + c) * N;
  const float* ap = p.A + (int64_t)c * N;
  const bool cont = n > qlen;
  float S[R], A2[R];
  if (N % 4 == 0) {
#pragma unroll
    for (int i = 0; i < R; i += 4) {
      const bool in = d0 + i < N;
      const f32x4 a = *reinterpret_cast<const f32x4*>(ap + (in ? d0 + i : 0));
      const f32x4 s = cont ? *reinterpret_cast<const f32x4*>(sp + (in ? d0 + i : 0)) : f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int k = 0; k < 4; ++k) {
        A2[i + k] = in ? a[k] * 1.4426950408889634f : 0.f;
        S[i + k] = in ? s[k] : 0.f;
      }
    }
  } else {
#pragma unroll
    for (int i = 0; i < R; ++i) {
      const bool in = d0 + i < N;
      A2[i] = in ? ap[d0 + i] * 1.4426950408889634f : 0.f;
      S[i] = in && cont ? sp[d0 + i] : 0.f;
    }
  }
  const float dtb = p.dt_bias[cs], Dc = p.D[cs];
  const T* xp = (const T*)p.x + (int64_t)t0 * p.ldx + cs;
  const T* zp = (const T*)p.z + (int64_t)t0 * p.ldz + cs;
  const float* dp = p.dt + (int64_t)t0 * p.ldt + cs;
  float rx[NI], rz[NI], rd[NI], rb[NB];
  auto fetch = [&](int j0) {  // rows past the portion's end repeat its last row: they are staged and never used
#pragma unroll
    for (int k = 0; k < NI; ++k) {
      const int64_t j = min(j0 + it + 4 * k, qlen - 1);
      rx[k] = El<T>::ld(xp + j * p.ldx);
      rz[k] = El<T>::ld(zp + j * p.ldz);
      rd[k] = dp[j * p.ldt];
    }
#pragma unroll
    for (int k = 0; k < NB; ++k) {
      const int e = tid + 256 * k, row = min(e / (2 * NP), CT - 1), q = e % (2 * NP), m = q % NP;
      const int64_t j = t0 + min(j0 + row, qlen - 1);
      const float v = El<T>::ld((q < NP ? (const T*)p.Bm : (const T*)p.Cm) + j * p.ldb + min(m, N - 1));
      rb[k] = m < N ? v : 0.f;
    }
  };
  fetch(0);
  for (int j0 = 0; j0 < qlen; j0 += CT) {
    const int nt = min(CT, qlen - j0);
#pragma unroll
    for (int k = 0; k < NI; ++k) {
      const int j = it + 4 * k;
      const float d = j < nt ? ss_softplus<T>(rd[k] + dtb) : 0.f;
      *reinterpret_cast<f32x2*>(&sdx[(j * SS_CH + ic) * 2]) = f32x2{d, d * rx[k]};
      sy[j * SS_LDY + ic] = Dc * rx[k];
      sg[j * SS_CH + ic] = ss_silu<T>(rz[k]);
    }
#pragma unroll
    for (int k = 0; k < NB; ++k) {
      const int e = tid + 256 * k;
      if (e < CT * 2 * NP) sbc[e] = rb[k];
    }
    __syncthreads();
    if (j0 + CT < qlen) fetch(j0 + CT);
    constexpr int UNR = R <= 8 ? CT / 4 : 1;
#pragma unroll UNR
    for (int m = 0; m < CT / 4; ++m) {
      float yv[4];
#pragma unroll
      for (int q = 0; q < 4; ++q) {
        const int jj = 4 * m + q;
        const f32x2 dx = *reinterpret_cast<const f32x2*>(&sdx[(jj * SS_CH + ch) * 2]);
        const float* bp = sbc + jj * 2 * NP + d0;
        float y = 0.f, y2 = 0.f;
#pragma unroll
        for (int i = 0; i < R; i += 4) {
          const f32x4 bv = *reinterpret_cast<const f32x4*>(bp + i), cv = *reinterpret_cast<const f32x4*>(bp + NP + i);
#pragma unroll
          for (int k = 0; k < 4; ++k) {
            S[i + k] = fmaf(__builtin_amdgcn_exp2f(dx[0] * A2[i + k]), S[i + k], dx[1] * bv[k]);
            if (k & 1) y2 = fmaf(S[i + k], cv[k], y2);
            else y = fmaf(S[i + k], cv[k], y);
          }
        }
        y += y2;
        y += ss_swap<0xB1>(y);  // lanes 0 <-> 1, 2 <-> 3
        y += ss_swap<0x4E>(y);  // lanes 0 <-> 2, 1 <-> 3
        yv[q] = y;
      }
      // every lane of the channel holds the four tokens' sums; each adds one of them to its row
      sy[(4 * m + part) * SS_LDY + ch] += part & 2 ? (part & 1 ? yv[3] : yv[2]) : (part & 1 ? yv[1] : yv[0]);
    }
    __syncthreads();  // the rows' sums are complete, and every reader of the staged numbers is done
    if (live_s) {
#pragma unroll
      for (int k = 0; k < NI; ++k) {
        const int j = it + 4 * k;
        if (j < nt) El<T>::st(outp + (int64_t)(j0 + j) * p.ldo, sy[j * SS_LDY + ic] * sg[j * SS_CH + ic]);
      }
    }
  }
  if (!live) return;
  if (N % 4 == 0) {
#pragma unroll
    for (int i = 0; i < R; i += 4)
      if (d0 + i < N) *reinterpret_cast<f32x4*>(sp + d0 + i) = f32x4{S[i], S[i + 1], S[i + 2], S[i + 3]};
  } else {
#pragma unroll
    for (int i = 0; i < R; ++i)
      if (d0 + i < N) sp[d0 + i] = S[i];
  }
}

// all_single: every sequence of the step has one row
template <typename T>
static void selective_scan_t(const ScanArgs& p, int B, int all_single, hipStream_t st) {
  dim3 g((p.inner + SS_CH - 1) / SS_CH, B);
#define LAUNCH_SS(R_)                                                            \
  do {                                                                           \
    if (all_single) selective_scan_kernel<T, R_, 4><<<g, 256, 0, st>>>(p);       \
    else selective_scan_kernel<T, R_, 16><<<g, 256, 0, st>>>(p);                 \
  } while (0)
  if (p.N <= 16) LAUNCH_SS(4);
  else if (p.N <= 32) LAUNCH_SS(8);
  else if (p.N <= 64) LAUNCH_SS(16);
  else if (p.N <= 128) LAUNCH_SS(32);
  else LAUNCH_SS(64);
#undef LAUNCH_SS
}

void launch_selective_scan(const void* x, int64_t ldx, const void* dt, int64_t ldt, const void* dt_bias, const void* Bm,
                           const void* Cm, int64_t ldb, const void* A, const void* D, const void* z, int64_t ldz,
                           void* state, const void* cu, const void* ctx, const void* sslots, void* out, int64_t ldo, int B,
                           int inner, int N, int all_single, int dtype, hipStream_t st) {
  if (B == 0) return;
  if (N < 1 || N > 256) throw std::runtime_error("selective_scan: 1 to 256 state numbers per channel");
  if (B > 65535 || inner < 1) throw std::runtime_error("selective_scan: too many sequences");
  if (N % 4 == 0 && (((uintptr_t)A | (uintptr_t)state) & 15)) throw std::runtime_error("selective_scan: A, state 16-byte aligned");
  ScanArgs p{x, ldx, (const float*)dt, ldt, (const float*)dt_bias, Bm, Cm, ldb, (const float*)A, (const float*)D, z, ldz,
             (float*)state, (const int*)cu, (const int*)ctx, (const int*)sslots, out, ldo, inner, N};
  DISPATCH_T(dtype, T, (selective_scan_t<T>(p, B, all_single, st)));
  HIP_CHECK_LAUNCH();
}
