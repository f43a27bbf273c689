// Query, key and value heads of an attention layer on their way into the paged cache, one launch from the projection row:
//
//   u = projection row (q | k | v columns), or a short causal convolution over time of it (no activation):
//       u[t, c] = sum_k w[k, c] x[t - (taps - 1) + k, c], inputs before the portion from the sequence's tail
//   q, k: per head  x <- x / sqrt(mean(x^2) + eps) * weight  (optional), then the first 2 * half numbers turned by the
//         row's angles cs [T, half, 2], number i paired with i + half (optional)
//   v:    the key columns as they were projected where there is no value projection (off_v == off_k); per head
//         v <- v / sqrt(mean(v^2) + eps) (optional), then all vdim numbers turned by vcs [T, vdim / 2, 2] (optional)
//
// q leaves in fp32 [T, H * dim] or, for the matrix-core attention kernel, in bf16; k and v go into the paged caches at slots[t] (< 0: not cached), in the storage type.
// Norms, angles and the convolution's sum are fp32. One workgroup per row: the row's numbers are formed in LDS, then a wave
// takes a head at a time. In a step of single rows (tail_here) the workgroup also renews its sequence's tail - nobody
// else reads it; portions renew theirs in a second launch, after every row has read the old one.
#include "anytype.h"
#include "seqrows.h"

struct HeadPrepArgs {
  const void* proj;
  int64_t ldp;
  int off_q, off_k, off_v;
  const void* conv;  // [taps, nq + nk + nv] (columns q | k | v, contiguous in the projection) or null
  int taps;
  float* tail;  // [slots, taps - 1, nq + nk + nv]
  int tail_here;
  const int* cu;
  const int* ctx;
  const int* sslots;
  int B;
  const float* qw;  // [dim] or null
  const float* kw;
  int vnorm;
  float eps;
  const float* cs;
  int half;
  const float* vcs;
  void* q;
  int q_bf;
  void* kc;
  void* vc;
  const int64_t* slots;
  int H, G, dim, vdim;
};

template <typename T, int V>
__device__ __forceinline__ void hp_ld(const T* p, float* v) {
  if constexpr (V == 8) {
    const u16x8 x = *reinterpret_cast<const u16x8*>(p);
#pragma unroll
    for (int i = 0; i < 8; ++i) v[i] = bf2f(x[i]);
  } else if constexpr (V == 4) {
    const f32x4 x = *reinterpret_cast<const f32x4*>(p);
#pragma unroll
    for (int i = 0; i < 4; ++i) v[i] = x[i];
  } else {
    v[0] = El<T>::ld(p);
  }
}

// Heads whose vectors are whole 16-byte pieces: N / 8 neighbouring lanes (a power of two) share a vector, each lane takes
// eight numbers and, where they are turned, the eight they are paired with; the sum of squares is added up over the lanes.
template <typename T>
__device__ __forceinline__ void head_vec(const HeadPrepArgs& A, const float* x0, int heads, int N, const float* w, bool norm,
                                         int half, const float* tab, int kind, int64_t dst) {
  const int L = N >> 3, sub = threadIdx.x & (L - 1), per = blockDim.x / L, d = 8 * sub;
  const bool turn = d < 2 * half, lo = d < half;
  const int od = lo ? d + half : d - half;
  for (int n = threadIdx.x / L; n < heads; n += per) {
    const float* x = x0 + n * N;
    float a[8], o[8];
    *reinterpret_cast<f32x4*>(a) = *reinterpret_cast<const f32x4*>(x + d);
    *reinterpret_cast<f32x4*>(a + 4) = *reinterpret_cast<const f32x4*>(x + d + 4);
    float inv = 1.f;
    if (norm) {
      float s = 0.f;
#pragma unroll
      for (int i = 0; i < 8; ++i) s = fmaf(a[i], a[i], s);
      for (int m = L >> 1; m > 0; m >>= 1) s += __shfl_xor(s, m, 64);
      inv = 1.0f / sqrtf(s / (float)N + A.eps);
    }
    if (w) {
#pragma unroll
      for (int i = 0; i < 8; ++i) a[i] *= inv * w[d + i];
    } else {
#pragma unroll
      for (int i = 0; i < 8; ++i) a[i] *= inv;
    }
    if (turn) {
      *reinterpret_cast<f32x4*>(o) = *reinterpret_cast<const f32x4*>(x + od);
      *reinterpret_cast<f32x4*>(o + 4) = *reinterpret_cast<const f32x4*>(x + od + 4);
      const float* tb = tab + 2 * (lo ? d : od);
#pragma unroll
      for (int i = 0; i < 8; i += 2) {
        const f32x4 cs = *reinterpret_cast<const f32x4*>(tb + 2 * i);
        const float o0 = o[i] * inv * (w ? w[od + i] : 1.0f), o1 = o[i + 1] * inv * (w ? w[od + i + 1] : 1.0f);
        a[i] = lo ? a[i] * cs[0] - o0 * cs[1] : a[i] * cs[0] + o0 * cs[1];
        a[i + 1] = lo ? a[i + 1] * cs[2] - o1 * cs[3] : a[i + 1] * cs[2] + o1 * cs[3];
      }
    }
    const int64_t at = dst + (int64_t)n * N + d;
    if (sizeof(T) == 2 && (kind != 0 || A.q_bf)) {
      u16x8 y;
#pragma unroll
      for (int i = 0; i < 8; ++i) y[i] = f2bf(a[i]);
      *reinterpret_cast<u16x8*>((bf16_t*)(kind == 0 ? A.q : kind == 1 ? A.kc : A.vc) + at) = y;
    } else {
      float* p = (float*)(kind == 0 ? A.q : kind == 1 ? A.kc : A.vc) + at;
      *reinterpret_cast<f32x4*>(p) = *reinterpret_cast<f32x4*>(a);
      *reinterpret_cast<f32x4*>(p + 4) = *reinterpret_cast<f32x4*>(a + 4);
    }
  }
}

// V numbers of a tail row (fp32; whole 16-byte pieces where V is one)
template <int V>
__device__ __forceinline__ void hp_ldf(const float* p, float* v) {
  if constexpr (V >= 4) {
#pragma unroll
    for (int i = 0; i < V; i += 4) *reinterpret_cast<f32x4*>(v + i) = *reinterpret_cast<const f32x4*>(p + i);
  } else {
    v[0] = p[0];
  }
}
template <int V>
__device__ __forceinline__ void hp_stf(float* p, const float* v) {
  if constexpr (V >= 4) {
#pragma unroll
    for (int i = 0; i < V; i += 4) *reinterpret_cast<f32x4*>(p + i) = *reinterpret_cast<const f32x4*>(v + i);
  } else {
    p[0] = v[0];
  }
}

// V: numbers per thread and access while the row is formed (8 bf16 or 4 fp32 numbers = 16 bytes, or 1)
template <typename T, int V>
__global__ __launch_bounds__(512) void head_prep_kernel(HeadPrepArgs A, int vec) {
  extern __shared__ __attribute__((aligned(16))) float us[];
  const int t = blockIdx.x, lane = threadIdx.x & 63, wv = threadIdx.x >> 6, nw = blockDim.x >> 6;
  const int dim = A.dim, vdim = A.vdim, H = A.H, G = A.G;
  const int nq = H * dim, nk = G * dim, nv = G * vdim;
  const bool sharev = A.off_v == A.off_k;  // the values are the projected keys
  const T* row = (const T*)A.proj + (int64_t)t * A.ldp;
  const int64_t slot = A.slots[t];
  if (A.conv) {
    const RowSeq r = row_seq(A.cu, A.ctx, A.B, t);
    const int C = nq + nk + nv, R = A.taps - 1;
    const int ss = r.pos >= 0 ? A.sslots[r.b] : -1;
    float* st = A.tail + (int64_t)max(ss, 0) * R * C;
    for (int c = threadIdx.x * V; c < C; c += blockDim.x * V) {
      float acc[V];
#pragma unroll
      for (int i = 0; i < V; ++i) acc[i] = 0.f;
      if (r.pos >= 0) {
        for (int k = 0; k <= R; ++k) {
          const int d = R - k;
          if (r.pos - d < 0) continue;
          float x[V], w[V];
          hp_ld<T, V>((const T*)A.conv + (int64_t)k * C + c, w);
          if (r.j - d >= 0) {
            hp_ld<T, V>(row - (int64_t)d * A.ldp + A.off_q + c, x);
          } else {
            hp_ldf<V>(st + (int64_t)(r.j - d + R) * C + c, x);  // (a row without a slot reads slot 0 and is not used)
          }
#pragma unroll
          for (int i = 0; i < V; ++i) acc[i] = fmaf(w[i], x[i], acc[i]);
        }
        if (A.tail_here && ss >= 0) {  // one row per sequence: the tail moves up by one and takes this row
          for (int i = 0; i < R; ++i) {
            float x[V];
            if (i + 1 < R) {
              if (r.pos > 0) {
                hp_ldf<V>(st + (int64_t)(i + 1) * C + c, x);
              } else {
#pragma unroll
                for (int e = 0; e < V; ++e) x[e] = 0.f;
              }
            } else {
              hp_ld<T, V>(row + A.off_q + c, x);
            }
            hp_stf<V>(st + (int64_t)i * C + c, x);
          }
        }
      }
#pragma unroll
      for (int i = 0; i < V; ++i) us[c + i] = acc[i];
    }
  } else {
    for (int c = threadIdx.x * V; c < nq + nk + (sharev ? 0 : nv); c += blockDim.x * V) {
      const int src = c < nq ? A.off_q + c : (c < nq + nk ? A.off_k + c - nq : A.off_v + c - nq - nk);
      float x[V];
      hp_ld<T, V>(row + src, x);
#pragma unroll
      for (int i = 0; i < V; ++i) us[c + i] = x[i];
    }
  }
  __syncthreads();
  if (vec) {
    const float* kt = A.cs ? A.cs + (int64_t)t * A.half * 2 : nullptr;
    head_vec<T>(A, us, H, dim, A.qw, A.qw != nullptr, kt ? A.half : 0, kt, 0, (int64_t)t * nq);
    if (slot < 0) return;
    head_vec<T>(A, us + nq, G, dim, A.kw, A.kw != nullptr, kt ? A.half : 0, kt, 1, slot * (int64_t)nk);
    const float* vt = A.vcs ? A.vcs + (int64_t)t * vdim : nullptr;
    head_vec<T>(A, us + (sharev ? nq : nq + nk), G, vdim, nullptr, A.vnorm != 0, vt ? vdim >> 1 : 0, vt, 2,
                slot * (int64_t)nv);
    return;
  }
  const int nvec = H + G + (slot >= 0 ? G : 0);
  for (int n = wv; n < nvec; n += nw) {
    const int kind = n < H ? 0 : (n < H + G ? 1 : 2);  // query, key, value
    if (kind == 1 && slot < 0) continue;
    const int idx = kind == 0 ? n : (kind == 1 ? n - H : n - H - G);
    const int N = kind == 2 ? vdim : dim;
    const float* x = us + (kind == 0 ? idx * dim : (kind == 1 ? nq + idx * dim : (sharev ? nq : nq + nk) + idx * vdim));
    const float* w = kind == 0 ? A.qw : (kind == 1 ? A.kw : nullptr);
    float inv = 1.f;
    if (w || (kind == 2 && A.vnorm)) {
      float s = 0.f;
      for (int d = lane; d < N; d += 64) s = fmaf(x[d], x[d], s);
      inv = 1.0f / sqrtf(warp_sum(s) / (float)N + A.eps);
    }
    const float* tab = nullptr;
    int half = 0;
    if (kind == 2) {
      if (A.vcs) half = vdim >> 1, tab = A.vcs + (int64_t)t * half * 2;
    } else if (A.cs) {
      half = A.half, tab = A.cs + (int64_t)t * half * 2;
    }
    const int64_t qd = (int64_t)t * nq + idx * dim;
    T* cd = kind == 2 ? (T*)A.vc + slot * (int64_t)nv + idx * vdim : (T*)A.kc + slot * (int64_t)nk + idx * dim;
    for (int d = lane; d < N; d += 64) {
      float v = x[d] * inv * (w ? w[d] : 1.0f);
      if (d < 2 * half) {
        const bool lo = d < half;
        const int i = lo ? d : d - half, od = lo ? d + half : d - half;
        const float o = x[od] * inv * (w ? w[od] : 1.0f);
        const float c = tab[2 * i], s = tab[2 * i + 1];
        v = lo ? v * c - o * s : v * c + o * s;
      }
      if (kind == 0 && A.q_bf) ((bf16_t*)A.q)[qd + d] = f2bf(v);
      else if (kind == 0) ((float*)A.q)[qd + d] = v;
      else El<T>::st(cd + d, v);
    }
  }
}

void launch_conv_tail(const void* in, int64_t ldi, void* state, const void* cu, const void* ctx, const void* sslots, int B,
                      int C, int taps, int di, hipStream_t st);

void launch_head_prep(const void* proj, int64_t ldp, int off_q, int off_k, int off_v, const void* conv, int taps,
                      void* tail, int single, const void* cu, const void* ctx, const void* sslots, int B, const void* qw,
                      const void* kw, int vnorm, float eps, const void* cs, int half, const void* vcs, void* q, int q_bf,
                      void* kc, void* vc, const void* slots, int T_, int H, int G, int dim, int vdim, int dt,
                      hipStream_t st) {
  if (T_ == 0) return;
  if (G < 1 || H % G) throw std::runtime_error("head_prep: heads must be a multiple of the key heads");
  if (half < 0 || 2 * half > dim || (vcs && vdim % 2)) throw std::runtime_error("head_prep: rotation wider than a head");
  const int nq = H * dim, nk = G * dim, nv = G * vdim, C = nq + nk + nv;
  if (off_v == off_k && (conv || vdim != dim)) throw std::runtime_error("head_prep: shared keys need vdim == dim");
  if (conv && (off_k != off_q + nq || off_v != off_k + nk || taps < 1 || !sslots || (taps > 1 && !tail)))
    throw std::runtime_error("head_prep: the convolution takes contiguous q | k | v columns and a tail");
  const size_t lds = (size_t)C * 4;
  if (lds > 64 * 1024) throw std::runtime_error("head_prep: rows wider than 16384");
  HeadPrepArgs A{proj, ldp, off_q, off_k, off_v, conv, taps, (float*)tail, single, (const int*)cu, (const int*)ctx,
                 (const int*)sslots, B, (const float*)qw, (const float*)kw, vnorm, eps, (const float*)cs, half,
                 (const float*)vcs, q, q_bf, kc, vc, (const int64_t*)slots, H, G, dim, vdim};
  const int vn = dt == 0 ? 8 : 4;
  const auto al16 = [](const void* p) { return ((uintptr_t)p & 15) == 0; };
  const bool vec = al16(proj) && al16(conv) && al16(tail) && ldp % vn == 0 && off_q % vn == 0 && off_k % vn == 0 && off_v % vn == 0 &&
                   nq % vn == 0 && nk % vn == 0 && nv % vn == 0;
  // whole 16-byte pieces per head: sizes 8 to 512 that are powers of two, turned parts of whole pieces
  const auto pow2 = [](int n) { return n >= 8 && n <= 512 && (n & (n - 1)) == 0; };
  const int hv = pow2(dim) && pow2(vdim) && half % 8 == 0 && (!vcs || vdim % 16 == 0) && al16(q) && al16(kc) && al16(vc) &&
                 al16(cs) && al16(vcs) && (dt == 0 || !q_bf);
  const int th = T_ <= 512 ? 512 : 256;  // few rows: more waves to a row
  if (q_bf && dt != 0) throw std::runtime_error("head_prep: bf16 queries come from bf16 rows");
  if (dt == 0) {
    if (vec) head_prep_kernel<bf16_t, 8><<<T_, th, lds, st>>>(A, hv);
    else head_prep_kernel<bf16_t, 1><<<T_, th, lds, st>>>(A, hv);
  } else if (dt == 1) {
    if (vec) head_prep_kernel<float, 4><<<T_, th, lds, st>>>(A, hv);
    else head_prep_kernel<float, 1><<<T_, th, lds, st>>>(A, hv);
  } else {
    throw std::runtime_error("bad dtype code");
  }
  HIP_CHECK_LAUNCH();
  if (conv && taps > 1 && !single) {
    const int es = dt == 0 ? 2 : 4;
    launch_conv_tail((const char*)proj + (int64_t)off_q * es, ldp, tail, cu, ctx, sslots, B, C, taps, dt, st);
  }
}
