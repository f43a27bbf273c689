// Mixture-of-experts feed-forward: routing, grouping of (token, expert) pairs and the grouped expert GEMMs.
//
//   z = W_router h (fp32, gemm_any)                                   [T, E]
//   moe_route:   s = sigmoid(z), or softmax(z) over all experts; the `top` experts with the largest s + correction are chosen (ties: the lower
//                index); weights = chosen s / (their sum + 1e-20)     -> idx [T, top] int32, wts [T, top] fp32
//                or (score 2) s = z, the chosen ones weighted by a softmax over themselves. A bias may be added to z; one
//                more column of z after the E routed ones may hold a gate, whose sigmoid goes to sg [T]
//                A router may have more outputs than there are experts: the outputs from E on are identity experts,
//                whose output is the layer's input row; their pairs are left out of the grouping (place -1).
//   moe_group:   pairs p = t * top + j are bucketed by expert: off [E + 1], order [P] (pair at each sorted row),
//                place [P] (sorted row of each pair) and a flat list of row tiles (expert, first row; 64 or 128 rows each) so the
//                grouped GEMMs launch a grid whose size is known on the host (ceil(P / rows) + E tiles at most)
//   moe_gate_up: act[r, f] = glu(h[token(r)] . gate_e[f], h[token(r)] . up_e[f])   for sorted row r of expert e
//   moe_down:    y[r, n] = act[r, :] . down_e[n, :]                   (fp32)
//   moe_combine: out[t, :] = sum_j wts[t, j] * y[place[t * top + j], :] (+ (sw[t] *) shared[t, :])   (fp32, j ascending;
//                no wts: the plain sum, for layers whose weights went onto the experts' inputs in moe_gate_up)
//
// Expert activation (clamped, gated): g = min(g, limit), u = clamp(u, -limit, limit),
// glu = g * sigmoid(alpha * g) * (u + 1). glu_clamp applies the same to a dense [T, 2F] gate|up product (the
// shared expert, which runs through the ordinary GEMMs).
//
// Nothing here synchronises with the host: group sizes stay on the device, so a decode step with experts can be
// captured into a HIP graph. Every pair's row is computed alone, so a token's result does not depend on what else
// is in the step.
#include "anytype.h"
#include "tile_valu.h"

__device__ __forceinline__ float glu_clamped(float g, float u, float limit, float alpha) {
  g = fminf(g, limit);
  u = fminf(fmaxf(u, -limit), limit);
  return g / (1.f + expf(-alpha * g)) * (u + 1.f);
}
// silu: the plain gated form silu(g) * u, no clamps
__device__ __forceinline__ float glu_value(float g, float u, float limit, float alpha, int silu) {
  return silu ? g / (1.f + expf(-g)) * u : glu_clamped(g, u, limit, alpha);
}

// ------------------------------------------------------------------------------------------------ routing
// A wave routes one token of up to 128 outputs: lane e holds the logits of e and e + 64 (bias added; -inf past the last); an
// output's rank among all choice values (ties: the lower index first) says whether and where it is chosen. row: LDS, 16-byte
// aligned, room for the outputs in whole fours.
__device__ __forceinline__ void route_ranked(float (&sc)[2], float* row, const float* __restrict__ corr, int* __restrict__ idx,
                                             float* __restrict__ wts, int E, int top, int norm, int smax) {
  const int lane = threadIdx.x & 63;
  float ch[2];
  float mx = -INFINITY, den = 0.f;
  if (smax) mx = warp_max(fmaxf(sc[0], sc[1]));
  if (smax == 1) {
#pragma unroll
    for (int j = 0; j < 2; ++j) den += lane + 64 * j < E ? expf(sc[j] - mx) : 0.f;
    den = warp_sum(den);
  }
#pragma unroll
  for (int j = 0; j < 2; ++j) {
    const int e = lane + 64 * j;
    if (smax != 2 && e < E) sc[j] = smax ? expf(sc[j] - mx) / den : 1.f / (1.f + expf(-sc[j]));
    ch[j] = e < E ? sc[j] + (corr ? corr[e] : 0.f) : -INFINITY;
    if (!(ch[j] == ch[j])) ch[j] = -INFINITY;  // (a NaN ranks last: the ranks stay a permutation)
    if (e < ((E + 3) & ~3)) row[e] = ch[j];
  }
  __builtin_amdgcn_wave_barrier();
  __threadfence_block();
  int rank[2] = {0, 0};
  for (int e0 = 0; e0 < E; e0 += 4) {
    const f32x4 o = *reinterpret_cast<const f32x4*>(row + e0);
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      if (e0 + i >= E) continue;
#pragma unroll
      for (int j = 0; j < 2; ++j) rank[j] += o[i] > ch[j] || (o[i] == ch[j] && e0 + i < lane + 64 * j) ? 1 : 0;
    }
  }
  float sum = 0.f;
  bool in[2];
#pragma unroll
  for (int j = 0; j < 2; ++j) {
    in[j] = lane + 64 * j < E && rank[j] < top;
    if (smax == 2) sc[j] = expf(sc[j] - mx);  // (the largest is always chosen)
    sum += in[j] ? sc[j] : 0.f;
  }
  sum = warp_sum(sum);
  const float inv = smax == 2 ? 1.f / sum : norm ? 1.f / (sum + 1e-20f) : 1.f;
#pragma unroll
  for (int j = 0; j < 2; ++j)
    if (in[j]) {
      idx[rank[j]] = lane + 64 * j;
      wts[rank[j]] = sc[j] * inv;
    }
}

// one wave per token; lanes over experts
__global__ __launch_bounds__(64) void moe_route_kernel(const float* __restrict__ z, const float* __restrict__ corr,
                                                       int* __restrict__ idx, float* __restrict__ wts, int E, int top,
                                                       int norm, int smax, const float* __restrict__ zb,
                                                       float* __restrict__ sg) {
  extern __shared__ __attribute__((aligned(16))) float sc[];  // [E] scores, [E] choice values
  float* ch = sc + E;
  const int t = blockIdx.x, lane = threadIdx.x;
  const float* zr = z + (int64_t)t * (E + (sg ? 1 : 0));
  if (sg && lane == 0) sg[t] = 1.f / (1.f + expf(-zr[E]));
  if (E <= 128) {
    float v[2];
#pragma unroll
    for (int j = 0; j < 2; ++j) v[j] = lane + 64 * j < E ? zr[lane + 64 * j] + (zb ? zb[lane + 64 * j] : 0.f) : -INFINITY;
    route_ranked(v, sc, corr, idx + (int64_t)t * top, wts + (int64_t)t * top, E, top, norm, smax);
    return;
  }
  float mx = 0.f, den = 1.f;
  if (smax == 1) {
    mx = -INFINITY, den = 0.f;
    for (int e = lane; e < E; e += 64) mx = fmaxf(mx, zr[e] + (zb ? zb[e] : 0.f));
    mx = warp_max(mx);
    for (int e = lane; e < E; e += 64) den += expf(zr[e] + (zb ? zb[e] : 0.f) - mx);
    den = warp_sum(den);
  }
  for (int e = lane; e < E; e += 64) {
    const float ze = zr[e] + (zb ? zb[e] : 0.f);
    const float s = smax == 2 ? ze : smax ? expf(ze - mx) / den : 1.f / (1.f + expf(-ze));
    sc[e] = s;
    ch[e] = s + (corr ? corr[e] : 0.f);
  }
  __syncthreads();
  float sum = 0.f, first = 0.f;
  for (int j = 0; j < top; ++j) {
    float best = -INFINITY;
    int bi = 0x7fffffff;
    for (int e = lane; e < E; e += 64) {
      const float v = ch[e];
      if (v > best || (v == best && e < bi)) {
        best = v;
        bi = e;
      }
    }
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) {
      const float ov = __shfl_xor(best, o, 64);
      const int oi = __shfl_xor(bi, o, 64);
      if (ov > best || (ov == best && oi < bi)) {
        best = ov;
        bi = oi;
      }
    }
    if (bi >= E) bi = 0;  // every value NaN: keep indices in range
    float s = sc[bi];
    if (smax == 2) {  // the first one chosen is the largest
      if (j == 0) first = s;
      s = expf(s - first);
    }
    sum += s;
    if (lane == 0) {
      idx[(int64_t)t * top + j] = bi;
      wts[(int64_t)t * top + j] = s;
      ch[bi] = -INFINITY;
    }
    __syncthreads();
  }
  if (!norm && smax != 2) return;  // the chosen scores themselves
  const float inv = 1.f / (sum + (smax == 2 ? 0.f : 1e-20f));
  for (int j = lane; j < top; j += 64) wts[(int64_t)t * top + j] *= inv;
}

void launch_moe_route(const void* z, const void* corr, void* idx, void* wts, int T_, int E, int top, int norm,
                      int smax, const void* zb, void* sg, hipStream_t st) {
  if (T_ == 0) return;
  if (top > E || top <= 0) throw std::runtime_error("moe_route: top must be in [1, experts]");
  moe_route_kernel<<<T_, 64, (2 * E + 4) * sizeof(float), st>>>((const float*)z, (const float*)corr, (int*)idx, (float*)wts,
                                                           E, top, norm, smax, (const float*)zb, (float*)sg);
  HIP_CHECK_LAUNCH();
}

// Router logits and routing in one launch, for steps of few tokens (a decode step): one workgroup per token, its waves
// share the experts' dot products z_e = h . W_r[e] (fp32 accumulation over lanes), then the token is routed
// as moe_route_kernel does. A prompt's thousands of tokens take the matrix-core GEMM and moe_route instead.
template <typename T>
__global__ __launch_bounds__(1024) void moe_router_kernel(const T* __restrict__ h, int64_t ldh, const T* __restrict__ wr,
                                                         const float* __restrict__ corr, int* __restrict__ idx,
                                                         float* __restrict__ wts, int E, int K, int top, bool vec,
                                                         int norm, int smax, const float* __restrict__ zb,
                                                         float* __restrict__ sg) {
  extern __shared__ __attribute__((aligned(16))) float sc[];  // [E] scores, [E] choice values
  float* ch = sc + E;
  const bool ranked = E <= 128;
  const int t = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wv = tid >> 6, nw = blockDim.x >> 6;
  const T* x = h + (int64_t)t * ldh;
  for (int e = wv; e < E + (sg ? 1 : 0); e += nw) {
    const T* w = wr + (int64_t)e * K;
    float acc = 0.f;
    if (vec) {  // K % 8 == 0, rows 16-byte aligned - eight elements per lane, two or four 16-byte accesses
      typedef T vec8 __attribute__((ext_vector_type(8)));
#pragma unroll 4
      for (int k = lane * 8; k < K; k += 512) {
        const vec8 xv = *reinterpret_cast<const vec8*>(x + k), wv = *reinterpret_cast<const vec8*>(w + k);
#pragma unroll
        for (int i = 0; i < 8; ++i) {
          const T xi = xv[i], wi = wv[i];
          acc = fmaf(El<T>::ld(&xi), El<T>::ld(&wi), acc);
        }
      }
    } else {
      for (int k = lane; k < K; k += 64) acc = fmaf(El<T>::ld(x + k), El<T>::ld(w + k), acc);
    }
    acc = warp_sum(acc);
    if (lane == 0) {
      if (e == E) {
        sg[t] = 1.f / (1.f + expf(-acc));
        continue;
      }
      if (zb) acc += zb[e];
      if (ranked) {
        sc[e] = acc;
        continue;
      }
      const float s = smax ? acc : 1.f / (1.f + expf(-acc));
      sc[e] = s;
      ch[e] = s + (corr ? corr[e] : 0.f);
    }
  }
  __syncthreads();
  if (ranked) {
    if (wv) return;
    float v[2];
#pragma unroll
    for (int j = 0; j < 2; ++j) v[j] = lane + 64 * j < E ? sc[lane + 64 * j] : -INFINITY;
    __builtin_amdgcn_wave_barrier();
    route_ranked(v, sc, corr, idx + (int64_t)t * top, wts + (int64_t)t * top, E, top, norm, smax);
    return;
  }
  if (smax == 1) {  // sc holds the logits: every wave forms their maximum and sum, then the scores replace them
    float mx = -INFINITY, den = 0.f;
    for (int e = lane; e < E; e += 64) mx = fmaxf(mx, sc[e]);
    mx = warp_max(mx);
    for (int e = lane; e < E; e += 64) den += expf(sc[e] - mx);
    den = warp_sum(den);
    __syncthreads();
    for (int e = tid; e < E; e += blockDim.x) {
      const float s = expf(sc[e] - mx) / den;
      sc[e] = s;
      ch[e] = s + (corr ? corr[e] : 0.f);
    }
    __syncthreads();
  }
  float sum = 0.f, first = 0.f;
  for (int j = 0; j < top; ++j) {
    float best = -INFINITY;
    int bi = 0x7fffffff;
    for (int e = lane; e < E; e += 64) {
      const float v = ch[e];
      if (v > best || (v == best && e < bi)) {
        best = v;
        bi = e;
      }
    }
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) {
      const float ov = __shfl_xor(best, o, 64);
      const int oi = __shfl_xor(bi, o, 64);
      if (ov > best || (ov == best && oi < bi)) {
        best = ov;
        bi = oi;
      }
    }
    if (bi >= E) bi = 0;
    float s = sc[bi];
    if (smax == 2) {
      if (j == 0) first = s;
      s = expf(s - first);
    }
    sum += s;
    __syncthreads();  // every wave has read ch before the winner is struck out
    if (tid == 0) {
      idx[(int64_t)t * top + j] = bi;
      wts[(int64_t)t * top + j] = s;
      ch[bi] = -INFINITY;
    }
    __syncthreads();
  }
  if (!norm && smax != 2) return;
  const float inv = 1.f / (sum + (smax == 2 ? 0.f : 1e-20f));
  for (int j = tid; j < top; j += blockDim.x) wts[(int64_t)t * top + j] *= inv;
}

void launch_moe_router(const void* h, int64_t ldh, const void* wr, const void* corr, void* idx, void* wts, int T_,
                       int E, int K, int top, int dt, int norm, int smax, const void* zb, void* sg, hipStream_t st) {
  if (T_ == 0) return;
  if (top > E || top <= 0) throw std::runtime_error("moe_router: top must be in [1, experts]");
  const int es = dt == 0 ? 2 : 4;
  const bool vec = K % 8 == 0 && ((uintptr_t)h % 16) == 0 && ((uintptr_t)wr % 16) == 0 && (ldh * es) % 16 == 0;
  const int threads = E >= 16 ? 1024 : (E >= 8 ? 512 : 256);  // a wave per expert up to 16 waves
  DISPATCH_T(dt, T, (moe_router_kernel<T><<<T_, threads, (2 * E + 4) * sizeof(float), st>>>(
                        (const T*)h, ldh, (const T*)wr, (const float*)corr, (int*)idx, (float*)wts, E, K, top, vec,
                        norm, smax, (const float*)zb, (float*)sg)));
  HIP_CHECK_LAUNCH();
}

// The same for bf16 rows on the matrix cores, at any number of rows: a workgroup takes 16 tokens and all outputs (up to 16 *
// MR_NT), its eight waves an eighth of K each (fragments straight from memory: lane (li, g) holds k = 8 g .. 8 g + 7 of row li);
// the parts meet in LDS and every wave routes two of the tokens, a score per lane (lane e: outputs e, e + 64) whose rank among
// all decides whether and where it is chosen.
#define MR_NT 8
template <int NT>
__global__ __launch_bounds__(512) void moe_router_mfma_kernel(const bf16_t* __restrict__ h, int64_t ldh,
                                                              const bf16_t* __restrict__ wr, const float* __restrict__ corr,
                                                              int* __restrict__ idx, float* __restrict__ wts, int T_, int E,
                                                              int K, int top, int norm, int smax,
                                                              const float* __restrict__ zb, float* __restrict__ sg) {
  constexpr int LD = 16 * NT + 4;
  __shared__ __attribute__((aligned(16))) float part[4][16][LD];
  const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6, li = lane & 15, g = lane >> 4;
  const int t0 = blockIdx.x * 16, EG = E + (sg ? 1 : 0);
  f32x4 acc[NT];
#pragma unroll
  for (int j = 0; j < NT; ++j) acc[j] = f32x4{0.f, 0.f, 0.f, 0.f};
  const bf16_t* a = h + (int64_t)min(t0 + li, T_ - 1) * ldh + 8 * g;
  const bf16_t* b[NT];
#pragma unroll
  for (int j = 0; j < NT; ++j) b[j] = wr + (int64_t)min(16 * j + li, EG - 1) * K + 8 * g;
  const int ks = K / 32;  // (neighbouring waves take neighbouring steps: the halves of a 128-byte line meet in the cache)
  constexpr int U = NT <= 4 ? 8 : 4;  // steps whose loads are in flight together
  for (int k0 = w; k0 < ks; k0 += 8 * U) {  // (K a multiple of 32; steps past the end repeat the last one with a zero row)
    s16x8 av[U], bv[U][NT];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int k = min(k0 + 8 * u, ks - 1);
      av[u] = *reinterpret_cast<const s16x8*>(a + 32 * k);
#pragma unroll
      for (int j = 0; j < NT; ++j) bv[u][j] = *reinterpret_cast<const s16x8*>(b[j] + 32 * k);
    }
    __builtin_amdgcn_sched_barrier(0);  // all loads are issued before the first product waits for one
#pragma unroll
    for (int u = 0; u < U; ++u) {
      if (k0 + 8 * u >= ks) av[u] = s16x8{0, 0, 0, 0, 0, 0, 0, 0};
#pragma unroll
      for (int j = 0; j < NT; ++j) acc[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(av[u], bv[u][j], acc[j], 0, 0, 0);
    }
  }
  if (w >= 4) {
#pragma unroll
    for (int j = 0; j < NT; ++j)
#pragma unroll
      for (int i = 0; i < 4; ++i) part[w - 4][4 * g + i][16 * j + li] = acc[j][i];
  }
  __syncthreads();
  if (w < 4) {
#pragma unroll
    for (int j = 0; j < NT; ++j)
#pragma unroll
      for (int i = 0; i < 4; ++i) part[w][4 * g + i][16 * j + li] += acc[j][i];
  }
  __syncthreads();
  auto z_of = [&](int r, int e) { return (part[0][r][e] + part[1][r][e]) + (part[2][r][e] + part[3][r][e]); };
  for (int r = 2 * w; r < 2 * w + 2; ++r) {
    const int64_t t = t0 + r;
    if (t >= T_) return;
    float sc[2];
#pragma unroll
    for (int j = 0; j < 2; ++j) {
      const int e = lane + 64 * j;
      sc[j] = e < E ? z_of(r, e) + (zb ? zb[e] : 0.f) : -INFINITY;
    }
    if (sg && lane == 0) sg[t] = 1.f / (1.f + expf(-z_of(r, E)));
    __builtin_amdgcn_wave_barrier();
    route_ranked(sc, &part[0][r][0], corr, idx + t * top, wts + t * top, E, top, norm, smax);  // (the row is this wave's alone)
  }
}

// may a router of E outputs (+ gate) over bf16 rows of K numbers take the matrix-core form?
bool moe_router_mfma_ok(int E, int gate, int K) { return E + (gate ? 1 : 0) <= 16 * MR_NT && E <= 128 && K % 32 == 0; }

void launch_moe_router_mfma(const void* h, int64_t ldh, const void* wr, const void* corr, void* idx, void* wts, int T_,
                            int E, int K, int top, int norm, int smax, const void* zb, void* sg, hipStream_t st) {
  if (T_ == 0) return;
  if (top > E || top <= 0) throw std::runtime_error("moe_router: top must be in [1, experts]");
  if (!moe_router_mfma_ok(E, sg != nullptr, K) || (((uintptr_t)h | (uintptr_t)wr) & 15) || ldh % 8)
    throw std::runtime_error("moe_router: shape of the matrix-core form");
#define LAUNCH_MR(NT_)                                                                                                      \
  moe_router_mfma_kernel<NT_><<<(T_ + 15) / 16, 512, 0, st>>>((const bf16_t*)h, ldh, (const bf16_t*)wr, (const float*)corr, \
                                                              (int*)idx, (float*)wts, T_, E, K, top, norm, smax,            \
                                                              (const float*)zb, (float*)sg)
  const int nt = (E + (sg ? 1 : 0) + 15) / 16;
  if (nt <= 1) LAUNCH_MR(1);
  else if (nt <= 2) LAUNCH_MR(2);
  else if (nt <= 3) LAUNCH_MR(3);
  else if (nt <= 5) LAUNCH_MR(5);
  else LAUNCH_MR(MR_NT);
#undef LAUNCH_MR
  HIP_CHECK_LAUNCH();
}

// ------------------------------------------------------------------------------------------------ grouping
// One workgroup. meta = [ntiles | off[E + 1] | tile_expert[maxt] | tile_row0[maxt]], order [P], place [P].
__global__ __launch_bounds__(1024) void moe_group_kernel(const int* __restrict__ idx, int P, int E, int maxt,
                                                         int* __restrict__ meta, int* __restrict__ order,
                                                         int* __restrict__ place, int tile_rows) {
  extern __shared__ int sm[];  // cnt[E], cur[E]
  int* cnt = sm;
  int* cur = sm + E;
  int* off = meta + 1;
  int* tile_e = meta + 1 + (E + 1);
  int* tile_r = tile_e + maxt;
  for (int e = threadIdx.x; e < E; e += blockDim.x) cnt[e] = 0;
  __syncthreads();
  constexpr int U = 8;  // pairs per thread whose loads and atomics are in flight together
  for (int p0 = threadIdx.x; p0 < P; p0 += blockDim.x * U) {
    int e[U];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int p = p0 + u * blockDim.x;
      e[u] = p < P ? idx[p] : E;
    }
#pragma unroll
    for (int u = 0; u < U; ++u)
      if (e[u] < E) atomicAdd(&cnt[e[u]], 1);
  }
  __syncthreads();
  if (threadIdx.x == 0) {
    int o = 0, nt = 0;
    for (int e = 0; e < E; ++e) {
      off[e] = o;
      cur[e] = o;
      for (int r = 0; r < cnt[e]; r += tile_rows) {
        if (nt < maxt) {
          tile_e[nt] = e;
          tile_r[nt] = o + r;
        }
        ++nt;
      }
      o += cnt[e];
    }
    off[E] = o;
    meta[0] = nt < maxt ? nt : maxt;
  }
  __syncthreads();
  // rows within an expert take whatever order the atomics give: every pair's row is computed on its own, so the
  // values do not depend on where the row lands
  for (int p0 = threadIdx.x; p0 < P; p0 += blockDim.x * U) {
    int e[U], o[U];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int p = p0 + u * blockDim.x;
      e[u] = p < P ? idx[p] : E;
    }
#pragma unroll
    for (int u = 0; u < U; ++u) o[u] = e[u] < E ? atomicAdd(&cur[e[u]], 1) : -1;  // (-1: an identity expert, no row of its own)
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int p = p0 + u * blockDim.x;
      if (p >= P) continue;
      if (o[u] >= 0) order[o[u]] = p;
      place[p] = o[u];
    }
  }
}

void launch_moe_group(const void* idx, int P, int E, int maxt, void* meta, void* order, void* place, int tile_rows,
                      hipStream_t st) {
  if (P == 0) return;
  if (tile_rows <= 0) throw std::runtime_error("moe_group: tile rows");
  if (E > 4096) throw std::runtime_error("moe_group: more than 4096 experts");
  moe_group_kernel<<<1, 1024, 2 * E * sizeof(int), st>>>((const int*)idx, P, E, maxt, (int*)meta, (int*)order,
                                                          (int*)place, tile_rows);
  HIP_CHECK_LAUNCH();
}

// ------------------------------------------------------------------------------------------------ grouped GEMMs
// (wg null: experts without a gate, act = gelu(up), the error-function form)
// grid (ceil(F / 64), maxt): tile y of the list covers sorted rows [row0, min(row0 + 64, off[e + 1])) of expert e.
template <typename T>
__global__ __launch_bounds__(256) void moe_gate_up_kernel(const T* __restrict__ h, int64_t ldh,
                                                          const T* __restrict__ wg, const T* __restrict__ wu,
                                                          const int* __restrict__ meta, const int* __restrict__ order,
                                                          T* __restrict__ act, int E, int maxt, int top, int F, int K,
                                                          float limit, float alpha, const float* __restrict__ pw,
                                                          int silu) {
  __shared__ float As[TV_BK][TV_LD];
  __shared__ float Gs[TV_BK][TV_LD];
  __shared__ float Us[TV_BK][TV_LD];
  if ((int)blockIdx.y >= meta[0]) return;
  const int* off = meta + 1;
  const int e = meta[1 + (E + 1) + blockIdx.y];
  const int row0 = meta[1 + (E + 1) + maxt + blockIdx.y];
  const int rows = min(TV_BM, off[e + 1] - row0);
  const int n0 = blockIdx.x * TV_BN;
  const int tid = threadIdx.x;
  const T* G = wg ? wg + (int64_t)e * F * K : nullptr;
  const T* U = wu + (int64_t)e * F * K;
  const int r = tid >> 2, kq = (tid & 3) * 4;
  const T* arow = r < rows ? h + (int64_t)(order[row0 + r] / top) * ldh : nullptr;
  const int n = n0 + r;
  float ag[4][4] = {}, au[4][4] = {};
  for (int k0 = 0; k0 < K; k0 += TV_BK) {
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int k = k0 + kq + i;
      const bool kin = k < K;
      As[kq + i][r] = (arow && kin) ? El<T>::ld(arow + k) : 0.f;
      Gs[kq + i][r] = (G && n < F && kin) ? El<T>::ld(G + (int64_t)n * K + k) : 0.f;
      Us[kq + i][r] = (n < F && kin) ? El<T>::ld(U + (int64_t)n * K + k) : 0.f;
    }
    __syncthreads();
    tv_mac(ag, As, Gs, tid);
    tv_mac(au, As, Us, tid);
    __syncthreads();
  }
  const int tx = tid & 15, ty = tid >> 4;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int m = ty * 4 + i;
    if (m >= rows) continue;
    const float sw = pw ? pw[order[row0 + m]] : 1.0f;  // the pair's weight on the expert's input
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int f = n0 + tx * 4 + j;
      if (f >= F) continue;
      const float v = wg ? glu_value(ag[i][j] * sw, au[i][j] * sw, limit, alpha, silu) : gelu_erf(au[i][j] * sw);
      El<T>::st(act + (int64_t)(row0 + m) * F + f, v);
    }
  }
}

template <typename T>
__global__ __launch_bounds__(256) void moe_down_kernel(const T* __restrict__ act, const T* __restrict__ wd,
                                                       const int* __restrict__ meta, float* __restrict__ y, int E,
                                                       int maxt, int N, int F) {
  __shared__ float As[TV_BK][TV_LD];
  __shared__ float Bs[TV_BK][TV_LD];
  if ((int)blockIdx.y >= meta[0]) return;
  const int* off = meta + 1;
  const int e = meta[1 + (E + 1) + blockIdx.y];
  const int row0 = meta[1 + (E + 1) + maxt + blockIdx.y];
  const int rows = min(TV_BM, off[e + 1] - row0);
  const int n0 = blockIdx.x * TV_BN;
  const int tid = threadIdx.x;
  const T* W = wd + (int64_t)e * N * F;
  const int r = tid >> 2, kq = (tid & 3) * 4;
  const T* arow = r < rows ? act + (int64_t)(row0 + r) * F : nullptr;
  const int n = n0 + r;
  float acc[4][4] = {};
  for (int k0 = 0; k0 < F; k0 += TV_BK) {
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int k = k0 + kq + i;
      const bool kin = k < F;
      As[kq + i][r] = (arow && kin) ? El<T>::ld(arow + k) : 0.f;
      Bs[kq + i][r] = (n < N && kin) ? El<T>::ld(W + (int64_t)n * F + k) : 0.f;
    }
    __syncthreads();
    tv_mac(acc, As, Bs, tid);
    __syncthreads();
  }
  const int tx = tid & 15, ty = tid >> 4;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int m = ty * 4 + i;
    if (m >= rows) continue;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int c = n0 + tx * 4 + j;
      if (c < N) y[(int64_t)(row0 + m) * N + c] = acc[i][j];
    }
  }
}

void launch_moe_gate_up(const void* h, int64_t ldh, const void* wg, const void* wu, const void* meta,
                        const void* order, void* act, int E, int maxt, int top, int F, int K, float limit,
                        float alpha, int dt, const void* pw, int silu, hipStream_t st) {
  if (maxt <= 0) return;
  if (maxt > 65535) throw std::runtime_error("moe_gate_up: too many row tiles");
  dim3 g((F + TV_BN - 1) / TV_BN, maxt);
  DISPATCH_T(dt, T, (moe_gate_up_kernel<T><<<g, 256, 0, st>>>((const T*)h, ldh, (const T*)wg, (const T*)wu,
                                                               (const int*)meta, (const int*)order, (T*)act, E, maxt,
                                                               top, F, K, limit, alpha, (const float*)pw, silu)));
  HIP_CHECK_LAUNCH();
}

void launch_moe_down(const void* act, const void* wd, const void* meta, void* y, int E, int maxt, int N, int F,
                     int dt, hipStream_t st) {
  if (maxt <= 0) return;
  if (maxt > 65535) throw std::runtime_error("moe_down: too many row tiles");
  dim3 g((N + TV_BN - 1) / TV_BN, maxt);
  DISPATCH_T(dt, T, (moe_down_kernel<T><<<g, 256, 0, st>>>((const T*)act, (const T*)wd, (const int*)meta, (float*)y,
                                                            E, maxt, N, F)));
  HIP_CHECK_LAUNCH();
}

// ------------------------------------------------------------------------------------------------ combine
template <typename T>
__global__ __launch_bounds__(256) void moe_combine_kernel(const float* __restrict__ y, const int* __restrict__ place,
                                                          const float* __restrict__ wts, const T* __restrict__ shared_,
                                                          int64_t lds_, float* __restrict__ out, int N, int top,
                                                          const T* __restrict__ ident, int64_t ldi,
                                                          const float* __restrict__ sw) {
  const int t = blockIdx.x;
  for (int c = threadIdx.x; c < N; c += blockDim.x) {
    float a = 0.f;
    for (int j = 0; j < top; ++j) {
      const int pl = place[(int64_t)t * top + j];
      const float e = pl >= 0 ? y[(int64_t)pl * N + c] : (ident ? El<T>::ld(ident + (int64_t)t * ldi + c) : 0.f);
      a = fmaf(wts ? wts[(int64_t)t * top + j] : 1.0f, e, a);
    }
    if (shared_) a = fmaf(sw ? sw[t] : 1.0f, El<T>::ld(shared_ + (int64_t)t * lds_ + c), a);
    out[(int64_t)t * N + c] = a;
  }
}

void launch_moe_combine(const void* y, const void* place, const void* wts, const void* shared_, int64_t lds_,
                        void* out, int T_, int N, int top, int dt, const void* ident, int64_t ldi, const void* sw,
                        hipStream_t st) {
  if (T_ == 0) return;
  DISPATCH_T(dt, T, (moe_combine_kernel<T><<<T_, 256, 0, st>>>((const float*)y, (const int*)place, (const float*)wts,
                                                                (const T*)shared_, lds_, (float*)out, N, top,
                                                                (const T*)ident, ldi, (const float*)sw)));
  HIP_CHECK_LAUNCH();
}

// ------------------------------------------------------------------------------------------------ dense GLU
// out[t, f] = glu(gu[t, f], gu[t, F + f])
template <typename T>
__global__ __launch_bounds__(256) void glu_clamp_kernel(const T* __restrict__ gu, int64_t ldg, T* __restrict__ out,
                                                        int64_t ldo, int F, float limit, float alpha) {
  const int t = blockIdx.x;
  const T* g = gu + (int64_t)t * ldg;
  for (int f = threadIdx.x; f < F; f += blockDim.x)
    El<T>::st(out + (int64_t)t * ldo + f, glu_clamped(El<T>::ld(g + f), El<T>::ld(g + F + f), limit, alpha));
}

void launch_glu_clamp(const void* gu, int64_t ldg, void* out, int64_t ldo, int T_, int F, float limit, float alpha,
                      int dt, hipStream_t st) {
  if (T_ == 0) return;
  DISPATCH_T(dt, T, (glu_clamp_kernel<T><<<T_, 256, 0, st>>>((const T*)gu, ldg, (T*)out, ldo, F, limit, alpha)));
  HIP_CHECK_LAUNCH();
}
