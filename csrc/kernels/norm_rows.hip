// Row kernels of layers whose attention values are its projected keys and whose routed feed-forward runs beside the mixer:
//
//   qk_row_norm_cache      biases, RMS norms over the whole query and key projections, query temperature, paged write of the
//                          projected key and its norm's statistic (the key norm's weight goes into the query)
//   residual_routed_norm   x += mixer output + weighted expert rows + a vector, in fp32, and the next layer's normalised input
//                          from the same pass
//
// One workgroup per row; any width, four or eight columns per access where sizes and bases allow it.  Statistics, sums and
// temperatures are fp32; only the stored activations take the activation dtype T (bf16 or float).
#include "common.h"
#include "hybrid_launchers.h"

namespace {

bool aligned16(const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; }

template <int V>
SYM_DEV void ldv(const bf16* p, float* f) {
  if constexpr (V == 8) load8(p, f);
  else if constexpr (V == 4) {
    const bf16x4 v = *reinterpret_cast<const bf16x4*>(p);
#pragma unroll
    for (int i = 0; i < 4; ++i) f[i] = (float)v[i];
  } else f[0] = (float)p[0];
}
template <int V>
SYM_DEV void ldv(const float* p, float* f) {
  if constexpr (V == 8) load8f(p, f);
  else if constexpr (V == 4) {
    const float4 v = *reinterpret_cast<const float4*>(p);
    f[0] = v.x, f[1] = v.y, f[2] = v.z, f[3] = v.w;
  } else f[0] = p[0];
}
template <int V>
SYM_DEV void stv(bf16* p, const float* f) {
  if constexpr (V == 8) store8(p, f);
  else if constexpr (V == 4) {
    bf16x4 v;
#pragma unroll
    for (int i = 0; i < 4; ++i) v[i] = (bf16)f[i];
    *reinterpret_cast<bf16x4*>(p) = v;
  } else p[0] = (bf16)f[0];
}
template <int V>
SYM_DEV void stv(float* p, const float* f) {
  if constexpr (V == 8) store8f(p, f);
  else if constexpr (V == 4) *reinterpret_cast<float4*>(p) = make_float4(f[0], f[1], f[2], f[3]);
  else p[0] = f[0];
}

// sums of two values over the workgroup
template <int BT>
SYM_DEV void block_sum2(float& a, float& b, float* scratch) {
  a = wave_sum(a), b = wave_sum(b);
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6;
  if (lane == 0) scratch[2 * w] = a, scratch[2 * w + 1] = b;
  __syncthreads();
  a = b = 0.f;
#pragma unroll
  for (int i = 0; i < BT / 64; ++i) a += scratch[2 * i], b += scratch[2 * i + 1];
}

template <typename T, int BT, int V>
__global__ __launch_bounds__(BT) void qk_row_norm_cache_kernel(QkRowNormArgs a) {
  __shared__ float scratch[2 * (BT / 64)];
  const int row = blockIdx.x, nq = a.H * a.dk, nk = a.G * a.dk, n = nq + nk;
  const T* z = reinterpret_cast<const T*>(a.z) + (long long)row * a.ldz;
  float sq = 0.f, sk = 0.f;
  for (int c = V * threadIdx.x; c < n; c += V * BT) {
    float v[V], b[V], s = 0.f;
    ldv<V>(z + c, v);
    if (a.bias) ldv<V>(a.bias + c, b);
#pragma unroll
    for (int i = 0; i < V; ++i) {
      if (a.bias) v[i] += b[i];
      s += v[i] * v[i];
    }
    if (c < nq) sq += s;
    else sk += s;
  }
  block_sum2<BT>(sq, sk, scratch);
  const int p = a.positions[row], slot = a.slots[row];
  const float rk = 1.f / sqrtf(sk / (float)nk + a.eps);
  const float rq = 1.f / sqrtf(sq / (float)nq + a.eps) * (1.f + a.coef * logf((float)((p + 1) / a.every + 1)));
  if (threadIdx.x == 0 && slot >= 0) a.key_scale[slot] = rk;
  T* q = reinterpret_cast<T*>(a.q_out) + (long long)row * nq;
  T* kv = reinterpret_cast<T*>(a.kv_cache) + (long long)slot * nk;
  const int rep = a.H / a.G;
  for (int c = V * threadIdx.x; c < n; c += V * BT) {
    if (c >= nq && slot < 0) break;
    float v[V], b[V];
    ldv<V>(z + c, v);
    if (a.bias) {
      ldv<V>(a.bias + c, b);
#pragma unroll
      for (int i = 0; i < V; ++i) v[i] += b[i];
    }
    if (c < nq) {
      const int head = c / a.dk;
      float w[V], wk[V];
      ldv<V>(a.wq + c, w);
      ldv<V>(a.wk + (head / rep) * a.dk + (c - head * a.dk), wk);
#pragma unroll
      for (int i = 0; i < V; ++i) v[i] *= rq * w[i] * wk[i];
      stv<V>(q + c, v);
    } else {
      stv<V>(kv + (c - nq), v);
    }
  }
}

// VPT > 0: the row's sums stay in registers, VPT vectors of four columns per thread (d <= 4 BT VPT); VPT == 0: any width
template <typename T, int BT, int VPT>
__global__ __launch_bounds__(BT) void residual_routed_norm_kernel(RoutedSumArgs a) {
  __shared__ float scratch[BT / 64];
  __shared__ float wts[64];
  __shared__ int rows[64];
  constexpr int V = VPT > 0 ? 4 : 1, P = VPT > 0 ? VPT : 1;
  const int row = blockIdx.x, d = a.d;
  const long long o = (long long)row * d;
  float* x = a.x + o;
  const T* ya = reinterpret_cast<const T*>(a.a);
  const T* yr = reinterpret_cast<const T*>(a.y);
  const int k = a.y ? a.k : 0;
  if (k) {
    if ((int)threadIdx.x < k) {
      rows[threadIdx.x] = a.dst[(long long)row * k + threadIdx.x];
      wts[threadIdx.x] = a.w[(long long)row * k + threadIdx.x];
    }
    __syncthreads();
  }
  float sq = 0.f, keep[P][V];
  const auto sum = [&](int c, float* s) {
    float t[V];
    ldv<V>(x + c, s);
    if (a.a) {
      ldv<V>(ya + o + c, t);
#pragma unroll
      for (int i = 0; i < V; ++i) s[i] += t[i];
    }
#pragma unroll 4
    for (int j = 0; j < k; ++j) {
      ldv<V>(yr + (long long)rows[j] * d + c, t);
      const float w = wts[j];
#pragma unroll
      for (int i = 0; i < V; ++i) s[i] += w * t[i];
    }
    if (a.bias) {
      ldv<V>(a.bias + c, t);
#pragma unroll
      for (int i = 0; i < V; ++i) s[i] += t[i];
    }
#pragma unroll
    for (int i = 0; i < V; ++i) sq += s[i] * s[i];
    stv<V>(x + c, s);
  };
  if constexpr (VPT > 0) {
#pragma unroll
    for (int i = 0; i < VPT; ++i) {
      const int c = 4 * (threadIdx.x + BT * i);
      if (c < d) sum(c, keep[i]);
    }
  } else {
    for (int c = threadIdx.x; c < d; c += BT) sum(c, keep[0]);
  }
  if (!a.out) return;      // (launch-uniform)
  const float r = 1.f / sqrtf(block_sum<BT>(sq, scratch) / (float)d + a.eps);
  T* out = reinterpret_cast<T*>(a.out) + o;
  if constexpr (VPT > 0) {
#pragma unroll
    for (int i = 0; i < VPT; ++i) {
      const int c = 4 * (threadIdx.x + BT * i);
      if (c < d) {
        float w[4];
        ldv<4>(a.wn + c, w);
#pragma unroll
        for (int u = 0; u < 4; ++u) w[u] *= keep[i][u] * r;
        stv<4>(out + c, w);
      }
    }
  } else {      // (each thread re-reads the columns it wrote itself)
    for (int c = threadIdx.x; c < d; c += BT) out[c] = (T)(x[c] * r * a.wn[c]);
  }
}

}  // namespace

#define DISPATCH_T(f32, ...)      \
  if (f32) {                      \
    using T = float;              \
    __VA_ARGS__                   \
  } else {                        \
    using T = bf16;               \
    __VA_ARGS__                   \
  }

void launch_qk_row_norm_cache(const QkRowNormArgs& a, int T_, int f32, hipStream_t s) {
  if (T_ <= 0) return;
  const bool vec = a.dk % 8 == 0 && a.ldz % 8 == 0 && aligned16(a.z) && aligned16(a.bias) && aligned16(a.wq) &&
                   aligned16(a.wk) && aligned16(a.q_out) && aligned16(a.kv_cache);
#define QK(BT, V) DISPATCH_T(f32, (qk_row_norm_cache_kernel<T, BT, V><<<T_, BT, 0, s>>>(a));)
  if (!vec) { QK(256, 1) }
  else if (T_ <= 256 && (a.H + a.G) * a.dk > 2048) { QK(512, 8) }
  else { QK(256, 8) }
#undef QK
}

void launch_residual_routed_norm(const RoutedSumArgs& a, int f32, hipStream_t s) {
  if (a.T <= 0) return;
  const bool vec = a.d % 4 == 0 && aligned16(a.x) && aligned16(a.a) && aligned16(a.y) && aligned16(a.bias) &&
                   aligned16(a.wn) && aligned16(a.out);
#define RN(BT, VPT) DISPATCH_T(f32, (residual_routed_norm_kernel<T, BT, VPT><<<a.T, BT, 0, s>>>(a));)
  const int q = a.d / 4;
  if (!vec || q > 4 * 1024) { RN(256, 0) }
  else if (q <= 256) { RN(256, 1) }
  else if (q <= 512) { if (a.T <= 256) { RN(512, 1) } else { RN(256, 2) } }
  else if (q <= 1024) { if (a.T <= 256) { RN(1024, 1) } else { RN(256, 4) } }
  else if (q <= 2048) { RN(1024, 2) }
  else { RN(1024, 4) }
#undef RN
}
