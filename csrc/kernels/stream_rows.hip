// Row kernels of models with several residual streams, a hashed token-pair embedding, convolved attention projections
// and a matrix memory with a normaliser:
//
//   embed_pair_hash      every stream = table[token] + pair_table[hash(previous token, token)]   (fp32 streams)
//   token_state_update   a run's last token into its sequence's state slot
//   hyper_mix_norm       streams <- streams M + c_out y (all at once), and the next sublayer's input rms_norm(c_in . streams)
//                        from the same pass; also the plain gathered sum + norm in front of the output head
//   conv_qkv_cache       causal per-channel convolution of q | k | v with carried taps, unit-RMS value heads, paged cache write
//                        (a workgroup per (row, head))
//   memory_norm_gate     o / (max(|n . q|, exp(-m)) + 1e-6), unit RMS per head, weight, sigmoid gate
//   logit_softcap        cap tanh(logits / cap)
//   residual_layer_norm  x = base + a + b on the fp32 stream and the next sublayer's layer norm (weight, bias) from the same
//                        pass; also the gathered norm in front of the output head
//   conv_silu_qkv        causal per-channel convolution of q | k | v with carried taps, silu, unit-vector q / k heads (a wave
//                        per (rows, head)); in decode-sized steps also a few fp32 projections of the same input
//
// One workgroup per row unless noted; columns strided over the threads (coalesced), any width.  All statistics, mixing
// and sums are fp32; only the stored activations take the activation dtype T (bf16 or float).
#include "common.h"
#include "hybrid_launchers.h"
#include "wave_dot.h"

namespace {

constexpr int NT = 256;
constexpr int MAX_S = 8;      // residual streams
constexpr int MAX_TAPS = 16;

SYM_DEV float ldf(const void* p, int f32, long long i) {
  return f32 ? reinterpret_cast<const float*>(p)[i] : (float)reinterpret_cast<const bf16*>(p)[i];
}
SYM_DEV float sigmoidf(float v) { return 1.f / (1.f + expf(-v)); }

SYM_DEV long long token_of(const int* ids, const int* src, const int* prev, int row) {
  const int sr = src ? src[row] : -1;
  return sr >= 0 ? prev[sr] : ids[row];
}

template <typename T, int BT>
__global__ __launch_bounds__(BT) void embed_pair_hash_kernel(PairHashArgs a) {
  const int row = blockIdx.x, d = a.d, S = a.S;
  const long long tok = token_of(a.ids, a.src, a.prev, row);
  long long prow = -1;
  if (a.pair_table) {
    const int pr = a.prev_row[row];
    if (pr == -1) {
      prow = a.buckets;
    } else {
      const long long ptok = pr >= 0 ? token_of(a.ids, a.src, a.prev, pr) : a.tok_state[-(pr + 2)];
      const long long n = a.buckets;
      prow = ((ptok * a.mul_prev + tok * a.mul_cur) % n + n) % n;
    }
  }
  const T* t = reinterpret_cast<const T*>(a.table) + tok * d;
  const T* pt = prow >= 0 ? reinterpret_cast<const T*>(a.pair_table) + prow * d : nullptr;
  float* x = a.x + (long long)row * S * d;
  for (int c = threadIdx.x; c < d; c += BT) {
    float v = (float)t[c];
    if (pt) v += (float)pt[c];
    for (int s = 0; s < S; ++s) x[(long long)s * d + c] = v;
  }
  // rows that are runs of their own: the row's token becomes the carried one (after every thread has read the old one)
  if (a.save_slot) {
    __syncthreads();
    const int sv = a.save_slot[row];
    if (threadIdx.x == 0 && sv >= 0) a.tok_state[sv] = (int)tok;
  }
}

__global__ __launch_bounds__(NT) void token_state_update_kernel(const int* __restrict__ ids, int* __restrict__ tok_state,
                                                                const int* __restrict__ cu_q,
                                                                const int* __restrict__ save_slot, int runs) {
  const int run = blockIdx.x * NT + threadIdx.x;
  if (run >= runs) return;
  const int s0 = cu_q ? cu_q[run] : run, s1 = cu_q ? cu_q[run + 1] : run + 1;
  if (s1 <= s0) return;
  const int sv = save_slot[s1 - 1];
  if (sv >= 0) tok_state[sv] = ids[s1 - 1];
}

// Dynamic LDS: d floats (the mixed input u of the row, kept between the two passes) + S S + 2 S floats.
template <typename T, int BT>
__global__ __launch_bounds__(BT) void hyper_mix_norm_kernel(HyperMixArgs a) {
  extern __shared__ float lds[];
  __shared__ float scratch[BT / 64];
  const int row = blockIdx.x, d = a.d, S = a.S;
  float* us = lds;                 // [d]
  float* ms = lds + d;             // [S][S] mix, then [S] outc, [S] inc
  const bool upd = a.a != nullptr && row < a.T;
  const bool emit = a.out != nullptr && row < a.n;
  for (int i = threadIdx.x; i < S * S + 2 * S; i += BT) {
    float v = 1.f;
    if (i < S * S) v = a.mix ? a.mix[i] : 0.f;
    else if (i < S * S + S) v = a.outc ? a.outc[i - S * S] : 0.f;
    else v = a.inc ? a.inc[i - S * S - S] : 1.f;
    ms[i] = v;
  }
  __syncthreads();
  const float* outc = ms + S * S;
  const float* inc = outc + S;
  const long long xrow = a.rows ? a.rows[row] : (long long)row;
  float* x = a.xs + xrow * S * d;
  const long long o = (long long)row * d;
  float sq = 0.f;
  for (int c = threadIdx.x; c < d; c += BT) {
    float xv[MAX_S];
#pragma unroll
    for (int s = 0; s < MAX_S; ++s)
      if (s < S) xv[s] = x[(long long)s * d + c];
    if (upd) {
      float y = a.sa * ldf(a.a, a.a_f32, o + c);
      if (a.b) y += a.sb * ldf(a.b, a.b_f32, o + c);
      float nv[MAX_S];
#pragma unroll
      for (int t = 0; t < MAX_S; ++t) {
        if (t < S) {
          float acc = outc[t] * y;
#pragma unroll
          for (int s = 0; s < MAX_S; ++s)
            if (s < S) acc += ms[s * S + t] * xv[s];
          nv[t] = acc;
        }
      }
#pragma unroll
      for (int t = 0; t < MAX_S; ++t)
        if (t < S) {
          xv[t] = nv[t];
          x[(long long)t * d + c] = nv[t];
        }
    }
    if (emit) {
      float u = 0.f;
#pragma unroll
      for (int s = 0; s < MAX_S; ++s)
        if (s < S) u += inc[s] * xv[s];
      us[c] = u;
      sq += u * u;
    }
  }
  if (!emit) return;     // (row-uniform)
  const float r = 1.f / sqrtf(block_sum<BT>(sq, scratch) / (float)d + a.eps);
  T* out = reinterpret_cast<T*>(a.out) + o;
  // (each thread re-reads the columns it wrote itself)
  for (int c = threadIdx.x; c < d; c += BT) out[c] = (T)(us[c] * r * a.w[c]);
}

// grid (T, H + 2 G): one workgroup of CQ threads per (row, head of q | k | v), a thread per channel (wider heads: several).
// A value head is brought to unit RMS before it is stored.  The small workgroups give a decode step's few rows a few
// hundred of them; a thread's taps and carried inputs are loads that do not depend on one another.
constexpr int CQ = 128;
constexpr int CQ_PER = 4;     // channels per thread kept in registers: heads up to 512 wide
template <typename T>
__global__ __launch_bounds__(CQ) void conv_qkv_cache_kernel(ConvQkvArgs a) {
  __shared__ float scratch[CQ / 64];
  const int row = blockIdx.x, unit = blockIdx.y, C = a.C, taps = a.taps;
  const int nq = a.H * a.dk, nk = a.G * a.dk;
  // the unit's channels [c0, c0 + width) and where they go
  int c0, width;
  T* dst_out;
  const int slot = a.slots[row];
  bool vhead = false;
  if (unit < a.H) {
    c0 = unit * a.dk, width = a.dk;
    dst_out = reinterpret_cast<T*>(a.q_out) + (long long)row * nq + c0;
  } else if (unit < a.H + a.G) {
    const int g = unit - a.H;
    c0 = nq + g * a.dk, width = a.dk;
    dst_out = slot >= 0 ? reinterpret_cast<T*>(a.k_cache) + (long long)slot * nk + g * a.dk : nullptr;
  } else {
    const int g = unit - a.H - a.G;
    c0 = nq + nk + g * a.dv, width = a.dv;
    dst_out = slot >= 0 ? reinterpret_cast<T*>(a.v_cache) + ((long long)slot * a.G + g) * a.dv : nullptr;
    vhead = true;
  }
  const int s0 = a.cu_q ? a.cu_q[a.row_seq[row]] : row;
  const int j = row - s0;
  const int pr = a.prev_row[s0];
  const T* st = pr <= -2 ? reinterpret_cast<const T*>(a.state) + (long long)(-(pr + 2)) * a.state_stride : nullptr;
  const T* z = reinterpret_cast<const T*>(a.z);
  const T* w = reinterpret_cast<const T*>(a.w);
  const int sv = (!a.cu_q && a.save_slot) ? a.save_slot[row] : -1;
  T* dst = sv >= 0 ? reinterpret_cast<T*>(a.state) + (long long)sv * a.state_stride : nullptr;
  float y[CQ_PER];
  float sq = 0.f;
#pragma unroll
  for (int u = 0; u < CQ_PER; ++u) {
    const int e = threadIdx.x + u * CQ;
    y[u] = 0.f;
    if (e < width) {
      const int c = c0 + e;
      float acc = 0.f;
      for (int i = 0; i < taps; ++i) {       // i positions back
        float v = 0.f;
        if (i <= j) v = (float)z[(long long)(row - i) * a.ldz + c];
        else if (st) v = (float)st[(long long)(taps - 1 - (i - j)) * C + c];
        acc += (float)w[(long long)c * taps + taps - 1 - i] * v;
      }
      y[u] = acc;
      sq += acc * acc;
      // rows that are runs of their own: this thread alone reads and writes its channel of the row's slot, so the
      // carried taps move on here (older ones one place down, the row's input on top)
      if (dst && taps > 1) {
        const int keep = taps - 1;
        T vals[MAX_TAPS];
#pragma unroll
        for (int m = 0; m < MAX_TAPS; ++m)
          if (m < keep) vals[m] = m + 1 < keep ? (st ? st[(long long)(m + 1) * C + c] : (T)0.f) : z[(long long)row * a.ldz + c];
#pragma unroll
        for (int m = 0; m < MAX_TAPS; ++m)
          if (m < keep) dst[(long long)m * C + c] = vals[m];
      }
    }
  }
  float r = 1.f;
  if (vhead) r = 1.f / sqrtf(block_sum<CQ>(sq, scratch) / (float)a.dv + a.v_eps);     // (unit-uniform branch)
  if (!dst_out) return;
#pragma unroll
  for (int u = 0; u < CQ_PER; ++u) {
    const int e = threadIdx.x + u * CQ;
    if (e < width) dst_out[e] = (T)(y[u] * r);
  }
}

// grid (T, H), one wave per (row, head)
template <typename T>
__global__ __launch_bounds__(64) void memory_norm_gate_kernel(const float* __restrict__ y, const float* __restrict__ m,
                                                              const T* __restrict__ gate, long long ldg,
                                                              const float* __restrict__ w, float eps, T* __restrict__ out,
                                                              int H, int P) {
  const int row = blockIdx.x, h = blockIdx.y, lane = threadIdx.x;
  const float* yr = y + ((long long)row * H + h) * (P + 1);
  const float den = fmaxf(fabsf(yr[P]), expf(-m[(long long)row * H + h])) + 1e-6f;
  float sq = 0.f;
  for (int c = lane; c < P; c += 64) {
    const float o = yr[c] / den;
    sq += o * o;
  }
  const float r = 1.f / sqrtf(wave_sum(sq) / (float)P + eps);
  const T* gr = gate + (long long)row * ldg + (long long)h * P;
  T* orow = out + ((long long)row * H + h) * P;
  for (int c = lane; c < P; c += 64)
    orow[c] = (T)(yr[c] / den * r * w[(long long)h * P + c] * sigmoidf((float)gr[c]));
}

// Four columns of a row, fp32 or bf16
SYM_DEV float4 ld4(const void* p, int f32, long long i) {
  if (f32) return *reinterpret_cast<const float4*>(reinterpret_cast<const float*>(p) + i);
  const bf16x4 v = *reinterpret_cast<const bf16x4*>(reinterpret_cast<const bf16*>(p) + i);
  return make_float4((float)v[0], (float)v[1], (float)v[2], (float)v[3]);
}
SYM_DEV void st4(float* p, const float4& v) { *reinterpret_cast<float4*>(p) = v; }
SYM_DEV void st4(bf16* p, const float4& v) {
  bf16x4 o;
  o[0] = (bf16)v.x, o[1] = (bf16)v.y, o[2] = (bf16)v.z, o[3] = (bf16)v.w;
  *reinterpret_cast<bf16x4*>(p) = o;
}

// One workgroup per row; VPT > 0: the row in registers, VPT vectors of four columns per thread (d % 4 == 0, d <= 4 BT VPT);
// VPT == 0: any width, columns strided over the threads and re-read (each thread those it wrote itself)
template <typename T, int BT, int VPT>
__global__ __launch_bounds__(BT) void residual_layer_norm_kernel(ResidualLnArgs a) {
  __shared__ float scratch[BT / 64];
  const int row = blockIdx.x, d = a.d;
  const long long xrow = a.rows ? a.rows[row] : (long long)row;
  const long long o = (long long)row * d;
  float* x = a.x + xrow * d;
  const float* base = a.base ? a.base + xrow * d : x;
  const bool upd = a.base || a.a || a.b;
  float sum = 0.f, sq = 0.f;
  if constexpr (VPT > 0) {
    float4 v[VPT];
#pragma unroll
    for (int i = 0; i < VPT; ++i) {
      const int c = 4 * (threadIdx.x + BT * i);
      v[i] = make_float4(0.f, 0.f, 0.f, 0.f);
      if (c < d) {
        v[i] = *reinterpret_cast<const float4*>(base + c);
        if (a.a) {
          const float4 t = ld4(a.a, a.a_f32, o + c);
          v[i].x += t.x, v[i].y += t.y, v[i].z += t.z, v[i].w += t.w;
        }
        if (a.b) {
          const float4 t = ld4(a.b, a.b_f32, o + c);
          v[i].x += t.x, v[i].y += t.y, v[i].z += t.z, v[i].w += t.w;
        }
        if (upd) st4(x + c, v[i]);
        sum += (v[i].x + v[i].y) + (v[i].z + v[i].w);
      }
    }
    if (!a.out) return;     // (launch-uniform)
    float4 w[VPT], bs[VPT];   // (loads under the reductions)
#pragma unroll
    for (int i = 0; i < VPT; ++i) {
      const int c = 4 * (threadIdx.x + BT * i);
      if (c < d) {
        w[i] = *reinterpret_cast<const float4*>(a.w + c);
        bs[i] = *reinterpret_cast<const float4*>(a.bias + c);
      }
    }
    const float mean = block_sum<BT>(sum, scratch) / (float)d;
#pragma unroll
    for (int i = 0; i < VPT; ++i) {
      if (4 * (int)(threadIdx.x + BT * i) < d) {
        v[i].x -= mean, v[i].y -= mean, v[i].z -= mean, v[i].w -= mean;
        sq += v[i].x * v[i].x + v[i].y * v[i].y + v[i].z * v[i].z + v[i].w * v[i].w;
      }
    }
    const float r = 1.f / sqrtf(block_sum<BT>(sq, scratch) / (float)d + a.eps);
    T* out = reinterpret_cast<T*>(a.out) + o;
#pragma unroll
    for (int i = 0; i < VPT; ++i) {
      const int c = 4 * (threadIdx.x + BT * i);
      if (c < d)
        st4(out + c, make_float4(v[i].x * r * w[i].x + bs[i].x, v[i].y * r * w[i].y + bs[i].y, v[i].z * r * w[i].z + bs[i].z,
                                 v[i].w * r * w[i].w + bs[i].w));
    }
  } else {
    for (int c = threadIdx.x; c < d; c += BT) {
      float v = base[c];
      if (a.a) v += ldf(a.a, a.a_f32, o + c);
      if (a.b) v += ldf(a.b, a.b_f32, o + c);
      if (upd) x[c] = v;
      sum += v;
    }
    if (!a.out) return;
    const float mean = block_sum<BT>(sum, scratch) / (float)d;
    for (int c = threadIdx.x; c < d; c += BT) sq += (x[c] - mean) * (x[c] - mean);
    const float r = 1.f / sqrtf(block_sum<BT>(sq, scratch) / (float)d + a.eps);
    T* out = reinterpret_cast<T*>(a.out) + o;
    for (int c = threadIdx.x; c < d; c += BT) out[c] = (T)((x[c] - mean) * r * a.w[c] + a.bias[c]);
  }
}

// One head's share of conv_silu_qkv: which channels of the projection a unit covers, and where its row goes
struct ConvUnit {
  int kind, hd, width, c0;     // kind 0: q, 1: k, 2: v
};
SYM_DEV ConvUnit conv_unit(const ConvSiluArgs& a, int unit) {
  ConvUnit u;
  u.kind = unit < a.G ? 0 : (unit < 2 * a.G ? 1 : 2);
  u.hd = unit - u.kind * a.G;
  u.width = u.kind == 2 ? a.P : a.N;
  u.c0 = u.kind * a.G * a.N + u.hd * u.width;
  return u;
}

// silu, unit length (q, k), store.  y: the wave's PER x VC convolved channels of the row's head
template <typename T, int VC, int PER>
SYM_DEV void conv_silu_store(const ConvSiluArgs& a, const ConvUnit& un, int row, int lane, float (&y)[PER][VC]) {
  float sq = 0.f;
#pragma unroll
  for (int u = 0; u < PER; ++u)
#pragma unroll
    for (int i = 0; i < VC; ++i) {
      y[u][i] *= sigmoidf(y[u][i]);      // (channels past the head's width are 0)
      sq += y[u][i] * y[u][i];
    }
  float r = 1.f;
  if (un.kind < 2) r = 1.f / sqrtf(wave_sum(sq) + a.eps) * (un.kind == 0 ? a.q_scale : 1.f);
#pragma unroll
  for (int u = 0; u < PER; ++u) {
    const int e = VC * (lane + 64 * u);
    if (e < un.width) {
      if (un.kind < 2) {
        float* o = (un.kind == 0 ? a.q_out : a.k_out) + (long long)row * a.G * a.N + un.hd * un.width + e;
        if constexpr (VC == 4) st4(o, make_float4(y[u][0] * r, y[u][1] * r, y[u][2] * r, y[u][3] * r));
        else o[0] = y[u][0] * r;
      } else {
        T* o = reinterpret_cast<T*>(a.v_out) + ((long long)row * a.H + un.hd) * un.width + e;
        if constexpr (VC == 4) st4(o, make_float4(y[u][0], y[u][1], y[u][2], y[u][3]));
        else o[0] = (T)y[u][0];
      }
    }
  }
}

// A wave past the heads: one output of the small projection that rides along (one row per wave)
template <typename T>
SYM_DEV void conv_gate_unit(const ConvSiluArgs& a, int j, int row, int lane) {
  if (j >= a.gn) return;
  const float v = wave_dot<T>(reinterpret_cast<const T*>(a.gx) + (long long)row * a.ldgx,
                              reinterpret_cast<const T*>(a.gw) + (long long)j * a.gd, a.gd, lane);
  if (lane == 0) a.gout[(long long)row * a.gn + j] = v;
}

// The usual tap counts, heads up to 256 wide, four channels per lane: the taps are loaded once per wave and the inputs
// slide through registers from row to row (a run's start reloads them from the slot).  A wave per (ROWS rows, head).
template <typename T, int TAPS, int ROWS>
__global__ void conv_silu_qkv_taps_kernel(ConvSiluArgs a) {
  const int lane = threadIdx.x & 63;
  const int unit = blockIdx.y * (blockDim.x >> 6) + (threadIdx.x >> 6);
  if (unit >= 2 * a.G + a.H) {
    if (ROWS == 1 && a.gn) conv_gate_unit<T>(a, unit - 2 * a.G - a.H, blockIdx.x, lane);
    return;
  }
  const ConvUnit un = conv_unit(a, unit);
  const int C = a.C, e = 4 * lane, c = un.c0 + e;
  const bool in = e < un.width;
  const T* z = reinterpret_cast<const T*>(a.z);
  T wr[4 * TAPS];              // [channel][tap]
  if (in) {
    const T* w = reinterpret_cast<const T*>(a.w) + (long long)c * TAPS;
#pragma unroll
    for (int i = 0; i < TAPS; ++i)
      __builtin_memcpy(wr + 4 * i, __builtin_assume_aligned(w + 4 * i, 4 * sizeof(T)), 4 * sizeof(T));
  }
  T hist[TAPS][4];             // hist[b]: the input b places back
  int run0 = -1;
  const int r0 = blockIdx.x * ROWS, r1 = min(a.T, r0 + ROWS);
  for (int row = r0; row < r1; ++row) {
    const int s0 = a.cu_q ? a.cu_q[a.row_seq[row]] : row;
    float y[1][4] = {{0.f, 0.f, 0.f, 0.f}};
    if (in) {
      if (s0 != run0) {
        const int j = row - s0;
        const int pr = j < TAPS - 1 ? a.prev_row[s0] : -1;
        const T* st = pr <= -2 ? reinterpret_cast<const T*>(a.state) + (long long)(-(pr + 2)) * a.state_stride : nullptr;
#pragma unroll
        for (int b = 1; b < TAPS; ++b) {
          const T* src = b <= j ? z + (long long)(row - b) * a.ldz + c : (st ? st + (long long)(TAPS - 1 - (b - j)) * C + c : nullptr);
          if (src) {
            __builtin_memcpy(hist[b], __builtin_assume_aligned(src, 4 * sizeof(T)), 4 * sizeof(T));
          } else {
#pragma unroll
            for (int i = 0; i < 4; ++i) hist[b][i] = (T)0.f;
          }
        }
      } else {
#pragma unroll
        for (int b = TAPS - 1; b > 0; --b)
#pragma unroll
          for (int i = 0; i < 4; ++i) hist[b][i] = hist[b - 1][i];
      }
      __builtin_memcpy(hist[0], __builtin_assume_aligned(z + (long long)row * a.ldz + c, 4 * sizeof(T)), 4 * sizeof(T));
#pragma unroll
      for (int b = 0; b < TAPS; ++b)
#pragma unroll
        for (int i = 0; i < 4; ++i) y[0][i] += (float)wr[i * TAPS + TAPS - 1 - b] * (float)hist[b][i];
      // (as in the general kernel: a row that is a run of its own moves the carried taps on)
      if (!a.cu_q && a.save_slot && a.save_slot[row] >= 0) {
        T* dst = reinterpret_cast<T*>(a.state) + (long long)a.save_slot[row] * a.state_stride;
#pragma unroll
        for (int b = 0; b < TAPS - 1; ++b)
          __builtin_memcpy(__builtin_assume_aligned(dst + (long long)(TAPS - 2 - b) * C + c, 4 * sizeof(T)), hist[b],
                           4 * sizeof(T));
      }
    }
    run0 = s0;
    conv_silu_store<T, 4, 1>(a, un, row, lane, y);
  }
}

// Any tap count: a wave per (ROWS consecutive rows, head); a lane owns VC neighbouring channels of the head, PER times
// over (64 VC PER >= the widest head).  VC = 4: eight- or sixteen-byte accesses (strides, head sizes and bases permitting).
template <typename T, int VC, int PER, int ROWS>
__global__ void conv_silu_qkv_kernel(ConvSiluArgs a) {
  const int lane = threadIdx.x & 63;
  const int unit = blockIdx.y * (blockDim.x >> 6) + (threadIdx.x >> 6);
  if (unit >= 2 * a.G + a.H) {
    if (ROWS == 1 && a.gn) conv_gate_unit<T>(a, unit - 2 * a.G - a.H, blockIdx.x, lane);
    return;
  }
  const int taps = a.taps, C = a.C, keep = taps - 1;
  const ConvUnit un = conv_unit(a, unit);
  const T* z = reinterpret_cast<const T*>(a.z);
  const T* w = reinterpret_cast<const T*>(a.w);
  for (int row = blockIdx.x * ROWS; row < min(a.T, (int)(blockIdx.x + 1) * ROWS); ++row) {
    const int s0 = a.cu_q ? a.cu_q[a.row_seq[row]] : row;
    const int j = row - s0;
    const int pr = j < keep ? a.prev_row[s0] : -1;
    const T* st = pr <= -2 ? reinterpret_cast<const T*>(a.state) + (long long)(-(pr + 2)) * a.state_stride : nullptr;
    const int sv = (!a.cu_q && a.save_slot) ? a.save_slot[row] : -1;
    T* dst = sv >= 0 && keep ? reinterpret_cast<T*>(a.state) + (long long)sv * a.state_stride : nullptr;
    float y[PER][VC];
#pragma unroll
    for (int u = 0; u < PER; ++u) {
      const int e = VC * (lane + 64 * u);
#pragma unroll
      for (int i = 0; i < VC; ++i) y[u][i] = 0.f;
      if (e < un.width) {
        const int c = un.c0 + e;
        T hist[MAX_TAPS][VC];     // hist[b]: the input b places back (b = 0: this row's)
#pragma unroll
        for (int b = 0; b < MAX_TAPS; ++b) {
          if (b < taps) {
            const T* src = b <= j ? z + (long long)(row - b) * a.ldz + c : (st ? st + (long long)(keep - (b - j)) * C + c : nullptr);
            if (src) {
              if constexpr (VC == 4) __builtin_memcpy(hist[b], __builtin_assume_aligned(src, 4 * sizeof(T)), 4 * sizeof(T));
              else hist[b][0] = src[0];
            } else {
#pragma unroll
              for (int i = 0; i < VC; ++i) hist[b][i] = (T)0.f;
            }
          }
        }
#pragma unroll
        for (int b = 0; b < MAX_TAPS; ++b)
          if (b < taps)
#pragma unroll
            for (int i = 0; i < VC; ++i) y[u][i] += (float)w[(long long)(c + i) * taps + keep - b] * (float)hist[b][i];
        // rows that are runs of their own: this lane alone reads and writes its channels of the row's slot, so the carried
        // taps move on here (place m holds the input keep - m back from the next token)
        if (dst) {
#pragma unroll
          for (int b = 0; b < MAX_TAPS - 1; ++b)
            if (b < keep) {
              T* o = dst + (long long)(keep - 1 - b) * C + c;
              if constexpr (VC == 4) __builtin_memcpy(__builtin_assume_aligned(o, 4 * sizeof(T)), hist[b], 4 * sizeof(T));
              else o[0] = hist[b][0];
            }
        }
      }
    }
    conv_silu_store<T, VC, PER>(a, un, row, lane, y);
  }
}

__global__ __launch_bounds__(NT) void logit_softcap_kernel(float* __restrict__ x, long long n, float cap) {
  for (long long i = (long long)blockIdx.x * NT + threadIdx.x; i < n; i += (long long)gridDim.x * NT)
    x[i] = cap * tanhf(x[i] / cap);
}

// a decode-sized launch of wide rows: more threads per row (fewer passes over the columns)
bool wide_rows(int rows, int d) { return rows <= 256 && d >= 2048; }

}  // namespace

#define DISPATCH_T(f32, ...)      \
  if (f32) {                      \
    using T = float;              \
    __VA_ARGS__                   \
  } else {                        \
    using T = bf16;               \
    __VA_ARGS__                   \
  }

void launch_embed_pair_hash(const PairHashArgs& a, int f32, hipStream_t s) {
  if (a.T <= 0) return;
  if (wide_rows(a.T, a.d)) {
    DISPATCH_T(f32, (embed_pair_hash_kernel<T, 1024><<<a.T, 1024, 0, s>>>(a));)
  } else {
    DISPATCH_T(f32, (embed_pair_hash_kernel<T, NT><<<a.T, NT, 0, s>>>(a));)
  }
}

void launch_token_state_update(const int* ids, int* tok_state, const int* cu_q, const int* save_slot, int runs,
                               hipStream_t s) {
  if (runs <= 0) return;
  token_state_update_kernel<<<(runs + NT - 1) / NT, NT, 0, s>>>(ids, tok_state, cu_q, save_slot, runs);
}

void launch_hyper_mix_norm(const HyperMixArgs& a, int f32, hipStream_t s) {
  const int rows = a.a ? (a.out && a.n > a.T ? a.n : a.T) : (a.out ? a.n : 0);
  if (rows <= 0) return;
  const size_t lds = (size_t)(a.d + a.S * a.S + 2 * a.S) * sizeof(float);
  if (wide_rows(rows, a.d)) {
    DISPATCH_T(f32, (hyper_mix_norm_kernel<T, 1024><<<rows, 1024, lds, s>>>(a));)
  } else {
    DISPATCH_T(f32, (hyper_mix_norm_kernel<T, NT><<<rows, NT, lds, s>>>(a));)
  }
}

void launch_conv_qkv_cache(const ConvQkvArgs& a, int f32, hipStream_t s) {
  if (a.T <= 0) return;
  dim3 grid(a.T, a.H + 2 * a.G);
  DISPATCH_T(f32, conv_qkv_cache_kernel<T><<<grid, CQ, 0, s>>>(a);)
}

void launch_memory_norm_gate(const float* y, const float* m, const void* gate, long long ldg, const float* w, float eps,
                             void* out, int T_, int H, int P, int f32, hipStream_t s) {
  if (T_ <= 0) return;
  dim3 grid(T_, H);
  DISPATCH_T(f32, memory_norm_gate_kernel<T><<<grid, 64, 0, s>>>(y, m, (const T*)gate, ldg, w, eps, (T*)out, H, P);)
}

void launch_logit_softcap(float* x, long long n, float cap, hipStream_t s) {
  if (n <= 0) return;
  const long long blocks = (n + NT - 1) / NT;
  logit_softcap_kernel<<<(unsigned)(blocks < 4096 ? blocks : 4096), NT, 0, s>>>(x, n, cap);
}

void launch_residual_layer_norm(const ResidualLnArgs& a, int f32, hipStream_t s) {
  if (a.n <= 0) return;
  const auto al = [](const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; };
  const bool vec = a.d % 4 == 0 && al(a.x) && al(a.base) && al(a.a) && al(a.b) && al(a.w) && al(a.bias) && al(a.out);
#define LN(BT, VPT) DISPATCH_T(f32, (residual_layer_norm_kernel<T, BT, VPT><<<a.n, BT, 0, s>>>(a));)
  const int q = a.d / 4;
  if (!vec || q > 8 * 256) {
    if (wide_rows(a.n, a.d)) { LN(1024, 0) } else { LN(256, 0) }
  } else if (q <= 256) {
    LN(256, 1)
  } else if (a.n <= 256) {      // a decode-sized launch: more threads per row
    if (q <= 512) { LN(512, 1) } else if (q <= 1024) { LN(1024, 1) } else { LN(1024, 2) }
  } else if (q <= 512) {
    LN(256, 2)
  } else if (q <= 1024) {
    LN(256, 4)
  } else {
    LN(256, 8)
  }
#undef LN
}

// grid of a kernel with a wave per (rows, head): decode-sized launches one row and one wave per workgroup
#define CONV_ROWS(KERNEL1, KERNELN, ROWS)                                                                     \
  if (a.T <= 256) {                                                                                           \
    DISPATCH_T(f32, (KERNEL1<<<dim3(a.T, units + a.gn), 64, 0, s>>>(a));)                                          \
  } else {                                                                                                    \
    DISPATCH_T(f32, (KERNELN<<<dim3((a.T + ROWS - 1) / ROWS, (units + 3) / 4), 256, 0, s>>>(a));)             \
  }

void launch_conv_silu_qkv(const ConvSiluArgs& a, int f32, hipStream_t s) {
  if (a.T <= 0) return;
  const auto al = [](const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; };
  const int wide = a.N > a.P ? a.N : a.P, units = 2 * a.G + a.H;
  const bool vec = a.N % 4 == 0 && a.P % 4 == 0 && a.ldz % 4 == 0 && al(a.z) && al(a.w) && al(a.state) &&
                   a.state_stride % 4 == 0 && al(a.q_out) && al(a.k_out) && al(a.v_out);
  if (vec && wide <= 256 && a.taps == 4) {
    CONV_ROWS((conv_silu_qkv_taps_kernel<T, 4, 1>), (conv_silu_qkv_taps_kernel<T, 4, 8>), 8)
  } else if (vec && wide <= 256 && a.taps == 3) {
    CONV_ROWS((conv_silu_qkv_taps_kernel<T, 3, 1>), (conv_silu_qkv_taps_kernel<T, 3, 8>), 8)
  } else if (vec && wide <= 256 && a.taps == 2) {
    CONV_ROWS((conv_silu_qkv_taps_kernel<T, 2, 1>), (conv_silu_qkv_taps_kernel<T, 2, 8>), 8)
  } else if (vec) {      // heads up to 512 wide (checked by the op layer)
    CONV_ROWS((conv_silu_qkv_kernel<T, 4, 2, 1>), (conv_silu_qkv_kernel<T, 4, 2, 4>), 4)
  } else {
    CONV_ROWS((conv_silu_qkv_kernel<T, 1, 8, 1>), (conv_silu_qkv_kernel<T, 1, 8, 4>), 4)
  }
}
#undef CONV_ROWS
