// Gated delta rule: a linear recurrence whose state [N x P] (fp32, per sequence and head) is corrected towards every new
// key / value pair,
//
//     S <- diag(g_t) S;   u_t = beta_t (v_t - S^T k_t);   S <- S + k_t u_t^T;   o_t = S^T q_t
//
//     beta_t = sigmoid(bz_t),   log g_t = -exp(A_log) softplus(dz_t + dt_bias)     per head, or per head and key channel
//
// q, k fp32 (unit vectors: see conv_silu_qkv), v in the activation dtype; decays, step sizes, states and sums fp32.  A run
// of rows (one sequence's tokens of a step) starts from its state slot (or zero at position 0) and ends in it; each (slot,
// head, column) is read and written by one lane group of one workgroup.
//
// Two forms:
//
// 1. Token by token (decode steps, the 32-bit model): grid (P / columns, heads, runs).  A wave's lanes are PCOLS value
//    columns x SLICES slices of the key channels, the slices in neighbouring lanes: S^T k sits on the serial path of every
//    token, and a sum over neighbouring lanes is two or three cross-lane adds on the vector unit (no LDS round trip).  The
//    vectors that all columns share are staged through LDS for CH tokens at a time, the next batch's loads in flight.
//
// 2. Chunked (prompt steps): with chunks of C = 32 tokens, G_i the running sum of log g inside the chunk and S_0 the state
//    in front of it,
//        u_i = beta_i (v_i - (k_i e^(G_i))^T S_0 - sum_{j < i} Akk_ij u_j),      Akk_ij = sum_n k_i k_j e^(G_i - G_j)
//        o_i = (q_i e^(G_i))^T S_0 + sum_{j <= i} Aqk_ij u_j                      (every exponent <= 0: nothing overflows)
//        S_C = e^(G_C) S_0 + sum_j (k_j e^(G_C - G_j)) u_j^T
//    delta_chunk_prep_kernel (one workgroup per chunk and head, all chunks at once) evaluates Akk, Aqk -- the exponents of
//    differences taken per (i, j, channel), so strong decays are exact -- and T = (I + diag(beta) Akk)^-1 diag(beta) by
//    forward substitution.  delta_chunk_scan_kernel (grid (P / 64, heads, runs)) then walks a run's chunks with
//        R = V - Kt S,   U = T R,   O = Qt S + Aqk U,   S <- D S + Kh^T U
//    as fp32 matrix products (v_mfma_f32_16x16x4_f32).  A wave owns 16 value columns and ALL of N: its state stays in
//    accumulator registers for the whole run, and since an accumulator's rows are 4 (lane / 16) + r and a B operand's
//    contraction index is lane / 16, register r of the state IS the B operand of a step that contracts over the rows
//    4 g + r (the A operand is read in the same order: one 16-byte LDS read feeds four steps).  The same holds for R and U.
#include "common.h"
#include "hybrid_launchers.h"

namespace {

constexpr int NT = 256;
constexpr float LOG2E = 1.4426950408889634f;

SYM_DEV float softplus_exact(float v) { return fmaxf(v, 0.f) + log1pf(expf(-fabsf(v))); }
SYM_DEV float sigmoidf(float v) { return 1.f / (1.f + expf(-v)); }

template <int CTRL>
SYM_DEV float dpp_add(float v) {
  return v + __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(v), CTRL, 0xf, 0xf, true));
}
// sum over groups of 4 or 8 neighbouring lanes (quad_perm xor 1, xor 2, then the half row mirrored)
template <int SLICES>
SYM_DEV float slice_sum(float v) {
  v = dpp_add<0xB1>(v);
  v = dpp_add<0x4E>(v);
  if (SLICES == 8) v = dpp_add<0x141>(v);
  return v;
}

// NPL: state entries per lane (>= ceil(N / SLICES)); CH: tokens staged per batch
template <typename T, bool CHANNEL, int NPL, int CH, int SLICES>
__global__ __launch_bounds__(NT) void delta_scan_kernel(DeltaRuleArgs a) {
  extern __shared__ float lds[];
  constexpr int PCOLS = 64 / SLICES;
  constexpr int NPAD = NPL * SLICES;
  constexpr int LROW = SLICES * (NPL + 4);           // slices 16 bytes apart in bank space
  constexpr int EPT = (CH * NPAD + NT - 1) / NT;     // staged (token, channel) entries per thread
  constexpr int ASZ = CHANNEL ? CH * LROW : CH;
  constexpr int BUF = 2 * CH * LROW + ASZ + CH;      // q, k, decays, step sizes
  const int N = a.N, P = a.P;
  const int h = blockIdx.y, run = blockIdx.z;
  const int s0 = a.cu_q ? a.cu_q[run] : run, s1 = a.cu_q ? a.cu_q[run + 1] : run + 1;
  if (s1 <= s0) return;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int ns = lane & (SLICES - 1), pc = lane / SLICES;
  const int p = blockIdx.x * (PCOLS * (NT / 64)) + wave * PCOLS + pc;
  const bool pin = p < P;
  const int n0 = ns * NPL, l0 = ns * (NPL + 4);
  const int pr = a.prev_row[s0];
  const int sv = a.save_slot[s1 - 1];
  const long long gn = (long long)a.G * N;
  const float* q = a.q + (long long)(h / a.hpg) * N;
  const float* k = a.k + (long long)(h / a.hpg) * N;
  const T* v = reinterpret_cast<const T*>(a.v) + (long long)h * P + p;
  const float rate = expf(a.A_log[h]);
  float rq[EPT], rk[EPT], rz[EPT], vn[CH], rb = 0.f, rd = 0.f;
  auto fetch = [&](int t0) {
    const int nt = min(CH, s1 - t0);
#pragma unroll
    for (int u = 0; u < EPT; ++u) {
      const int i = threadIdx.x + NT * u;
      const int tt = i / NPAD, n = i - tt * NPAD;
      const bool in = tt < nt && n < N;
      const long long r = t0 + tt;
      rq[u] = in ? q[r * gn + n] : 0.f;
      rk[u] = in ? k[r * gn + n] : 0.f;
      if (CHANNEL) rz[u] = in ? a.dz[r * a.ldd + (long long)h * N + n] + a.dt_bias[(long long)h * N + n] : 0.f;
    }
    if (threadIdx.x < CH) {
      const bool in = (int)threadIdx.x < nt;
      const long long r = t0 + threadIdx.x;
      rb = in ? a.bz[r * a.ldb + h] : 0.f;
      if (!CHANNEL) rd = in ? a.dz[r * a.ldd + h] + a.dt_bias[h] : 0.f;
    }
#pragma unroll
    for (int tt = 0; tt < CH; ++tt)
      vn[tt] = tt < nt && pin ? (float)v[(long long)(t0 + tt) * a.H * P] : 0.f;
  };
  auto commit = [&](float* buf) {
    float* qS = buf;
    float* kS = buf + CH * LROW;
    float* aS = kS + CH * LROW;
    float* bS = aS + ASZ;
#pragma unroll
    for (int u = 0; u < EPT; ++u) {
      const int i = threadIdx.x + NT * u;
      const int tt = i / NPAD, n = i - tt * NPAD;
      if (tt < CH) {
        const int o = tt * LROW + (n / NPL) * (NPL + 4) + n % NPL;
        qS[o] = rq[u];
        kS[o] = rk[u];
        if (CHANNEL) aS[o] = expf(-rate * softplus_exact(rz[u]));   // (padding channels: k = q = 0, the state stays 0)
      }
    }
    if (threadIdx.x < CH) {
      bS[threadIdx.x] = sigmoidf(rb);
      if (!CHANNEL) aS[threadIdx.x] = expf(-rate * softplus_exact(rd));
    }
  };
  fetch(s0);
  float S[NPL];
  const bool old = pr <= -2 && pin;
  const float* st = a.state + (old ? (long long)(-(pr + 2)) * a.state_stride + (long long)h * N * P + p : 0);
#pragma unroll
  for (int i = 0; i < NPL; ++i) S[i] = old && n0 + i < N ? st[(long long)(n0 + i) * P] : 0.f;
  int flip = 0;
  for (int t0 = s0; t0 < s1; t0 += CH, flip ^= 1) {
    const int nt = min(CH, s1 - t0);
    float* buf = lds + flip * BUF;
    commit(buf);
    float vr[CH], po[CH];
#pragma unroll
    for (int tt = 0; tt < CH; ++tt) vr[tt] = vn[tt];
    __syncthreads();   // this batch is in LDS; every thread has finished the batch before the last (same buffer)
    if (t0 + CH < s1) fetch(t0 + CH);
    const float* qS = buf;
    const float* kS = buf + CH * LROW;
    const float* aS = kS + CH * LROW;
    const float* bS = aS + ASZ;
#pragma unroll
    for (int tt = 0; tt < CH; ++tt) {
      po[tt] = 0.f;
      if (tt < nt) {
        const float4* q4 = reinterpret_cast<const float4*>(qS + tt * LROW + l0);
        const float4* k4 = reinterpret_cast<const float4*>(kS + tt * LROW + l0);
        const float4* a4 = reinterpret_cast<const float4*>(aS + tt * LROW + l0);
        const float at = CHANNEL ? 0.f : aS[tt];
        float d0 = 0.f, d1 = 0.f, d2 = 0.f, d3 = 0.f;
#pragma unroll
        for (int i = 0; i < NPL / 4; ++i) {
          const float4 kv = k4[i];
          float4 av;
          if (CHANNEL) av = a4[i];
          else av = make_float4(at, at, at, at);
          S[4 * i + 0] *= av.x, S[4 * i + 1] *= av.y, S[4 * i + 2] *= av.z, S[4 * i + 3] *= av.w;
          d0 += S[4 * i + 0] * kv.x, d1 += S[4 * i + 1] * kv.y, d2 += S[4 * i + 2] * kv.z, d3 += S[4 * i + 3] * kv.w;
        }
        const float u = bS[tt] * (vr[tt] - slice_sum<SLICES>((d0 + d1) + (d2 + d3)));
        float o0 = 0.f, o1 = 0.f, o2 = 0.f, o3 = 0.f;
#pragma unroll
        for (int i = 0; i < NPL / 4; ++i) {
          const float4 kv = k4[i], qv = q4[i];
          S[4 * i + 0] += kv.x * u, S[4 * i + 1] += kv.y * u, S[4 * i + 2] += kv.z * u, S[4 * i + 3] += kv.w * u;
          o0 += S[4 * i + 0] * qv.x, o1 += S[4 * i + 1] * qv.y, o2 += S[4 * i + 2] * qv.z, o3 += S[4 * i + 3] * qv.w;
        }
        po[tt] = (o0 + o1) + (o2 + o3);
      }
    }
#pragma unroll
    for (int tt = 0; tt < CH; ++tt) po[tt] = slice_sum<SLICES>(po[tt]);
    if (ns == 0 && pin)
#pragma unroll
      for (int tt = 0; tt < CH; ++tt)
        if (tt < nt) a.out[((long long)(t0 + tt) * a.H + h) * P + p] = po[tt];
  }
  if (sv >= 0 && pin) {
    float* so = a.state + (long long)sv * a.state_stride + (long long)h * N * P + p;
#pragma unroll
    for (int i = 0; i < NPL; ++i)
      if (n0 + i < N) so[(long long)(n0 + i) * P] = S[i];
  }
}

// ---- chunked form ------------------------------------------------------------------------------------------------
constexpr int C = 32;            // tokens per chunk
constexpr int LC = C + 4;        // LDS pitch of a [.][C] matrix
// scratch per (row, head): row of T [C] | row of Aqk [C] | G: N key channels, or one value in four
SYM_DEV int ws_cols(bool channel, int N) { return 2 * C + (channel ? N : 4); }

// grid (64-row tiles x 2 chunks, heads)
template <bool CHANNEL>
__global__ __launch_bounds__(NT) void delta_chunk_prep_kernel(DeltaRuleArgs a) {
  extern __shared__ float lds[];
  const int N = a.N, N4 = (N + 3) & ~3, ld = N4 + 4;
  const int h = blockIdx.y, tile = blockIdx.x >> 1, sub = blockIdx.x & 1;
  const int seq = a.tiles[2 * tile], off = a.tiles[2 * tile + 1];
  const int q0 = a.cu_q[seq], qlen = a.cu_q[seq + 1] - q0;
  if (off >= qlen) return;                     // padding tile
  const int nt = min(C, qlen - off - C * sub);
  if (nt <= 0) return;
  const long long r0 = q0 + off + C * sub;
  float* kS = lds;                             // [C][ld]
  float* qS = kS + C * ld;
  float* GS = qS + C * ld;                     // CHANNEL: [C][ld], else [C]
  float* LS = GS + (CHANNEL ? C * ld : C);     // [C][LC] beta_i Akk_ij below the diagonal
  float* TS = LS + C * LC;                     // [C][LC]
  float* bS = TS + C * LC;                     // [C]
  const long long gn = (long long)a.G * N;
  const float* q = a.q + (long long)(h / a.hpg) * N;
  const float* k = a.k + (long long)(h / a.hpg) * N;
  const float rate2 = expf(a.A_log[h]) * LOG2E;
  const int tid = threadIdx.x;
  for (int i = tid; i < C * N4; i += NT) {
    const int tt = i / N4, n = i - tt * N4;
    const bool in = tt < nt && n < N;
    const long long r = r0 + tt;
    kS[tt * ld + n] = in ? k[r * gn + n] : 0.f;
    qS[tt * ld + n] = in ? q[r * gn + n] : 0.f;
    if (CHANNEL)
      GS[tt * ld + n] = in ? -rate2 * softplus_exact(a.dz[r * a.ldd + (long long)h * N + n] + a.dt_bias[(long long)h * N + n])
                           : 0.f;
  }
  if (tid < C) {
    const bool in = tid < nt;
    bS[tid] = in ? sigmoidf(a.bz[(r0 + tid) * a.ldb + h]) : 0.f;
    if (!CHANNEL) {
      float g = in ? -rate2 * softplus_exact(a.dz[(r0 + tid) * a.ldd + h] + a.dt_bias[h]) : 0.f;
#pragma unroll
      for (int o = 1; o < C; o <<= 1) {        // running sum over the chunk's tokens
        const float up = __shfl_up(g, o, 64);
        if (tid >= o) g += up;
      }
      GS[tid] = g;
    }
  }
  __syncthreads();
  const int wc = ws_cols(CHANNEL, N);
  float* ws = a.ws + (r0 * a.H + h) * wc;      // row stride H * wc
  const long long wrow = (long long)a.H * wc;
  if (CHANNEL) {
    for (int n = tid; n < N; n += NT) {
      float g = 0.f;
#pragma unroll 8
      for (int tt = 0; tt < C; ++tt) {
        g += GS[tt * ld + n];
        GS[tt * ld + n] = g;
        if (tt < nt) ws[tt * wrow + 2 * C + n] = g;
      }
    }
    __syncthreads();
  } else if (tid < nt) {
    ws[tid * wrow + 2 * C] = GS[tid];
  }
  // scores of a 2 x 2 block of (i, j) per thread
  const int ib = tid >> 4, jb = tid & 15;
  float kk[2][2] = {{0.f, 0.f}, {0.f, 0.f}}, qk[2][2] = {{0.f, 0.f}, {0.f, 0.f}};
  if (jb <= ib) {
    for (int n = 0; n < N4; n += 4) {
      float4 ki[2], qi[2], kj[2], gi[2], gj[2];
#pragma unroll
      for (int e = 0; e < 2; ++e) {
        ki[e] = *reinterpret_cast<const float4*>(kS + (2 * ib + e) * ld + n);
        qi[e] = *reinterpret_cast<const float4*>(qS + (2 * ib + e) * ld + n);
        kj[e] = *reinterpret_cast<const float4*>(kS + (2 * jb + e) * ld + n);
        if (CHANNEL) {
          gi[e] = *reinterpret_cast<const float4*>(GS + (2 * ib + e) * ld + n);
          gj[e] = *reinterpret_cast<const float4*>(GS + (2 * jb + e) * ld + n);
        }
      }
#pragma unroll
      for (int e = 0; e < 2; ++e)
#pragma unroll
        for (int f = 0; f < 2; ++f) {
          float4 w = kj[f];
          if (CHANNEL) {   // (entries above the diagonal: exponent clamped, never used)
            w.x *= __builtin_amdgcn_exp2f(fminf(gi[e].x - gj[f].x, 0.f));
            w.y *= __builtin_amdgcn_exp2f(fminf(gi[e].y - gj[f].y, 0.f));
            w.z *= __builtin_amdgcn_exp2f(fminf(gi[e].z - gj[f].z, 0.f));
            w.w *= __builtin_amdgcn_exp2f(fminf(gi[e].w - gj[f].w, 0.f));
          }
          kk[e][f] += ki[e].x * w.x + ki[e].y * w.y + ki[e].z * w.z + ki[e].w * w.w;
          qk[e][f] += qi[e].x * w.x + qi[e].y * w.y + qi[e].z * w.z + qi[e].w * w.w;
        }
    }
  }
#pragma unroll
  for (int e = 0; e < 2; ++e)
#pragma unroll
    for (int f = 0; f < 2; ++f) {
      const int i = 2 * ib + e, j = 2 * jb + f;
      float w = 1.f;
      if (!CHANNEL) w = __builtin_amdgcn_exp2f(fminf(GS[i] - GS[j], 0.f));
      LS[i * LC + j] = j < i ? bS[i] * kk[e][f] * w : 0.f;
      if (i < nt) ws[i * wrow + C + j] = j <= i ? qk[e][f] * w : 0.f;
    }
  __syncthreads();
  // T = (I + L)^-1 diag(beta): thread c solves column c by forward substitution
  if (tid < C) {
    float t[C];
#pragma unroll
    for (int i = 0; i < C; ++i) {
      float s0 = i == tid ? bS[i] : 0.f, s1 = 0.f;
#pragma unroll
      for (int j = 0; j < i; ++j) {
        const float l = LS[i * LC + j];
        if (j & 1) s1 -= l * t[j];
        else s0 -= l * t[j];
      }
      t[i] = s0 + s1;
      TS[i * LC + tid] = t[i];
    }
  }
  __syncthreads();
  for (int i = tid; i < C * C; i += NT) {
    const int tt = i / C, c = i - tt * C;
    if (tt < nt) ws[tt * wrow + c] = TS[tt * LC + c];
  }
}

// v_mfma_f32_16x16x4_f32: lane l holds A[l % 16][l / 16], B[l / 16][l % 16], D[4 (l / 16) + r][l % 16] in register r
SYM_DEV f32x4 mfma4(float x, float y, f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(x, y, c, 0, 0, 0); }

// grid (P / 64, heads, runs); NN: 16-row tiles of the state (N <= 16 NN)
template <typename T, bool CHANNEL, int NN>
__global__ __launch_bounds__(NT) void delta_chunk_scan_kernel(DeltaRuleArgs a) {
  extern __shared__ float lds[];
  constexpr int NP = 16 * NN;                  // padded key channels
  constexpr int LD = NP + 4;
  constexpr int EPT = C * NP / NT;             // staged (token, channel) entries per thread
  const int N = a.N, P = a.P;
  const int h = blockIdx.y, run = blockIdx.z;
  const int s0 = a.cu_q[run], s1 = a.cu_q[run + 1];
  if (s1 <= s0) return;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int col = lane & 15, g = lane >> 4;
  const int p = blockIdx.x * 64 + wave * 16 + col;
  const bool pin = p < P;
  float* Kt = lds;                             // [C][LD]  k e^G
  float* Qt = Kt + C * LD;                     // [C][LD]  q e^G
  float* Kh = Qt + C * LD;                     // [NP][LC] k e^(G_C - G), channel-major
  float* Tm = Kh + NP * LC;                    // [C][LC]
  float* Aq = Tm + C * LC;                     // [C][LC]
  float* D = Aq + C * LC;                      // [NP]     G_C
  const long long gn = (long long)a.G * N;
  const float* q = a.q + (long long)(h / a.hpg) * N;
  const float* k = a.k + (long long)(h / a.hpg) * N;
  const T* v = reinterpret_cast<const T*>(a.v) + (long long)h * P + p;
  const int wc = ws_cols(CHANNEL, N);
  const float* wsh = a.ws + (long long)h * wc;
  const long long wrow = (long long)a.H * wc;
  const int pr = a.prev_row[s0];
  const int sv = a.save_slot[s1 - 1];
  float rk[EPT], rq[EPT], rg[EPT], rt[C * C / NT], ra[C * C / NT], vn[8];
  float rgl[CHANNEL ? (NP + NT - 1) / NT : 1];   // G of the chunk's last token
  auto fetch = [&](int t0) {
    const int nt = min(C, s1 - t0);
#pragma unroll
    for (int u = 0; u < EPT; ++u) {
      const int i = tid + NT * u;
      const int tt = i / NP, n = i % NP;
      const bool in = tt < nt && n < N;
      const long long r = t0 + tt;
      rk[u] = in ? k[r * gn + n] : 0.f;
      rq[u] = in ? q[r * gn + n] : 0.f;
      if (CHANNEL) rg[u] = in ? wsh[r * wrow + 2 * C + n] : 0.f;
      else rg[u] = tt < nt ? wsh[r * wrow + 2 * C] : 0.f;
    }
    const float* last = wsh + (long long)(t0 + nt - 1) * wrow + 2 * C;
    if (CHANNEL) {
#pragma unroll
      for (int u = 0; u < (NP + NT - 1) / NT; ++u) {
        const int n = tid + NT * u;
        rgl[u] = n < N ? last[n] : 0.f;
      }
    } else {
      rgl[0] = last[0];
    }
#pragma unroll
    for (int u = 0; u < C * C / NT; ++u) {
      const int i = tid + NT * u, tt = i / C, j = i % C;
      const bool in = tt < nt && j < nt;
      rt[u] = in ? wsh[(long long)(t0 + tt) * wrow + j] : 0.f;
      ra[u] = in ? wsh[(long long)(t0 + tt) * wrow + C + j] : 0.f;
    }
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      const int tt = 16 * (i >> 2) + 4 * g + (i & 3);
      vn[i] = tt < nt && pin ? (float)v[(long long)(t0 + tt) * a.H * P] : 0.f;
    }
  };
  f32x4 S[NN];
  const bool old = pr <= -2 && pin;
  const float* st = a.state + (old ? (long long)(-(pr + 2)) * a.state_stride + (long long)h * N * P + p : 0);
#pragma unroll
  for (int t = 0; t < NN; ++t)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int n = 16 * t + 4 * g + r;
      S[t][r] = old && n < N ? st[(long long)n * P] : 0.f;
    }
  fetch(s0);
  for (int t0 = s0; t0 < s1; t0 += C) {
    const int nt = min(C, s1 - t0);
    __syncthreads();   // everyone is done with the previous chunk
    // G of the last token first: the entries' exponents need it
    if (CHANNEL) {
#pragma unroll
      for (int u = 0; u < (NP + NT - 1) / NT; ++u)
        if (tid + NT * u < NP) D[tid + NT * u] = rgl[u];
      __syncthreads();
    }
#pragma unroll
    for (int u = 0; u < EPT; ++u) {
      const int i = tid + NT * u;
      const int tt = i / NP, n = i % NP;
      const float gl = CHANNEL ? D[n] : rgl[0];
      const float eg = __builtin_amdgcn_exp2f(rg[u]);
      Kt[tt * LD + n] = rk[u] * eg;
      Qt[tt * LD + n] = rq[u] * eg;
      Kh[n * LC + tt] = rk[u] * __builtin_amdgcn_exp2f(fminf(gl - rg[u], 0.f));   // (rows past the run's end: k = 0)
    }
#pragma unroll
    for (int u = 0; u < C * C / NT; ++u) {
      const int i = tid + NT * u, tt = i / C, j = i % C;
      Tm[tt * LC + j] = rt[u];
      Aq[tt * LC + j] = ra[u];
    }
    f32x4 V0 = {vn[0], vn[1], vn[2], vn[3]}, V1 = {vn[4], vn[5], vn[6], vn[7]};
    const float dh = CHANNEL ? 0.f : __builtin_amdgcn_exp2f(rgl[0]);
    __syncthreads();
    if (t0 + C < s1) fetch(t0 + C);
    f32x4 K0 = {0.f, 0.f, 0.f, 0.f}, K1 = K0, O0 = K0, O1 = K0;
#pragma unroll
    for (int t = 0; t < NN; ++t) {
      const f32x4 x0 = *reinterpret_cast<const f32x4*>(Kt + col * LD + 16 * t + 4 * g);
      const f32x4 x1 = *reinterpret_cast<const f32x4*>(Kt + (16 + col) * LD + 16 * t + 4 * g);
      const f32x4 y0 = *reinterpret_cast<const f32x4*>(Qt + col * LD + 16 * t + 4 * g);
      const f32x4 y1 = *reinterpret_cast<const f32x4*>(Qt + (16 + col) * LD + 16 * t + 4 * g);
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        K0 = mfma4(x0[r], S[t][r], K0);
        K1 = mfma4(x1[r], S[t][r], K1);
        O0 = mfma4(y0[r], S[t][r], O0);
        O1 = mfma4(y1[r], S[t][r], O1);
      }
    }
    const f32x4 R0 = V0 - K0, R1 = V1 - K1;
    f32x4 U0 = {0.f, 0.f, 0.f, 0.f}, U1 = U0;
    {
      const f32x4 x00 = *reinterpret_cast<const f32x4*>(Tm + col * LC + 4 * g);
      const f32x4 x10 = *reinterpret_cast<const f32x4*>(Tm + (16 + col) * LC + 4 * g);
      const f32x4 x11 = *reinterpret_cast<const f32x4*>(Tm + (16 + col) * LC + 16 + 4 * g);
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        U0 = mfma4(x00[r], R0[r], U0);
        U1 = mfma4(x10[r], R0[r], U1);
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) U1 = mfma4(x11[r], R1[r], U1);
    }
    {
      const f32x4 x00 = *reinterpret_cast<const f32x4*>(Aq + col * LC + 4 * g);
      const f32x4 x10 = *reinterpret_cast<const f32x4*>(Aq + (16 + col) * LC + 4 * g);
      const f32x4 x11 = *reinterpret_cast<const f32x4*>(Aq + (16 + col) * LC + 16 + 4 * g);
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        O0 = mfma4(x00[r], U0[r], O0);
        O1 = mfma4(x10[r], U0[r], O1);
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) O1 = mfma4(x11[r], U1[r], O1);
    }
#pragma unroll
    for (int t = 0; t < NN; ++t) {
      if (CHANNEL) {
        const f32x4 d = *reinterpret_cast<const f32x4*>(D + 16 * t + 4 * g);
#pragma unroll
        for (int r = 0; r < 4; ++r) S[t][r] *= __builtin_amdgcn_exp2f(d[r]);
      } else {
        S[t] = S[t] * dh;
      }
    }
#pragma unroll
    for (int t = 0; t < NN; ++t) {
      const f32x4 x0 = *reinterpret_cast<const f32x4*>(Kh + (16 * t + col) * LC + 4 * g);
      const f32x4 x1 = *reinterpret_cast<const f32x4*>(Kh + (16 * t + col) * LC + 16 + 4 * g);
#pragma unroll
      for (int r = 0; r < 4; ++r) S[t] = mfma4(x0[r], U0[r], S[t]);
#pragma unroll
      for (int r = 0; r < 4; ++r) S[t] = mfma4(x1[r], U1[r], S[t]);
    }
    if (pin) {
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int i0 = 4 * g + r, i1 = 16 + i0;
        if (i0 < nt) a.out[((long long)(t0 + i0) * a.H + h) * P + p] = O0[r];
        if (i1 < nt) a.out[((long long)(t0 + i1) * a.H + h) * P + p] = O1[r];
      }
    }
  }
  if (sv >= 0 && pin) {
    float* so = a.state + (long long)sv * a.state_stride + (long long)h * N * P + p;
#pragma unroll
    for (int t = 0; t < NN; ++t)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int n = 16 * t + 4 * g + r;
        if (n < N) so[(long long)n * P] = S[t][r];
      }
  }
}

void raise_lds(const void* f) { hipFuncSetAttribute(f, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024); }

template <typename T, bool CHANNEL, int NPL, int CH, int SLICES>
void launch_serial(const DeltaRuleArgs& a, hipStream_t s) {
  const int cols = (64 / SLICES) * (NT / 64);
  const int lrow = SLICES * (NPL + 4);
  const size_t lds = (size_t)2 * (2 * CH * lrow + (CHANNEL ? CH * lrow : CH) + CH) * sizeof(float);
  static bool raised = false;
  if (!raised && lds > 64 * 1024) raise_lds(reinterpret_cast<const void*>(&delta_scan_kernel<T, CHANNEL, NPL, CH, SLICES>));
  raised = true;
  delta_scan_kernel<T, CHANNEL, NPL, CH, SLICES><<<dim3((a.P + cols - 1) / cols, a.H, a.runs), NT, lds, s>>>(a);
}

template <typename T, bool CHANNEL>
void serial(const DeltaRuleArgs& a, hipStream_t s) {
  const int need = (a.N + 3) / 4;
  if (a.T == a.runs) {        // one token per run: the state's traffic is the launch
    if (need <= 4) launch_serial<T, CHANNEL, 4, 1, 4>(a, s);
    else if (need <= 8) launch_serial<T, CHANNEL, 8, 1, 4>(a, s);
    else if (need <= 16) launch_serial<T, CHANNEL, 16, 1, 4>(a, s);
    else if (need <= 32) launch_serial<T, CHANNEL, 32, 1, 4>(a, s);
    else launch_serial<T, CHANNEL, 64, 1, 4>(a, s);
    return;
  }
  if (need <= 4) launch_serial<T, CHANNEL, 4, 16, 4>(a, s);
  else if (need <= 8) launch_serial<T, CHANNEL, 8, 16, 4>(a, s);
  else if (need <= 16) launch_serial<T, CHANNEL, 8, 16, 8>(a, s);
  else if (need <= 32) launch_serial<T, CHANNEL, 16, 16, 8>(a, s);
  else launch_serial<T, CHANNEL, 32, 8, 8>(a, s);      // N <= 256 (checked by the op layer)
}

template <typename T, bool CHANNEL, int NN>
void launch_scan(const DeltaRuleArgs& a, hipStream_t s) {
  constexpr int NP = 16 * NN;
  const size_t lds = (size_t)(2 * C * (NP + 4) + NP * LC + 2 * C * LC + NP) * sizeof(float);
  static bool raised = false;
  if (!raised && lds > 64 * 1024) raise_lds(reinterpret_cast<const void*>(&delta_chunk_scan_kernel<T, CHANNEL, NN>));
  raised = true;
  delta_chunk_scan_kernel<T, CHANNEL, NN><<<dim3((a.P + 63) / 64, a.H, a.runs), NT, lds, s>>>(a);
}

template <typename T, bool CHANNEL>
void chunked(const DeltaRuleArgs& a, hipStream_t s) {
  const int ld = ((a.N + 3) & ~3) + 4;
  const size_t lds = (size_t)(2 * C * ld + (CHANNEL ? C * ld : C) + 2 * C * LC + C) * sizeof(float);
  static bool raised = false;
  if (!raised) raise_lds(reinterpret_cast<const void*>(&delta_chunk_prep_kernel<CHANNEL>));
  raised = true;
  delta_chunk_prep_kernel<CHANNEL><<<dim3(2 * a.ntiles, a.H), NT, lds, s>>>(a);
  const int nn = (a.N + 15) / 16;
  if (nn <= 1) launch_scan<T, CHANNEL, 1>(a, s);
  else if (nn <= 2) launch_scan<T, CHANNEL, 2>(a, s);
  else if (nn <= 4) launch_scan<T, CHANNEL, 4>(a, s);
  else if (nn <= 8) launch_scan<T, CHANNEL, 8>(a, s);
  else launch_scan<T, CHANNEL, 16>(a, s);
}

}  // namespace

int launch_delta_rule(const DeltaRuleArgs& a, int channel, int f32, int impl, hipStream_t s) {
  if (a.runs <= 0 || a.T <= 0) return 1;
  const bool chunk = impl == 0 && a.tiles && a.ntiles > 0 && a.ws && a.cu_q;
  if (f32) {
    if (chunk) channel ? chunked<float, true>(a, s) : chunked<float, false>(a, s);
    else channel ? serial<float, true>(a, s) : serial<float, false>(a, s);
  } else {
    if (chunk) channel ? chunked<bf16, true>(a, s) : chunked<bf16, false>(a, s);
    else channel ? serial<bf16, true>(a, s) : serial<bf16, false>(a, s);
  }
  return chunk ? 0 : 1;
}
