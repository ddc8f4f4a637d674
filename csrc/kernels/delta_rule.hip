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
//    delta_chunk_prep_kernel (one workgroup per chunk and head, all chunks at once) evaluates Akk, Aqk and T = (I +
//    diag(beta) Akk)^-1 diag(beta) by forward substitution.  One decay per head: the scores are matrix products, times
//    e^(G_i - G_j).  Decays per channel: inside the two diagonal 16 x 16 tiles the exponents of differences are taken per
//    (i, j, channel) on the vector unit; the tile below them factors at the end of the first half, e^(G_i - G_15) e^(G_15 -
//    G_j), both exponents <= 0, and is a matrix product again.
//    delta_chunk_scan_kernel (grid (P / 64, heads, runs)) then walks a run's chunks with
//        R = V - Kt S,   U = T R,   O = Qt S + Aqk U,   S <- D S + Kh^T U
//    as fp32 matrix products (v_mfma_f32_16x16x4_f32).  A wave owns 16 value columns and ALL of N: its state stays in
//    accumulator registers for the whole run, and since an accumulator's rows are 4 (lane / 16) + r and a B operand's
//    contraction index is lane / 16, register r of the state IS the B operand of a step that contracts over the rows
//    4 g + r (the A operand is read in the same order: one 16-byte LDS read feeds four steps).  The same holds for R and U.
//    Four waves multiply, four others stage the next chunk (loads, exponentials, LDS) on the same SIMDs meanwhile.
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

// v_mfma_f32_16x16x4_f32: lane l holds A[l % 16][l / 16], B[l / 16][l % 16], D[4 (l / 16) + r][l % 16] in register r
SYM_DEV f32x4 mfma4(float x, float y, f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(x, y, c, 0, 0, 0); }
SYM_DEV f32x4 lds4(const float* p) { return *reinterpret_cast<const f32x4*>(p); }
SYM_DEV f32x4 exp2_neg(f32x4 v) {       // 2^v for exponents that are <= 0 where they matter
  f32x4 r;
#pragma unroll
  for (int i = 0; i < 4; ++i) r[i] = __builtin_amdgcn_exp2f(fminf(v[i], 0.f));
  return r;
}

// grid (64-row tiles x 2 chunks, heads); NN: 16-channel tiles (N <= 16 NN)
template <bool CHANNEL, int NN>
__global__ __launch_bounds__(NT) void delta_chunk_prep_kernel(DeltaRuleArgs a) {
  extern __shared__ float lds[];
  constexpr int NP = 16 * NN, LD = NP + 4;
  constexpr int TSTEP = NT / NP, EPT = C / TSTEP;      // a thread stages channel n of the tokens tt0, tt0 + TSTEP, ..
  const int N = a.N;
  const int h = blockIdx.y, tile = blockIdx.x >> 1, sub = blockIdx.x & 1;
  const int seq = a.tiles[2 * tile], off = a.tiles[2 * tile + 1];
  const int q0 = a.cu_q[seq], qlen = a.cu_q[seq + 1] - q0;
  if (off >= qlen) return;                     // padding tile
  const int nt = min(C, qlen - off - C * sub);
  if (nt <= 0) return;
  const long long r0 = q0 + off + C * sub;
  float* kS = lds;                             // [C][LD]
  float* qS = kS + C * LD;                     // [C][LD]
  float* GS = qS + C * LD;                     // CHANNEL: [C][LD], else [C]
  float* XS = GS + (CHANNEL ? C * LD : C);     // [2 halves of the channels][Akk, Aqk][C][LC]
  float* bS = XS + 4 * C * LC;                 // [C]
  float* LS = XS;                              // afterwards: [C][LC] beta_i Akk_ij below the diagonal
  float* TS = XS + 2 * C * LC;                 // [C][LC]
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int n = tid % NP, tt0 = tid / NP;
  const int gn = a.G * N;
  const float rate2 = expf(a.A_log[h]) * LOG2E;
  {
    const float* k = a.k + (r0 + tt0) * gn + (h / a.hpg) * N + n;
    const float* q = a.q + (r0 + tt0) * gn + (h / a.hpg) * N + n;
    const float* dz = CHANNEL ? a.dz + (r0 + tt0) * a.ldd + h * N + n : nullptr;
    const float db = CHANNEL && n < N ? a.dt_bias[h * N + n] : 0.f;
    float rk[EPT], rq[EPT], rz[EPT];
#pragma unroll
    for (int u = 0; u < EPT; ++u) {
      const bool in = tt0 + TSTEP * u < nt && n < N;
      rk[u] = in ? k[(long long)TSTEP * u * gn] : 0.f;
      rq[u] = in ? q[(long long)TSTEP * u * gn] : 0.f;
      if (CHANNEL) rz[u] = in ? dz[TSTEP * u * a.ldd] : 0.f;
    }
#pragma unroll
    for (int u = 0; u < EPT; ++u) {
      const int o = (tt0 + TSTEP * u) * LD + n;
      kS[o] = rk[u];
      qS[o] = rq[u];
      if (CHANNEL) GS[o] = tt0 + TSTEP * u < nt && n < N ? -rate2 * softplus_exact(rz[u] + db) : 0.f;
    }
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
    if (tid < NP) {
      float g[C];
#pragma unroll
      for (int tt = 0; tt < C; ++tt) g[tt] = GS[tt * LD + tid];
#pragma unroll
      for (int tt = 1; tt < C; ++tt) g[tt] += g[tt - 1];
#pragma unroll
      for (int tt = 0; tt < C; ++tt) {
        GS[tt * LD + tid] = g[tt];
        if (tt < nt && tid < N) ws[tt * wrow + 2 * C + tid] = g[tt];
      }
    }
    __syncthreads();
  } else if (tid < nt) {
    ws[tid * wrow + 2 * C] = GS[tid];
  }
  // scores.  A wave takes one half of the channels (half) of Akk or Aqk (kind) for the matrix products
  constexpr int NH = NN > 1 ? NN / 2 : 1;      // 16-channel tiles per half
  const int half = wave >> 1, kind = wave & 1;
  const int col = lane & 15, g = lane >> 4;
  {
    const float* iS = kind ? qS : kS;
    f32x4 d00 = {0.f, 0.f, 0.f, 0.f}, d10 = d00, d11 = d00;
    if (NN > 1 || half == 0) {
#pragma unroll
      for (int t = 0; t < NH; ++t) {
        const int c = 16 * (half * NH + t) + 4 * g;
        f32x4 i1 = lds4(iS + (16 + col) * LD + c);
        f32x4 j0 = lds4(kS + col * LD + c);
        if (CHANNEL) {
          const f32x4 mid = lds4(GS + 15 * LD + c);
          i1 = i1 * exp2_neg(lds4(GS + (16 + col) * LD + c) - mid);
          j0 = j0 * exp2_neg(mid - lds4(GS + col * LD + c));
#pragma unroll
          for (int r = 0; r < 4; ++r) d10 = mfma4(i1[r], j0[r], d10);
        } else {
          const f32x4 i0 = lds4(iS + col * LD + c), j1 = lds4(kS + (16 + col) * LD + c);
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            d00 = mfma4(i0[r], j0[r], d00);
            d10 = mfma4(i1[r], j0[r], d10);
            d11 = mfma4(i1[r], j1[r], d11);
          }
        }
      }
    }
    float* X = XS + (half * 2 + kind) * C * LC;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      X[(16 + 4 * g + r) * LC + col] = d10[r];
      if (!CHANNEL) {
        X[(4 * g + r) * LC + col] = d00[r];
        X[(16 + 4 * g + r) * LC + 16 + col] = d11[r];
      }
    }
  }
  if (CHANNEL) {
    // diagonal tiles: wave (half, tile), a 2 x 2 block of (i, j) per lane, both kinds
    const int dt = wave & 1, ib = lane >> 3, jb = lane & 7;
    const int i0 = 16 * dt + 2 * ib, j0 = 16 * dt + 2 * jb;
    float kk[2][2] = {{0.f, 0.f}, {0.f, 0.f}}, qk[2][2] = {{0.f, 0.f}, {0.f, 0.f}};
    if (jb <= ib && (NN > 1 || half == 0)) {
#pragma unroll 2
      for (int c = 16 * NH * half; c < 16 * NH * (half + 1); c += 4) {
        f32x4 ki[2], qi[2], kj[2], gi[2], gj[2];
#pragma unroll
        for (int e = 0; e < 2; ++e) {
          ki[e] = lds4(kS + (i0 + e) * LD + c);
          qi[e] = lds4(qS + (i0 + e) * LD + c);
          gi[e] = lds4(GS + (i0 + e) * LD + c);
          kj[e] = lds4(kS + (j0 + e) * LD + c);
          gj[e] = lds4(GS + (j0 + e) * LD + c);
        }
#pragma unroll
        for (int e = 0; e < 2; ++e)
#pragma unroll
          for (int f = 0; f < 2; ++f) {
            const f32x4 w = kj[f] * exp2_neg(gi[e] - gj[f]);    // (above the diagonal: clamped, never used)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
              kk[e][f] += ki[e][r] * w[r];
              qk[e][f] += qi[e][r] * w[r];
            }
          }
      }
    }
    float* X = XS + half * 2 * C * LC;
#pragma unroll
    for (int e = 0; e < 2; ++e)
#pragma unroll
      for (int f = 0; f < 2; ++f) {
        X[(i0 + e) * LC + j0 + f] = kk[e][f];
        X[C * LC + (i0 + e) * LC + j0 + f] = qk[e][f];
      }
  }
  __syncthreads();
  // the halves meet; Akk goes on as beta_i Akk_ij (the threads hold their sums across a barrier: LS lies on XS)
  float lv[C * C / NT];
#pragma unroll
  for (int u = 0; u < C * C / NT; ++u) {
    const int i = (tid + NT * u) / C, j = (tid + NT * u) % C;
    const int o = i * LC + j;
    float w = 1.f;
    if (!CHANNEL) w = __builtin_amdgcn_exp2f(fminf(GS[i] - GS[j], 0.f));
    const bool stored = !(i < 16 && j >= 16);
    lv[u] = j < i ? bS[i] * w * (XS[o] + XS[2 * C * LC + o]) : 0.f;
    const float av = stored && j <= i ? w * (XS[C * LC + o] + XS[3 * C * LC + o]) : 0.f;
    if (i < nt) ws[i * wrow + C + j] = av;
  }
  __syncthreads();
#pragma unroll
  for (int u = 0; u < C * C / NT; ++u) LS[(tid + NT * u) / C * LC + (tid + NT * u) % C] = lv[u];
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
#pragma unroll
  for (int u = 0; u < C * C / NT; ++u) {
    const int i = (tid + NT * u) / C, c = (tid + NT * u) % C;
    if (i < nt) ws[i * wrow + c] = TS[i * LC + c];
  }
}

// grid (P / 64, heads, runs), 512 threads: waves 0 .. 3 multiply (16 value columns each), waves 4 .. 7 stage.  NN: 16-row
// tiles of the state (N <= 16 NN); NBUF: LDS stages (two where they fit)
template <typename T, bool CHANNEL, int NN, int NBUF>
__global__ __launch_bounds__(2 * NT) void delta_chunk_scan_kernel(DeltaRuleArgs a) {
  extern __shared__ float lds[];
  constexpr int NP = 16 * NN;                  // padded key channels
  constexpr int LD = NP + 4;
  constexpr int TSTEP = NT / NP, EPT = C / TSTEP;      // a staging thread owns channel n of the tokens tt0, tt0 + TSTEP, ..
  constexpr int oQ = C * LD, oH = 2 * C * LD, oT = oH + NP * LC, oA = oT + C * LC, oD = oA + C * LC, STAGE = oD + NP;
  const int N = a.N, P = a.P;
  const int h = blockIdx.y, run = blockIdx.z;
  const int s0 = a.cu_q[run], s1 = a.cu_q[run + 1];
  if (s1 <= s0) return;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int chunks = (s1 - s0 + C - 1) / C;
  const int wc = ws_cols(CHANNEL, N);
  const long long wrow = (long long)a.H * wc;
  if (wave >= 4) {
    // ---- staging waves -----------------------------------------------------------------------------------------
    const int tid = threadIdx.x - NT, n = tid % NP, tt0 = tid / NP;
    const bool nin = n < N;
    const int gn = a.G * N;
    const float* k = a.k + (long long)(s0 + tt0) * gn + (h / a.hpg) * N + n;
    const float* q = a.q + (long long)(s0 + tt0) * gn + (h / a.hpg) * N + n;
    const float* wsh = a.ws + (long long)s0 * wrow + (long long)h * wc;
    const float* G = wsh + tt0 * wrow + 2 * C + (CHANNEL ? n : 0);
    const int mj = tid % C, mt = tid / C;      // the [C][C] matrices: column mj of the rows mt, mt + NT / C, ..
    const float* M = wsh + mt * wrow + mj;
    constexpr int MSTEP = NT / C, MPT = C / MSTEP;
    // a chunk waits in registers until its stage is free; at sizes where that does not fit (one stage), it is loaded a few
    // rows at a time instead
    constexpr bool AHEAD = NBUF == 2;
    constexpr int EB = AHEAD ? EPT : 4;
    float rk[EB], rq[EB], rg[EB], gl, rt[MPT], ra[MPT];
    auto fetch = [&](int c, int u0) {
      const int t0 = c * C, nt = min(C, s1 - s0 - t0);
      const float* kc = k + (long long)t0 * gn;
      const float* qc = q + (long long)t0 * gn;
      const float* Gc = G + t0 * wrow;
#pragma unroll
      for (int e = 0; e < EB; ++e) {
        const int u = u0 + e;
        const bool row = tt0 + TSTEP * u < nt;
        rk[e] = row && nin ? kc[(long long)TSTEP * u * gn] : 0.f;
        rq[e] = row && nin ? qc[(long long)TSTEP * u * gn] : 0.f;
        rg[e] = row && (nin || !CHANNEL) ? Gc[TSTEP * u * wrow] : 0.f;
      }
      if (u0) return;
      gl = nin || !CHANNEL ? wsh[(long long)(t0 + nt - 1) * wrow + 2 * C + (CHANNEL ? n : 0)] : 0.f;
      const float* Mc = M + t0 * wrow;
#pragma unroll
      for (int u = 0; u < MPT; ++u) {
        const bool in = mt + MSTEP * u < nt && mj < nt;
        rt[u] = in ? Mc[MSTEP * u * wrow] : 0.f;
        ra[u] = in ? Mc[MSTEP * u * wrow + C] : 0.f;
      }
    };
    auto put = [&](float* st, int u0) {
#pragma unroll
      for (int e = 0; e < EB; ++e) {
        const int tt = tt0 + TSTEP * (u0 + e);
        const float eg = __builtin_amdgcn_exp2f(rg[e]);
        st[tt * LD + n] = rk[e] * eg;
        st[oQ + tt * LD + n] = rq[e] * eg;
        st[oH + n * LC + tt] = rk[e] * __builtin_amdgcn_exp2f(fminf(gl - rg[e], 0.f));   // (rows past the run's end: k = 0)
      }
    };
    auto stash = [&](float* st, int c) {
      if (AHEAD) {
        put(st, 0);
      } else {
#pragma unroll 1
        for (int u0 = 0; u0 < EPT; u0 += EB) {
          fetch(c, u0);
          put(st, u0);
        }
      }
      if (tt0 == 0) st[oD + n] = __builtin_amdgcn_exp2f(gl);
#pragma unroll
      for (int u = 0; u < MPT; ++u) {
        st[oT + (mt + MSTEP * u) * LC + mj] = rt[u];
        st[oA + (mt + MSTEP * u) * LC + mj] = ra[u];
      }
    };
    if (AHEAD) fetch(0, 0);
    stash(lds, 0);
    if (AHEAD && chunks > 1) fetch(1, 0);
    __syncthreads();                           // chunk 0 is staged
    for (int c = 0; c < chunks; ++c) {
      if (NBUF == 1) __syncthreads();          // chunk c has been read
      if (c + 1 < chunks) {
        stash(lds + (NBUF == 2 ? ((c + 1) & 1) * STAGE : 0), c + 1);
        if (AHEAD && c + 2 < chunks) fetch(c + 2, 0);
      }
      __syncthreads();                         // chunk c + 1 is staged (two stages: and chunk c has been read)
    }
    return;
  }
  // ---- multiplying waves -----------------------------------------------------------------------------------------
  const int col = lane & 15, g = lane >> 4;
  const int p = blockIdx.x * 64 + wave * 16 + col;
  const bool pin = p < P;
  const int pr = a.prev_row[s0];
  const int sv = a.save_slot[s1 - 1];
  const long long hp = (long long)a.H * P;
  const T* v = reinterpret_cast<const T*>(a.v) + (long long)s0 * hp + (long long)h * P + p;
  float* out = a.out + (long long)s0 * hp + (long long)h * P + p;
  float vn[8];
  auto fetch_v = [&](int c) {
    const int nt = min(C, s1 - s0 - c * C);
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      const int tt = 16 * (i >> 2) + 4 * g + (i & 3);
      vn[i] = tt < nt && pin ? (float)v[(long long)(c * C + tt) * hp] : 0.f;
    }
  };
  f32x4 S[NN];
  const bool old = pr <= -2 && pin;
  const float* st0 = a.state + (old ? (long long)(-(pr + 2)) * a.state_stride + (long long)h * N * P + p : 0);
#pragma unroll
  for (int t = 0; t < NN; ++t)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int n = 16 * t + 4 * g + r;
      S[t][r] = old && n < N ? st0[(long long)n * P] : 0.f;
    }
  fetch_v(0);
  __syncthreads();                             // chunk 0 is staged
  for (int c = 0; c < chunks; ++c) {
    const float* st = lds + (NBUF == 2 ? (c & 1) * STAGE : 0);
    const float* Kt = st + col * LD + 4 * g;
    const float* Qt = st + oQ + col * LD + 4 * g;
    const float* Kh = st + oH + col * LC + 4 * g;
    const float* Tm = st + oT + col * LC + 4 * g;
    const float* Aq = st + oA + col * LC + 4 * g;
    const float* D = st + oD + 4 * g;
    const f32x4 V0 = {vn[0], vn[1], vn[2], vn[3]}, V1 = {vn[4], vn[5], vn[6], vn[7]};
    if (c + 1 < chunks) fetch_v(c + 1);
    f32x4 K0 = {0.f, 0.f, 0.f, 0.f}, K1 = K0, O0 = K0, O1 = K0;
#pragma unroll
    for (int t = 0; t < NN; ++t) {
      const f32x4 x0 = lds4(Kt + 16 * t), x1 = lds4(Kt + 16 * LD + 16 * t);
      const f32x4 y0 = lds4(Qt + 16 * t), y1 = lds4(Qt + 16 * LD + 16 * t);
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
      const f32x4 x00 = lds4(Tm), x10 = lds4(Tm + 16 * LC), x11 = lds4(Tm + 16 * LC + 16);
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        U0 = mfma4(x00[r], R0[r], U0);
        U1 = mfma4(x10[r], R0[r], U1);
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) U1 = mfma4(x11[r], R1[r], U1);
    }
    {
      const f32x4 x00 = lds4(Aq), x10 = lds4(Aq + 16 * LC), x11 = lds4(Aq + 16 * LC + 16);
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        O0 = mfma4(x00[r], U0[r], O0);
        O1 = mfma4(x10[r], U0[r], O1);
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) O1 = mfma4(x11[r], U1[r], O1);
    }
#pragma unroll
    for (int t = 0; t < NN; ++t) S[t] = S[t] * lds4(D + 16 * t);
#pragma unroll
    for (int t = 0; t < NN; ++t) {
      const f32x4 x0 = lds4(Kh + 16 * t * LC), x1 = lds4(Kh + 16 * t * LC + 16);
#pragma unroll
      for (int r = 0; r < 4; ++r) S[t] = mfma4(x0[r], U0[r], S[t]);
#pragma unroll
      for (int r = 0; r < 4; ++r) S[t] = mfma4(x1[r], U1[r], S[t]);
    }
    if (pin) {
      const int nt = min(C, s1 - s0 - c * C);
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int i0 = 4 * g + r, i1 = 16 + i0;
        if (i0 < nt) out[(long long)(c * C + i0) * hp] = O0[r];
        if (i1 < nt) out[(long long)(c * C + i1) * hp] = O1[r];
      }
    }
    if (NBUF == 1) __syncthreads();            // chunk c has been read
    __syncthreads();                           // chunk c + 1 is staged (two stages: and chunk c has been read)
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
void launch_chunks(const DeltaRuleArgs& a, hipStream_t s) {
  constexpr int NP = 16 * NN, LD = NP + 4;
  constexpr int STAGE = 2 * C * LD + NP * LC + 2 * C * LC + NP;
  constexpr int NBUF = 2 * STAGE * (int)sizeof(float) <= 160 * 1024 ? 2 : 1;
  const size_t prep = (size_t)((CHANNEL ? 3 : 2) * C * LD + 4 * C * LC + 2 * C) * sizeof(float);
  const size_t scan = (size_t)NBUF * STAGE * sizeof(float);
  static bool raised = false;
  if (!raised) {
    raise_lds(reinterpret_cast<const void*>(&delta_chunk_prep_kernel<CHANNEL, NN>));
    raise_lds(reinterpret_cast<const void*>(&delta_chunk_scan_kernel<T, CHANNEL, NN, NBUF>));
    raised = true;
  }
  delta_chunk_prep_kernel<CHANNEL, NN><<<dim3(2 * a.ntiles, a.H), NT, prep, s>>>(a);
  delta_chunk_scan_kernel<T, CHANNEL, NN, NBUF><<<dim3((a.P + 63) / 64, a.H, a.runs), 2 * NT, scan, s>>>(a);
}

template <typename T, bool CHANNEL>
void chunked(const DeltaRuleArgs& a, hipStream_t s) {
  const int nn = (a.N + 15) / 16;
  if (nn <= 1) launch_chunks<T, CHANNEL, 1>(a, s);
  else if (nn <= 2) launch_chunks<T, CHANNEL, 2>(a, s);
  else if (nn <= 4) launch_chunks<T, CHANNEL, 4>(a, s);
  else if (nn <= 8) launch_chunks<T, CHANNEL, 8>(a, s);
  else launch_chunks<T, CHANNEL, 16>(a, s);
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
