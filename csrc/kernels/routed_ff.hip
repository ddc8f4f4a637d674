// Routed feed-forward with squared-ReLU (or plain) experts: router, expert segments, expert products.
//
//   route_topk      logits x . Wr[e] + bias in fp32, the k largest, weights = softmax over the chosen ones, and the places of
//                   the routed rows in expert order (segment bounds, token of every place, place of every choice)
//   expert_linear   y[place] = act(W[e] x[src[place]]) over the expert segments; rows are gathered where they are read, so no
//                   permuted copy of the activations exists, and the squared ReLU is the epilogue of the up product
//
// Router in bf16: 16 tokens x 16 experts per MFMA, the waves of a workgroup split the width and meet in LDS (the products of
// bf16 values and their sums are exact to fp32 accumulation).  A step of at most 16 tokens is one workgroup, which then also
// lays out the segments; larger steps take one more launch.
// Expert products in bf16: a weight-streaming kernel for few rows per expert (a wave per 16 weight rows and width slice, the
// rows of the segment as the other MFMA operand), and a 128 x 128 or 256 x 256 tile kernel staged through LDS by direct loads
// for prompt steps.  Other shapes and fp32: the all-shapes segment product of glu_moe.hip.
#include "common.h"
#include "direct_lds.h"
#include "hybrid_launchers.h"
#include "latent_launchers.h"
#include "wave_dot.h"

namespace {

constexpr int NT = 256;
constexpr int MAX_E = 1024;      // experts the segment layout handles
constexpr int PLAN_NT = 1024;

// ---- router --------------------------------------------------------------------------------------------------------------
// One wave: the k largest of z[0 .. E) (LDS), ties to the lowest index; ids / softmax weights of the chosen to global
SYM_DEV void choose(float* z, int E, int k, int lane, int* ids, float* w) {
  float zmax = 0.f, sum = 0.f;
  for (int j = 0; j < k; ++j) {
    float best = -INFINITY;
    int bi = 0x7fffffff;
    for (int e = lane; e < E; e += 64) {
      const float v = z[e];
      if (v > best) { best = v; bi = e; }
    }
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) {
      const float ob = __shfl_xor(best, o, 64);
      const int oi = __shfl_xor(bi, o, 64);
      if (ob > best || (ob == best && oi < bi)) { best = ob; bi = oi; }
    }
    if (bi >= E) bi = j;       // only with non-finite logits: keep the id a valid segment index for the kernels downstream
    if (j == 0) zmax = best;
    const float p = j == 0 ? 1.f : expf(best - zmax);
    sum += p;
    if (lane == 0) {
      ids[j] = bi;
      w[j] = p;
    }
    if ((bi & 63) == lane) z[bi] = -INFINITY;      // (the lane that scans this entry)
  }
  const float inv = 1.f / sum;
  if (lane == 0)
    for (int j = 0; j < k; ++j) w[j] *= inv;
}

// Segment layout by one workgroup of BT threads.  Items lo .. hi - 1 of the R choices get their places; the counts run over
// all of them (tot) and over those before lo (before), so workgroups that share the items out agree on every segment.
// LDS: 3 E ints.
template <int BT>
SYM_DEV void layout_segments(const int* __restrict__ ids, int R, int E, int k, int lo, int hi, int* lds,
                             int* __restrict__ offsets, int* __restrict__ dst, int* __restrict__ src) {
  int *tot = lds, *before = lds + E, *cur = lds + 2 * E;
  for (int e = threadIdx.x; e < E; e += BT) tot[e] = 0, before[e] = 0;
  __syncthreads();
  for (int a = threadIdx.x; a < R; a += BT) {
    const int e = ids[a];
    atomicAdd(&tot[e], 1);
    if (a < lo) atomicAdd(&before[e], 1);
  }
  __syncthreads();
  if (threadIdx.x < 64) {        // exclusive sums, 64 experts at a time
    const int lane = threadIdx.x;
    int carry = 0;
    for (int e0 = 0; e0 < E; e0 += 64) {
      const int e = e0 + lane;
      const int n = e < E ? tot[e] : 0;
      int s = n;
#pragma unroll
      for (int o = 1; o < 64; o <<= 1) {
        const int t = __shfl_up(s, o, 64);
        if (lane >= o) s += t;
      }
      if (e < E) {
        cur[e] = carry + s - n + before[e];
        if (lo == 0) offsets[e] = carry + s - n;
      }
      carry += __shfl(s, 63, 64);
    }
    if (lo == 0 && lane == 0) offsets[E] = carry;
  }
  __syncthreads();
  for (int a = lo + threadIdx.x; a < hi; a += BT) {
    const int pos = atomicAdd(&cur[ids[a]], 1);
    dst[a] = pos;
    src[pos] = a / k;
  }
}

__global__ __launch_bounds__(PLAN_NT) void expert_layout_kernel(const int* __restrict__ ids, int R, int E, int k,
                                                                int* __restrict__ offsets, int* __restrict__ dst,
                                                                int* __restrict__ src) {
  extern __shared__ int plds[];
  const int lo = blockIdx.x * 4 * PLAN_NT;
  layout_segments<PLAN_NT>(ids, R, E, k, lo, min(R, lo + 4 * PLAN_NT), plds, offsets, dst, src);
}

// grid ceil(T / 16), NW waves; NE expert tiles of 16 (E <= 16 NE), d % 32 == 0.  Dynamic LDS: NW NE 256 floats (partial
// logits) or, reused, 16 E floats + the layout's counters; PLAN: the single workgroup lays out the segments as well.
template <int NW, int NE, bool PLAN>
__global__ __launch_bounds__(64 * NW) void route_mfma_kernel(RouteArgs a) {
  extern __shared__ float part[];
  __shared__ int chosen[PLAN ? 1024 : 1];      // PLAN: the workgroup's choices (at most 16 tokens x 64)
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, j = lane & 15, hq = lane >> 4;
  const int t0 = 16 * blockIdx.x, d = a.d, E = a.E;
  const bf16* x = reinterpret_cast<const bf16*>(a.x) + (long long)min(t0 + j, a.T - 1) * d + 8 * hq;
  const bf16* w[NE];
  f32x4 acc[NE];
#pragma unroll
  for (int n = 0; n < NE; ++n) {
    w[n] = reinterpret_cast<const bf16*>(a.Wr) + (long long)min(16 * n + j, E - 1) * d + 8 * hq;
    acc[n] = f32x4{0.f, 0.f, 0.f, 0.f};
  }
#pragma unroll 4
  for (int c = 32 * wave; c < d; c += 32 * NW) {
    Pack8 xf;
    xf.u = *reinterpret_cast<const uint4*>(x + c);
#pragma unroll
    for (int n = 0; n < NE; ++n) {
      Pack8 wf;
      wf.u = *reinterpret_cast<const uint4*>(w[n] + c);
      acc[n] = mfma16(wf.v, xf.v, acc[n]);      // lane: token j, experts 16 n + 4 hq + 0..3
    }
  }
#pragma unroll
  for (int n = 0; n < NE; ++n)
    *reinterpret_cast<f32x4*>(part + (((wave * NE + n) * 16 + j) * 16 + 4 * hq)) = acc[n];
  __syncthreads();
  // the waves' partial logits of (token, expert) meet in the first slab: [NE][16 tokens][16 experts]
  for (int i = threadIdx.x; i < NE * 256; i += 64 * NW) {
    float s = part[i];
    for (int v = 1; v < NW; ++v) s += part[v * NE * 256 + i];
    const int e = 16 * (i >> 8) + (i & 15);
    part[i] = e < E ? s + (a.bias ? a.bias[e] : 0.f) : -INFINITY;
  }
  __syncthreads();
  for (int t = wave; t < 16; t += NW) {
    if (t0 + t >= a.T) break;
    float z = lane < 16 * NE ? part[((lane >> 4) * 16 + t) * 16 + (lane & 15)] : -INFINITY;   // (E <= 64: one per lane)
    float zmax = 0.f, sum = 0.f, mine = 0.f;
    int my = 0;
    for (int q = 0; q < a.k; ++q) {
      float best = z;
      int bi = lane;
#pragma unroll
      for (int o = 32; o > 0; o >>= 1) {
        const float ob = __shfl_xor(best, o, 64);
        const int oi = __shfl_xor(bi, o, 64);
        if (ob > best || (ob == best && oi < bi)) { best = ob; bi = oi; }
      }
      if (!(best > -INFINITY) || bi >= E) bi = q;   // only with non-finite logits: a valid segment index
      if (q == 0) zmax = best;
      const float p = q == 0 ? 1.f : expf(best - zmax);
      sum += p;
      if (lane == q) my = bi, mine = p;
      if (lane == bi) z = -INFINITY;
    }
    if (lane < a.k) {
      const long long o = (long long)(t0 + t) * a.k + lane;
      a.ids[o] = my;
      a.w[o] = mine / sum;
      if constexpr (PLAN) chosen[t * a.k + lane] = my;
    }
  }
  if constexpr (PLAN) {
    __syncthreads();      // (the partial logits are done with)
    layout_segments<64 * NW>(chosen, a.T * a.k, E, a.k, 0, a.T * a.k, reinterpret_cast<int*>(part), a.offsets, a.dst, a.src);
  }
}

// any width, both dtypes, E <= MAX_E: a workgroup per token, a wave per expert in turn
template <typename T>
__global__ __launch_bounds__(NT) void route_rows_kernel(RouteArgs a) {
  extern __shared__ float z[];
  const int t = blockIdx.x, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const T* x = reinterpret_cast<const T*>(a.x) + (long long)t * a.d;
  for (int e = wave; e < a.E; e += NT / 64) {
    const float s = wave_dot<T>(x, reinterpret_cast<const T*>(a.Wr) + (long long)e * a.d, a.d, lane);
    if (lane == 0) z[e] = s + (a.bias ? a.bias[e] : 0.f);
  }
  __syncthreads();
  if (wave == 0) choose(z, a.E, a.k, lane, a.ids + (long long)t * a.k, a.w + (long long)t * a.k);
}

// ---- expert products -----------------------------------------------------------------------------------------------------
SYM_DEV float relu2f(float v) {
  v = fmaxf(v, 0.f);
  return v * v;
}

// Few rows per expert: grid (ceil(N / 16), E), NW waves.  A workgroup owns 16 weight rows of one expert; its waves take the
// width's 64-element steps in turn (weights streamed once, straight into registers), multiply them with up to 16 MT rows of
// the segment per pass, and their sums meet in LDS.  K % 32 == 0.
template <int MT, int NW>
__global__ __launch_bounds__(64 * NW) void expert_stream_kernel(ExpertArgs a) {
  __shared__ float part[NW][MT * 256];
  const int e = blockIdx.y, n0 = 16 * blockIdx.x;
  const int s0 = a.offsets[e], s1 = min(a.offsets[e + 1], a.R);
  if (s0 >= s1) return;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, j = lane & 15, hq = lane >> 4;
  const int K = a.K, N = a.N;
  const bf16* w = reinterpret_cast<const bf16*>(a.W) + ((long long)e * N + min(n0 + j, N - 1)) * K + 8 * hq;
  for (int r0 = s0; r0 < s1; r0 += 16 * MT) {
    const bf16* x[MT];
    f32x4 acc[MT];
#pragma unroll
    for (int m = 0; m < MT; ++m) {
      const int r = min(r0 + 16 * m + j, s1 - 1);
      x[m] = reinterpret_cast<const bf16*>(a.x) + (long long)(a.src ? a.src[r] : r) * K + 8 * hq;
      acc[m] = f32x4{0.f, 0.f, 0.f, 0.f};
    }
    // 64 elements of every weight row per step: whole 128-byte lines
    constexpr int U = MT == 1 ? 4 : 2;
    int c = 64 * wave;
    for (; c + 64 * NW * (U - 1) + 64 <= K; c += 64 * NW * U) {
      Pack8 wf[U][2];
#pragma unroll
      for (int u = 0; u < U; ++u)
#pragma unroll
        for (int v = 0; v < 2; ++v) wf[u][v].w = ld_nt16(w + c + 64 * NW * u + 32 * v);
#pragma unroll
      for (int u = 0; u < U; ++u)
#pragma unroll
        for (int v = 0; v < 2; ++v)
#pragma unroll
          for (int m = 0; m < MT; ++m) {
            Pack8 xf;
            xf.u = *reinterpret_cast<const uint4*>(x[m] + c + 64 * NW * u + 32 * v);
            acc[m] = mfma16(wf[u][v].v, xf.v, acc[m]);     // lane: row j, outputs n0 + 4 hq + 0..3
          }
    }
    for (; c < K; c += 64 * NW)
#pragma unroll
      for (int v = 0; v < 2; ++v) {
        if (c + 32 * v >= K) break;
        Pack8 wf;
        wf.w = ld_nt16(w + c + 32 * v);
#pragma unroll
        for (int m = 0; m < MT; ++m) {
          Pack8 xf;
          xf.u = *reinterpret_cast<const uint4*>(x[m] + c + 32 * v);
          acc[m] = mfma16(wf.v, xf.v, acc[m]);
        }
      }
#pragma unroll
    for (int m = 0; m < MT; ++m) *reinterpret_cast<f32x4*>(&part[wave][m * 256 + j * 16 + 4 * hq]) = acc[m];
    __syncthreads();
    for (int i = threadIdx.x; i < MT * 256; i += 64 * NW) {
      float s = part[0][i];
#pragma unroll
      for (int v = 1; v < NW; ++v) s += part[v][i];
      const int r = r0 + (i >> 4), n = n0 + (i & 15);
      if (r < s1 && n < N) reinterpret_cast<bf16*>(a.y)[(long long)r * N + n] = (bf16)(a.relu2 ? relu2f(s) : s);
    }
    __syncthreads();
  }
}

// Prompt steps: BM x BN output tiles, waves in WR rows x WC columns, K in steps of 64 through two LDS stages filled by direct
// global -> LDS loads.  LDS rows are 128 B with the 16-byte chunk c stored at c ^ ((row >> 1) & 7) (swizzled on the load's
// source), so fragment reads do not conflict.  The tile list is walked on the device: a slot past the last tile exits before
// any barrier.  K % 64 == 0.
SYM_DEV int chunk_swz(int row) { return (row >> 1) & 7; }

template <int BM, int BN, int WR, int WC>
__global__ __launch_bounds__(64 * WR * WC) void expert_tile_kernel(ExpertArgs a) {
  constexpr int NWV = WR * WC, MS = BM / WR / 16, NS = BN / WC / 16;   // 16-row subtiles of a wave
  constexpr int AB = BM * 128, BB = BN * 128, STAGE = AB + BB;         // bytes of a stage
  constexpr int AL = BM / 8 / NWV, BL = BN / 8 / NWV;                  // direct loads (8 rows each) per wave and stage
  extern __shared__ __attribute__((aligned(16))) char smem[];
  int e = -1, r0 = 0, rows = 0;
  {
    int slot = blockIdx.y;
    for (int i = 0; i < a.E; ++i) {
      const int s0 = a.offsets[i], s1 = min(a.offsets[i + 1], a.R);
      const int t = (max(0, s1 - s0) + BM - 1) / BM;
      if (slot < t) {
        e = i;
        r0 = s0 + slot * BM;
        rows = min(BM, s1 - r0);
        break;
      }
      slot -= t;
    }
  }
  if (e < 0) return;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, wr = wave / WC, wc = wave % WC;
  const int n0 = BN * blockIdx.x, K = a.K, N = a.N;
  const bf16* asrc[AL];
  const bf16* bsrc[BL];
#pragma unroll
  for (int i = 0; i < AL; ++i) {
    const int row = 8 * (NWV * i + wave) + (lane >> 3), ch = (lane & 7) ^ chunk_swz(row);
    const int p = r0 + min(row, rows - 1);          // rows past the segment re-read its last one (never stored)
    asrc[i] = reinterpret_cast<const bf16*>(a.x) + (long long)(a.src ? a.src[p] : p) * K + 8 * ch;
  }
#pragma unroll
  for (int i = 0; i < BL; ++i) {
    const int row = 8 * (NWV * i + wave) + (lane >> 3), ch = (lane & 7) ^ chunk_swz(row);
    bsrc[i] = reinterpret_cast<const bf16*>(a.W) + ((long long)e * N + min(n0 + row, N - 1)) * K + 8 * ch;
  }
  const unsigned int lds0 = lds_address(smem) + __builtin_amdgcn_readfirstlane(wave) * 1024;
  auto stage = [&](int kt, int buf) {
    const unsigned int base = lds0 + buf * STAGE;
#pragma unroll
    for (int i = 0; i < AL; ++i) direct_load16(asrc[i] + kt * 64, base + NWV * i * 1024);
#pragma unroll
    for (int i = 0; i < BL; ++i) direct_load16(bsrc[i] + kt * 64, base + AB + NWV * i * 1024);
  };
  f32x4 acc[NS][MS];
#pragma unroll
  for (int i = 0; i < NS; ++i)
#pragma unroll
    for (int q = 0; q < MS; ++q) acc[i][q] = f32x4{0.f, 0.f, 0.f, 0.f};
  const int j = lane & 15, hq = lane >> 4;
  const int nk = K / 64;
  stage(0, 0);
  for (int kt = 0; kt < nk; ++kt) {
    wait_direct_loads();
    __syncthreads();      // stage kt has landed for every wave, and every wave is done reading the other stage
    if (kt + 1 < nk) stage(kt + 1, (kt + 1) & 1);
    const char* A = smem + (kt & 1) * STAGE;
    const char* B = A + AB;
#pragma unroll
    for (int ks = 0; ks < 2; ++ks) {
      const int c = 4 * ks + hq;
      Pack8 bf[NS], af[MS];
#pragma unroll
      for (int i = 0; i < NS; ++i) {
        const int row = (BN / WC) * wc + 16 * i + j;
        bf[i].u = *reinterpret_cast<const uint4*>(B + row * 128 + 16 * (c ^ chunk_swz(row)));
      }
#pragma unroll
      for (int q = 0; q < MS; ++q) {
        const int row = (BM / WR) * wr + 16 * q + j;
        af[q].u = *reinterpret_cast<const uint4*>(A + row * 128 + 16 * (c ^ chunk_swz(row)));
      }
#pragma unroll
      for (int i = 0; i < NS; ++i)
#pragma unroll
        for (int q = 0; q < MS; ++q) acc[i][q] = mfma16(bf[i].v, af[q].v, acc[i][q]);
    }
  }
  // lane (j, hq): output row 16 q + j of the wave's rows, columns 16 i + 4 hq + 0..3 of its columns
  bf16* y = reinterpret_cast<bf16*>(a.y);
  const bool vec = (N & 3) == 0;
#pragma unroll
  for (int q = 0; q < MS; ++q) {
    const int m = (BM / WR) * wr + 16 * q + j;
    if (m >= rows) continue;
#pragma unroll
    for (int i = 0; i < NS; ++i) {
      const int n = n0 + (BN / WC) * wc + 16 * i + 4 * hq;
      bf16* o = y + (long long)(r0 + m) * N + n;
      bf16x4 v;
#pragma unroll
      for (int u = 0; u < 4; ++u) v[u] = (bf16)(a.relu2 ? relu2f(acc[i][q][u]) : acc[i][q][u]);
      if (vec) {
        if (n < N) *reinterpret_cast<bf16x4*>(o) = v;
      } else {
#pragma unroll
        for (int u = 0; u < 4; ++u)
          if (n + u < N) o[u] = v[u];
      }
    }
  }
}

template <int BM, int BN, int WR, int WC>
void launch_tile(const ExpertArgs& a, hipStream_t s) {
  constexpr int lds = 2 * (BM + BN) * 128;
  static bool once = false;
  if (lds > 64 * 1024 && !once) {
    hipFuncSetAttribute(reinterpret_cast<const void*>(&expert_tile_kernel<BM, BN, WR, WC>),
                        hipFuncAttributeMaxDynamicSharedMemorySize, lds);
    once = true;
  }
  dim3 grid((a.N + BN - 1) / BN, (a.R + BM - 1) / BM + a.E);
  expert_tile_kernel<BM, BN, WR, WC><<<grid, 64 * WR * WC, lds, s>>>(a);
}

template <int NW, int NE>
void launch_route(const RouteArgs& a, hipStream_t s) {
  const int tiles = (a.T + 15) / 16;
  const size_t lds = (size_t)NW * NE * 256 * sizeof(float);
  if (tiles == 1) route_mfma_kernel<NW, NE, true><<<1, 64 * NW, lds, s>>>(a);
  else route_mfma_kernel<NW, NE, false><<<tiles, 64 * NW, lds, s>>>(a);
}

template <int NE>
void launch_route_ne(const RouteArgs& a, hipStream_t s) {
  if (a.T <= 512 && NE <= 4) launch_route<16 / (NE > 2 ? 2 : 1), NE>(a, s);   // decode-sized: the width over more waves
  else launch_route<4, NE>(a, s);
}

bool aligned16(const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; }

}  // namespace

void launch_route_topk(const RouteArgs& a, int f32, hipStream_t s) {
  if (a.T <= 0) return;
  const bool mfma = !f32 && a.d % 32 == 0 && a.E <= 64 && a.k <= 64 && aligned16(a.x) && aligned16(a.Wr);
  if (mfma) {
    if (a.E <= 16) launch_route_ne<1>(a, s);
    else if (a.E <= 32) launch_route_ne<2>(a, s);
    else launch_route_ne<4>(a, s);
    if (a.T <= 16) return;      // the single workgroup laid out the segments
  } else {
    const size_t lds = (size_t)a.E * sizeof(float);
    if (f32) route_rows_kernel<float><<<a.T, NT, lds, s>>>(a);
    else route_rows_kernel<bf16><<<a.T, NT, lds, s>>>(a);
  }
  const int R = a.T * a.k;
  expert_layout_kernel<<<(R + 4 * PLAN_NT - 1) / (4 * PLAN_NT), PLAN_NT, 3 * a.E * sizeof(int), s>>>(a.ids, R, a.E, a.k,
                                                                                                   a.offsets, a.dst, a.src);
}

// Returns the form used: 0 all shapes, 1 weight stream, 2 / 3 tiles of 128 / 256
int launch_expert_linear(const ExpertArgs& a, int f32, int impl, hipStream_t s) {
  if (a.R <= 0) return 0;
  const bool mfma = !f32 && aligned16(a.x) && aligned16(a.W) && aligned16(a.y);
  const int per = (a.R + a.E - 1) / a.E;      // rows per expert if they are spread evenly
  const bool stream = mfma && a.K % 32 == 0 && a.E <= 65535, tile = mfma && a.K % 64 == 0;
  if (impl < 0) impl = stream && (per <= 8 || !tile) ? 1 : (tile ? (per >= 512 && a.N >= 256 ? 3 : 2) : (stream ? 1 : 0));
  if (impl == 1 && stream) {
    dim3 grid((a.N + 15) / 16, a.E);
    if (per <= 8) expert_stream_kernel<1, 8><<<grid, 512, 0, s>>>(a);      // (8 waves: 31 us, 4 waves: 33 us at 16 x 2304 x 2048)
    else if (per <= 24) expert_stream_kernel<2, 4><<<grid, 256, 0, s>>>(a);
    else expert_stream_kernel<4, 4><<<grid, 256, 0, s>>>(a);
    return 1;
  }
  if (impl == 2 && tile) {
    launch_tile<128, 128, 2, 2>(a, s);
    return 2;
  }
  if (impl == 3 && tile) {
    launch_tile<256, 256, 2, 4>(a, s);
    return 3;
  }
  launch_grouped_linear(a.x, a.W, a.offsets, a.E, a.R, a.N, a.K, a.y, f32, s, a.src, a.relu2);
  return 0;
}
