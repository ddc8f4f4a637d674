// Causal softmax attention for single rows (decode steps, bf16): one workgroup per (row, key / value head, range of keys), the
// query heads of the group together, so a cached row is read once.  Same arguments as window_attention.hip's kernels for a
// window that never ends; optional sink, soft cap, per-key score factor and output gate (per head or per column).
//
// Four waves, 32 keys per wave and step.  A step's key and value rows go to the wave's own LDS by direct loads (KEYV: the
// values are the keys, one set of rows serves both products); the workgroups that share a CU cover each other's loads (a second
// stage per wave halves their number and measured slower: 64 rows x 1060 keys 60 us against 40 us).  Scores are S^T = K Q^T on
// v_mfma_f32_16x16x32_bf16 (16 query heads as columns), the weights go back as they lie into O^T = V^T P^T with transposed value
// fragments from the row-major rows (LDS transpose read).  Waves meet in LDS, ranges through write-through partial results and
// an arrival counter per (row, group): the workgroup that arrives last sums them in order, writes the output and sets the
// counter back to zero (nobody waits).  Softmax statistics and partial sums are fp32.
#include "attn_tiles.h"
#include "hybrid_launchers.h"

namespace {

constexpr int NW = 4, STEP = 32, MAX_REP = 16, MAX_PARTS = 64;

SYM_DEV void wait_loads() { asm volatile("s_waitcnt vmcnt(0) lgkmcnt(0)" ::: "memory"); }   // rows landed, LDS reads done

SYM_DEV void publish(float* p, float a, float b) {
  const unsigned long long v = (unsigned long long)__float_as_uint(a) | ((unsigned long long)__float_as_uint(b) << 32);
  __hip_atomic_store(reinterpret_cast<unsigned long long*>(p), v, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
}
SYM_DEV float2 collect(const float* p) {
  const unsigned long long v = __hip_atomic_load(reinterpret_cast<const unsigned long long*>(p), __ATOMIC_RELAXED,
                                                 __HIP_MEMORY_SCOPE_AGENT);
  return make_float2(__uint_as_float((unsigned int)v), __uint_as_float((unsigned int)(v >> 32)));
}

template <int D, bool KEYV, bool ONE>
__global__ __launch_bounds__(64 * NW) void split_attn_kernel(WindowAttnArgs a) {
  constexpr int CH = row_chunks(D), KD = (D + 31) / 32, VT = D / 16, ROWS = STEP * CH * 16;   // bytes of a step's rows
  constexpr int NL = STEP * CH / 64;                   // direct loads of a step's keys (and as many of its values)
  constexpr int STAGE = (KEYV ? 1 : 2) * ROWS + 256, LDO = D + 4;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  const int part = blockIdx.x, g = blockIdx.y, row = blockIdx.z;
  const int ctx = a.positions[row] + 1, lo = part * a.part_keys;
  if (lo >= ctx) return;
  const int hi_key = min(ctx, lo + a.part_keys), nparts = (ctx + a.part_keys - 1) / a.part_keys;
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int j = lane & 15, hq = lane >> 4, rep = a.H / a.G;
  const int* bt = a.block_tables + (long long)a.row_seq[row] * a.max_blocks;
  const bf16* kc = reinterpret_cast<const bf16*>(a.k_cache) + g * D;
  const bf16* vc = reinterpret_cast<const bf16*>(a.v_cache) + g * D;
  const long long ld = (long long)a.G * D;
  const unsigned int lds0 = lds_address(smem) + wave * STAGE;
  const bool scaled = a.key_scale != nullptr;

  auto stage = [&](int k0) {
    const int blk = ONE ? bt[k0 >> a.bs_shift] : 0;
    auto row_of = [&](int kp) {
      kp = min(kp, ctx - 1);
      return ONE ? ((long long)blk << a.bs_shift) + (kp & (a.BS - 1)) : cache_row(bt, kp, a.BS, a.bs_shift);
    };
    if (scaled) direct_load4(a.key_scale + row_of(k0 + (lane & 31)), lds0 + STAGE - 256);
    long long src[NL];
#pragma unroll
    for (int i = 0; i < NL; ++i) {
      const int r = (64 / CH) * i + lane / CH;
      int c = (lane & (CH - 1)) ^ swz<CH>(r);
      if (D < 8 * CH && c >= D / 8) c = 0;             // (places past the head's end are never used)
      src[i] = row_of(k0 + r) * ld + 8 * c;
    }
#pragma unroll
    for (int i = 0; i < NL; ++i) direct_load16(kc + src[i], lds0 + i * 1024);
    if constexpr (!KEYV)
#pragma unroll
      for (int i = 0; i < NL; ++i) direct_load16(vc + src[i], lds0 + ROWS + i * 1024);
  };

  const int k_first = lo + STEP * wave;
  if (k_first < hi_key) stage(k_first);
  bf16x8 qf[KD];       // column j: query head g rep + j
#pragma unroll
  for (int kk = 0; kk < KD; ++kk) {
    Pack8 t;
    t.u = make_uint4(0, 0, 0, 0);
    if (j < rep && 32 * kk + 8 * hq < D)
      t.u = *reinterpret_cast<const uint4*>(reinterpret_cast<const bf16*>(a.q) + ((long long)row * a.H + g * rep + j) * D +
                                            32 * kk + 8 * hq);
    qf[kk] = t.v;
  }
  f32x4 o[VT];
#pragma unroll
  for (int t = 0; t < VT; ++t) o[t] = f32x4{0.f, 0.f, 0.f, 0.f};
  float m = -INFINITY, l = 0.f;
  const float sl2 = a.scale * ATT_LOG2E, cap2 = a.softcap * ATT_LOG2E;
  const float c1 = a.softcap > 0.f ? 2.f * sl2 / a.softcap : 0.f;
  const char* S = smem + wave * STAGE;
  for (int k0 = k_first; k0 < hi_key; k0 += STEP * NW) {
    wait_loads();
    float p[2][4];
#pragma unroll
    for (int s = 0; s < 2; ++s) {
      f32x4 acc = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int kk = 0; kk < KD; ++kk) {
        const int r = 16 * s + j;
        Pack8 kf;
        kf.u = *reinterpret_cast<const uint4*>(S + r * CH * 16 + 16 * ((4 * kk + hq) ^ swz<CH>(r)));
        acc = mfma16(kf.v, qf[kk], acc);
      }
      // keys k0 + 16 s + 4 hq + i of head j
      float4 ks = make_float4(1.f, 1.f, 1.f, 1.f);
      if (scaled) ks = *reinterpret_cast<const float4*>(S + STAGE - 256 + 4 * (16 * s + 4 * hq));
      p[s][0] = acc[0] * ks.x, p[s][1] = acc[1] * ks.y, p[s][2] = acc[2] * ks.z, p[s][3] = acc[3] * ks.w;
    }
    float mx = -INFINITY;
#pragma unroll
    for (int s = 0; s < 2; ++s)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        float v = p[s][i];
        if (a.softcap > 0.f) v = cap2 - 2.f * cap2 * __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(c1 * v));
        else v *= sl2;
        p[s][i] = k0 + 16 * s + 4 * hq + i < hi_key ? v : -INFINITY;
        mx = fmaxf(mx, p[s][i]);
      }
    mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
    mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
    const float mt = fmaxf(m, mx);                     // (the step's first key is in range: finite)
    const float corr = __builtin_amdgcn_exp2f(m - mt);
    l *= corr;
#pragma unroll
    for (int t = 0; t < VT; ++t) o[t] *= corr;
    m = mt;
    Pack8 pf;
#pragma unroll
    for (int s = 0; s < 2; ++s)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const float w = __builtin_amdgcn_exp2f(p[s][i] - mt);
        l += w;
        pf.h[4 * s + i] = (bf16)w;
      }
#pragma unroll
    for (int t = 0; t < VT; ++t) {
      uint2 x[2];
#pragma unroll
      for (int s = 0; s < 2; ++s) {
        const int r = 16 * s + 4 * hq + (j >> 2), c = 2 * t + ((j & 3) >> 1);
        x[s] = read_tr(S + (KEYV ? 0 : ROWS) + r * CH * 16 + 16 * (c ^ swz<CH>(r)) + 8 * (j & 1));
      }
      Pack8 vf;
      vf.u = make_uint4(x[0].x, x[0].y, x[1].x, x[1].y);
      o[t] = mfma16(vf.v, pf.v, o[t]);                 // head j, columns 16 t + 4 hq + 0..3
    }
    if (k0 + STEP * NW < hi_key) {
      asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");     // (this step's rows have been read)
      stage(k0 + STEP * NW);
    }
  }
  l += __shfl_xor(l, 16, 64);
  l += __shfl_xor(l, 32, 64);

  // the waves meet: [NW][rep][LDO] sums, [NW][rep][2] statistics
  __syncthreads();
  float* so = reinterpret_cast<float*>(smem);
  float* sm = so + NW * rep * LDO;
  if (j < rep) {
#pragma unroll
    for (int t = 0; t < VT; ++t)
      *reinterpret_cast<f32x4*>(so + (wave * rep + j) * LDO + 16 * t + 4 * hq) = o[t];
    if (hq == 0) sm[2 * (wave * rep + j)] = m, sm[2 * (wave * rep + j) + 1] = l;
  }
  __syncthreads();
  const int items = rep * (D / 4);
  auto finish = [&](int r, int c, float4 v, float M, float L) {      // (M in units of log2 e)
    const int h = g * rep + r;
    float fac = 1.f;
    const bf16* gp = a.gate ? reinterpret_cast<const bf16*>(a.gate) + (long long)row * a.ldg + (a.gate_cols ? h * D : h)
                            : nullptr;
    if (a.gate && !a.gate_cols) fac = 1.f / (1.f + expf(-(float)gp[0]));
    if (a.sink) {     // one more term in the denominator
      const float sk = a.sink[h] * ATT_LOG2E, M2 = fmaxf(M, sk), f = exp2f(M - M2);
      L = L * f + exp2f(sk - M2);
      fac *= f;
    }
    fac /= L;
    float y[4] = {v.x * fac, v.y * fac, v.z * fac, v.w * fac};
    bf16x4 w;
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      if (a.gate_cols) y[u] /= 1.f + expf(-(float)gp[c + u]);
      w[u] = (bf16)y[u];
    }
    *reinterpret_cast<bf16x4*>(reinterpret_cast<bf16*>(a.out) + ((long long)row * a.H + h) * D + c) = w;
  };
  const long long group = (long long)row * a.G + g;
  for (int i = threadIdx.x; i < items; i += 64 * NW) {
    const int r = i / (D / 4), c = 4 * (i % (D / 4));
    float M = -INFINITY;
#pragma unroll
    for (int w = 0; w < NW; ++w) M = fmaxf(M, sm[2 * (w * rep + r)]);
    float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
    float L = 0.f;
#pragma unroll
    for (int w = 0; w < NW; ++w) {
      const float f = exp2f(sm[2 * (w * rep + r)] - M);       // a wave without keys: 0
      const float4 x = *reinterpret_cast<const float4*>(so + (w * rep + r) * LDO + c);
      L += f * sm[2 * (w * rep + r) + 1];
      v.x += f * x.x, v.y += f * x.y, v.z += f * x.z, v.w += f * x.w;
    }
    if (nparts == 1) {
      finish(r, c, v, M, L);
    } else {
      float* po = a.part_o + ((group * a.max_parts + part) * rep + r) * D + c;
      publish(po, v.x, v.y);
      publish(po + 2, v.z, v.w);
      if (c == 0) publish(a.part_ml + ((group * a.max_parts + part) * rep + r) * 2, M, L);
    }
  }
  if (nparts == 1) return;
  asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
  __shared__ int last;
  __syncthreads();
  if (threadIdx.x == 0)
    last = __hip_atomic_fetch_add(a.counters + group, 1, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT) == nparts - 1;
  __syncthreads();
  if (!last) return;
  float* pm = so;      // [nparts][rep][2]
  for (int i = threadIdx.x; i < nparts * rep; i += 64 * NW) {
    const float2 v = collect(a.part_ml + (group * a.max_parts * rep + i) * 2);
    pm[2 * i] = v.x, pm[2 * i + 1] = v.y;
  }
  __syncthreads();
  for (int i = threadIdx.x; i < items; i += 64 * NW) {
    const int r = i / (D / 4), c = 4 * (i % (D / 4));
    float M = -INFINITY, L = 0.f;
    for (int p = 0; p < nparts; ++p) M = fmaxf(M, pm[2 * (p * rep + r)]);
    float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll 8
    for (int p = 0; p < nparts; ++p) {
      const float* po = a.part_o + ((group * a.max_parts + p) * rep + r) * D + c;
      const float2 x = collect(po), y = collect(po + 2);
      const float f = exp2f(pm[2 * (p * rep + r)] - M);
      L += f * pm[2 * (p * rep + r) + 1];
      v.x += f * x.x, v.y += f * x.y, v.z += f * y.x, v.w += f * y.y;
    }
    finish(r, c, v, M, L);
  }
  if (threadIdx.x == 0) __hip_atomic_store(a.counters + group, 0, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
}

template <int D, bool KEYV, bool ONE>
void launch(const WindowAttnArgs& a, hipStream_t s) {
  constexpr int stage = (KEYV ? 1 : 2) * STEP * row_chunks(D) * 16 + 256;
  const int rep = a.H / a.G;
  int lds = NW * stage;
  lds = max(lds, (int)(NW * rep * (D + 6) * sizeof(float)));
  lds = max(lds, (int)(a.max_parts * rep * 2 * sizeof(float)));
  static bool once = false;
  if (!once) {
    hipFuncSetAttribute(reinterpret_cast<const void*>(&split_attn_kernel<D, KEYV, ONE>),
                        hipFuncAttributeMaxDynamicSharedMemorySize, 150 * 1024);
    once = true;
  }
  split_attn_kernel<D, KEYV, ONE><<<dim3(a.max_parts, a.G, a.T), 64 * NW, lds, s>>>(a);
}

template <int D, bool KEYV>
void launch_kv(const WindowAttnArgs& a, hipStream_t s) {
  if (a.bs_shift >= 5) launch<D, KEYV, true>(a, s);      // cache blocks of 32 tokens or a larger power of two
  else launch<D, KEYV, false>(a, s);
}

template <int D>
void launch_d(const WindowAttnArgs& a, hipStream_t s) {
  if (a.k_cache == a.v_cache) launch_kv<D, true>(a, s);
  else launch_kv<D, false>(a, s);
}

}  // namespace

bool launch_split_attn(const WindowAttnArgs& a, hipStream_t s) {
  const auto al = [](const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; };
  if (!a.part_o || !a.part_ml || !a.counters || a.part_keys < STEP || a.part_keys % STEP || a.max_parts < 1 ||
      a.max_parts > MAX_PARTS || a.dk != a.dv || a.bias || a.window < (1 << 30) || a.H / a.G > MAX_REP || a.T > 65535 ||
      a.G > 65535 || !al(a.q) || !al(a.k_cache) || !al(a.v_cache) || !al(a.out) || !al(a.part_o))
    return false;
  switch (a.dk) {
    case 32: launch_d<32>(a, s); return true;
    case 48: launch_d<48>(a, s); return true;
    case 64: launch_d<64>(a, s); return true;
    case 80: launch_d<80>(a, s); return true;
    case 96: launch_d<96>(a, s); return true;
    case 112: launch_d<112>(a, s); return true;
    case 128: launch_d<128>(a, s); return true;
    default: return false;
  }
}
