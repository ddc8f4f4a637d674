// Causal softmax attention for prompt rows (bf16): one workgroup per (128 consecutive rows of a sequence's run, query head),
// grouped key / value heads over the paged token-major cache.  Same arguments as window_attention.hip's kernels for a window
// that never ends; optional sink, soft cap, per-key score factor and output gate (per head or per column).
//
// Four waves of 32 rows each; keys walk in tiles of 64 up to the last row's own position.  A tile's rows go from the cache to
// LDS by direct loads, one tile ahead of the products (two stages), in 16-byte chunks whose place within the row is XORed with
// the row number so that neither fragment read conflicts.  Scores are S^T = K Q^T on v_mfma_f32_32x32x16_bf16: a lane ends with
// one query row's scores of 32 keys, in exactly the order in which they go back, as bf16 weights, into O^T = V^T P^T.  The
// transposed value fragments come from the row-major tile through the LDS transpose read (ds_read_b64_tr_b16), so values are
// neither transposed while staged nor -- where the values ARE the keys (KEYV) -- staged at all: one tile serves both products.
//
// Softmax statistics are fp32.  Without a cap: running maximum (one cross-lane step per tile), sums combined at the end.  With
// a cap c <= 60 the scores lie in [-c, c], so e^s needs no maximum: p = 2^(c' - 2 c' / (1 + 2^(2 s log2(e) / c))), c' = c log2 e.
#include "attn_tiles.h"
#include "hybrid_launchers.h"

namespace {

constexpr float MAX_CAP = 60.f;      // e^60 times any number of keys and e^-60 are well inside fp32 and bf16
constexpr int PW = 4, ROWS = 32 * PW;

SYM_DEV f32x16 mfma32(bf16x8 a, bf16x8 b, f32x16 c) { return __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, b, c, 0, 0, 0); }

template <int D, bool CAP, bool KEYV, bool ONE>
__global__ __launch_bounds__(64 * PW, 2) void prompt_attn_kernel(WindowAttnArgs a) {
  constexpr int CH = row_chunks(D), KD = D / 16, VT = (D + 31) / 32, TILE = 64 * CH * 16;   // bytes of a staged tile
  constexpr int NL = CH / PW;                          // direct loads per wave and tile (64 / CH rows each)
  constexpr int STAGE = (KEYV ? 1 : 2) * TILE + 256;   // keys, values, 64 key factors
  extern __shared__ __attribute__((aligned(16))) char smem[];
  const int tile = blockIdx.y, h = blockIdx.x;
  const int seq = a.tiles[2 * tile], row0 = a.tiles[2 * tile + 1];
  const int r_hi = a.cu_q[seq + 1], first = a.cu_q[seq] + row0;
  if (first >= r_hi || (row0 & 64)) return;            // padding tile / the second half of a pair (whole workgroup)
  const int nrows = min(ROWS, r_hi - first);
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, j = lane & 31, hi = lane >> 5;
  const int g = h / (a.H / a.G);
  const int my_row = first + 32 * wave + j;
  const bool rv = 32 * wave + j < nrows;
  const int p_first = a.positions[first], p_last = p_first + nrows - 1;
  const int wq_lo = p_first + 32 * wave, wq_hi = wq_lo + 31, qp = wq_lo + j;
  const int* bt = a.block_tables + (long long)a.row_seq[first] * a.max_blocks;
  const bf16* kc = reinterpret_cast<const bf16*>(a.k_cache) + g * D;
  const bf16* vc = reinterpret_cast<const bf16*>(a.v_cache) + g * D;
  const long long ld = (long long)a.G * D;

  bf16x8 qf[KD];
  {
    const bf16* q = reinterpret_cast<const bf16*>(a.q) + ((long long)my_row * a.H + h) * D + 8 * hi;
#pragma unroll
    for (int kk = 0; kk < KD; ++kk) {
      Pack8 t;
      t.u = rv ? *reinterpret_cast<const uint4*>(q + 16 * kk) : make_uint4(0, 0, 0, 0);
      qf[kk] = t.v;
    }
  }
  // staging: load i of a wave fills the rows (64 / CH) (PW i + wave) .. of the tile.  ONE: a tile lies in one cache block, whose
  // number is read one tile ahead (a scalar load: no wait of the direct loads in flight); else every row is looked up.
  const unsigned int lds0 = lds_address(smem);
  const int uw = __builtin_amdgcn_readfirstlane(wave);
  int blk = 0;
  auto row_of = [&](int kp) {
    kp = min(kp, p_last);
    return ONE ? ((long long)blk << a.bs_shift) + (kp & (a.BS - 1)) : cache_row(bt, kp, a.BS, a.bs_shift);
  };
  auto stage = [&](int kt, int buf) {
    const unsigned int base = lds0 + buf * STAGE;
#pragma unroll
    for (int i = 0; i < NL; ++i) {
      const int r = (64 / CH) * (PW * i + wave) + lane / CH;
      int c = (lane & (CH - 1)) ^ swz<CH>(r);
      if (D < 8 * CH && c >= D / 8) c = 0;             // (places past the head's end are never used)
      const long long src = row_of(kt + r) * ld + 8 * c;
      direct_load16(kc + src, base + (PW * i + uw) * 1024);
      if constexpr (!KEYV) direct_load16(vc + src, base + TILE + (PW * i + uw) * 1024);
    }
    if (a.key_scale && uw == 0) direct_load4(a.key_scale + row_of(kt + lane), base + STAGE - 256);
  };

  // fragment addresses within a stage: key rows 32 b + j (chunk 2 kk + hi); value rows 16 c' + 8 s + 4 hi' + (l >> 2), entries
  // 32 dt + 16 (group & 1) + 4 (l & 3) .. (group = lane / 16, l = lane % 16, hi' = group / 2)
  int ka[KD], va[VT][2];
#pragma unroll
  for (int kk = 0; kk < KD; ++kk) ka[kk] = j * CH * 16 + 16 * ((2 * kk + hi) ^ swz<CH>(j));
#pragma unroll
  for (int dt = 0; dt < VT; ++dt)
#pragma unroll
    for (int s = 0; s < 2; ++s) {
      const int l = lane & 15, grp = lane >> 4, r = 8 * s + 4 * (grp >> 1) + (l >> 2);
      const int c = 4 * dt + 2 * (grp & 1) + ((l & 3) >> 1);
      va[dt][s] = (KEYV ? 0 : TILE) + r * CH * 16 + 16 * (c ^ swz<CH>(r)) + 8 * (l & 1);
    }

  f32x16 o[VT];
#pragma unroll
  for (int i = 0; i < VT; ++i)
#pragma unroll
    for (int e = 0; e < 16; ++e) o[i][e] = 0.f;
  float m = CAP ? 0.f : -INFINITY, l = 0.f;            // l: this lane's keys only, the two lanes of a row meet at the end
  const float sl2 = a.scale * ATT_LOG2E;
  const float c1 = CAP ? 2.f * sl2 / a.softcap : 0.f, c2 = CAP ? a.softcap * ATT_LOG2E : 0.f;
  const bool scaled = a.key_scale != nullptr;

  if (ONE) blk = bt[0];
  stage(0, 0);
  if (ONE && 64 <= p_last) blk = bt[64 >> a.bs_shift];
  int buf = 0;
  for (int kt = 0; kt <= p_last; kt += 64, buf ^= 1) {
    wait_direct_loads();
    __syncthreads();                                   // the tile has landed; every wave is done with the other stage
    if (kt + 64 <= p_last) {
      stage(kt + 64, buf ^ 1);
      if (ONE && kt + 128 <= p_last) blk = bt[(kt + 128) >> a.bs_shift];
    }
    if (kt > wq_hi || 32 * wave >= nrows) continue;    // (wave-uniform) nothing of this tile is visible here
    const char* S = smem + buf * STAGE;
    float p[2][16];
    {
      // all key fragments are in flight before the first product waits for its own
      Pack8 kf[2][KD];
#pragma unroll
      for (int b = 0; b < 2; ++b)
#pragma unroll
        for (int kk = 0; kk < KD; ++kk) kf[b][kk].u = *reinterpret_cast<const uint4*>(S + ka[kk] + b * 32 * CH * 16);
      __builtin_amdgcn_sched_barrier(0);
#pragma unroll
      for (int b = 0; b < 2; ++b) {
        f32x16 acc;
#pragma unroll
        for (int e = 0; e < 16; ++e) acc[e] = 0.f;
#pragma unroll
        for (int kk = 0; kk < KD; ++kk) acc = mfma32(kf[b][kk].v, qf[kk], acc);
#pragma unroll
        for (int e = 0; e < 16; ++e) p[b][e] = acc[e];   // key kt + 32 b + 8 (e / 4) + 4 hi + e % 4 of row qp
      }
    }
    if (scaled) {
      const float* ks = reinterpret_cast<const float*>(S + STAGE - 256) + 4 * hi;
#pragma unroll
      for (int b = 0; b < 2; ++b)
#pragma unroll
        for (int e4 = 0; e4 < 4; ++e4) {
          const float4 f = *reinterpret_cast<const float4*>(ks + 32 * b + 8 * e4);
          p[b][4 * e4] *= f.x, p[b][4 * e4 + 1] *= f.y, p[b][4 * e4 + 2] *= f.z, p[b][4 * e4 + 3] *= f.w;
        }
    }
    const bool edge = kt + 63 > wq_lo;                 // (wave-uniform) some row does not see the whole tile
    const int vis = qp - kt - 4 * hi;                  // key offsets <= vis are visible
    if constexpr (CAP) {
#pragma unroll
      for (int b = 0; b < 2; ++b)
#pragma unroll
        for (int e = 0; e < 16; ++e) {
          const float t = __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(c1 * p[b][e]));
          p[b][e] = __builtin_amdgcn_exp2f(c2 - 2.f * c2 * t);
        }
      if (edge) {
#pragma unroll
        for (int b = 0; b < 2; ++b)
#pragma unroll
          for (int e = 0; e < 16; ++e)
            if (32 * b + 8 * (e / 4) + e % 4 > vis) p[b][e] = 0.f;
      }
    } else {
      if (edge) {
#pragma unroll
        for (int b = 0; b < 2; ++b)
#pragma unroll
          for (int e = 0; e < 16; ++e)
            if (32 * b + 8 * (e / 4) + e % 4 > vis) p[b][e] = -INFINITY;
      }
      float mx = p[0][0];
#pragma unroll
      for (int b = 0; b < 2; ++b)
#pragma unroll
        for (int e = 0; e < 16; ++e) mx = fmaxf(mx, p[b][e]);
      mx = fmaxf(mx, __shfl_xor(mx, 32, 64)) * sl2;    // (scale > 0: checked by the launcher)
      const float mt = fmaxf(m, mx);
      const float mref = mt == -INFINITY ? 0.f : mt;   // a row that sees nothing of the tile yet
      if (__any(mt > m)) {                             // some row's maximum moved: rescale (else every factor is 1)
        const float corr = __builtin_amdgcn_exp2f(m - mref);
        l *= corr;
#pragma unroll
        for (int i = 0; i < VT; ++i) o[i] *= corr;
        m = mt;
      }
#pragma unroll
      for (int b = 0; b < 2; ++b)
#pragma unroll
        for (int e = 0; e < 16; ++e) p[b][e] = __builtin_amdgcn_exp2f(p[b][e] * sl2 - mref);
    }
    float sum = 0.f;
    bf16x8 pf[4];
#pragma unroll
    for (int b = 0; b < 2; ++b)
#pragma unroll
      for (int e = 0; e < 16; ++e) {
        sum += p[b][e];
        pf[2 * b + e / 8][e % 8] = (bf16)p[b][e];
      }
    l += sum;
#pragma unroll
    for (int c = 0; c < 4; ++c)
#pragma unroll
      for (int dt = 0; dt < VT; ++dt) {
        const uint2 x0 = read_tr(S + va[dt][0] + c * 16 * CH * 16), x1 = read_tr(S + va[dt][1] + c * 16 * CH * 16);
        Pack8 vf;
        vf.u = make_uint4(x0.x, x0.y, x1.x, x1.y);
        o[dt] = mfma32(vf.v, pf[c], o[dt]);
      }
  }
  l += __shfl_xor(l, 32, 64);
  if (!rv) return;
  float fac = 1.f;
  const bf16* gp = a.gate ? reinterpret_cast<const bf16*>(a.gate) + (long long)my_row * a.ldg + (a.gate_cols ? h * D : h)
                          : nullptr;
  if (a.gate && !a.gate_cols) fac = 1.f / (1.f + expf(-(float)gp[0]));
  if (a.sink) {     // one more term in the denominator (m is in units of log2 e)
    const float sk = a.sink[h] * ATT_LOG2E, M = fmaxf(m, sk), f = exp2f(m - M);
    l = l * f + exp2f(sk - M);
    fac *= f;
  }
  const float inv = fac / l;
  bf16* out = reinterpret_cast<bf16*>(a.out) + ((long long)my_row * a.H + h) * D;
  bf16x4 gv[VT][4];      // all gates in flight before the first store (which the loads could not pass)
  if (a.gate_cols) {
    const bool vec = (a.ldg & 3) == 0 && (reinterpret_cast<uintptr_t>(a.gate) & 7) == 0;
#pragma unroll
    for (int dt = 0; dt < VT; ++dt)
#pragma unroll
      for (int e4 = 0; e4 < 4; ++e4) {
        const int c = 32 * dt + 8 * e4 + 4 * hi;
        if (D % 32 && c >= D) continue;
        if (vec) gv[dt][e4] = *reinterpret_cast<const bf16x4*>(gp + c);
        else
#pragma unroll
          for (int u = 0; u < 4; ++u) gv[dt][e4][u] = gp[c + u];
      }
  }
#pragma unroll
  for (int dt = 0; dt < VT; ++dt)
#pragma unroll
    for (int e4 = 0; e4 < 4; ++e4) {
      const int c = 32 * dt + 8 * e4 + 4 * hi;
      if (D % 32 && c >= D) continue;
      bf16x4 w;
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        float v = o[dt][4 * e4 + u] * inv;
        if (a.gate_cols) v *= __builtin_amdgcn_rcpf(1.f + __expf(-(float)gv[dt][e4][u]));
        w[u] = (bf16)v;
      }
      *reinterpret_cast<bf16x4*>(out + c) = w;
    }
}

template <int D, bool CAP, bool KEYV, bool ONE>
void launch(const WindowAttnArgs& a, hipStream_t s) {
  constexpr int lds = 2 * ((KEYV ? 1 : 2) * 64 * row_chunks(D) * 16 + 256);
  static bool once = false;
  if (lds > 64 * 1024 && !once) {
    hipFuncSetAttribute(reinterpret_cast<const void*>(&prompt_attn_kernel<D, CAP, KEYV, ONE>),
                        hipFuncAttributeMaxDynamicSharedMemorySize, lds);
    once = true;
  }
  prompt_attn_kernel<D, CAP, KEYV, ONE><<<dim3(a.H, a.ntiles), 64 * PW, lds, s>>>(a);
}

template <int D>
void launch_d(const WindowAttnArgs& a, hipStream_t s) {
  const bool one = a.bs_shift >= 6;      // cache blocks of 64 tokens or a larger power of two
  if (a.softcap > 0.f) one ? launch<D, true, false, true>(a, s) : launch<D, true, false, false>(a, s);
  else if (a.k_cache == a.v_cache) one ? launch<D, false, true, true>(a, s) : launch<D, false, true, false>(a, s);
  else one ? launch<D, false, false, true>(a, s) : launch<D, false, false, false>(a, s);
}

}  // namespace

bool launch_prompt_attn(const WindowAttnArgs& a, hipStream_t s) {
  const auto al = [](const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; };
  if (!a.tiles || !a.cu_q || a.ntiles <= 0 || a.ntiles > 65535 || a.dk != a.dv || a.bias || a.window < (1 << 30) ||
      !(a.scale > 0.f) || a.softcap > MAX_CAP || !al(a.q) || !al(a.k_cache) || !al(a.v_cache) || !al(a.out))
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
