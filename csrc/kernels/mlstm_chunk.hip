// Chunk-parallel form of the mLSTM recurrence for prompt portions of bf16 models (gfx950, wave64); the
// token-by-token form, which decode steps and f32 models run, is in outer_scan.hip.
//
// With f_t <= 0 the log forget gate, i_t the input gate, m the running maximum before a chunk of L
// tokens and F_t the sum of f over the chunk up to t:
//
//     E_s = i_s - F_s,   R_t = max(m, max_{s <= t} E_s),   m_t = F_t + R_t
//     P_ts = (q_t . k_s) exp(E_s - R_t)  for s <= t
//     o_t = sum_s P_ts v_s + exp(m - R_t) S^T q_t,     n_t . q_t likewise with v = 1
//     y_t = o_t / (max(|n_t . q_t|, exp(-m_t)) + 1e-6)
//     S <- exp(m - R_L) S + sum_s k_s (exp(E_s - R_L) v_s)^T,     m <- F_L + R_L
//
// One workgroup per (32 value columns, head, sequence) walks the chunks in order; the chunk's products
// run on v_mfma_f32_16x16x32_bf16.  q, k and v are bf16 as they come; every other operand is an f32 number
// split into bf16 hi + lo parts (two MFMAs, 16 bits of mantissa): the weights P, the weighted values, the
// state as the queries read it.  The state itself stays in f32 accumulators from chunk to chunk.  The
// normaliser is a 33rd value column whose values are 1.  The next chunk's rows are fetched into registers
// under the current chunk's products.  Exponents are kept in base 2 (E, R, m, F times log2 e), gates use the
// hardware exponential, logarithm and reciprocal.
#include "common.h"

namespace {

constexpr int MC_L = 64, MC_V = 32, MC_PS = MC_L + 8;     // tokens per chunk, value columns, stride of [.][token] tiles
typedef float f32x2v __attribute__((ext_vector_type(2)));
typedef __bf16 bf16x2v __attribute__((ext_vector_type(2)));

// inclusive scans over the 64 lanes (DPP row shifts, then row broadcasts)
template <int CTRL, int ROWS> __device__ __forceinline__ float dpp_from(float old, float v) {
  return __int_as_float(__builtin_amdgcn_update_dpp(__float_as_int(old), __float_as_int(v), CTRL, ROWS, 0xf, false));
}
__device__ __forceinline__ float scan_add(float v) {
  v += dpp_from<0x111, 0xf>(0.f, v);
  v += dpp_from<0x112, 0xf>(0.f, v);
  v += dpp_from<0x114, 0xf>(0.f, v);
  v += dpp_from<0x118, 0xf>(0.f, v);
  v += dpp_from<0x142, 0xa>(0.f, v);
  v += dpp_from<0x143, 0xc>(0.f, v);
  return v;
}
__device__ __forceinline__ float scan_max(float v) {
  v = fmaxf(v, dpp_from<0x111, 0xf>(-INFINITY, v));
  v = fmaxf(v, dpp_from<0x112, 0xf>(-INFINITY, v));
  v = fmaxf(v, dpp_from<0x114, 0xf>(-INFINITY, v));
  v = fmaxf(v, dpp_from<0x118, 0xf>(-INFINITY, v));
  v = fmaxf(v, dpp_from<0x142, 0xa>(-INFINITY, v));
  v = fmaxf(v, dpp_from<0x143, 0xc>(-INFINITY, v));
  return v;
}
__device__ __forceinline__ float last_lane(float v) { return __int_as_float(__builtin_amdgcn_readlane(__float_as_int(v), 63)); }

__device__ __forceinline__ uint32_t pack2(float a, float b) {
  return __builtin_bit_cast(uint32_t, __builtin_convertvector(f32x2v{a, b}, bf16x2v));
}
// four f32 numbers as bf16 hi and lo parts
__device__ __forceinline__ void split4(const float (&x)[4], uint2& hi, uint2& lo) {
  hi = make_uint2(pack2(x[0], x[1]), pack2(x[2], x[3]));
  lo = make_uint2(pack2(x[0] - __uint_as_float(hi.x << 16), x[1] - __uint_as_float(hi.x & 0xffff0000u)),
                  pack2(x[2] - __uint_as_float(hi.y << 16), x[3] - __uint_as_float(hi.y & 0xffff0000u)));
}
__device__ __forceinline__ bf16x8 frag(const u16* p) { return __builtin_bit_cast(bf16x8, *reinterpret_cast<const uint4*>(p)); }

constexpr float LOG2E = 1.44269504088896f;
__device__ __forceinline__ float ex2(float x) { return __builtin_amdgcn_exp2f(x); }
// log2(e) cap tanh(x / cap), from cap - 2 cap / (exp(2 x / cap) + 1); an overflowing exponential gives cap
__device__ __forceinline__ float cap2(float x, float cap) {
  return LOG2E * cap * (1.f - 2.f * __builtin_amdgcn_rcpf(ex2(2.f * LOG2E * x / cap) + 1.f));
}
// log2 sigmoid(y / log2 e)
__device__ __forceinline__ float logsigmoid2(float y) { return fminf(y, 0.f) - __builtin_amdgcn_logf(1.f + ex2(-fabsf(y))); }

template <int KD> constexpr long mc_lds() {
  return 2L * (2 * MC_L * (KD + 8) + KD * MC_PS + 3 * MC_V * MC_PS + 4 * 2 * 16 * MC_PS + 2 * (MC_V + 1) * (KD + 8) + 2 * MC_L) +
         4L * 4 * MC_L;
}

// KD >= d (the padded dims are zeros).  MFMA operand layout: with lr = lane & 15, g4 = lane >> 4, A holds
// row lr, contraction indices 8 g4 .. 8 g4 + 7; B column lr, the same indices; the accumulator rows
// 4 g4 .. 4 g4 + 3 of column lr.
template <int KD>
__global__ void __launch_bounds__(256) mlstm_chunk_kernel(const u16* __restrict__ proj, long ld, int H, int d, int dv,
                                                          const float* __restrict__ gate_b, float cap, float qs,
                                                          float* __restrict__ state, float* __restrict__ nm, int NCB,
                                                          const int* __restrict__ qstart, const int* __restrict__ qlen,
                                                          const int* __restrict__ ctx, const int* __restrict__ rows,
                                                          float* __restrict__ raw) {
  constexpr int KST = KD + 8, DS = KD / 32, NT = KD / 64, NF = KD / 32, KCH = KD / 8;
  extern __shared__ __attribute__((aligned(16))) unsigned char smraw[];
  const int s = blockIdx.z, h = blockIdx.y, v0 = blockIdx.x * MC_V;
  const int n = qlen[s];
  if (n <= 0) return;
  const int q0 = qstart[s], p0 = ctx[s] - n, slot = rows[s];
  u16* qsh = reinterpret_cast<u16*>(smraw);        // [L][KST]
  u16* ksh = qsh + MC_L * KST;                     // [L][KST]: token t in row 16 (t & 3) + (t >> 2)
  u16* kt = ksh + MC_L * KST;                      // [KD][PS]: keys transposed
  u16* vt = kt + KD * MC_PS;                       // [V][PS]: values transposed
  u16* wh = vt + MC_V * MC_PS;                     // [V][PS]: values times exp(E_s - R_L), hi and lo
  u16* wl = wh + MC_V * MC_PS;
  u16* pw = wl + MC_V * MC_PS;                     // [4 waves][hi | lo][16][PS]: weights P
  u16* sth = pw + 4 * 2 * 16 * MC_PS;              // [V + 1][KST]: state before the chunk, transposed, hi and lo
  u16* stl = sth + (MC_V + 1) * KST;
  u16* wnh = stl + (MC_V + 1) * KST;               // [L]: exp(E_s - R_L), hi and lo
  u16* wnl = wnh + MC_L;
  float* Es = reinterpret_cast<float*>(wnl + MC_L);   // [L] each: E + log2 qs, R, qs exp(m - R), exp(-m_t)
  float* Rs = Es + MC_L;
  float* Xs = Rs + MC_L;
  float* Ds = Xs + MC_L;
  const int tid = threadIdx.x, lane = tid & 63;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int lr = lane & 15, g4 = lane >> 4;
  u16* phi = pw + wave * (2 * 16 * MC_PS);
  u16* plo = phi + 16 * MC_PS;
  const float bi = gate_b[h], bf = gate_b[H + h];
  const int kcol = H * d, vcol = 2 * H * d, icol = vcol + 2 * H * dv + h;
  // state tiles of this wave: rows 16 (wave + 4 j) .., value blocks 0, 1 and the normaliser's
  f32x4 S[NT][3];
  const long sh0 = (long)slot * H + h;
  float* sp = state + sh0 * d * dv;
  float* np = nm + (sh0 * NCB + 2 * blockIdx.x) * (d + 1);
#pragma unroll
  for (int j = 0; j < NT; ++j)
#pragma unroll
    for (int cb = 0; cb < 3; ++cb)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int r = 16 * (wave + 4 * j) + 4 * g4 + i, c = v0 + 16 * cb + lr;
        float v = 0.f;
        if (p0 > 0 && r < d) {
          if (cb < 2) { if (c < dv) v = sp[(long)r * dv + c]; }
          else if (lr == 0) v = np[r];
        }
        S[j][cb][i] = v;
      }
  float m = p0 > 0 ? np[d] * LOG2E : 0.f;
  const float lqs = __builtin_amdgcn_logf(qs);
  const bf16x8 zero8 = __builtin_bit_cast(bf16x8, make_uint4(0u, 0u, 0u, 0u));
  const bf16x8 ones8 = __builtin_bit_cast(bf16x8, lr == 0 ? make_uint4(0x3f803f80u, 0x3f803f80u, 0x3f803f80u, 0x3f803f80u)
                                                          : make_uint4(0u, 0u, 0u, 0u));
  // a thread moves the same (token, 8 dims) of every chunk
  uint4 pq[NF], pk[NF], pv;
  u16 gi, gf;
  const int vtok = tid >> 2, vc8 = 8 * (tid & 3);
  auto fetch = [&](int t0) {
    const u16* base = proj + (long)(q0 + t0) * ld;
    const int nt = min(MC_L, n - t0);
#pragma unroll
    for (int f = 0; f < NF; ++f) {
      const int e = tid + 256 * f, t = e / KCH, c = (e % KCH) * 8;
      pq[f] = pk[f] = make_uint4(0u, 0u, 0u, 0u);
      if (t < nt && c < d) {
        const u16* r = base + t * ld + h * d + c;
        pq[f] = *reinterpret_cast<const uint4*>(r);
        pk[f] = *reinterpret_cast<const uint4*>(r + kcol);
      }
    }
    pv = make_uint4(0u, 0u, 0u, 0u);
    if (vtok < nt && v0 + vc8 < dv) pv = *reinterpret_cast<const uint4*>(base + vtok * ld + vcol + h * dv + v0 + vc8);
    gi = gf = 0;
    if (lane < nt) {
      gi = base[lane * ld + icol];
      gf = base[lane * ld + icol + H];
    }
  };
  fetch(0);
  for (int t0 = 0; t0 < n; t0 += MC_L) {
    const int nt = min(MC_L, n - t0);
    // gates, a lane per token (every wave for itself)
    float ig = -INFINITY, fg = 0.f;
    if (lane < nt) {
      ig = cap2(bf2f(gi) + bi, cap);
      fg = logsigmoid2(cap2(bf2f(gf) + bf, cap));
    }
    const float F = scan_add(fg), E = ig - F, R = fmaxf(m, scan_max(E));
    const float RL = last_lane(R), decay = ex2(m - RL), wlast = ex2(E - RL);
    const float wv = __shfl(wlast, 16 * wave + (lane >> 2));     // the weight of the token whose values this thread moves
    __syncthreads();     // the previous chunk is consumed
    if (wave == 0) {
      Es[lane] = E + lqs;
      Rs[lane] = R;
      Xs[lane] = qs * ex2(m - R);
      Ds[lane] = ex2(-(F + R));
    } else if (wave == 1) {
      const uint32_t hi = pack2(wlast, 0.f);
      wnh[lane] = (u16)hi;
      wnl[lane] = (u16)pack2(wlast - __uint_as_float(hi << 16), 0.f);
    }
    m = last_lane(F) + RL;
#pragma unroll
    for (int f = 0; f < NF; ++f) {
      const int e = tid + 256 * f, t = e / KCH, c = (e % KCH) * 8;
      *reinterpret_cast<uint4*>(qsh + t * KST + c) = pq[f];
      *reinterpret_cast<uint4*>(ksh + (16 * (t & 3) + (t >> 2)) * KST + c) = pk[f];
    }
    {
      const uint32_t pe[4] = {pv.x, pv.y, pv.z, pv.w};
#pragma unroll
      for (int x = 0; x < 4; ++x) {
        const float w0 = wv * __uint_as_float(pe[x] << 16), w1 = wv * __uint_as_float(pe[x] & 0xffff0000u);
        const uint32_t hi = pack2(w0, w1), lo = pack2(w0 - __uint_as_float(hi << 16), w1 - __uint_as_float(hi & 0xffff0000u));
        const int o = (vc8 + 2 * x) * MC_PS + vtok;
        vt[o] = (u16)pe[x];
        vt[o + MC_PS] = (u16)(pe[x] >> 16);
        wh[o] = (u16)hi;
        wh[o + MC_PS] = (u16)(hi >> 16);
        wl[o] = (u16)lo;
        wl[o + MC_PS] = (u16)(lo >> 16);
      }
    }
#pragma unroll
    for (int j = 0; j < NT; ++j)
#pragma unroll
      for (int cb = 0; cb < 3; ++cb) {
        if (cb == 2 && lr != 0) continue;
        const float x[4] = {S[j][cb][0], S[j][cb][1], S[j][cb][2], S[j][cb][3]};
        uint2 hi, lo;
        split4(x, hi, lo);
        const int o = (16 * cb + (cb < 2 ? lr : 0)) * KST + 16 * (wave + 4 * j) + 4 * g4;
        *reinterpret_cast<uint2*>(sth + o) = hi;
        *reinterpret_cast<uint2*>(stl + o) = lo;
      }
    if (t0 + MC_L < n) fetch(t0 + MC_L);
    __syncthreads();
    // keys once more, [dim][token] (8 tokens of a dim as one 16-byte vector)
#pragma unroll
    for (int f = 0; f < NF; ++f) {
      const int e = tid + 256 * f, kg = e / KD, c = e % KD;
      const u16* col = ksh + 2 * kg * KST + c;
      uint32_t w4[4];
#pragma unroll
      for (int x = 0; x < 4; ++x) {
        const int r0 = 16 * ((2 * x) & 3) + ((2 * x) >> 2), r1 = 16 * ((2 * x + 1) & 3) + ((2 * x + 1) >> 2);
        w4[x] = (uint32_t)col[r0 * KST] | ((uint32_t)col[r1 * KST] << 16);
      }
      *reinterpret_cast<uint4*>(kt + c * MC_PS + 8 * kg) = make_uint4(w4[0], w4[1], w4[2], w4[3]);
    }
    // scores of the wave's 16 rows; block kb, column lr stands for token 4 lr + kb
    bf16x8 qa[DS];
    f32x4 sacc[4];
#pragma unroll
    for (int kb = 0; kb < 4; ++kb) sacc[kb] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int st = 0; st < DS; ++st) {
      qa[st] = frag(qsh + (16 * wave + lr) * KST + 8 * g4 + 32 * st);
#pragma unroll
      for (int kb = 0; kb < 4; ++kb)
        sacc[kb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qa[st], frag(ksh + (16 * kb + lr) * KST + 8 * g4 + 32 * st), sacc[kb], 0, 0, 0);
    }
    const int row0 = 16 * wave + 4 * g4;
    const float4 e4 = *reinterpret_cast<const float4*>(Es + 4 * lr), r4 = *reinterpret_cast<const float4*>(Rs + row0);
    const float ev[4] = {e4.x, e4.y, e4.z, e4.w}, rv[4] = {r4.x, r4.y, r4.z, r4.w};
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      float p[4];
#pragma unroll
      for (int kb = 0; kb < 4; ++kb) {
        const float w = sacc[kb][i] * ex2(ev[kb] - rv[i]);
        p[kb] = 4 * lr + kb <= row0 + i ? w : 0.f;
      }
      uint2 hi, lo;
      split4(p, hi, lo);
      *reinterpret_cast<uint2*>(phi + (4 * g4 + i) * MC_PS + 4 * lr) = hi;
      *reinterpret_cast<uint2*>(plo + (4 * g4 + i) * MC_PS + 4 * lr) = lo;
    }
    // the patch is this wave's own: its LDS accesses are in order, the fence keeps the compiler's order too
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    __builtin_amdgcn_wave_barrier();
    f32x4 oi[3], os[3];
#pragma unroll
    for (int cb = 0; cb < 3; ++cb) oi[cb] = os[cb] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int st = 0; st < DS; ++st) {      // what the state holds of earlier chunks
      const int o = 8 * g4 + 32 * st;
#pragma unroll
      for (int cb = 0; cb < 2; ++cb) {
        os[cb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qa[st], frag(sth + (16 * cb + lr) * KST + o), os[cb], 0, 0, 0);
        os[cb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qa[st], frag(stl + (16 * cb + lr) * KST + o), os[cb], 0, 0, 0);
      }
      const bf16x8 nh = lr == 0 ? frag(sth + MC_V * KST + o) : zero8, nl = lr == 0 ? frag(stl + MC_V * KST + o) : zero8;
      os[2] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qa[st], nh, os[2], 0, 0, 0);
      os[2] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qa[st], nl, os[2], 0, 0, 0);
    }
#pragma unroll
    for (int ks = 0; ks < MC_L; ks += 32) {      // tokens of this chunk
      const bf16x8 ah = frag(phi + lr * MC_PS + 8 * g4 + ks), al = frag(plo + lr * MC_PS + 8 * g4 + ks);
#pragma unroll
      for (int cb = 0; cb < 3; ++cb) {
        const bf16x8 b = cb < 2 ? frag(vt + (16 * cb + lr) * MC_PS + 8 * g4 + ks) : ones8;
        oi[cb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ah, b, oi[cb], 0, 0, 0);
        oi[cb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(al, b, oi[cb], 0, 0, 0);
      }
    }
    {
      const float4 x4 = *reinterpret_cast<const float4*>(Xs + row0), d4 = *reinterpret_cast<const float4*>(Ds + row0);
      const float xv[4] = {x4.x, x4.y, x4.z, x4.w}, dn[4] = {d4.x, d4.y, d4.z, d4.w};
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const float nq = __shfl(oi[2][i] + xv[i] * os[2][i], lane & 48);      // the row's normaliser: column 0 of its block
        const float inv = __builtin_amdgcn_rcpf(fmaxf(fabsf(nq), dn[i]) + 1e-6f);
        const int t = row0 + i;
        if (t >= nt) continue;
        float* dst = raw + (long)(q0 + t0 + t) * ((long)H * dv) + (long)h * dv + v0 + lr;
#pragma unroll
        for (int cb = 0; cb < 2; ++cb)
          if (v0 + 16 * cb + lr < dv) dst[16 * cb] = (oi[cb][i] + xv[i] * os[cb][i]) * inv;
      }
    }
    __syncthreads();     // the transposed keys are there
#pragma unroll
    for (int j = 0; j < NT; ++j) {
#pragma unroll
      for (int cb = 0; cb < 3; ++cb)
#pragma unroll
        for (int i = 0; i < 4; ++i) S[j][cb][i] *= decay;
#pragma unroll
      for (int ks = 0; ks < MC_L; ks += 32) {
        const int o = 8 * g4 + ks;
        const bf16x8 a = frag(kt + (16 * (wave + 4 * j) + lr) * MC_PS + o);
#pragma unroll
        for (int cb = 0; cb < 3; ++cb) {
          const bf16x8 bh = cb < 2 ? frag(wh + (16 * cb + lr) * MC_PS + o) : lr == 0 ? frag(wnh + o) : zero8;
          const bf16x8 bl = cb < 2 ? frag(wl + (16 * cb + lr) * MC_PS + o) : lr == 0 ? frag(wnl + o) : zero8;
          S[j][cb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, bh, S[j][cb], 0, 0, 0);
          S[j][cb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, bl, S[j][cb], 0, 0, 0);
        }
      }
    }
  }
  // back to the slot; every 16-column block keeps its own copy of normaliser and maximum
#pragma unroll
  for (int j = 0; j < NT; ++j)
#pragma unroll
    for (int cb = 0; cb < 3; ++cb)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int r = 16 * (wave + 4 * j) + 4 * g4 + i, c = v0 + 16 * cb + lr;
        if (r >= d) continue;
        if (cb < 2) {
          if (c < dv) sp[(long)r * dv + c] = S[j][cb][i];
        } else if (lr == 0) {
          np[r] = S[j][cb][i];
          if (2 * (int)blockIdx.x + 1 < NCB) np[d + 1 + r] = S[j][cb][i];
        }
      }
  if (tid == 0) {
    np[d] = m / LOG2E;
    if (2 * (int)blockIdx.x + 1 < NCB) np[2 * d + 1] = m / LOG2E;
  }
}

}  // namespace

// 1 when the chunk form takes the shape: bf16 rows of whole 16-byte vectors, key width <= 128
extern "C" int dllm_mlstm_chunk_ok(int f32, long ld, int d, int dv) {
  return !f32 && d >= 8 && d <= 128 && d % 8 == 0 && dv >= 8 && dv % 8 == 0 && ld % 8 == 0;
}

// NCB: 16-column blocks of the value width, each with a copy of normaliser and maximum in nm
extern "C" int dllm_mlstm_chunk(const void* proj, long ld, int H, int d, int dv, const float* gate_b, float cap, float* state,
                                float* nm, int NCB, const int* qstart, const int* qlen, const int* ctx, const int* rows, int S,
                                float* raw, hipStream_t st) {
  if (S <= 0) return 0;
  if (!dllm_mlstm_chunk_ok(0, ld, d, dv) || H < 1 || NCB != (dv + 15) / 16 || (uintptr_t)proj % 16) return -1;
  const dim3 grid((dv + MC_V - 1) / MC_V, H, S);
  const float qs = 1.f / sqrtf((float)d);
#define MC(KD)                                                                                                                \
  do {                                                                                                                        \
    static bool set_ = false; /* raised once: no attribute call inside a later stream capture */                             \
    if (!set_) {                                                                                                              \
      (void)hipFuncSetAttribute((const void*)mlstm_chunk_kernel<KD>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)mc_lds<KD>()); \
      set_ = true;                                                                                                            \
    }                                                                                                                         \
    hipLaunchKernelGGL((mlstm_chunk_kernel<KD>), grid, dim3(256), mc_lds<KD>(), st, (const u16*)proj, ld, H, d, dv, gate_b, cap, qs, \
                       state, nm, NCB, qstart, qlen, ctx, rows, raw);                                                         \
  } while (0)
  if (d <= 64) MC(64); else MC(128);
#undef MC
  return (int)hipGetLastError();
}
