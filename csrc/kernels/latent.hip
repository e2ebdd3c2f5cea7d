// Latent attention: softmax attention whose keys and values are one shared compressed vector per
// token (a normed latent of `rank` dims plus a rotated key part of `rot` dims that every head
// shares).  The per-head key up-projection is absorbed into the query on the host side, so a row
// (token, head) scores key j as  q_lat . c_j + q_rot . kr_j  and returns  sum_j p_j c_j  (the value
// up-projection follows as a per-head batched GEMM).  Only [c_j | kr_j] is cached, paged in
// 16-token blocks.
//
//   latent_kv_write   one workgroup per token: RMS-norm the latent (f32), rotate the shared key part
//                     (pairs (2i, 2i + 1) or (i, i + rot / 2)), write both into the token's cache slot, and
//                     norm the query latent that the same projection made
//   latent_q_prep     queries of the expanded form: the rotated part rotated, everything scaled
//   latent_prep       latent_kv_write without a rotated part for a layer whose feed-forward shares the
//                     projection: the same launch squares the relu of the up columns
//   latent_expand     keys and values of every head from the cached latents of a step's sequences, into
//                     pages of their own (prompt portions then run the grouped-query attention kernel); the
//                     shared rotated part is copied behind every head's key
//   gate_heads        per-head outputs [H, T, dv] times sigmoid(gate), laid out token-major; one logit per
//                     entry or one per head
//   latent_attention  one workgroup per 16 rows (token-major (token, head) rows of one sequence):
//                     the rows' queries staged once in LDS as f32 (rotation and the score scale
//                     applied while staging); keys walk in tiles staged in LDS as f32;
//                     phase 1: a lane owns a key and sums q . k over the dims (q read as LDS
//                     broadcasts, k with an odd row stride: no bank conflicts) -> f32 scores, causal
//                     mask, online softmax per row (wave reductions);
//                     phase 2: a lane owns latent dims lane, lane + 64, ... and accumulates p . c.
//                     Each wave owns 4 of the 16 rows through both phases.  Small grids (decode) split
//                     a row's keys over several workgroups; latent_combine merges their partials.
//                     sinks: one more term exp(sinks[head]) of the softmax denominator, without a value.
// Activations and the cache are bf16 or f32 (template); scores, softmax and sums are f32.
#include "common.h"

namespace {

template <typename T> __device__ __forceinline__ float ldf(const T* p);
template <> __device__ __forceinline__ float ldf<u16>(const u16* p) { return bf2f(*p); }
template <> __device__ __forceinline__ float ldf<float>(const float* p) { return *p; }
template <typename T> __device__ __forceinline__ void stf(T* p, float v);
template <> __device__ __forceinline__ void stf<u16>(u16* p, float v) { *p = f2bf(v); }
template <> __device__ __forceinline__ void stf<float>(float* p, float v) { *p = v; }

// Rotary pair of the rotated part's entry c (of `rot`): its partner, its angle index, and whether it is
// the pair's first.  hf: pairs (i, i + rot / 2), else (2i, 2i + 1).
__device__ __forceinline__ void rot_pair(int c, int half, int hf, int& partner, int& ang, bool& first) {
  if (hf) { first = c < half; ang = first ? c : c - half; partner = first ? c + half : c - half; }
  else { first = !(c & 1); ang = c >> 1; partner = c ^ 1; }
}
template <typename T>
__device__ __forceinline__ float rotated(const T* r, int c, int half, int hf, const float* cs) {
  int p, a;
  bool first;
  rot_pair(c, half, hf, p, a, first);
  const float v = ldf(r + c), w = ldf(r + p);
  return first ? v * cs[a] - w * cs[half + a] : v * cs[a] + w * cs[half + a];
}

// wave 0: the token's latent and shared key part into its cache slot.  waves 1 to 3 (launched when qsrc):
// qdst = rmsnorm(qsrc row) qw, the query latent.  Rows of up to 8 values a lane stay in registers between
// the sum and the store.  zl (optional, [zh, tokens, rank]): a padding token's rows, which no attention
// tile writes, are cleared.
template <typename T>
__global__ void __launch_bounds__(256) latent_kv_write_kernel(const T* __restrict__ ckv, long ld, int rank, int rot,
                                                              const float* __restrict__ w, float eps,
                                                              const int* __restrict__ pos,
                                                              const float* __restrict__ cos_sin, int tab_w,
                                                              const int* __restrict__ slots, T* __restrict__ cache, int hf,
                                                              const T* __restrict__ qsrc, long ldqs, int qn,
                                                              const float* __restrict__ qw, T* __restrict__ qdst,
                                                              T* __restrict__ zl, int zh) {
  constexpr int NR = 8;      // values a lane keeps
  __shared__ float red[3];
  const int t = blockIdx.x, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int slot = slots[t];
  if (zl && slot < 0)
    for (int i = threadIdx.x; i < zh * rank; i += blockDim.x) stf(zl + ((long)(i / rank) * gridDim.x + t) * rank + i % rank, 0.f);
  const bool is_q = wave > 0;
  const T* r = is_q ? qsrc + (long)t * ldqs : ckv + (long)t * ld;
  const int n = is_q ? qn : rank, i0 = is_q ? threadIdx.x - 64 : lane, step = is_q ? 192 : 64;
  float v[NR], s = 0.f;
#pragma unroll
  for (int j = 0; j < NR; ++j) {
    v[j] = i0 + j * step < n ? ldf(r + i0 + j * step) : 0.f;
    s += v[j] * v[j];
  }
  for (int i = i0 + NR * step; i < n; i += step) { const float x = ldf(r + i); s += x * x; }
  s = wave_sum(s);
  if (qsrc) {      // uniform: the query latent's sum over its three waves
    if (is_q && lane == 0) red[wave - 1] = s;
    __syncthreads();
    if (is_q) s = red[0] + red[1] + red[2];
  }
  if (!is_q && slot < 0) return;
  const float rs = 1.f / sqrtf(s / (float)n + eps);
  const float* g = is_q ? qw : w;
  T* dst = is_q ? qdst + (long)t * qn : cache + (long)slot * (rank + rot);
#pragma unroll
  for (int j = 0; j < NR; ++j)
    if (i0 + j * step < n) stf(dst + i0 + j * step, v[j] * rs * g[i0 + j * step]);
  for (int i = i0 + NR * step; i < n; i += step) stf(dst + i, ldf(r + i) * rs * g[i]);
  if (is_q) return;
  const float* cs = cos_sin + (long)pos[t] * tab_w;
  const int half = rot >> 1;
  for (int i = lane; i < rot; i += 64) stf(dst + rank + i, rotated(r + rank, i, half, hf, cs));
}

// out[t, h, :] = [q_h | rotated part] * scale for queries q [T, H (dim + rot)]; x over the columns, y over
// the tokens
template <typename T>
__global__ void __launch_bounds__(256) latent_q_prep_kernel(const T* __restrict__ q, long ldq, int H, int dim, int rot, int hf,
                                                            const int* __restrict__ pos, const float* __restrict__ cos_sin,
                                                            int tab_w, float scale, T* __restrict__ out, long Tn) {
  const int c = blockIdx.x * 256 + threadIdx.x, w = dim + rot;
  if (c >= H * w) return;
  const int h = c / w, i = c - h * w, half = rot >> 1;
  for (long t = blockIdx.y; t < Tn; t += gridDim.y) {
    const T* r = q + t * ldq + (long)h * w;
    const float v = i < dim ? ldf(r + i) : rotated(r + dim, i - dim, half, hf, cos_sin + (long)pos[t] * tab_w);
    stf(out + t * (long)(H * w) + c, v * scale);
  }
}

// The same for bf16 rows of whole 16-byte vectors and rotate-half pairs (dim % 8 == 0, rot % 16 == 0): a
// thread owns 8 neighbouring unrotated dims, or 8 rotary pairs.
__global__ void __launch_bounds__(256) latent_q_prep_vec_kernel(const u16* __restrict__ q, long ldq, int H, int dim, int rot,
                                                                const int* __restrict__ pos, const float* __restrict__ cos_sin,
                                                                int tab_w, float scale, u16* __restrict__ out, long Tn) {
  const int w = dim + rot, half = rot >> 1, per = (dim + half) >> 3;      // vectors (or pairs of vectors) of a head
  const int u = blockIdx.x * 256 + threadIdx.x;
  if (u >= H * per) return;
  const int h = u / per, c = 8 * (u - h * per);
  for (long t = blockIdx.y; t < Tn; t += gridDim.y) {
    const u16* r = q + t * ldq + (long)h * w;
    u16* o = out + t * (long)(H * w) + (long)h * w;
    float a[8];
    unpack8(ld16(r + c), a);
    if (c >= dim) {
      float b[8];
      unpack8(ld16(r + c + half), b);
      const float* cs = cos_sin + (long)pos[t] * tab_w + (c - dim);
#pragma unroll
      for (int x = 0; x < 8; ++x) {
        const float cc = cs[x] * scale, sn = cs[half + x] * scale, va = a[x];
        a[x] = va * cc - b[x] * sn;
        b[x] = b[x] * cc + va * sn;
      }
      st16(o + c + half, pack8(b));
    } else {
#pragma unroll
      for (int x = 0; x < 8; ++x) a[x] *= scale;
    }
    st16(o + c, pack8(a));
  }
}

// proj row: ... | latent (column ccol, rank wide) | ... | up (column ucol, ff wide) | ...: the latent's RMS
// norm into the token's cache slot (wave 0 of the token's first workgroup), act[tok] = relu(up)^2
// (shared by the token's workgroups; vec: rows of whole 16-byte vectors).
template <typename T>
__global__ void __launch_bounds__(256) latent_prep_kernel(const T* __restrict__ proj, long ld, int ccol, int rank,
                                                          const float* __restrict__ w, float eps,
                                                          const int* __restrict__ slots, T* __restrict__ cache, int ucol,
                                                          int ff, T* __restrict__ act, long lda, int vec,
                                                          T* __restrict__ q, int nq, float qscale, T* __restrict__ zl, int zh) {
  // q (optional): the row's first nq columns times qscale, as rows of a matrix of their own
  const long tok = blockIdx.x;
  const int tid = threadIdx.x;
  const T* row = proj + tok * ld;
  const int slot = slots[tok];
  // zl (optional, [H, T, rank]): a padding token's rows, which no attention tile writes, are cleared
  if (zl && slot < 0)
    for (int i = blockIdx.y * 256 + tid; i < zh * rank; i += gridDim.y * 256)
      stf(zl + ((long)(i / rank) * gridDim.x + tok) * rank + i % rank, 0.f);
  if (blockIdx.y == 0 && tid < 64 && slot >= 0) {
    const T* r = row + ccol;
    float s = 0.f;
    for (int i = tid; i < rank; i += 64) { const float v = ldf(r + i); s += v * v; }
    const float rs = 1.f / sqrtf(wave_sum(s) / (float)rank + eps);
    T* dst = cache + (long)slot * rank;
    for (int i = tid; i < rank; i += 64) stf(dst + i, ldf(r + i) * rs * w[i]);
  }
  if (q)
    for (int i = blockIdx.y * 256 + tid; i < nq; i += gridDim.y * 256) stf(q + tok * nq + i, ldf(row + i) * qscale);
  if (!act) return;
  const T* up = row + ucol;
  T* a = act + tok * lda;
  if constexpr (sizeof(T) == 2) {
    if (vec) {
      for (int i = 8 * (blockIdx.y * 256 + tid); i < ff; i += 8 * gridDim.y * 256) {
        float f[8];
        unpack8(ld16(up + i), f);
#pragma unroll
        for (int x = 0; x < 8; ++x) { f[x] = fmaxf(f[x], 0.f); f[x] *= f[x]; }
        st16(a + i, pack8(f));
      }
      return;
    }
  }
  for (int i = blockIdx.y * 256 + tid; i < ff; i += gridDim.y * 256) {
    const float v = fmaxf(ldf(up + i), 0.f);
    stf(a + i, v * v);
  }
}

// Keys and values of one head from 64 cached latents (four pages of one sequence): K = C Wk^T, V = C Wv^T
// with C [64, rank] staged in LDS, Wk [H d, rank], Wv [H dv, rank] (rank % 32 == 0, d % 8 == 0).  A wave
// owns groups of NB 16-column blocks, first the key columns', then the value columns', over all 64 latents.
// Operands of v_mfma_f32_16x16x32_bf16 hold rows of either matrix alike (row lane & 15, contraction
// 8 (lane >> 4) ..), so keys are made as W C^T (four key dims of a latent per lane) and values as C W^T (four
// latents of a value dim per lane): both leave as 8-byte vectors.  Cache rows are [latent | rot rotated
// dims]; output pages: K [S nb, H, 16, d + rot] (the rotated dims copied behind every head's key), V
// [S nb, H, dv, 16], page (s, j) at s nb + j.
template <int NB>
__global__ void __launch_bounds__(256) latent_expand_kernel(const u16* __restrict__ cache, const int* __restrict__ bt, int bt_ld,
                                                            int nb, int pages, const int* __restrict__ ctx, int rank, int H,
                                                            int d, int dv, const u16* __restrict__ wk,
                                                            const u16* __restrict__ wv, u16* __restrict__ kc,
                                                            u16* __restrict__ vc, int rot) {
  extern __shared__ __attribute__((aligned(16))) unsigned char smx[];
  u16* csh = reinterpret_cast<u16*>(smx);      // [64][rank + 8]
  const int s = blockIdx.z, h = blockIdx.y, j0 = blockIdx.x * 4;
  if (j0 * 16 >= ctx[s]) return;               // nothing of the sequence lies here (uniform)
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int lr = lane & 15, g4 = lane >> 4;
  const int str = rank + 8, ch = rank >> 3, Dp = rank + rot, kd = d + rot;
  for (int e = tid; e < 64 * (rot >> 3); e += 256) {      // the shared rotated part (rot % 8 == 0)
    const int t = e / (rot >> 3), c = 8 * (e - t * (rot >> 3)), j = j0 + (t >> 4);
    if (j >= nb) continue;
    const int pg = bt[(long)s * bt_ld + j];
    uint4 v = make_uint4(0u, 0u, 0u, 0u);
    if (pg >= 0 && pg < pages) v = ld16(cache + ((long)pg * 16 + (t & 15)) * Dp + rank + c);
    st16(kc + ((((long)s * nb + j) * H + h) * 16 + (t & 15)) * kd + d + c, v);
  }
  for (int e = tid; e < 64 * ch; e += 256) {
    const int t = e / ch, c = e - t * ch, j = j0 + (t >> 4);
    uint4 v = make_uint4(0u, 0u, 0u, 0u);
    if (j < nb) {
      const int pg = bt[(long)s * bt_ld + j];
      if (pg >= 0 && pg < pages) v = ld16(cache + ((long)pg * 16 + (t & 15)) * Dp + 8 * c);
    }
    st16(csh + t * str + 8 * c, v);
  }
  __syncthreads();
  const int kblk = (d + 15) >> 4, vblk = (dv + 15) >> 4;
  const int kgr = (kblk + NB - 1) / NB, ngr = kgr + (vblk + NB - 1) / NB;
  for (int gi = wave; gi < ngr; gi += 4) {
    const bool key = gi < kgr;                 // wave-uniform
    const int b0 = (key ? gi : gi - kgr) * NB, cols = key ? d : dv;
    const u16* w = (key ? wk : wv) + (long)h * cols * rank;
    const u16* wp[NB];
#pragma unroll
    for (int b = 0; b < NB; ++b) wp[b] = w + (long)min((b0 + b) * 16 + lr, cols - 1) * rank + 8 * g4;   // rows past the end: any
    f32x4 acc[4][NB];
#pragma unroll
    for (int t = 0; t < 4; ++t)
#pragma unroll
      for (int b = 0; b < NB; ++b) acc[t][b] = f32x4{0.f, 0.f, 0.f, 0.f};
    const u16* cp = csh + lr * str + 8 * g4;
    if (key) {
#pragma unroll 2
      for (int k = 0; k < rank; k += 32) {
        bf16x8 wf[NB];
#pragma unroll
        for (int b = 0; b < NB; ++b) wf[b] = __builtin_bit_cast(bf16x8, ld16(wp[b] + k));
#pragma unroll
        for (int t = 0; t < 4; ++t) {
          const bf16x8 cf = __builtin_bit_cast(bf16x8, ld16(cp + 16 * t * str + k));
#pragma unroll
          for (int b = 0; b < NB; ++b) acc[t][b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf[b], cf, acc[t][b], 0, 0, 0);
        }
      }
    } else {
#pragma unroll 2
      for (int k = 0; k < rank; k += 32) {
        bf16x8 wf[NB];
#pragma unroll
        for (int b = 0; b < NB; ++b) wf[b] = __builtin_bit_cast(bf16x8, ld16(wp[b] + k));
#pragma unroll
        for (int t = 0; t < 4; ++t) {
          const bf16x8 cf = __builtin_bit_cast(bf16x8, ld16(cp + 16 * t * str + k));
#pragma unroll
          for (int b = 0; b < NB; ++b) acc[t][b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(cf, wf[b], acc[t][b], 0, 0, 0);
        }
      }
    }
#pragma unroll
    for (int t = 0; t < 4; ++t) {
      if (j0 + t >= nb) continue;
      const long page = ((long)s * nb + j0 + t) * H + h;
#pragma unroll
      for (int b = 0; b < NB; ++b) {
        const f32x4 a = acc[t][b];
        const uint2 v = make_uint2((uint32_t)f2bf(a[0]) | ((uint32_t)f2bf(a[1]) << 16), (uint32_t)f2bf(a[2]) | ((uint32_t)f2bf(a[3]) << 16));
        const int c0 = (b0 + b) * 16;
        if (key) {
          if (c0 + 4 * g4 < d) *reinterpret_cast<uint2*>(kc + (page * 16 + lr) * kd + c0 + 4 * g4) = v;
        } else {
          if (c0 + lr < dv) *reinterpret_cast<uint2*>(vc + (page * dv + c0 + lr) * 16 + 4 * g4) = v;
        }
      }
    }
  }
}

// out[t, h dv + i] = o[h, t, i] sigmoid(gate[t, h dv + i]), or gate[t, h] with `ghead`: x over the columns,
// y over the tokens
template <typename T>
__global__ void __launch_bounds__(256) gate_heads_kernel(const T* __restrict__ o, const T* __restrict__ gate, long ldg,
                                                         T* __restrict__ out, long ldo, int H, int dv, long Tn, int ghead) {
  const int c = blockIdx.x * 256 + threadIdx.x;
  if (c >= H * dv) return;
  const int h = c / dv, i = c - h * dv;
  for (long t = blockIdx.y; t < Tn; t += gridDim.y)
    stf(out + t * ldo + c, ldf(o + ((long)h * Tn + t) * dv + i) / (1.f + expf(-ldf(gate + t * ldg + (ghead ? h : c)))));
}

// ... for bf16 rows of whole 16-byte vectors (dv % 8 == 0): a thread owns 8 neighbouring entries of a head
__global__ void __launch_bounds__(256) gate_heads_vec_kernel(const u16* __restrict__ o, const u16* __restrict__ gate, long ldg,
                                                             u16* __restrict__ out, long ldo, int H, int dv, long Tn, int ghead) {
  const int c = 8 * (blockIdx.x * 256 + threadIdx.x);
  if (c >= H * dv) return;
  const int h = c / dv, i = c - h * dv;
  for (long t = blockIdx.y; t < Tn; t += gridDim.y) {
    float v[8], g[8];
    unpack8(ld16(o + ((long)h * Tn + t) * dv + i), v);
    if (ghead) {
      const float s = 1.f / (1.f + __expf(-bf2f(gate[t * ldg + h])));
#pragma unroll
      for (int x = 0; x < 8; ++x) v[x] *= s;
    } else {
      unpack8(ld16(gate + t * ldg + c), g);
#pragma unroll
      for (int x = 0; x < 8; ++x) v[x] *= __builtin_amdgcn_rcpf(1.f + __expf(-g[x]));
    }
    st16(out + t * ldo + c, pack8(v));
  }
}

constexpr int LROWS = 16;

// one cache row -> f32 in LDS, lanes along the row (bf16 rows of even length move 4 bytes per lane)
__device__ __forceinline__ void stage_row(const float* src, float* dst, int Dp, int lane) {
  for (int c = lane; c < Dp; c += 64) dst[c] = src[c];
}
__device__ __forceinline__ void stage_row(const u16* src, float* dst, int Dp, int lane) {
  if ((Dp & 1) == 0) {
    const uint32_t* s2 = reinterpret_cast<const uint32_t*>(src);
    for (int c = lane; c < (Dp >> 1); c += 64) {
      const uint32_t w = s2[c];
      dst[2 * c] = __uint_as_float(w << 16);
      dst[2 * c + 1] = __uint_as_float(w & 0xffff0000u);
    }
  } else {
    for (int c = lane; c < Dp; c += 64) dst[c] = bf2f(src[c]);
  }
}

// RI: latent dims per lane in phase 2 (rank <= 64 RI)
template <typename T, int RI>
__global__ void __launch_bounds__(256) latent_attention_kernel(
    const T* __restrict__ qa, const T* __restrict__ q, long ldq, int H, int dim, int rot, int rank, long Ttot,
    const float* __restrict__ cos_sin, int tab_w, const T* __restrict__ cache, const int* __restrict__ bt, int bt_w,
    const int* __restrict__ qstart, const int* __restrict__ qlen, const int* __restrict__ ctx,
    const int* __restrict__ tile_seq, const int* __restrict__ tile_tok0, float scale, T* __restrict__ out, int KT,
    int tpe, int kstride, int vec, int splits, float* __restrict__ part_o, float* __restrict__ part_ml, int hf,
    const float* __restrict__ sinks) {
  extern __shared__ float sm[];
  const int entry = blockIdx.y;
  const int s = tile_seq[entry];
  const int n = qlen[s];
  if (n <= 0) return;
  const int tok0 = tile_tok0[entry];
  if (tok0 >= n) return;
  const int ntok = min(tpe, n - tok0);
  const int nrows = ntok * H;                  // rows of this entry, token-major
  const int row0 = blockIdx.x * LROWS;
  if (row0 >= nrows) return;
  const int q0 = qstart[s], p0 = ctx[s] - n;
  const int Dp = rank + rot;
  float* qsh = sm;                              // [16][Dp]
  float* ksh = qsh + LROWS * Dp;                // [KT][kstride]
  float* psh = ksh + KT * kstride;              // [16][64]
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int half = rot >> 1;
  // stage the rows' queries (f32, scaled): latent part from qa [H, T, rank], rotated part from q
  for (int e = tid; e < LROWS * Dp; e += 256) {
    const int rr = e / Dp, c = e % Dp, row = row0 + rr;
    float v = 0.f;
    if (row < nrows) {
      const int tl = tok0 + row / H, h = row % H;
      const long tok = q0 + tl;
      if (c < rank) {
        v = ldf(qa + ((long)h * Ttot + tok) * rank + c);
      } else {
        v = rotated(q + tok * ldq + (long)h * (dim + rot) + dim, c - rank, half, hf, cos_sin + (long)(p0 + tl) * tab_w);
      }
      v *= scale;
    }
    qsh[e] = v;
  }
  // causal horizon of the block: the last row's position
  const int last_row = min(row0 + LROWS, nrows) - 1;
  const int kmax = p0 + tok0 + last_row / H + 1;
  int rpos[4];
  bool rok[4];
#pragma unroll
  for (int a = 0; a < 4; ++a) {
    const int row = row0 + wave * 4 + a;
    rok[a] = row < nrows;
    rpos[a] = p0 + tok0 + (rok[a] ? row / H : 0);
  }
  float m[4], l[4], acc[4][RI];
#pragma unroll
  for (int a = 0; a < 4; ++a) {
    m[a] = -INFINITY;
    l[a] = 0.f;
#pragma unroll
    for (int i = 0; i < RI; ++i) acc[a][i] = 0.f;
  }
  const int* btr = bt + (long)s * bt_w;
  // split over keys (small grids): split z of `splits` walks its share of the key tiles and leaves
  // unnormalised partials; latent_combine merges them
  const int ntiles = (kmax + KT - 1) / KT;
  const int kbeg = (int)((long)ntiles * blockIdx.z / splits) * KT;
  const int kend = min(kmax, (int)((long)ntiles * (blockIdx.z + 1) / splits) * KT);
  for (int k0 = kbeg; k0 < kend; k0 += KT) {
    const int nk = min(KT, kend - k0);
    __syncthreads();   // the previous tile is consumed (and the queries are staged)
    // the tile's pages: read once, so the row loads below do not each wait for a block-table entry
    const int pg0 = k0 >> 4, npg = ((k0 + nk - 1) >> 4) - pg0 + 1;
    const int pg = lane < npg ? btr[pg0 + lane] : 0;
#pragma unroll 4
    for (int kk = wave; kk < nk; kk += 4) {          // a wave per key row, lanes along the row
      const int kidx = k0 + kk;
      const long page = __shfl(pg, (kidx >> 4) - pg0);
      stage_row(cache + (page * 16 + (kidx & 15)) * Dp, ksh + kk * kstride, Dp, lane);
    }
    __syncthreads();
    // phase 1: lane = key
    float sc[4] = {0.f, 0.f, 0.f, 0.f};
    if (lane < nk) {
      const float* kr = ksh + lane * kstride;
      const float* qr = qsh + (wave * 4) * Dp;
      if (vec) {          // 16-byte LDS reads: rows are 16-byte aligned, kstride / 4 is odd (no bank conflicts)
#pragma unroll 8
        for (int c = 0; c < Dp; c += 4) {
          const float4 kv = *reinterpret_cast<const float4*>(kr + c);
#pragma unroll
          for (int a = 0; a < 4; ++a) {
            const float4 qv = *reinterpret_cast<const float4*>(qr + a * Dp + c);
            sc[a] += qv.x * kv.x + qv.y * kv.y + qv.z * kv.z + qv.w * kv.w;
          }
        }
      } else {
        for (int c = 0; c < Dp; ++c) {
          const float kv = kr[c];
#pragma unroll
          for (int a = 0; a < 4; ++a) sc[a] += qr[a * Dp + c] * kv;
        }
      }
    }
    float alpha[4];
#pragma unroll
    for (int a = 0; a < 4; ++a) {
      const bool vis = lane < nk && rok[a] && (k0 + lane) <= rpos[a];
      const float sv = vis ? sc[a] : -INFINITY;
      const float mn = fmaxf(m[a], wave_max(sv));
      float p = 0.f;
      alpha[a] = 1.f;
      if (mn != -INFINITY) {
        p = vis ? expf(sv - mn) : 0.f;
        alpha[a] = expf(m[a] - mn);     // m = -inf -> 0
        m[a] = mn;
      }
      l[a] = l[a] * alpha[a] + wave_sum(p);
      psh[(wave * 4 + a) * 64 + lane] = p;
    }
    __syncthreads();
    // phase 2: lane = latent dim
#pragma unroll
    for (int a = 0; a < 4; ++a)
#pragma unroll
      for (int i = 0; i < RI; ++i) acc[a][i] *= alpha[a];
#pragma unroll 4
    for (int kk = 0; kk < nk; ++kk) {
      float kv[RI];
#pragma unroll
      for (int i = 0; i < RI; ++i) {
        const int c = lane + 64 * i;
        kv[i] = c < rank ? ksh[kk * kstride + c] : 0.f;
      }
#pragma unroll
      for (int a = 0; a < 4; ++a) {
        const float p = psh[(wave * 4 + a) * 64 + kk];
#pragma unroll
        for (int i = 0; i < RI; ++i) acc[a][i] += p * kv[i];
      }
    }
  }
  if (splits > 1) {
#pragma unroll
    for (int a = 0; a < 4; ++a) {
      const long pr = (((long)entry * gridDim.x + blockIdx.x) * LROWS + wave * 4 + a) * splits + blockIdx.z;
      if (lane == 0) { part_ml[2 * pr] = m[a]; part_ml[2 * pr + 1] = l[a]; }
#pragma unroll
      for (int i = 0; i < RI; ++i) {
        const int c = lane + 64 * i;
        if (c < rank) part_o[pr * rank + c] = acc[a][i];
      }
    }
    return;
  }
#pragma unroll
  for (int a = 0; a < 4; ++a) {
    const int row = row0 + wave * 4 + a;
    if (row >= nrows) continue;
    const long tok = q0 + tok0 + row / H;
    const int h = row % H;
    const float inv = l[a] > 0.f ? 1.f / (l[a] + (sinks ? expf(sinks[h] - m[a]) : 0.f)) : 0.f;
#pragma unroll
    for (int i = 0; i < RI; ++i) {
      const int c = lane + 64 * i;
      if (c < rank) stf(out + ((long)h * Ttot + tok) * rank + c, acc[a][i] * inv);
    }
  }
}

// ---------------------------------------------------------------- bf16 models: matrix-core form
// Same row blocks, key tiles, causal mask, online softmax and key splits as above, with both products
// on v_mfma_f32_16x16x32_bf16 (operands bf16 from the cache, f32 accumulation):
//   scores   S[16 rows x 16 keys] per wave (wave w: keys 16w..16w+15 of the tile): A = query rows
//            (LDS, bf16, the rotation applied while staging, the score scale applied to the f32 sums),
//            B = key rows (LDS, row-major copy of the tile);
//   softmax  in the accumulator layout (a lane holds rows 4g..4g+3 of one key): row maxima by DPP
//            over the 16 lanes of a row group, then across the waves through LDS; a lane keeps a
//            partial row sum of its own keys until the end;
//   weights  written to LDS as bf16 hi + lo parts (p = hi + lo to 2^-17), so the second product sees
//            f32 weights to 16 bits of mantissa through two MFMAs;
//   output   O[16 rows x rank]: wave w owns latent column blocks w, w + 4, ...; A = weights (hi, lo),
//            B = a TRANSPOSED copy of the tile's latent part in LDS ([dim][key], made from the
//            row-major tile by a second pass), because the product contracts over keys and an operand
//            holds 8 consecutive contraction indices per lane.
__device__ __forceinline__ float row16_max(float v) {
  v = fmaxf(v, __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x128, 0xf, 0xf, false)));
  v = fmaxf(v, __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x124, 0xf, 0xf, false)));
  v = fmaxf(v, __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x122, 0xf, 0xf, false)));
  v = fmaxf(v, __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x121, 0xf, 0xf, false)));
  return v;
}
__device__ __forceinline__ float row16_add(float v) {
  v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x128, 0xf, 0xf, false));
  v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x124, 0xf, 0xf, false));
  v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x122, 0xf, 0xf, false));
  v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x121, 0xf, 0xf, false));
  return v;
}

struct MfmaLds { int Dpad, qstr, ktstr, pstr, RB; long bytes; };
static inline MfmaLds mfma_lds(int rank, int rot, int KT, int rows = LROWS) {
  MfmaLds L;
  L.Dpad = (rank + rot + 31) & ~31;
  L.qstr = L.Dpad + 8;
  L.ktstr = KT + 8;
  L.pstr = KT + 8;
  L.RB = (rank + 15) / 16;
  L.bytes = 2L * (rows * L.qstr + (long)KT * L.qstr + (long)L.RB * 16 * L.ktstr + 2L * rows * L.pstr) + 4L * 4 * rows;
  return L;
}

// A key tile's rows into registers: wave w takes rows w, w + 4, ..., a lane 16 bytes of a row (two per
// row cover up to 1024 entries); rows past `kend` and lanes past the row's end get zeros.
template <int KT>
__device__ __forceinline__ void fetch_tile(uint4 (&pf)[KT / 4][2], const u16* __restrict__ cache,
                                           const int* __restrict__ btr, int k0, int kend, int Dp, int lane, int wave) {
  const int nk = min(KT, kend - k0);
  const int pg0 = k0 >> 4, npg = ((k0 + nk - 1) >> 4) - pg0 + 1;
  const int pg = lane < npg ? btr[pg0 + lane] : 0;
#pragma unroll
  for (int r = 0; r < KT / 4; ++r) {
    const int kk = wave + 4 * r, kidx = k0 + kk;
    const bool live = kk < nk;
    const long page = __shfl(pg, live ? (kidx >> 4) - pg0 : 0);
    const uint4* src = reinterpret_cast<const uint4*>(cache + (page * 16 + (kidx & 15)) * Dp);
#pragma unroll
    for (int j = 0; j < 2; ++j) {
      const int c8 = lane + 64 * j;
      pf[r][j] = (live && c8 < (Dp >> 3)) ? src[c8] : make_uint4(0u, 0u, 0u, 0u);
    }
  }
}

// LR: 16-row blocks per workgroup (1: decode steps and short portions; 2: prompt portions, where the
// tile's staging, transposition and barriers then serve 32 rows and every wave has a score task at
// 32-key tiles).  Score tasks (row block, 16 keys) are dealt to the waves round-robin.
template <int CB, int KT, int LR>
__global__ void __launch_bounds__(256) latent_attention_mfma_kernel(
    const u16* __restrict__ qa, const u16* __restrict__ q, long ldq, int H, int dim, int rot, int rank, long Ttot,
    const float* __restrict__ cos_sin, int tab_w, const u16* __restrict__ cache, const int* __restrict__ bt, int bt_w,
    const int* __restrict__ qstart, const int* __restrict__ qlen, const int* __restrict__ ctx,
    const int* __restrict__ tile_seq, const int* __restrict__ tile_tok0, float scale, u16* __restrict__ out,
    int tpe, int splits, float* __restrict__ part_o, float* __restrict__ part_ml, int Dpad, int qstr, int ktstr,
    int pstr, int RB, int hf, const float* __restrict__ sinks) {
  constexpr int RPB = 16 * LR;                      // rows per workgroup
  constexpr int NKB = KT >> 4;                      // 16-key blocks per tile
  constexpr int NT = (LR * NKB + 3) / 4;            // score tasks per wave
  extern __shared__ __attribute__((aligned(16))) unsigned char smraw[];
  const int entry = blockIdx.y;
  const int s = tile_seq[entry];
  const int n = qlen[s];
  if (n <= 0) return;
  const int tok0 = tile_tok0[entry];
  if (tok0 >= n) return;
  const int ntok = min(tpe, n - tok0);
  const int nrows = ntok * H;
  const int row0 = blockIdx.x * RPB;
  if (row0 >= nrows) return;
  const int q0 = qstart[s], p0 = ctx[s] - n;
  const int Dp = rank + rot;
  u16* qsh = reinterpret_cast<u16*>(smraw);             // [RPB][qstr]
  u16* ksh = qsh + RPB * qstr;                          // [KT][qstr]
  u16* ktr = ksh + KT * qstr;                           // [RB * 16][ktstr]: latent part transposed
  u16* phi = ktr + RB * 16 * ktstr;                     // [RPB][pstr]
  u16* plo = phi + RPB * pstr;
  float* wred = reinterpret_cast<float*>(plo + RPB * pstr);   // [4][RPB]
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int lr = lane & 15, g = lane >> 4;
  const int half = rot >> 1;
  // queries: the latent part as 16-byte vectors where rows allow it, the rest (rotated part, padding) alone
  const int cs0 = (rank & 7) == 0 ? rank : 0;
  for (int e = tid; e < RPB * (cs0 >> 3); e += 256) {
    const int rr = e / (cs0 >> 3), c = 8 * (e - rr * (cs0 >> 3)), row = row0 + rr;
    uint4 v = make_uint4(0u, 0u, 0u, 0u);
    if (row < nrows) v = ld16(qa + ((long)(row % H) * Ttot + q0 + tok0 + row / H) * rank + c);
    st16(qsh + rr * qstr + c, v);
  }
  const int nrest = Dpad - cs0;
  for (int e = tid; e < RPB * nrest; e += 256) {
    const int rr = e / nrest, c = cs0 + e - rr * nrest, row = row0 + rr;
    float v = 0.f;
    if (row < nrows && c < Dp) {
      const int tl = tok0 + row / H, h = row % H;
      const long tok = q0 + tl;
      if (c < rank) {
        v = bf2f(qa[((long)h * Ttot + tok) * rank + c]);
      } else {
        v = rotated(q + tok * ldq + (long)h * (dim + rot) + dim, c - rank, half, hf, cos_sin + (long)(p0 + tl) * tab_w);
      }
    }
    qsh[rr * qstr + c] = f2bf(v);
  }
  // zero what no staging pass writes: the key rows' padded dims
  const int npad = Dpad - Dp;
  for (int e = tid; e < KT * npad; e += 256) ksh[(e / npad) * qstr + Dp + e % npad] = 0;
  const int last_row = min(row0 + RPB, nrows) - 1;
  const int kmax = p0 + tok0 + last_row / H + 1;
  int rpos[LR][4];
  bool rok[LR][4];
  float m[LR][4], l[LR][4];
  f32x4 acc[CB][LR];
#pragma unroll
  for (int b = 0; b < LR; ++b) {
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int row = row0 + 16 * b + 4 * g + i;
      rok[b][i] = row < nrows;
      rpos[b][i] = p0 + tok0 + (rok[b][i] ? row / H : 0);
      m[b][i] = -INFINITY;
      l[b][i] = 0.f;
    }
#pragma unroll
    for (int j = 0; j < CB; ++j) acc[j][b] = f32x4{0.f, 0.f, 0.f, 0.f};
  }
  const int* btr = bt + (long)s * bt_w;
  const int ntiles = (kmax + KT - 1) / KT;
  const int kbeg = (int)((long)ntiles * blockIdx.z / splits) * KT;
  const int kend = min(kmax, (int)((long)ntiles * (blockIdx.z + 1) / splits) * KT);
  // rows of a multiple of 8 entries (and at most 1024) move as 16-byte vectors, one tile ahead
  const bool pre = (Dp & 7) == 0 && Dp <= 1024;
  uint4 pf[KT / 4][2];
  if (pre && kbeg < kend) fetch_tile<KT>(pf, cache, btr, kbeg, kend, Dp, lane, wave);
  for (int k0 = kbeg; k0 < kend; k0 += KT) {
    const int nk = min(KT, kend - k0);
    __syncthreads();
    if (pre) {
      // this tile's rows were fetched into registers while the previous tile was computed; put them
      // in LDS and start the next tile's fetch, which the products below then hide
#pragma unroll
      for (int r = 0; r < KT / 4; ++r) {
        const int kk = wave + 4 * r;
#pragma unroll
        for (int j = 0; j < 2; ++j) {
          const int c8 = lane + 64 * j;
          if (c8 < (Dp >> 3)) *reinterpret_cast<uint4*>(ksh + kk * qstr + 8 * c8) = pf[r][j];
        }
      }
      if (k0 + KT < kend) fetch_tile<KT>(pf, cache, btr, k0 + KT, kend, Dp, lane, wave);
    } else {
      const int pg0 = k0 >> 4, npg = ((k0 + nk - 1) >> 4) - pg0 + 1;
      const int pg = lane < npg ? btr[pg0 + lane] : 0;
#pragma unroll
      for (int r = 0; r < KT / 4; ++r) {        // a wave per key row; rows past the tile's end are zeros
        const int kk = wave + 4 * r, kidx = k0 + kk;
        const bool live = kk < nk;
        const long page = __shfl(pg, live ? (kidx >> 4) - pg0 : 0);
        const uint32_t* src = reinterpret_cast<const uint32_t*>(cache + (page * 16 + (kidx & 15)) * Dp);
        for (int c2 = lane; c2 < (Dp >> 1); c2 += 64) {
          const uint32_t w = live ? src[c2] : 0u;
          *reinterpret_cast<uint32_t*>(ksh + kk * qstr + 2 * c2) = w;
        }
      }
    }
    __syncthreads();
    // the latent part once more, transposed ([dim][key]): threads along the dims read 8 keys' entries
    // (2-byte reads of consecutive halfwords) and write them as one 16-byte vector
    {
      const int ndim = RB * 16;
      for (int e = tid; e < ndim * (KT / 8); e += 256) {
        const int kg = e / ndim, c = e - kg * ndim;
        uint32_t w4[4] = {0u, 0u, 0u, 0u};
        if (c < rank) {
          const u16* col = ksh + (8 * kg) * qstr + c;
#pragma unroll
          for (int x = 0; x < 4; ++x)
            w4[x] = (uint32_t)col[(2 * x) * qstr] | ((uint32_t)col[(2 * x + 1) * qstr] << 16);
        }
        *reinterpret_cast<uint4*>(ktr + c * ktstr + 8 * kg) = make_uint4(w4[0], w4[1], w4[2], w4[3]);
      }
    }
    __syncthreads();
    // scores: task t of this wave is (row block, key block) number wave + 4 t
    float sv[NT][4];
    bool vis[NT][4];
    float wm[LR][4];
#pragma unroll
    for (int b = 0; b < LR; ++b)
#pragma unroll
      for (int i = 0; i < 4; ++i) wm[b][i] = -INFINITY;
#pragma unroll
    for (int t = 0; t < NT; ++t) {
      const int task = wave + 4 * t;
      const bool on = task < LR * NKB;
      const int rb = on ? task / NKB : 0, kb = on ? task % NKB : 0;
      f32x4 sacc = {0.f, 0.f, 0.f, 0.f};
      if (on) {
        const u16* ap = qsh + (16 * rb + lr) * qstr + 8 * g;
        const u16* bp = ksh + (16 * kb + lr) * qstr + 8 * g;
        for (int st = 0; st < Dpad; st += 32) {
          const bf16x8 a = __builtin_bit_cast(bf16x8, *reinterpret_cast<const uint4*>(ap + st));
          const bf16x8 b = __builtin_bit_cast(bf16x8, *reinterpret_cast<const uint4*>(bp + st));
          sacc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, sacc, 0, 0, 0);
        }
      }
      const int kidx = k0 + 16 * kb + lr;
#pragma unroll
      for (int b = 0; b < LR; ++b) {          // (static indexing of the per-row-block registers)
        if (b == rb) {
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            vis[t][i] = on && kidx < kend && rok[b][i] && kidx <= rpos[b][i];
            sv[t][i] = vis[t][i] ? sacc[i] * scale : -INFINITY;
            wm[b][i] = fmaxf(wm[b][i], row16_max(sv[t][i]));
          }
        }
      }
    }
    if (lr == 0) {
#pragma unroll
      for (int b = 0; b < LR; ++b)
#pragma unroll
        for (int i = 0; i < 4; ++i) wred[wave * RPB + 16 * b + 4 * g + i] = wm[b][i];
    }
    __syncthreads();
    float alpha[LR][4];
#pragma unroll
    for (int b = 0; b < LR; ++b)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int r = 16 * b + 4 * g + i;
        const float tm = fmaxf(fmaxf(wred[r], wred[RPB + r]), fmaxf(wred[2 * RPB + r], wred[3 * RPB + r]));
        const float mn = fmaxf(m[b][i], tm);
        alpha[b][i] = mn != -INFINITY ? expf(m[b][i] - mn) : 1.f;
        m[b][i] = mn;
        l[b][i] *= alpha[b][i];
      }
#pragma unroll
    for (int t = 0; t < NT; ++t) {
      const int task = wave + 4 * t;
      if (task < LR * NKB) {
        const int rb = task / NKB, kb = task % NKB;
#pragma unroll
        for (int b = 0; b < LR; ++b) {
          if (b == rb) {
#pragma unroll
            for (int i = 0; i < 4; ++i) {
              const float p = (vis[t][i] && m[b][i] != -INFINITY) ? expf(sv[t][i] - m[b][i]) : 0.f;
              l[b][i] += p;
              const u16 hi = f2bf(p);
              const int r = 16 * b + 4 * g + i;
              phi[r * pstr + 16 * kb + lr] = hi;
              plo[r * pstr + 16 * kb + lr] = f2bf(p - bf2f(hi));
            }
          }
        }
      }
    }
    __syncthreads();
    // weighted latents of this wave's column blocks
#pragma unroll
    for (int j = 0; j < CB; ++j) {
      const int cb = wave + 4 * j;
      if (cb < RB) {
#pragma unroll
        for (int b = 0; b < LR; ++b)
#pragma unroll
          for (int i = 0; i < 4; ++i) acc[j][b][i] *= alpha[b][i];
        const u16* bp = ktr + (cb * 16 + lr) * ktstr + 8 * g;
        for (int ks = 0; ks < KT; ks += 32) {
          const bf16x8 bv = __builtin_bit_cast(bf16x8, *reinterpret_cast<const uint4*>(bp + ks));
#pragma unroll
          for (int b = 0; b < LR; ++b) {
            const int ro = (16 * b + lr) * pstr + ks + 8 * g;
            const bf16x8 ah = __builtin_bit_cast(bf16x8, *reinterpret_cast<const uint4*>(phi + ro));
            const bf16x8 al = __builtin_bit_cast(bf16x8, *reinterpret_cast<const uint4*>(plo + ro));
            acc[j][b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ah, bv, acc[j][b], 0, 0, 0);
            acc[j][b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(al, bv, acc[j][b], 0, 0, 0);
          }
        }
      }
    }
  }
  // row sums: over the 16 lanes of a row group, then over the waves
  __syncthreads();
#pragma unroll
  for (int b = 0; b < LR; ++b)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const float t = row16_add(l[b][i]);
      if (lr == 0) wred[wave * RPB + 16 * b + 4 * g + i] = t;
    }
  __syncthreads();
#pragma unroll
  for (int b = 0; b < LR; ++b) {
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int r = 16 * b + 4 * g + i;
      const float lt = wred[r] + wred[RPB + r] + wred[2 * RPB + r] + wred[3 * RPB + r];
      if (splits > 1) {
        const long pr = (((long)entry * gridDim.x + blockIdx.x) * RPB + r) * splits + blockIdx.z;
        if (wave == 0 && lr == 0) { part_ml[2 * pr] = m[b][i]; part_ml[2 * pr + 1] = lt; }
#pragma unroll
        for (int j = 0; j < CB; ++j) {
          const int c = (wave + 4 * j) * 16 + lr;
          if (wave + 4 * j < RB && c < rank) part_o[pr * rank + c] = acc[j][b][i];
        }
      } else {
        const int row = row0 + r;
        if (row < nrows) {
          const long tok = q0 + tok0 + row / H;
          const int h = row % H;
          const float inv = lt > 0.f ? 1.f / (lt + (sinks ? expf(sinks[h] - m[b][i]) : 0.f)) : 0.f;
#pragma unroll
          for (int j = 0; j < CB; ++j) {
            const int c = (wave + 4 * j) * 16 + lr;
            if (wave + 4 * j < RB && c < rank) out[((long)h * Ttot + tok) * rank + c] = f2bf(acc[j][b][i] * inv);
          }
        }
      }
    }
  }
}

// one workgroup per (entry, row): merge the splits' (max, sum, weighted latent) partials.  Lane z of every
// wave holds split z's weight (splits <= 64), a thread owns latent dims tid, tid + 256, ...
template <typename T>
__global__ void __launch_bounds__(256) latent_combine_kernel(const float* __restrict__ part_o,
                                                             const float* __restrict__ part_ml, int splits, int gx,
                                                             int H, int rank, long Ttot, const int* __restrict__ qstart,
                                                             const int* __restrict__ qlen, const int* __restrict__ tile_seq,
                                                             const int* __restrict__ tile_tok0, int tpe,
                                                             T* __restrict__ out, int rpb,
                                                             const float* __restrict__ sinks) {
  const long r = blockIdx.x;
  const int tid = threadIdx.x, lane = tid & 63;
  const int rl = (int)(r % rpb);
  const long eb = r / rpb;
  const int bx = (int)(eb % gx), entry = (int)(eb / gx);
  const int s = tile_seq[entry];
  const int n = qlen[s], tok0 = tile_tok0[entry];
  if (n <= 0 || tok0 >= n) return;
  const int row = bx * rpb + rl;
  if (row >= min(tpe, n - tok0) * H) return;
  const float* ml = part_ml + 2 * r * splits;
  const float mz = lane < splits ? ml[2 * lane] : -INFINITY, lz = lane < splits ? ml[2 * lane + 1] : 0.f;
  const float M = wave_max(mz);
  const float ez = mz > -INFINITY ? expf(mz - M) : 0.f;
  float L = wave_sum(lz * ez);
  if (sinks && L > 0.f) L += expf(sinks[row % H] - M);
  const float wz = L > 0.f ? ez / L : 0.f;
  const long tok = qstart[s] + tok0 + row / H;
  const int h = row % H;
  const float* po = part_o + r * splits * rank;
  for (int c0 = 0; c0 < rank; c0 += 256) {     // every lane stays in the loop: the shuffles read all lanes
    const int c = c0 + tid;
    const bool on = c < rank;
    float o = 0.f;
#pragma unroll 8
    for (int z = 0; z < splits; ++z) {
      const float w = __shfl(wz, z, 64);
      if (on && w != 0.f) o += po[(long)z * rank + c] * w;     // a split that saw no key left nothing to read
    }
    if (on) stf(out + ((long)h * Ttot + tok) * rank + c, o);
  }
}

}  // namespace

extern "C" int dllm_latent_kv_write(const void* ckv, long ld, int f32, int rank, int rot, const float* w, float eps,
                                    const int* pos, const float* cos_sin, int tab_w, const int* slots, void* cache,
                                    int T, int hf, const void* qsrc, long ldqs, int qn, const float* qw, void* qdst, void* zl,
                                    int zh, hipStream_t st) {
  if (T <= 0) return 0;
  if (rot < 0 || (rot & 1) || rot > tab_w || rank < 1 || (qsrc && (qn < 1 || !qw || !qdst))) return -1;
  const dim3 block(qsrc ? 256 : 64);
  if (f32)
    hipLaunchKernelGGL(latent_kv_write_kernel<float>, dim3(T), block, 0, st, (const float*)ckv, ld, rank, rot, w, eps, pos,
                       cos_sin, tab_w, slots, (float*)cache, hf, (const float*)qsrc, ldqs, qn, qw, (float*)qdst, (float*)zl, zh);
  else
    hipLaunchKernelGGL(latent_kv_write_kernel<u16>, dim3(T), block, 0, st, (const u16*)ckv, ld, rank, rot, w, eps, pos,
                       cos_sin, tab_w, slots, (u16*)cache, hf, (const u16*)qsrc, ldqs, qn, qw, (u16*)qdst, (u16*)zl, zh);
  return (int)hipGetLastError();
}

extern "C" int dllm_latent_q_prep(const void* q, long ldq, int f32, int H, int dim, int rot, int hf, const int* pos,
                                  const float* cos_sin, int tab_w, float scale, void* out, long T, hipStream_t st) {
  if (T <= 0) return 0;
  if (H < 1 || dim < 0 || rot < 0 || (rot & 1) || rot > tab_w || dim + rot < 1) return -1;
  if (!f32 && (hf || !rot) && dim % 8 == 0 && rot % 16 == 0 && ldq % 8 == 0 && (uintptr_t)q % 16 == 0 && (uintptr_t)out % 16 == 0) {
    const int units = H * ((dim + rot / 2) / 8);
    hipLaunchKernelGGL(latent_q_prep_vec_kernel, dim3((units + 255) / 256, (unsigned)(T < 4096 ? T : 4096)), dim3(256), 0, st,
                       (const u16*)q, ldq, H, dim, rot, pos, cos_sin, tab_w, scale, (u16*)out, T);
    return (int)hipGetLastError();
  }
  const dim3 grid((H * (dim + rot) + 255) / 256, (unsigned)(T < 4096 ? T : 4096));
  if (f32)
    hipLaunchKernelGGL(latent_q_prep_kernel<float>, grid, dim3(256), 0, st, (const float*)q, ldq, H, dim, rot, hf, pos, cos_sin,
                       tab_w, scale, (float*)out, T);
  else
    hipLaunchKernelGGL(latent_q_prep_kernel<u16>, grid, dim3(256), 0, st, (const u16*)q, ldq, H, dim, rot, hf, pos, cos_sin,
                       tab_w, scale, (u16*)out, T);
  return (int)hipGetLastError();
}

namespace {
template <typename T>
int launch_latent(int ri, dim3 g, long lds, hipStream_t st, const T* qa, const T* q, long ldq, int H, int dim, int rot,
                  int rank, long Ttot, const float* cos_sin, int tab_w, const T* cache, const int* bt, int bt_w,
                  const int* qstart, const int* qlen, const int* ctx, const int* tile_seq, const int* tile_tok0,
                  float scale, T* out, int KT, int tpe, int kstride, int vec, int splits, float* part_o, float* part_ml, int hf,
                  const float* sinks) {
#define LAT(RI)                                                                                                        \
  do {                                                                                                                 \
    static long have_ = 48 * 1024; /* raised once per size: no attribute call inside a later stream capture */        \
    if (lds > have_) {                                                                                                 \
      hipFuncSetAttribute((const void*)latent_attention_kernel<T, RI>, hipFuncAttributeMaxDynamicSharedMemorySize,    \
                          (int)lds);                                                                                   \
      have_ = lds;                                                                                                     \
    }                                                                                                                  \
    hipLaunchKernelGGL((latent_attention_kernel<T, RI>), g, dim3(256), lds, st, qa, q, ldq, H, dim, rot, rank, Ttot,   \
                       cos_sin, tab_w, cache, bt, bt_w, qstart, qlen, ctx, tile_seq, tile_tok0, scale, out, KT, tpe,   \
                       kstride, vec, splits, part_o, part_ml, hf, sinks);                                              \
  } while (0)
  if (ri <= 1) LAT(1); else if (ri <= 2) LAT(2); else if (ri <= 4) LAT(4); else LAT(8);
#undef LAT
  if (splits > 1) {
    const long n_rows = (long)g.y * g.x * LROWS;
    hipLaunchKernelGGL(latent_combine_kernel<T>, dim3((unsigned)n_rows), dim3(256), 0, st, part_o, part_ml, splits, (int)g.x, H,
                       rank, Ttot, qstart, qlen, tile_seq, tile_tok0, tpe, out, LROWS, sinks);
  }
  return (int)hipGetLastError();
}
}  // namespace

namespace {
int launch_latent_mfma(dim3 g, hipStream_t st, const u16* qa, const u16* q, long ldq, int H, int dim, int rot, int rank,
                       long Ttot, const float* cos_sin, int tab_w, const u16* cache, const int* bt, int bt_w,
                       const int* qstart, const int* qlen, const int* ctx, const int* tile_seq, const int* tile_tok0,
                       float scale, u16* out, int KT, int tpe, int splits, float* part_o, float* part_ml, int rows, int hf,
                       const float* sinks) {
  const MfmaLds L = mfma_lds(rank, rot, KT, rows);
  const int cbs = (L.RB + 3) / 4;
#define LATM3(CB, KTC, LRC)                                                                                                 \
  do {                                                                                                                 \
    static long have_ = 48 * 1024;                                                                                     \
    if (L.bytes > have_) {                                                                                             \
      hipFuncSetAttribute((const void*)latent_attention_mfma_kernel<CB, KTC, LRC>,                                     \
                          hipFuncAttributeMaxDynamicSharedMemorySize, (int)L.bytes);                                   \
      have_ = L.bytes;                                                                                                 \
    }                                                                                                                  \
    hipLaunchKernelGGL((latent_attention_mfma_kernel<CB, KTC, LRC>), g, dim3(256), L.bytes, st, qa, q, ldq, H, dim, rot, \
                       rank, Ttot, cos_sin, tab_w, cache, bt, bt_w, qstart, qlen, ctx, tile_seq, tile_tok0, scale, out, \
                       tpe, splits, part_o, part_ml, L.Dpad, L.qstr, L.ktstr, L.pstr, L.RB, hf, sinks);                \
  } while (0)
#define LATM2(CB, KTC)                                                                                                 \
  do {                                                                                                                 \
    if (rows == 32) LATM3(CB, KTC, 2); else LATM3(CB, KTC, 1);                                                         \
  } while (0)
#define LATM(CB)                                                                                                       \
  do {                                                                                                                 \
    if (KT == 64) LATM2(CB, 64); else LATM2(CB, 32);                                                                   \
  } while (0)
  if (cbs <= 1) LATM(1); else if (cbs <= 2) LATM(2); else if (cbs <= 4) LATM(4); else LATM(8);
#undef LATM
#undef LATM2
#undef LATM3
  if (splits > 1) {
    const long n_rows = (long)g.y * g.x * rows;
    hipLaunchKernelGGL(latent_combine_kernel<u16>, dim3((unsigned)n_rows), dim3(256), 0, st, part_o, part_ml, splits, (int)g.x, H,
                       rank, Ttot, qstart, qlen, tile_seq, tile_tok0, tpe, out, rows, sinks);
  }
  return (int)hipGetLastError();
}
}  // namespace

// 1 when the matrix-core kernel takes this shape with `rows` (16 or 32) rows per workgroup (bf16, even
// widths, a 32-key tile fits the LDS)
extern "C" int dllm_latent_mfma_ok(int rank, int rot, int rows) {
  if ((rank & 1) || (rot & 1) || rank < 2 || rank > 512 || (rows != 16 && rows != 32)) return 0;
  return mfma_lds(rank, rot, 32, rows).bytes <= 150 * 1024;
}

extern "C" int dllm_latent_attention(const void* qa, const void* q, long ldq, int f32, int H, int dim, int rot, int rank,
                                     long Ttot, const float* cos_sin, int tab_w, const void* cache, const int* bt,
                                     int bt_w, const int* qstart, const int* qlen, const int* ctx, const int* tile_seq,
                                     const int* tile_tok0, int n_entries, float scale, void* out, int splits,
                                     float* part_o, float* part_ml, int mfma, int rows, int hf, const float* sinks,
                                     hipStream_t st) {
  if (n_entries <= 0 || Ttot <= 0) return 0;
  if (rank < 1 || rank > 512 || rot < 0 || (rot & 1) || rot > tab_w || H < 1) return -1;
  if (splits < 1 || (splits > 1 && (!part_o || !part_ml))) return -3;
  if (mfma && !f32 && dllm_latent_mfma_ok(rank, rot, rows)) {
    const int KTm = mfma_lds(rank, rot, 64, rows).bytes <= 150 * 1024 ? 64 : 32;
    const int tpe_m = H >= rows ? 1 : rows / H;
    const dim3 gm((tpe_m * H + rows - 1) / rows, n_entries, splits);
    return launch_latent_mfma(gm, st, (const u16*)qa, (const u16*)q, ldq, H, dim, rot, rank, Ttot, cos_sin, tab_w,
                              (const u16*)cache, bt, bt_w, qstart, qlen, ctx, tile_seq, tile_tok0, scale, (u16*)out, KTm,
                              tpe_m, splits, part_o, part_ml, rows, hf, sinks);
  }
  if (rows != LROWS) return -4;   // only the matrix-core kernel has the 32-row form
  // key rows in LDS: an odd stride for 4-byte reads; when the row length is a multiple of 4 a stride
  // that is 4 x odd, so a lane's 16-byte reads are aligned and spread over all banks
  const int Dp = rank + rot, vec = (Dp & 3) == 0;
  const int kstride = vec ? (((Dp >> 2) & 1) ? Dp : Dp + 4) : (Dp | 1);
  int KT = 64;
  while (KT > 8 && 4L * (LROWS * Dp + (long)KT * kstride + LROWS * 64) > 140 * 1024) KT >>= 1;
  const long lds = 4L * (LROWS * Dp + (long)KT * kstride + LROWS * 64);
  if (lds > 150 * 1024) return -2;
  const int tpe = H >= 16 ? 1 : 16 / H;
  if (splits < 1 || (splits > 1 && (!part_o || !part_ml))) return -3;
  const dim3 g((tpe * H + LROWS - 1) / LROWS, n_entries, splits);
  const int ri = (rank + 63) / 64;
  if (f32)
    return launch_latent<float>(ri, g, lds, st, (const float*)qa, (const float*)q, ldq, H, dim, rot, rank, Ttot, cos_sin,
                                tab_w, (const float*)cache, bt, bt_w, qstart, qlen, ctx, tile_seq, tile_tok0, scale,
                                (float*)out, KT, tpe, kstride, vec, splits, part_o, part_ml, hf, sinks);
  return launch_latent<u16>(ri, g, lds, st, (const u16*)qa, (const u16*)q, ldq, H, dim, rot, rank, Ttot, cos_sin, tab_w,
                            (const u16*)cache, bt, bt_w, qstart, qlen, ctx, tile_seq, tile_tok0, scale, (u16*)out, KT, tpe, kstride, vec, splits, part_o, part_ml, hf,
                            sinks);
}

extern "C" int dllm_latent_prep(const void* proj, long ld, int f32, int ccol, int rank, const float* w, float eps,
                                const int* slots, void* cache, int ucol, int ff, void* act, long lda, void* q, int nq,
                                float qscale, void* zl, int zh, long T, hipStream_t st) {
  if (T <= 0) return 0;
  if (rank < 1 || (act && ff < 1)) return -1;
  const dim3 grid((unsigned)T, act ? (ff + 2047) / 2048 : 1);
  const int vec = act && !f32 && ff % 8 == 0 && ucol % 8 == 0 && ld % 8 == 0 && lda % 8 == 0 && (uintptr_t)proj % 16 == 0 &&
                  (uintptr_t)act % 16 == 0;
  if (f32)
    hipLaunchKernelGGL(latent_prep_kernel<float>, grid, dim3(256), 0, st, (const float*)proj, ld, ccol, rank, w, eps, slots,
                       (float*)cache, ucol, ff, (float*)act, lda, vec, (float*)q, nq, qscale, (float*)zl, zh);
  else
    hipLaunchKernelGGL(latent_prep_kernel<u16>, grid, dim3(256), 0, st, (const u16*)proj, ld, ccol, rank, w, eps, slots,
                       (u16*)cache, ucol, ff, (u16*)act, lda, vec, (u16*)q, nq, qscale, (u16*)zl, zh);
  return (int)hipGetLastError();
}

extern "C" int dllm_gate_heads(const void* o, int f32, const void* gate, long ldg, void* out, long ldo, int H, int dv, long T,
                               int ghead, hipStream_t st) {
  if (T <= 0) return 0;
  if (H < 1 || dv < 1) return -1;
  if (!f32 && dv % 8 == 0 && ldo % 8 == 0 && (uintptr_t)o % 16 == 0 && (uintptr_t)out % 16 == 0 &&
      (ghead || (ldg % 8 == 0 && (uintptr_t)gate % 16 == 0))) {
    hipLaunchKernelGGL(gate_heads_vec_kernel, dim3((H * dv / 8 + 255) / 256, (unsigned)(T < 4096 ? T : 4096)), dim3(256), 0, st,
                       (const u16*)o, (const u16*)gate, ldg, (u16*)out, ldo, H, dv, T, ghead);
    return (int)hipGetLastError();
  }
  const dim3 grid((H * dv + 255) / 256, (unsigned)(T < 4096 ? T : 4096));
  if (f32)
    hipLaunchKernelGGL(gate_heads_kernel<float>, grid, dim3(256), 0, st, (const float*)o, (const float*)gate, ldg, (float*)out,
                       ldo, H, dv, T, ghead);
  else
    hipLaunchKernelGGL(gate_heads_kernel<u16>, grid, dim3(256), 0, st, (const u16*)o, (const u16*)gate, ldg, (u16*)out, ldo, H,
                       dv, T, ghead);
  return (int)hipGetLastError();
}

// 1 when latent_expand takes the shape (bf16; the 64 latents of a workgroup fit the LDS)
extern "C" int dllm_latent_expand_ok(int rank, int d, int dv, int rot) {
  return rank >= 32 && rank % 32 == 0 && rank <= 1024 && d >= 8 && d % 8 == 0 && dv >= 1 && rot >= 0 && rot % 8 == 0;
}

extern "C" int dllm_latent_expand(const void* cache, const int* bt, int bt_ld, int S, int nb, int pages, const int* ctx, int rank,
                                  int H, int d, int dv, const void* wk, const void* wv, void* kc, void* vc, int rot,
                                  hipStream_t st) {
  if (S <= 0 || nb <= 0) return 0;
  if (!dllm_latent_expand_ok(rank, d, dv, rot) || H < 1 || S > 65535 || H > 65535) return -1;
  const long lds = 64L * (rank + 8) * 2;
  const dim3 grid((nb + 3) / 4, H, S);
#define LEX(NB)                                                                                                        \
  do {                                                                                                                 \
    static long have_ = 48 * 1024;                                                                                     \
    if (lds > have_) {                                                                                                 \
      hipFuncSetAttribute((const void*)latent_expand_kernel<NB>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds); \
      have_ = lds;                                                                                                     \
    }                                                                                                                  \
    hipLaunchKernelGGL(latent_expand_kernel<NB>, grid, dim3(256), lds, st, (const u16*)cache, bt, bt_ld, nb, pages, ctx, rank, H, \
                       d, dv, (const u16*)wk, (const u16*)wv, (u16*)kc, (u16*)vc, rot);                                \
  } while (0)
  if (d >= 128 && dv >= 128) LEX(4); else if (d >= 64 || dv >= 64) LEX(2); else LEX(1);
#undef LEX
  return (int)hipGetLastError();
}
