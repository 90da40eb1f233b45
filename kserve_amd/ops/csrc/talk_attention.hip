// Softmax attention against the paged cache whose scores are mixed over the
// heads before the softmax, in fp32 end to end:
//
//   score_g(i, j) = q_g(i) . k(j) * k_scale(j) * scale
//   s_h = sum_g talk[h, g] score_g + bias[h, i - j]
//   p   = exp(s_h) / (1 + sum exp(s_h))     (keys 0 <= i - j < window)
//   o_h = sum_j p_j k(j), times sigmoid(gate) per element
//
// Pages hold the un-normed keys, which are the values too, and one factor per
// row (1/rms of the whole key projection). `bias` [heads, n] is already mixed
// over the heads and constant past distance n - 1.
//
//  * talk_prep_cache: whole-row RMS norm of the query projection times a weight
//    (fp32 out), keys to the pages, 1/rms of the key row to k_scale.
//  * talk_attention prefill: a block takes 16 consecutive tokens and ALL heads,
//    8 waves. Per tile of 16 NKT keys: (1) every wave computes its heads'
//    transposed scores S^T = K Q^T on the fp32 matrix cores
//    (v_mfma_f32_16x16x4_f32; keys and queries straight from the caches, 64
//    contiguous bytes per row and load) into LDS [head][key][query];
//    (2) every wave takes some keys and mixes over the heads, in place: per key
//    a [heads x heads] x [heads x 16 queries] product, again on the matrix
//    cores; (3) every wave reads its heads' mixed scores back in accumulator
//    layout (one query per lane column), adds the bias, masks, updates the
//    running softmax and multiplies with the keys as values, whose weights
//    never leave the registers. A wave works on NH heads at once; SHARE: they
//    belong to one key group, so every key fragment is loaded once for all.
//    Loads run ahead of the products that use them.
//    More heads than 8 NH: further blocks (grid z) take the next ones and
//    recompute the scores of all heads.
//  * talk_attention decode (one token per sequence): a block takes one split
//    of the sequence's keys, all heads: the heads of a key group are the
//    matrix product's columns, 64 keys per tile; the mixed scores go through
//    a [heads x heads] x [heads x 16 keys] product, the softmax runs with one
//    key per lane. Partial results go to scratch; talk_merge_kernel combines
//    the splits, adds the 1 of the denominator and applies the gate.
#include "cache_chunk.h"

namespace {

constexpr int NT = 512;
constexpr int NWV = NT / WAVE_SIZE;
constexpr int QS = 20;  // floats per key row of a score tile (16 queries + pad)
constexpr float LOG2E = 1.44269504088896340736f;

template <typename T>
__global__ void __launch_bounds__(256) talk_prep_cache_kernel(
    float* __restrict__ q_out, const T* __restrict__ q, long q_stride,
    const T* __restrict__ k, long k_stride, const float* __restrict__ w,
    const int* __restrict__ slot_mapping, T* __restrict__ k_cache,
    float* __restrict__ k_scale, float eps, int q_width, int kv_heads, int D,
    int block_size, int vec) {
  __shared__ float scratch[4];
  const long t = blockIdx.x;
  const T* qr = q + t * q_stride;
  const T* kr = k + t * k_stride;
  const int k_width = kv_heads * D;
  float sq = 0.f, sk = 0.f;
  for (int i = threadIdx.x * 4; i < q_width; i += 1024) {
    const f32x4 x = load4_f32(qr + i, vec, q_width - i);
    sq += x[0] * x[0] + x[1] * x[1] + x[2] * x[2] + x[3] * x[3];
  }
  for (int i = threadIdx.x * 4; i < k_width; i += 1024) {
    const f32x4 x = load4_f32(kr + i, vec, k_width - i);
    sk += x[0] * x[0] + x[1] * x[1] + x[2] * x[2] + x[3] * x[3];
  }
  sq = block_sum_sync<4>(sq, scratch);
  sk = block_sum_sync<4>(sk, scratch);
  const float qinv = 1.0f / sqrtf(sq / (float)q_width + eps);
  for (int i = threadIdx.x * 4; i < q_width; i += 1024) {
    const f32x4 x = load4_f32(qr + i, vec, q_width - i);
    const f32x4 ww = load4_f32(w + i, vec, q_width - i);
    if (vec) {
      *reinterpret_cast<f32x4*>(q_out + t * q_width + i) = x * ww * qinv;
    } else {
      for (int c = 0; c < 4; ++c)
        if (i + c < q_width) q_out[t * q_width + i + c] = x[c] * ww[c] * qinv;
    }
  }
  const long slot = slot_mapping[t];
  if (slot < 0) return;
  const long blk = slot / block_size, off = slot % block_size;
  if (threadIdx.x == 0)
    k_scale[blk * block_size + off] = 1.0f / sqrtf(sk / (float)k_width + eps);
  for (int i = threadIdx.x; i < k_width; i += 256) {
    const int g = i / D, d = i % D;
    k_cache[((blk * kv_heads + g) * block_size + off) * D + d] = kr[i];
  }
}

// loads of the first (contraction) and second (values) product; FULL: heads of
// exactly the padded width in aligned rows, no guards around the loads
template <bool FULL, typename T>
__device__ __forceinline__ void load_chunk(Chunk8<T>& c, const T* p, bool vec,
                                           int valid) {
  if constexpr (FULL) {
    c.load(p, true, 8);
  } else {
    if (valid > 0) c.load(p, vec, valid);
    else c.zero();
  }
}
// four values kept in the cache dtype until they are used
template <typename T>
struct Quad;
template <>
struct Quad<short> {
  short4_t x;
  __device__ __forceinline__ float get(int i) const { return bf16_bits_to_float(x[i]); }
};
template <>
struct Quad<float> {
  f32x4 x;
  __device__ __forceinline__ float get(int i) const { return x[i]; }
};
template <bool FULL, typename T>
__device__ __forceinline__ void load_quad(Quad<T>& q, const T* p, bool vec, int valid) {
  if (FULL || (vec && valid >= 4)) {
    q.x = *reinterpret_cast<const decltype(q.x)*>(p);
  } else {
#pragma unroll
    for (int i = 0; i < 4; ++i) q.x[i] = i < valid ? p[i] : (T)0;
  }
}

// Cache row (of kv head 0) and score factor of a tile's keys, one key per
// thread, in steps so that the dependent loads of the next tile hide behind
// this tile's work: find(), then load(), then store() to LDS. Keys past
// `last` repeat the last one (masked later).
struct KeyRows {
  int blk, po;
  float f;
  __device__ __forceinline__ void find(int k0, int last, int count, const int* bt,
                                       int block_size) {
    if ((int)threadIdx.x < count) {
      const int kp = min(k0 + (int)threadIdx.x, last);
      blk = bt[kp / block_size];
      po = kp % block_size;
    }
  }
  __device__ __forceinline__ void load(int count, int block_size,
                                       const float* k_scale) {
    if ((int)threadIdx.x < count) f = k_scale[(long)blk * block_size + po];
  }
  __device__ __forceinline__ void store(int* rows, float* ksc, int count,
                                        int block_size, int kv_heads,
                                        float mult) const {
    if ((int)threadIdx.x < count) {
      rows[threadIdx.x] = blk * kv_heads * block_size + po;
      ksc[threadIdx.x] = f * mult;
    }
  }
};

// 16-key tiles per step of the prefill kernel: two where the registers (heads
// of a wave times the head size) and the LDS (heads) allow
constexpr int key_tiles(int DP, int NH, int HT) {
  return HT <= 2 && DP * NH < 512 ? 2 : 1;
}

// LDS floats of the prefill kernel: scores [H4][16 NKT][QS] | talk^T [H4][16 HT]
// | rows [2][16 NKT] | factors [2][16 NKT]
template <typename T, int DP, int NH, int HT, bool SHARE, bool FULL>
__global__ void __launch_bounds__(NT) talk_prefill_kernel(
    T* __restrict__ out, const float* __restrict__ q,
    const T* __restrict__ k_cache, const float* __restrict__ k_scale,
    const int* __restrict__ block_tables, int bt_stride,
    const int* __restrict__ cu_q, const int* __restrict__ ctx_lens,
    const float* __restrict__ talk, const float* __restrict__ bias, int bias_n,
    const T* __restrict__ gate, long gate_stride, float scale, int heads,
    int kv_heads, int D, int block_size, int window) {
  constexpr int NKT = key_tiles(DP, NH, HT);
  constexpr int BK = 16 * NKT;
  extern __shared__ float lds[];
  const int H4 = (heads + 3) & ~3;
  float* S = lds;
  float* Tt = S + H4 * BK * QS;
  float* Ksc = Tt + H4 * 16 * HT;
  int* Rows = reinterpret_cast<int*>(Ksc + 2 * BK);

  const int s = blockIdx.y;
  const int q0 = cu_q[s];
  const int q_len = cu_q[s + 1] - q0;
  const int tok0 = blockIdx.x * 16;
  if (tok0 >= q_len) return;
  const int nq = min(16, q_len - tok0);
  const int base_pos = ctx_lens[s] - q_len + tok0;
  const int last_pos = base_pos + nq - 1;
  const int kbeg = window > 0 ? max(base_pos - window + 1, 0) : 0;
  const int lane = threadIdx.x & 63;
  const int wave = threadIdx.x >> 6;
  const int li = lane & 15, lg = lane >> 4;
  const int rep = heads / kv_heads;
  const int items = (heads + NH - 1) / NH;
  const int* bt = block_tables + (long)s * bt_stride;
  const bool vec = (D % 8) == 0;
  const float mult = scale * LOG2E;
  const int qpos = li < nq ? base_pos + li : -1;
  const int qstart = window > 0 ? qpos - window + 1 : 0;
  const float* qrow = q + (long)(q0 + tok0 + min(li, nq - 1)) * heads * D;

  for (int e = threadIdx.x; e < H4 * 16 * HT; e += NT) {
    const int g = e / (16 * HT), h = e % (16 * HT);
    Tt[e] = (g < heads && h < heads) ? talk[h * heads + g] : 0.f;
  }
  for (int e = heads * BK * QS + threadIdx.x; e < H4 * BK * QS; e += NT) S[e] = 0.f;
  KeyRows kr;
  kr.find(kbeg, last_pos, BK, bt, block_size);
  kr.load(BK, block_size, k_scale);
  kr.store(Rows, Ksc, BK, block_size, kv_heads, mult);

  // this wave's heads in steps (1) and (3) when one block covers all heads;
  // otherwise step (1) walks all of them and step (3) takes this block's
  const int item3 = blockIdx.z * NWV + wave;
  f32x4 o[NH][DP / 16];
  float m[NH], l[NH];
#pragma unroll
  for (int a = 0; a < NH; ++a) {
    m[a] = -INFINITY;
    l[a] = 0.f;
#pragma unroll
    for (int i = 0; i < DP / 16; ++i) o[a][i] = f32x4{0.f, 0.f, 0.f, 0.f};
  }
  __syncthreads();

  int buf = 0;
  for (int k0 = kbeg; k0 <= last_pos; k0 += BK, buf ^= 1) {
    const int* rows = Rows + buf * BK;
    const float* ksc = Ksc + buf * BK;
    kr.find(k0 + BK, last_pos, BK, bt, block_size);
    // (1) scores of all heads
    for (int item = wave; item < items; item += NWV) {
      int hh[NH];
#pragma unroll
      for (int a = 0; a < NH; ++a) hh[a] = min(item * NH + a, heads - 1);
      f32x4 acc[NH][NKT];
#pragma unroll
      for (int a = 0; a < NH; ++a)
#pragma unroll
        for (int t = 0; t < NKT; ++t) acc[a][t] = f32x4{0.f, 0.f, 0.f, 0.f};
      long krow[NKT];
#pragma unroll
      for (int t = 0; t < NKT; ++t) krow[t] = rows[16 * t + li];
      // Steps (k8, head) in order, the query fragment two steps ahead and the
      // key fragments one k8 ahead of their products. Contraction step c of
      // lane group lg stands for d = 32 k8 + 8 lg + c.
      constexpr int K8 = DP / 32, STEPS = K8 * NH, KB = SHARE ? 1 : NH;
      constexpr int KR = SHARE ? 2 : 1;  // key fragments in flight
      Chunk8<T> kf[KR][KB][NKT];
      Chunk8<float> qf[3];
      auto load_k = [&](int k8) {
        const int d0 = 32 * k8 + 8 * lg;
#pragma unroll
        for (int a = 0; a < KB; ++a) {
          const int g = hh[a] / rep;
#pragma unroll
          for (int t = 0; t < NKT; ++t)
            load_chunk<FULL>(kf[k8 % KR][a][t],
                             k_cache + (krow[t] + (long)g * block_size) * D + d0, vec,
                             D - d0);
        }
      };
      auto load_q = [&](int step) {
        const int d0 = 32 * (step / NH) + 8 * lg;
        load_chunk<FULL>(qf[step % 3], qrow + hh[step % NH] * D + d0, vec, D - d0);
      };
      load_k(0);
      load_q(0);
      if (STEPS > 1) load_q(1);
      f32x4 kfac[NKT];
#pragma unroll
      for (int t = 0; t < NKT; ++t)
        kfac[t] = *reinterpret_cast<const f32x4*>(ksc + 16 * t + 4 * lg);
#pragma unroll
      for (int st = 0; st < STEPS; ++st) {
        const int a = st % NH, k8 = st / NH;
        if (a == 0 && KR == 2 && k8 + 1 < K8) load_k(k8 + 1);
        if (a == 0 && KR == 1 && k8 > 0) load_k(k8);
        if (st + 2 < STEPS) load_q(st + 2);
        // keep the loads ahead of this step's products
        __builtin_amdgcn_sched_barrier(0);
#pragma unroll
        for (int c = 0; c < 8; ++c)
#pragma unroll
          for (int t = 0; t < NKT; ++t)
            acc[a][t] = __builtin_amdgcn_mfma_f32_16x16x4f32(
                kf[k8 % KR][SHARE ? 0 : a][t].get(c), qf[st % 3].get(c), acc[a][t], 0,
                0, 0);
      }
#pragma unroll
      for (int a = 0; a < NH; ++a) {
        if (item * NH + a < heads) {
#pragma unroll
          for (int t = 0; t < NKT; ++t)
#pragma unroll
            for (int v = 0; v < 4; ++v) {
              const int key = 16 * t + 4 * lg + v;
              S[(hh[a] * BK + key) * QS + li] = acc[a][t][v] * kfac[t][v];
            }
        }
      }
    }
    kr.load(BK, block_size, k_scale);
    __syncthreads();
    // (2) mix over the heads, in place: the wave reads its keys' scores of all
    // heads before it writes any
    {
      constexpr int KPW = BK / NWV;  // keys of a wave: wave * KPW ...
      f32x4 mx[KPW][HT];
#pragma unroll
      for (int k = 0; k < KPW; ++k)
#pragma unroll
        for (int t = 0; t < HT; ++t) mx[k][t] = f32x4{0.f, 0.f, 0.f, 0.f};
      for (int g4 = 0; g4 < H4; g4 += 4) {
        float ta[HT], sb[KPW];
#pragma unroll
        for (int t = 0; t < HT; ++t) ta[t] = Tt[(g4 + lg) * 16 * HT + 16 * t + li];
#pragma unroll
        for (int k = 0; k < KPW; ++k)
          sb[k] = S[((g4 + lg) * BK + wave * KPW + k) * QS + li];
#pragma unroll
        for (int k = 0; k < KPW; ++k)
#pragma unroll
          for (int t = 0; t < HT; ++t)
            mx[k][t] = __builtin_amdgcn_mfma_f32_16x16x4f32(ta[t], sb[k], mx[k][t], 0, 0, 0);
      }
#pragma unroll
      for (int t = 0; t < HT; ++t)
#pragma unroll
        for (int v = 0; v < 4; ++v) {
          const int h = 16 * t + 4 * lg + v;
          if (h < heads) {
#pragma unroll
            for (int k = 0; k < KPW; ++k)
              S[(h * BK + wave * KPW + k) * QS + li] = mx[k][t][v];
          }
        }
    }
    // every wave is past the previous tile's last use of the other buffer
    kr.store(Rows + (buf ^ 1) * BK, Ksc + (buf ^ 1) * BK, BK, block_size, kv_heads, mult);
    __syncthreads();
    // (3) softmax and values of this wave's heads
    if (item3 < items) {
      // values of 16 keys at a time, the next ones in flight
      constexpr int VJ = DP / 64;
      auto load_v = [&](Quad<T>(&dst)[VJ], int t, int v, int a) {
        const int g = min(item3 * NH + a, heads - 1) / rep;
        const T* row = k_cache + (rows[16 * t + 4 * lg + v] + (long)g * block_size) * D;
#pragma unroll
        for (int j = 0; j < VJ; ++j)
          load_quad<FULL>(dst[j], row + 64 * j + 4 * li, vec, D - (64 * j + 4 * li));
      };
      Quad<T> vs[SHARE ? NKT : 1][4][VJ];
      if (SHARE) {
#pragma unroll
        for (int v = 0; v < 4; ++v) load_v(vs[0][v], 0, v, 0);
      }
      // bias of every (head, key) of this lane, all loads in flight at once
      float p[NH][NKT][4], bs[NH][NKT][4];
#pragma unroll
      for (int a = 0; a < NH; ++a) {
        const int h = min(item3 * NH + a, heads - 1);
        const float* bh = bias + (long)h * bias_n;
#pragma unroll
        for (int t = 0; t < NKT; ++t)
#pragma unroll
          for (int v = 0; v < 4; ++v) {
            const int key = 16 * t + 4 * lg + v;
            bs[a][t][v] = bh[min(max(qpos - (k0 + key), 0), bias_n - 1)];
            p[a][t][v] = S[(h * BK + key) * QS + li];
          }
      }
      __builtin_amdgcn_sched_barrier(0);
#pragma unroll
      for (int a = 0; a < NH; ++a) {
        float mt = -INFINITY;
#pragma unroll
        for (int t = 0; t < NKT; ++t)
#pragma unroll
          for (int v = 0; v < 4; ++v) {
            const int kp = k0 + 16 * t + 4 * lg + v;
            float sc = p[a][t][v] + bs[a][t][v] * LOG2E;
            asm volatile("" : "+v"(sc));  // a select below, no branch around the loads
            p[a][t][v] = (kp <= qpos && kp >= qstart) ? sc : -INFINITY;
            mt = fmaxf(mt, p[a][t][v]);
          }
        mt = fmaxf(mt, __shfl_xor(mt, 16, WAVE_SIZE));
        mt = fmaxf(mt, __shfl_xor(mt, 32, WAVE_SIZE));
        const float mn = fmaxf(m[a], mt);
        // a column that has seen no visible key yet keeps mn = -inf
        const float corr = (mn == -INFINITY) ? 1.f : exp2f(m[a] - mn);
        float ps = 0.f;
#pragma unroll
        for (int t = 0; t < NKT; ++t)
#pragma unroll
          for (int v = 0; v < 4; ++v) {
            const float pv = p[a][t][v] == -INFINITY ? 0.f : exp2f(p[a][t][v] - mn);
            p[a][t][v] = pv;
            ps += pv;
          }
        ps += __shfl_xor(ps, 16, WAVE_SIZE);
        ps += __shfl_xor(ps, 32, WAVE_SIZE);
        l[a] = l[a] * corr + ps;
        m[a] = mn;
#pragma unroll
        for (int i = 0; i < DP / 16; ++i) o[a][i] *= corr;
      }
#pragma unroll
      for (int t = 0; t < NKT; ++t) {
        if (SHARE && t + 1 < NKT) {
#pragma unroll
          for (int v = 0; v < 4; ++v) load_v(vs[t + 1][v], t + 1, v, 0);
          __builtin_amdgcn_sched_barrier(0);
        }
        // row li of output tile 4 j + c is value column 64 j + 4 li + c
#pragma unroll
        for (int v = 0; v < 4; ++v)
#pragma unroll
          for (int a = 0; a < NH; ++a) {
            if (!SHARE) load_v(vs[0][0], t, v, a);
#pragma unroll
            for (int j = 0; j < VJ; ++j)
#pragma unroll
              for (int c = 0; c < 4; ++c)
                o[a][4 * j + c] = __builtin_amdgcn_mfma_f32_16x16x4f32(
                    vs[SHARE ? t : 0][SHARE ? v : 0][j].get(c), p[a][t][v], o[a][4 * j + c], 0, 0, 0);
          }
      }
    }
    // step (1) of the next tile writes other heads' scores than this wave's
    if (gridDim.z > 1) __syncthreads();
  }

  if (item3 >= items || li >= nq) return;
  const long tok = q0 + tok0 + li;
#pragma unroll
  for (int a = 0; a < NH; ++a) {
    const int h = item3 * NH + a;
    if (h < heads) {
      // the 1 in the denominator: a key with score 0 and no value
      const float mn = fmaxf(m[a], 0.f);
      const float corr = m[a] == -INFINITY ? 0.f : exp2f(m[a] - mn);
      const float f = corr / (l[a] * corr + exp2f(-mn));
#pragma unroll
      for (int j = 0; j < DP / 64; ++j)
#pragma unroll
        for (int v = 0; v < 4; ++v) {
          const int d0 = 64 * j + 4 * (4 * lg + v);
          if (d0 < D) {
            const long e = (tok * heads + h) * D + d0;
            f32x4 gv = f32x4{0.f, 0.f, 0.f, 0.f};
            if (gate) gv = load4_f32(gate + tok * gate_stride + (long)h * D + d0, false, D - d0);
#pragma unroll
            for (int c = 0; c < 4; ++c)
              if (d0 + c < D) {
                float r = o[a][4 * j + c][v] * f;
                if (gate) r *= 1.0f / (1.0f + expf(-gv[c]));
                st_f32(out, e + c, r);
              }
          }
        }
    }
  }
}

constexpr int DBK = 64;       // keys per decode tile
constexpr int DS = DBK + 4;   // floats per head row of a decode score tile

// LDS floats of the decode kernel: q [H][DP + 4] | scores [H4][DS] | mixed
// [H][DS] | talk^T [H4][HP] | max, sum, correction [H] each | factors [2][DBK]
// | rows [2][DBK]. Value work items: (kv head, 16 query heads, 64 columns).
template <typename T, int DP, int IPW, bool FULL>
__global__ void __launch_bounds__(NT) talk_decode_kernel(
    float* __restrict__ ws, const float* __restrict__ q,
    const T* __restrict__ k_cache, const float* __restrict__ k_scale,
    const int* __restrict__ block_tables, int bt_stride,
    const int* __restrict__ cu_q, const int* __restrict__ ctx_lens,
    const float* __restrict__ talk, const float* __restrict__ bias, int bias_n,
    float scale, int heads, int kv_heads, int D, int block_size, int window) {
  extern __shared__ float lds[];
  constexpr int QR = DP + 4;
  const int H4 = (heads + 3) & ~3;
  const int HP = (heads + 15) & ~15;
  float* Q = lds;
  float* S = Q + heads * QR;
  float* P = S + H4 * DS;
  float* Tt = P + heads * DS;
  float* Mx = Tt + H4 * HP;
  float* Sm = Mx + H4;
  float* Cr = Sm + H4;
  float* Ksc = Cr + H4;
  int* Rows = reinterpret_cast<int*>(Ksc + 2 * DBK);

  const int s = blockIdx.y;
  const int tok = cu_q[s];
  if (cu_q[s + 1] - tok < 1) return;
  const int split = blockIdx.x, nsplit = gridDim.x;
  const int pos = ctx_lens[s] - 1;
  const int kbeg = window > 0 ? max(pos - window + 1, 0) : 0;
  const int lane = threadIdx.x & 63;
  const int wave = threadIdx.x >> 6;
  const int li = lane & 15, lg = lane >> 4;
  const int rep = heads / kv_heads;
  const int ct = (rep + 15) / 16;  // column tiles of a key group
  const int nj = (D + 63) / 64;
  const int* bt = block_tables + (long)s * bt_stride;
  const bool vec = (D % 8) == 0;
  const float mult = scale * LOG2E;

  for (int e = threadIdx.x; e < heads * QR; e += NT) {
    const int h = e / QR, d = e % QR;
    Q[e] = d < D ? q[((long)tok * heads + h) * D + d] : 0.f;
  }
  for (int e = threadIdx.x; e < H4 * HP; e += NT) {
    const int g = e / HP, h = e % HP;
    Tt[e] = (g < heads && h < heads) ? talk[h * heads + g] : 0.f;
  }
  for (int e = heads * DS + threadIdx.x; e < H4 * DS; e += NT) S[e] = 0.f;
  for (int e = threadIdx.x; e < heads; e += NT) {
    Mx[e] = -INFINITY;
    Sm[e] = 0.f;
  }
  const int kfirst = kbeg + split * DBK;
  const int kstep = nsplit * DBK;
  KeyRows kr;
  kr.find(kfirst, pos, DBK, bt, block_size);
  kr.load(DBK, block_size, k_scale);
  kr.store(Rows, Ksc, DBK, block_size, kv_heads, mult);

  // value items of this wave: kv head, first query head, number of them, columns
  const int items = kv_heads * ct * nj;
  f32x4 o[IPW][4];
#pragma unroll
  for (int i = 0; i < IPW; ++i)
#pragma unroll
    for (int c = 0; c < 4; ++c) o[i][c] = f32x4{0.f, 0.f, 0.f, 0.f};
  const int item0 = (blockIdx.z * NWV + wave) * IPW;
  __syncthreads();

  int buf = 0;
  for (int k0 = kfirst; k0 <= pos; k0 += kstep, buf ^= 1) {
    const int* rows = Rows + buf * DBK;
    const float* ksc = Ksc + buf * DBK;
    kr.find(k0 + kstep, pos, DBK, bt, block_size);
    // (1) scores: 16 keys x the heads of one key group
    for (int u = wave; u < kv_heads * ct * 4; u += NWV) {
      const int kt = u & 3, gc = u >> 2;
      const int g = gc / ct, c0 = (gc % ct) * 16;
      const int h = g * rep + min(c0 + li, rep - 1);
      const long krow = rows[16 * kt + li] + (long)g * block_size;
      f32x4 acc = f32x4{0.f, 0.f, 0.f, 0.f}, acc2 = acc;
      Chunk8<T> kf[DP / 32];
#pragma unroll
      for (int k8 = 0; k8 < DP / 32; ++k8) {
        const int d0 = 32 * k8 + 8 * lg;
        load_chunk<FULL>(kf[k8], k_cache + krow * D + d0, vec, D - d0);
      }
#pragma unroll
      for (int k8 = 0; k8 < DP / 32; ++k8) {
        const float* qp = Q + h * QR + 32 * k8 + 8 * lg;
        const f32x4 qa = *reinterpret_cast<const f32x4*>(qp);
        const f32x4 qb = *reinterpret_cast<const f32x4*>(qp + 4);
#pragma unroll
        for (int c = 0; c < 4; ++c) {
          acc = __builtin_amdgcn_mfma_f32_16x16x4f32(kf[k8].get(c), qa[c], acc, 0, 0, 0);
          acc2 = __builtin_amdgcn_mfma_f32_16x16x4f32(kf[k8].get(4 + c), qb[c], acc2, 0, 0, 0);
        }
      }
      if (c0 + li < rep) {
        const f32x4 f = *reinterpret_cast<const f32x4*>(ksc + 16 * kt + 4 * lg);
        *reinterpret_cast<f32x4*>(S + h * DS + 16 * kt + 4 * lg) = (acc + acc2) * f;
      }
    }
    kr.load(DBK, block_size, k_scale);
    __syncthreads();
    // (2) mix over the heads: 16 heads x 16 keys a unit
    for (int u = wave; u < (HP / 16) * 4; u += NWV) {
      const int kt = u & 3, ht = u >> 2;
      f32x4 mx = f32x4{0.f, 0.f, 0.f, 0.f};
      for (int g4 = 0; g4 < H4; g4 += 4)
        mx = __builtin_amdgcn_mfma_f32_16x16x4f32(Tt[(g4 + lg) * HP + 16 * ht + li],
                                                  S[(g4 + lg) * DS + 16 * kt + li],
                                                  mx, 0, 0, 0);
#pragma unroll
      for (int v = 0; v < 4; ++v) {
        const int h = 16 * ht + 4 * lg + v;
        if (h < heads) P[h * DS + 16 * kt + li] = mx[v];
      }
    }
    kr.store(Rows + (buf ^ 1) * DBK, Ksc + (buf ^ 1) * DBK, DBK, block_size, kv_heads, mult);
    __syncthreads();
    // (3) softmax, one key per lane
    for (int h = wave; h < heads; h += NWV) {
      const int kp = k0 + lane;
      const int n = min(max(pos - kp, 0), bias_n - 1);
      const float sc = kp <= pos ? P[h * DS + lane] + bias[(long)h * bias_n + n] * LOG2E
                                 : -INFINITY;
      const float m = Mx[h];
      // the tile's first key is visible, so mn is finite
      const float mn = fmaxf(m, wave_reduce_max(sc));
      const float pv = sc == -INFINITY ? 0.f : exp2f(sc - mn);
      const float ps = wave_reduce_sum(pv);
      P[h * DS + lane] = pv;
      if (lane == 0) {
        const float corr = exp2f(m - mn);
        Cr[h] = corr;
        Sm[h] = Sm[h] * corr + ps;
        Mx[h] = mn;
      }
    }
    __syncthreads();
    // (4) values
#pragma unroll
    for (int i = 0; i < IPW; ++i) {
      const int item = item0 + i;
      if (item < items) {
        const int j = item % nj, gc = item / nj;
        const int g = gc / ct, c0 = (gc % ct) * 16;
        const int h = g * rep + min(c0 + li, rep - 1);
        const int d0 = 64 * j + 4 * li;
        const float corr = Cr[h];
#pragma unroll
        for (int c = 0; c < 4; ++c) o[i][c] *= corr;
#pragma unroll
        for (int kt = 0; kt < 4; ++kt) {
          const f32x4 p = *reinterpret_cast<const f32x4*>(P + h * DS + 16 * kt + 4 * lg);
          Quad<T> vv[4];
#pragma unroll
          for (int v = 0; v < 4; ++v) {
            const long vrow = rows[16 * kt + 4 * lg + v] + (long)g * block_size;
            load_quad<FULL>(vv[v], k_cache + vrow * D + d0, vec, D - d0);
          }
#pragma unroll
          for (int v = 0; v < 4; ++v)
#pragma unroll
            for (int c = 0; c < 4; ++c)
              o[i][c] = __builtin_amdgcn_mfma_f32_16x16x4f32(vv[v].get(c), p[v], o[i][c], 0, 0, 0);
        }
      }
    }
  }

  __syncthreads();
#pragma unroll
  for (int i = 0; i < IPW; ++i) {
    const int item = item0 + i;
    if (item < items) {
      const int j = item % nj, gc = item / nj;
      const int g = gc / ct, c0 = (gc % ct) * 16;
      if (c0 + li < rep) {
        const int h = g * rep + c0 + li;
        float* wr = ws + (((long)s * heads + h) * nsplit + split) * (D + 2);
#pragma unroll
        for (int v = 0; v < 4; ++v)
#pragma unroll
          for (int c = 0; c < 4; ++c) {
            const int d = 64 * j + 4 * (4 * lg + v) + c;
            if (d < D) wr[d] = o[i][c][v];
          }
      }
    }
  }
  if (blockIdx.z == 0)
    for (int h = threadIdx.x; h < heads; h += NT) {
      float* wr = ws + (((long)s * heads + h) * nsplit + split) * (D + 2);
      wr[D] = Mx[h];
      wr[D + 1] = Sm[h];
    }
}

template <typename T>
__global__ void talk_merge_kernel(T* __restrict__ out, const float* __restrict__ ws,
                                  const int* __restrict__ cu_q,
                                  const T* __restrict__ gate, long gate_stride,
                                  int heads, int D, int nsplit) {
  const int s = blockIdx.x / heads, h = blockIdx.x % heads;
  const long tok = cu_q[s];
  if (cu_q[s + 1] - tok < 1) return;
  const float* wr = ws + ((long)s * heads + h) * nsplit * (D + 2);
  // one more key with score 0 and no value
  float M = 0.f;
  for (int i = 0; i < nsplit; ++i) M = fmaxf(M, wr[i * (D + 2) + D]);
  float L = exp2f(-M);
  for (int i = 0; i < nsplit; ++i) {
    const float mi = wr[i * (D + 2) + D];
    if (mi != -INFINITY) L += wr[i * (D + 2) + D + 1] * exp2f(mi - M);
  }
  const float f = 1.0f / L;
  for (int d = threadIdx.x; d < D; d += blockDim.x) {
    float O = 0.f;
    for (int i = 0; i < nsplit; ++i) {
      const float mi = wr[i * (D + 2) + D];
      if (mi != -INFINITY) O += wr[i * (D + 2) + d] * exp2f(mi - M);
    }
    O *= f;
    if (gate) {
      const float gv = ld_f32(gate, tok * gate_stride + (long)h * D + d);
      O *= 1.0f / (1.0f + expf(-gv));
    }
    st_f32(out, (tok * heads + h) * D + d, O);
  }
}

struct TalkArgs {
  void* out;
  const void *q, *k_cache, *k_scale, *block_tables;
  int bt_stride;
  const void *cu_q, *ctx_lens, *talk, *bias;
  int bias_n;
  const void* gate;
  long gate_stride;
  float scale;
  int num_seqs, max_q_len, heads, kv_heads, D, block_size, window;
  void* ws;
  int nsplit;
  hipStream_t stream;
};

constexpr size_t LDS_MAX = 160 * 1024;

template <typename F>
hipError_t allow_lds(F fn, size_t smem) {
  if (smem > LDS_MAX) return hipErrorInvalidValue;
  if (smem <= 48 * 1024) return hipSuccess;
  return hipFuncSetAttribute((const void*)fn,
                             hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem);
}

template <typename T, int DP, int NH, int HT, bool SHARE, bool FULL = false>
hipError_t launch_prefill(const TalkArgs& a) {
  if constexpr (SHARE && !FULL && DP <= 128 && sizeof(T) == 2) {
    if (a.D == DP) return launch_prefill<T, DP, NH, HT, SHARE, true>(a);
  }
  constexpr int BK = 16 * key_tiles(DP, NH, HT);
  const int H4 = (a.heads + 3) & ~3;
  const size_t smem =
      sizeof(float) * ((size_t)H4 * BK * QS + (size_t)H4 * 16 * HT + 4 * BK);
  auto fn = talk_prefill_kernel<T, DP, NH, HT, SHARE, FULL>;
  hipError_t e = allow_lds(fn, smem);
  if (e != hipSuccess) return e;
  dim3 grid(cdiv(a.max_q_len, 16), a.num_seqs, cdiv(cdiv(a.heads, NH), NWV));
  hipLaunchKernelGGL(fn, grid, dim3(NT), smem, a.stream, (T*)a.out,
                     (const float*)a.q, (const T*)a.k_cache,
                     (const float*)a.k_scale, (const int*)a.block_tables,
                     a.bt_stride, (const int*)a.cu_q, (const int*)a.ctx_lens,
                     (const float*)a.talk, (const float*)a.bias, a.bias_n,
                     (const T*)a.gate, a.gate_stride, a.scale, a.heads,
                     a.kv_heads, a.D, a.block_size, a.window);
  return hipGetLastError();
}

// NH heads per wave so that 8 waves cover the heads where that fits the
// registers; HT: 16-head tiles of the mixing product
template <typename T, int DP>
hipError_t dispatch_prefill(const TalkArgs& a) {
  const int H = a.heads, rep = a.heads / a.kv_heads;
  if (H <= 8) return launch_prefill<T, DP, 1, 1, true>(a);
  if constexpr (DP <= 128) {
    // (fp32 pages: the exact-check dtype, one variant each)
    constexpr bool fast = sizeof(T) == 2;
    if (H <= 16)
      return fast && rep % 2 == 0 ? launch_prefill<T, DP, 2, 1, fast>(a)
                                  : launch_prefill<T, DP, 2, 1, false>(a);
    if (H <= 32)
      return fast && rep % 4 == 0 ? launch_prefill<T, DP, 4, 2, fast>(a)
                                  : launch_prefill<T, DP, 4, 2, false>(a);
    return launch_prefill<T, DP, 4, 6, false>(a);
  } else {
    if (H <= 16) return launch_prefill<T, DP, 2, 1, false>(a);
    if (H <= 32) return launch_prefill<T, DP, 2, 2, false>(a);
    return launch_prefill<T, DP, 2, 6, false>(a);
  }
}

template <typename T, int DP, int IPW, bool FULL = false>
hipError_t launch_decode(const TalkArgs& a, int items) {
  if constexpr (!FULL && DP <= 128 && sizeof(T) == 2) {
    if (a.D == DP) return launch_decode<T, DP, IPW, true>(a, items);
  }
  const int H4 = (a.heads + 3) & ~3, HP = (a.heads + 15) & ~15;
  const size_t smem =
      sizeof(float) * ((size_t)a.heads * (DP + 4) + (size_t)H4 * DS +
                       (size_t)a.heads * DS + (size_t)H4 * HP + 3 * (size_t)H4 +
                       4 * DBK);
  auto fn = talk_decode_kernel<T, DP, IPW, FULL>;
  hipError_t e = allow_lds(fn, smem);
  if (e != hipSuccess) return e;
  dim3 grid(a.nsplit, a.num_seqs, cdiv(items, NWV * IPW));
  hipLaunchKernelGGL(fn, grid, dim3(NT), smem, a.stream, (float*)a.ws,
                     (const float*)a.q, (const T*)a.k_cache,
                     (const float*)a.k_scale, (const int*)a.block_tables,
                     a.bt_stride, (const int*)a.cu_q, (const int*)a.ctx_lens,
                     (const float*)a.talk, (const float*)a.bias, a.bias_n,
                     a.scale, a.heads, a.kv_heads, a.D, a.block_size, a.window);
  e = hipGetLastError();
  if (e != hipSuccess) return e;
  hipLaunchKernelGGL(talk_merge_kernel<T>, dim3(a.num_seqs * a.heads), dim3(64),
                     0, a.stream, (T*)a.out, (const float*)a.ws,
                     (const int*)a.cu_q, (const T*)a.gate, a.gate_stride,
                     a.heads, a.D, a.nsplit);
  return hipGetLastError();
}

template <typename T, int DP>
hipError_t dispatch_decode(const TalkArgs& a) {
  const int ct = cdiv(a.heads / a.kv_heads, 16);
  const int items = a.kv_heads * ct * cdiv(a.D, 64);
  if (items <= NWV) return launch_decode<T, DP, 1>(a, items);
  if (items <= 2 * NWV) return launch_decode<T, DP, 2>(a, items);
  return launch_decode<T, DP, 4>(a, items);
}

template <typename T, int DP>
hipError_t dispatch(const TalkArgs& a) {
  return a.max_q_len == 1 ? dispatch_decode<T, DP>(a) : dispatch_prefill<T, DP>(a);
}

template <typename T>
hipError_t dispatch_d(const TalkArgs& a) {
  if (a.D <= 64) return dispatch<T, 64>(a);
  if (a.D <= 128) return dispatch<T, 128>(a);
  return dispatch<T, 256>(a);
}

}  // namespace

extern "C" hipError_t ks_talk_prep_cache(
    void* q_out, const void* q, long q_stride, const void* k, long k_stride,
    const void* w, const void* slot_mapping, void* k_cache, void* k_scale,
    float eps, int tokens, int q_width, int kv_heads, int D, int block_size,
    int is_f32, hipStream_t stream) {
  if (tokens == 0) return hipSuccess;
  const int ab = is_f32 ? 16 : 8;
  auto al = [](const void* p, int bytes) { return ((uintptr_t)p % bytes) == 0; };
  const int vec = q_width % 4 == 0 && (kv_heads * D) % 4 == 0 &&
                  q_stride % 4 == 0 && k_stride % 4 == 0 && al(q, ab) &&
                  al(k, ab) && al(w, 16) && al(q_out, 16);
#define TP_ARGS(TT)                                                            \
  (float*)q_out, (const TT*)q, q_stride, (const TT*)k, k_stride,               \
      (const float*)w, (const int*)slot_mapping, (TT*)k_cache,                 \
      (float*)k_scale, eps, q_width, kv_heads, D, block_size, vec
  if (is_f32)
    hipLaunchKernelGGL(talk_prep_cache_kernel<float>, dim3(tokens), dim3(256), 0,
                       stream, TP_ARGS(float));
  else
    hipLaunchKernelGGL(talk_prep_cache_kernel<short>, dim3(tokens), dim3(256), 0,
                       stream, TP_ARGS(short));
  HIP_CHECK_KERNEL();
  return hipSuccess;
}

// key splits of a decode launch: enough blocks for two or so on every compute
// unit, at most 8, with a window no more than it has tiles
extern "C" int ks_talk_decode_splits(int num_seqs, int window) {
  int n = cdiv(1024, num_seqs > 0 ? num_seqs : 1);
  if (n > 8) n = 8;
  if (window > 0 && n > cdiv(window, DBK)) n = cdiv(window, DBK);
  return n < 1 ? 1 : n;
}

extern "C" hipError_t ks_talk_attention(
    void* out, const void* q, const void* k_cache, const void* k_scale,
    const void* block_tables, int bt_stride, const void* cu_q,
    const void* ctx_lens, const void* talk, const void* bias, int bias_n,
    const void* gate, long gate_stride, float scale, int num_seqs,
    int max_q_len, int heads, int kv_heads, int D, int block_size, int window,
    int is_f32, void* ws, int nsplit, hipStream_t stream) {
  if (num_seqs == 0 || max_q_len == 0) return hipSuccess;
  if (D < 1 || D > 256 || kv_heads < 1 || heads < 1 || heads % kv_heads != 0 ||
      heads > 96 || window < 0 || bias_n < 1 ||
      (max_q_len == 1 && (!ws || nsplit < 1)))
    return hipErrorInvalidValue;
  const TalkArgs a{out, q, k_cache, k_scale, block_tables, bt_stride, cu_q,
                   ctx_lens, talk, bias, bias_n, gate, gate_stride, scale,
                   num_seqs, max_q_len, heads, kv_heads, D, block_size, window,
                   ws, nsplit, stream};
  return is_f32 ? dispatch_d<float>(a) : dispatch_d<short>(a);
}
