// Linear-attention recurrences with a matrix state per head, over a flat,
// variable-length token batch with per-sequence state slots (the layout of
// ssm_scan.hip: `positions[t]`, `cu_seqlens[s]`, `slots[s]`; a portion that
// starts at position 0 ignores what its slot held).
//
// The state of head h is S (K x V, fp32), stored per slot as [H, V, K] so
// that the contraction index is contiguous. Per token, with query q and key k
// of the head's q/k group and value v:
//
//   decay form (retention):   S <- d S + k v^T                 o = S^T q
//   delta form (gated delta): S <- g S;  u = b (v - S^T k);
//                             S <- S + k u^T                   o = S^T q
//
// A third form has one decay per head AND key channel, read per token from
// fp32 rows: S <- diag(g) S first (one multiplication per state element), then
// the delta form with g = 1.
//
// A fourth form is the decay form with such per-channel decays,
//   channel decay (gated linear attention): S <- diag(g) S + k v^T,
// and reads q, k, v in the activation dtype straight from the columns of a
// projection (q times q_scale).
//
// d is a constant per head; g = exp(-exp(A_log) softplus(a + dt_bias)) and
// b = sigmoid(beta_raw) are computed here in fp32 from raw per-token, per-head
// projection columns. Both forms are evaluated from the OLD state with two
// independent contractions, p1 = S^T k and p2 = S^T q:
//   u = b (v - g p1)   (decay form: u = v)
//   o = g p2 + u (k . q)
//   S <- g S + k u^T
// so a token costs one pass over the registers that hold the state.
//
// Lane (ns, pl) of a 256-thread block owns rows n = ns + 16 r of columns
// pl + 16 c of one head's tile; a 16-lane DPP tree sums the contractions.
// Tokens go through LDS a chunk at a time with the next chunk's loads in
// flight. Grid = column tiles x heads x sequences: prefill portions and
// single-token decode batches run the same kernel.
//
// The two decay forms have no correction by the old state, so a prompt portion
// takes 16 tokens at a time on the fp32 matrix cores (decay_chunk_kernel).
// With b_t the product of a chunk's decays up to token t (per key channel),
//   O = (Q b) S + mask(Q b (K / b)^T) V,   S <- diag(b_16) (S + (K / b)^T V).
// b_16 >= 2^-60 keeps every factor and product finite and each term's relative
// error at a few roundings; a chunk with a channel below that walks its tokens
// one by one on the same registers.
//
// Helpers for what precedes the recurrence:
//  * rope_scale_heads: rotary positions on the first 2*half coordinates of
//    every head (coordinate i pairs with i + half), times a constant, fp32
//    out; two runs of heads with a constant each (queries, keys), columns
//    after them are only widened to fp32 (values).
//  * unit_norm_heads: x / sqrt(sum(x^2) + eps) * scale per head, in place on
//    fp32 rows; two runs of heads with a scale each (queries, keys).
//  * lowrank_channel_decay: sigmoid(z)^(1/tau), z = W2 low + b, the decays of
//    the fourth form from a low-rank projection; fp32 after the first factor.
//  * delta_unit_decay: the unit norms, and for the third form the decays
//    g = exp(-exp(A_log) softplus(a + dt_bias)) per head and key channel.
#include "dtype_io.h"

#include <type_traits>

namespace {

constexpr int NT = 256;
constexpr int NW = NT / WAVE_SIZE;

__device__ __forceinline__ float row16_sum(float v) {
  auto swz = [](float x, auto ctrl) {
    return __builtin_bit_cast(
        float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, x),
                                           decltype(ctrl)::value, 0xF, 0xF, true));
  };
  v += swz(v, std::integral_constant<int, 0xB1>{});   // quad_perm [1,0,3,2]
  v += swz(v, std::integral_constant<int, 0x4E>{});   // quad_perm [2,3,0,1]
  v += swz(v, std::integral_constant<int, 0x141>{});  // row_half_mirror
  v += swz(v, std::integral_constant<int, 0x140>{});  // row_mirror
  return v;
}

template <typename T>
__global__ void rope_scale_heads_kernel(
    float* __restrict__ out, const T* __restrict__ in, long in_stride,
    const long* __restrict__ positions, const float* __restrict__ inv_freq,
    int half, int heads_a, float scale_a, int heads_b, float scale_b, int dim,
    int width) {
  extern __shared__ float cs[];  // [half][2] = (cos, sin)
  const long t = blockIdx.x;
  const float pos = (float)positions[t];
  for (int i = threadIdx.x; i < half; i += NT) {
    float sn, co;
    sincosf(pos * inv_freq[i], &sn, &co);
    cs[2 * i] = co;
    cs[2 * i + 1] = sn;
  }
  __syncthreads();
  const int na = heads_a * dim, n = (heads_a + heads_b) * dim;
  const T* row = in + t * in_stride;
  for (int e = threadIdx.x; e < width; e += NT) {
    float r = ld_f32(row, e);
    if (e < n) {
      const int i = e % dim;
      if (i < 2 * half) {
        const bool lo = i < half;
        const int fi = lo ? i : i - half;
        const float y = ld_f32(row, lo ? e + half : e - half);
        const float co = cs[2 * fi], sn = cs[2 * fi + 1];
        r = lo ? r * co - y * sn : r * co + y * sn;
      }
      r *= e < na ? scale_a : scale_b;
    }
    out[t * width + e] = r;
  }
}

__global__ void unit_norm_heads_kernel(float* __restrict__ x, long stride,
                                       int heads_a, float scale_a, int heads_b,
                                       float scale_b, int dim, float eps) {
  const long t = blockIdx.x;
  const int lane = threadIdx.x & 63;
  const int wave = threadIdx.x >> 6;
  for (int job = wave; job < heads_a + heads_b; job += NW) {
    float* p = x + t * stride + (long)job * dim;
    float ss = 0.f;
    for (int i = lane; i < dim; i += WAVE_SIZE) ss += p[i] * p[i];
    ss = wave_reduce_sum(ss);
    const float m = (job < heads_a ? scale_a : scale_b) / sqrtf(ss + eps);
    for (int i = lane; i < dim; i += WAVE_SIZE) p[i] *= m;
  }
}

// unit norms of q and k heads in place (as above, scale 1 for k), and the
// decay of every head and key channel
template <typename T>
__global__ void delta_unit_decay_kernel(
    float* __restrict__ x, long stride, float* __restrict__ g,
    const T* __restrict__ a_raw, long a_stride, const float* __restrict__ a_log,
    const float* __restrict__ dt_bias, int qk_heads, int dim, float q_scale,
    float eps, int decays) {
  const long t = blockIdx.x;
  const int lane = threadIdx.x & 63;
  const int wave = threadIdx.x >> 6;
  for (int job = wave; job < 2 * qk_heads; job += NW) {
    float* p = x + t * stride + (long)job * dim;
    float ss = 0.f;
    for (int i = lane; i < dim; i += WAVE_SIZE) ss += p[i] * p[i];
    ss = wave_reduce_sum(ss);
    const float m = (job < qk_heads ? q_scale : 1.0f) / sqrtf(ss + eps);
    for (int i = lane; i < dim; i += WAVE_SIZE) p[i] *= m;
  }
  for (int e = threadIdx.x; e < decays; e += NT) {
    const float z = ld_f32(a_raw, t * a_stride + e) + dt_bias[e];
    // softplus without a clamp; log1p(exp(z)) is z itself past z ~ 30
    const float sp = z > 30.f ? z : log1pf(expf(z));
    g[t * decays + e] = expf(-expf(a_log[e / dim]) * sp);
  }
}

// A block takes DT tokens (their low rows in LDS as fp32) x 256 columns; a lane
// keeps one column's sums of all DT tokens and reads that column's row of w2.
constexpr int DT = 16;

template <typename T>
__global__ void __launch_bounds__(NT) lowrank_channel_decay_kernel(
    float* __restrict__ out, const T* __restrict__ low, long low_stride,
    const float* __restrict__ w2, const float* __restrict__ bias, float inv_tau,
    int tokens, int r, int n) {
  extern __shared__ float ls[];  // [DT][r]
  const long t0 = (long)blockIdx.x * DT;
  const int cnt = min((long)DT, tokens - t0);
  for (int e = threadIdx.x; e < DT * r; e += NT) {
    const int tt = e / r;
    ls[e] = tt < cnt ? ld_f32(low, (t0 + tt) * low_stride + e % r) : 0.f;
  }
  __syncthreads();
  const int c = blockIdx.y * NT + threadIdx.x;
  if (c >= n) return;
  const float* w = w2 + (long)c * r;
  const bool vec = r % 4 == 0 && ((uintptr_t)w2 % 16) == 0;
  float acc[DT];
  const float b = bias[c];
#pragma unroll
  for (int a = 0; a < DT; ++a) acc[a] = b;
  if (vec) {
    for (int k = 0; k < r; k += 4) {
      const float4_t w4 = *reinterpret_cast<const float4_t*>(w + k);
#pragma unroll
      for (int a = 0; a < DT; ++a) {
        const float4_t x = *reinterpret_cast<const float4_t*>(ls + a * r + k);
        acc[a] += w4[0] * x[0] + w4[1] * x[1] + w4[2] * x[2] + w4[3] * x[3];
      }
    }
  } else {
    for (int k = 0; k < r; ++k) {
      const float wk = w[k];
#pragma unroll
      for (int a = 0; a < DT; ++a) acc[a] += wk * ls[a * r + k];
    }
  }
#pragma unroll
  for (int a = 0; a < DT; ++a) {
    if (a < cnt) {
      // log2 sigmoid(z) = min(z, 0) log2(e) - log2(1 + exp(-|z|)). The
      // logarithm's argument lies in [1, 2], so its absolute error is an ulp
      // of 1, no more than what rounding the decay itself costs.
      const float z2 = acc[a] * 1.44269504088896340736f;
      const float lg = fminf(z2, 0.f) -
                       __builtin_amdgcn_logf(1.0f + __builtin_amdgcn_exp2f(-fabsf(z2)));
      out[(t0 + a) * n + c] = __builtin_amdgcn_exp2f(lg * inv_tau);
    }
  }
}

constexpr int SCAN_TC = 16;  // tokens per chunk

// recurrence forms
constexpr int DECAY = 0, HEAD_DELTA = 1, CHANNEL_DELTA = 2, CHANNEL_DECAY = 3;

// R = state rows per lane (K <= 16 R), PC = columns per lane (a block covers
// 16 PC value columns of one head). TQ: dtype of q, k, v.
template <int R, int PC, int FORM, typename TQ>
__global__ void __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(4)))
linear_scan_kernel(
    float* __restrict__ o, const TQ* __restrict__ q, long q_stride,
    const TQ* __restrict__ k, long k_stride, const TQ* __restrict__ v,
    long v_stride, float q_scale, const float* __restrict__ decay,
    const float* __restrict__ a_f32, const short* __restrict__ a_bf16,
    const float* __restrict__ b_f32, const short* __restrict__ b_bf16,
    long ab_stride, const float* __restrict__ a_log,
    const float* __restrict__ dt_bias, const float* __restrict__ channel_decay,
    float* __restrict__ state,
    const long* __restrict__ positions, const int* __restrict__ cu_seqlens,
    const int* __restrict__ slots, int heads, int qk_heads, int V, int K) {
  extern __shared__ float lds[];
  constexpr bool DELTA = FORM == HEAD_DELTA || FORM == CHANNEL_DELTA;
  constexpr bool CHAN = FORM == CHANNEL_DELTA || FORM == CHANNEL_DECAY;
  constexpr int tc = SCAN_TC;
  constexpr int XS = 16 * PC;
  const int s = blockIdx.z;
  const int h = blockIdx.y;
  const int ns = threadIdx.x & 15;
  const int pl = threadIdx.x >> 4;
  const int p0 = blockIdx.x * XS;
  const int pt = min(XS, V - p0);  // columns of this tile
  const int first = cu_seqlens[s];
  const int len = cu_seqlens[s + 1] - first;
  if (len <= 0) return;
  const int hq = h / (heads / qk_heads);
  const int inner = heads * V;
  const long slot = slots[s];
  const bool fresh = positions[first] == 0;
  const float fixed = FORM == DECAY ? decay[h] : 1.f;
  const float A = FORM == HEAD_DELTA ? -expf(a_log[h]) : 0.f;
  const float bias = FORM == HEAD_DELTA ? dt_bias[h] : 0.f;

  // LDS: k[tc][K] | q[tc][K] | v[tc][XS] | g[tc] | beta[tc] | k.q[tc] | o[tc][XS]
  //      | channel decays [tc][K]
  float* Ks = lds;
  float* Qs = Ks + tc * K;
  float* Vs = Qs + tc * K;
  float* Gs = Vs + tc * XS;
  float* Bs = Gs + tc;
  float* Ds = Bs + tc;
  float* Os = Ds + tc;
  float* Cs = Os + tc * XS;
  float S[R][PC];
  float* sp = state + ((slot * heads + h) * (long)V) * K;
#pragma unroll
  for (int c = 0; c < PC; ++c) {
    const int p = p0 + pl + 16 * c;
#pragma unroll
    for (int r = 0; r < R; ++r) {
      const int n = ns + 16 * r;
      S[r][c] = (!fresh && p < V && n < K) ? sp[(long)p * K + n] : 0.f;
    }
  }

  // staging: 16 threads per token of the chunk, each takes every 16th
  // element of the token's k, q and v rows
  const int stk = threadIdx.x >> 4;
  const int sl = threadIdx.x & 15;
  float sK[R], sQ[R], sC[CHAN ? R : 1], sV[PC], sa = 0.f, sb = 0.f;
  auto prefetch = [&](int t0, int cnt) {
    const bool on = stk < cnt;
    const long t = first + t0 + (on ? stk : 0);
    const TQ* krow = k + t * k_stride + (long)hq * K;
    const TQ* qrow = q + t * q_stride + (long)hq * K;
    const TQ* vrow = v + t * v_stride + (long)h * V + p0;
#pragma unroll
    for (int r = 0; r < R; ++r) {
      const int n = sl + 16 * r;
      const bool ok = on && n < K;
      sK[r] = ok ? ld_f32(krow, n) : 0.f;
      sQ[r] = ok ? ld_f32(qrow, n) * q_scale : 0.f;
      if (CHAN) sC[r] = ok ? channel_decay[(t * heads + h) * K + n] : 0.f;
    }
#pragma unroll
    for (int c = 0; c < PC; ++c) {
      const int col = sl + 16 * c;
      sV[c] = (on && col < pt) ? ld_f32(vrow, col) : 0.f;
    }
    if (DELTA && on && sl == 0) {
      const long i = t * ab_stride + h;
      if (!CHAN) sa = (a_f32 ? a_f32[i] : bf16_bits_to_float(a_bf16[i])) + bias;
      sb = b_f32 ? b_f32[i] : bf16_bits_to_float(b_bf16[i]);
    }
  };
  auto commit = [&](int cnt) {
    float kq = 0.f;
#pragma unroll
    for (int r = 0; r < R; ++r) kq += sK[r] * sQ[r];
    kq = row16_sum(kq);  // every lane takes part, staged or not
    if (stk < cnt) {
#pragma unroll
      for (int r = 0; r < R; ++r) {
        const int n = sl + 16 * r;
        if (n < K) {
          Ks[stk * K + n] = sK[r];
          Qs[stk * K + n] = sQ[r];
          if (CHAN) Cs[stk * K + n] = sC[r];
        }
      }
#pragma unroll
      for (int c = 0; c < PC; ++c) Vs[stk * XS + sl + 16 * c] = sV[c];
      if (sl == 0) {
        Ds[stk] = kq;
        if (DELTA) {
          // softplus without a clamp; log1p(exp(x)) is x itself past x ~ 30
          const float sp_ = sa > 30.f ? sa : log1pf(expf(sa));
          Gs[stk] = CHAN ? 1.f : expf(A * sp_);
          Bs[stk] = 1.0f / (1.0f + expf(-sb));
        } else {
          Gs[stk] = fixed;
          Bs[stk] = 1.f;
        }
      }
    }
  };

  prefetch(0, min(tc, len));
  for (int t0 = 0; t0 < len; t0 += tc) {
    const int cnt = min(tc, len - t0);
    __syncthreads();  // previous chunk's LDS fully consumed
    commit(cnt);
    __syncthreads();
    if (t0 + tc < len) prefetch(t0 + tc, min(tc, len - t0 - tc));
    for (int tk = 0; tk < cnt; ++tk) {
      const float g = Gs[tk], bt = Bs[tk], kq = Ds[tk];
      float kk[R], qq[R];
#pragma unroll
      for (int r = 0; r < R; ++r) {
        const int n = ns + 16 * r;
        const bool ok = n < K;
        kk[r] = ok ? Ks[tk * K + n] : 0.f;
        qq[r] = ok ? Qs[tk * K + n] : 0.f;
        if (CHAN) {
          const float gc = ok ? Cs[tk * K + n] : 0.f;
#pragma unroll
          for (int c = 0; c < PC; ++c) S[r][c] *= gc;
        }
      }
#pragma unroll
      for (int c = 0; c < PC; ++c) {
        const int col = pl + 16 * c;
        const float vv = col < pt ? Vs[tk * XS + col] : 0.f;
        float p1 = 0.f, p2 = 0.f;
#pragma unroll
        for (int r = 0; r < R; ++r) {
          if (DELTA) p1 += S[r][c] * kk[r];
          p2 += S[r][c] * qq[r];
        }
        p2 = row16_sum(p2);
        float u = vv;
        if (DELTA) {
          p1 = row16_sum(p1);
          u = bt * (vv - (CHAN ? p1 : g * p1));
        }
#pragma unroll
        for (int r = 0; r < R; ++r) S[r][c] = (CHAN ? S[r][c] : g * S[r][c]) + kk[r] * u;
        if (ns == 0) Os[tk * XS + col] = (CHAN ? p2 : g * p2) + u * kq;
      }
    }
    __syncthreads();
    for (int e = threadIdx.x; e < cnt * pt; e += 256) {
      const int tk = e / pt, col = e % pt;
      o[(long)(first + t0 + tk) * inner + h * V + p0 + col] = Os[tk * XS + col];
    }
  }
#pragma unroll
  for (int c = 0; c < PC; ++c) {
    const int p = p0 + pl + 16 * c;
#pragma unroll
    for (int r = 0; r < R; ++r) {
      const int n = ns + 16 * r;
      if (p < V && n < K) sp[(long)p * K + n] = S[r][c];
    }
  }
}

typedef float f32x4 __attribute__((ext_vector_type(4)));

// KT: 16-row tiles of the key dimension (K <= 16 KT). 256 threads; a block
// takes 64 value columns of one head of one sequence, a wave 16 of them.
//
// State: s[kt], lane (li, lg) register r = S[k = 16 kt + 4 lg + r][v = li]. That
// is the accumulator layout of v_mfma_f32_16x16x4_f32 (rows k, columns v) and
// at the same time, with the contraction index of k-step r in lane group lg
// standing for 4 lg + r, the A operand of O^T = S^T (Q b)^T. The products:
//   O^T [v][t] += S^T (Q b)^T            A = s registers, B from LDS rows t
//   P^T [s][t]  = (K / b) (Q b)^T        A, B from LDS rows; the waves share
//                                        the key tiles and sum through LDS
//   O^T [v][t] += V^T mask(P)^T          A = v registers, B = P^T registers
//   S   [k][v] += (K / b)^T V            A from LDS (transposed), B = v registers
// V never passes through LDS: lane (li, lg) register r is v[token 4 lg + r][li].
//
// Staging: thread (n, g) takes key channel n of tokens g KT .. g KT + KT - 1
// (16 / KT threads per channel) and the decays of all 16 tokens. Tokens past
// the end and channels past K count as decay 1, q = k = v = 0.
// CHAN: per-channel decays, otherwise one constant per head.
template <int KT, bool CHAN, typename TQ>
__global__ void __launch_bounds__(NT)
__attribute__((amdgpu_waves_per_eu(KT > 8 ? 1 : 2)))
decay_chunk_kernel(
    float* __restrict__ o, const TQ* __restrict__ q, long q_stride,
    const TQ* __restrict__ k, long k_stride, const TQ* __restrict__ v,
    long v_stride, float q_scale, const float* __restrict__ decay,
    const float* __restrict__ channel_decay, float* __restrict__ state,
    const long* __restrict__ positions, const int* __restrict__ cu_seqlens,
    const int* __restrict__ slots, int heads, int qk_heads, int V, int K) {
  constexpr int TC = 16;         // tokens per chunk
  constexpr int KP = 16 * KT;
  constexpr int KS = KP + 4;     // row strides that spread rows over the banks
  constexpr int TS = TC + 4;
  constexpr float MIN_PRODUCT = 8.67361737988403547e-19f;  // 2^-60
  extern __shared__ float lds[];
  float* Qb = lds;               // [TC][KS]  q b        (slow chunk: q)
  float* Kb = Qb + TC * KS;      // [TC][KS]  k / b      (slow chunk: k)
  float* Kt = Kb + TC * KS;      // [KP][TS]  (k / b)^T  (slow chunk: decays^T)
  float* Bc = Kt + KP * TS;      // [KP]      b_16
  float* Ps = Bc + KP;           // [NW][64][4] partial P^T
  int* flag = reinterpret_cast<int*>(Ps + NW * WAVE_SIZE * 4);  // [NW]

  const int s = blockIdx.z, h = blockIdx.y;
  const int lane = threadIdx.x & 63;
  // a scalar, so that what one wave skips is skipped by a scalar branch (the
  // matrix instructions do not look at the execution mask)
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int li = lane & 15, lg = lane >> 4;
  const int first = cu_seqlens[s];
  const int len = cu_seqlens[s + 1] - first;
  if (len <= 0) return;
  const int hq = h / (heads / qk_heads);
  const int inner = heads * V;
  const int col = blockIdx.x * 64 + wave * 16;  // first value column of the wave
  const bool vok = col + li < V;
  const bool fresh = positions[first] == 0;
  const float fixed = CHAN ? 1.f : decay[h];

  // state rows are K floats; 4-element access where rows are aligned
  float* sp = state + (((long)slots[s] * heads + h) * V + col + li) * K;
  const bool kvec = K % 4 == 0;
  f32x4 st[KT];
#pragma unroll
  for (int kt = 0; kt < KT; ++kt) {
    const int m = 16 * kt + 4 * lg;
    st[kt] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (vok && !fresh) {
      if (kvec) {
        if (m < K) st[kt] = *reinterpret_cast<const f32x4*>(sp + m);
      } else {
#pragma unroll
        for (int r = 0; r < 4; ++r)
          if (m + r < K) st[kt][r] = sp[m + r];
      }
    }
  }

  const int n = threadIdx.x % KP;
  const int g = KP >= WAVE_SIZE ? wave * WAVE_SIZE / KP : threadIdx.x / KP;
  const bool nok = n < K;
  // A chunk's elements as they come from memory. The loads carry no condition
  // (clamped indexes instead; what is out of range is replaced in convert())
  // and nothing is computed from them in prefetch(), so all of them are in
  // flight together; rows are addressed by scalars where the token is one.
  float ra[TC];
  TQ rq[KT], rk[KT], rv[4];
  const unsigned nc = min(n, K - 1), vc = min(col + li, V - 1);
  // rows of one chunk are less than 2^31 elements apart (the host checks)
  const int a_row = heads * K, q_row = (int)q_stride, k_row = (int)k_stride,
            v_row = (int)v_stride;
  auto prefetch = [&](int t0) {
    const int last = min(TC, len - t0) - 1;
    const long t = first + t0;
    if (CHAN) {
      const float* ab = channel_decay + (t * heads + h) * K;
#pragma unroll
      for (int j = 0; j < TC; ++j) ra[j] = (ab + min(j, last) * a_row)[nc];
    }
    const TQ* qb = q + t * q_stride + (long)hq * K;
    const TQ* kb = k + t * k_stride + (long)hq * K;
#pragma unroll
    for (int j = 0; j < KT; ++j) {
      const int tk = min(g * KT + j, last);
      rq[j] = (qb + tk * q_row)[nc];
      rk[j] = (kb + tk * k_row)[nc];
    }
    const TQ* vb = v + t * v_stride + (long)h * V;
#pragma unroll
    for (int r = 0; r < 4; ++r)
      rv[r] = vb[(unsigned)(min(4 * lg + r, last) * v_row) + vc];
  };
  // widened, q scaled, decay products up to this thread's tokens
  float fq[KT], fk[KT], b[KT], prod;
  f32x4 vv;
  auto convert = [&](int t0) {
    const int cnt = min(TC, len - t0);
    // zero unless ok, without a branch
    auto keep = [](float x, bool ok) {
      return __builtin_bit_cast(float, __builtin_bit_cast(int, x) & (ok ? -1 : 0));
    };
#pragma unroll
    for (int j = 0; j < TC; ++j) {
      if (!CHAN) ra[j] = fixed;
      ra[j] = nok && j < cnt ? ra[j] : 1.f;
    }
#pragma unroll
    for (int j = 0; j < KT; ++j) {
      const bool ok = nok && g * KT + j < cnt;
      fq[j] = keep(ld_f32(rq, j) * q_scale, ok);
      fk[j] = keep(ld_f32(rk, j), ok);
    }
#pragma unroll
    for (int r = 0; r < 4; ++r)
      vv[r] = keep(ld_f32(rv, r), vok && 4 * lg + r < cnt);
    prod = 1.f;
#pragma unroll
    for (int j = 0; j < TC; ++j) {
      prod *= ra[j];
#pragma unroll
      for (int i = 0; i < KT; ++i)
        if (j % KT == i && j / KT == g) b[i] = prod;
    }
  };

  prefetch(0);
  convert(0);
  for (int t0 = 0; t0 < len; t0 += TC) {
    const int cnt = min(TC, len - t0);
    // the last chunk fetches itself once more: no condition around the loads
    const int tn = t0 + TC < len ? t0 + TC : t0;
    const bool bad = !(prod >= MIN_PRODUCT);
    __syncthreads();  // previous chunk consumed
    float kb[KT];
#pragma unroll
    for (int i = 0; i < KT; ++i) {
      kb[i] = fk[i] * __builtin_amdgcn_rcpf(b[i]);
      Qb[(g * KT + i) * KS + n] = fq[i] * b[i];
      Kb[(g * KT + i) * KS + n] = kb[i];
    }
    if constexpr (KT % 4 == 0) {
#pragma unroll
      for (int i = 0; i < KT; i += 4)
        *reinterpret_cast<f32x4*>(Kt + n * TS + g * KT + i) =
            f32x4{kb[i], kb[i + 1], kb[i + 2], kb[i + 3]};
    } else {
#pragma unroll
      for (int i = 0; i < KT; ++i) Kt[n * TS + g * KT + i] = kb[i];
    }
    if (g == 0) Bc[n] = prod;
    const bool wave_bad = __any(bad);
    if (lane == 0) flag[wave] = wave_bad;
    __syncthreads();
    int slow = 0;
#pragma unroll
    for (int w = 0; w < NW; ++w) slow |= flag[w];
    const f32x4 vcur = vv;

    if (__builtin_amdgcn_readfirstlane(slow)) {
      // every thread has read the flags before anything is overwritten
      __syncthreads();
#pragma unroll
      for (int i = 0; i < KT; ++i) {
        Qb[(g * KT + i) * KS + n] = fq[i];
        Kb[(g * KT + i) * KS + n] = fk[i];
      }
      if (g == 0) {
#pragma unroll
        for (int j = 0; j < TC; ++j) Kt[n * TS + j] = ra[j];
      }
      __syncthreads();
      for (int tk = 0; tk < cnt; ++tk) {
        const int r4 = tk & 3;
        const float vs = r4 == 0   ? vcur[0]
                         : r4 == 1 ? vcur[1]
                         : r4 == 2 ? vcur[2]
                                   : vcur[3];
        const float vt = __shfl(vs, (tk >> 2) * 16 + li, WAVE_SIZE);
        float acc = 0.f;
#pragma unroll
        for (int kt = 0; kt < KT; ++kt) {
          const int m = 16 * kt + 4 * lg;
          const f32x4 qq = *reinterpret_cast<const f32x4*>(Qb + tk * KS + m);
          const f32x4 kk = *reinterpret_cast<const f32x4*>(Kb + tk * KS + m);
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            st[kt][r] = st[kt][r] * Kt[(m + r) * TS + tk] + kk[r] * vt;
            acc += qq[r] * st[kt][r];
          }
        }
        acc += __shfl_xor(acc, 16, WAVE_SIZE);
        acc += __shfl_xor(acc, 32, WAVE_SIZE);
        if (lg == 0 && vok)
          o[(long)(first + t0 + tk) * inner + (long)h * V + col + li] = acc;
      }
      prefetch(tn);
      convert(tn);
      continue;
    }
    prefetch(tn);

    // Operands are read from LDS in groups ahead of their products (the
    // scheduling barriers keep the compiler from moving each read back to its
    // use, where every group of four products would wait for it).
    constexpr int PN = (KT + NW - 1) / NW;  // key tiles of P^T per wave
    const bool share = KT >= NW || wave < KT;
    f32x4 pa[PN], pc[PN], cq[KT];
#pragma unroll
    for (int i = 0; i < PN; ++i) {
      const int at = li * KS + 16 * (share ? wave + NW * i : 0) + 4 * lg;
      pa[i] = *reinterpret_cast<const f32x4*>(Kb + at);
      pc[i] = *reinterpret_cast<const f32x4*>(Qb + at);
    }
#pragma unroll
    for (int kt = 0; kt < KT; ++kt)
      cq[kt] = *reinterpret_cast<const f32x4*>(Qb + li * KS + 16 * kt + 4 * lg);
    __builtin_amdgcn_sched_barrier(0);
    // this wave's share of P^T and O^T from the old state: independent chains
    f32x4 p = f32x4{0.f, 0.f, 0.f, 0.f}, oa = p, ob = p;
    if (share) {
#pragma unroll
      for (int i = 0; i < PN; ++i)
#pragma unroll
        for (int r = 0; r < 4; ++r)
          p = __builtin_amdgcn_mfma_f32_16x16x4f32(pa[i][r], pc[i][r], p, 0, 0, 0);
    }
#pragma unroll
    for (int kt = 0; kt < KT; ++kt) {
      oa = __builtin_amdgcn_mfma_f32_16x16x4f32(st[kt][0], cq[kt][0], oa, 0, 0, 0);
      ob = __builtin_amdgcn_mfma_f32_16x16x4f32(st[kt][1], cq[kt][1], ob, 0, 0, 0);
      oa = __builtin_amdgcn_mfma_f32_16x16x4f32(st[kt][2], cq[kt][2], oa, 0, 0, 0);
      ob = __builtin_amdgcn_mfma_f32_16x16x4f32(st[kt][3], cq[kt][3], ob, 0, 0, 0);
    }
    *reinterpret_cast<f32x4*>(Ps + (wave * WAVE_SIZE + lane) * 4) = p;
    f32x4 bc[KT];
#pragma unroll
    for (int kt = 0; kt < KT; ++kt) {
      cq[kt] = *reinterpret_cast<const f32x4*>(Kt + (16 * kt + li) * TS + 4 * lg);
      bc[kt] = *reinterpret_cast<const f32x4*>(Bc + 16 * kt + 4 * lg);
    }
    __builtin_amdgcn_sched_barrier(0);
    // the state takes the chunk
#pragma unroll
    for (int r = 0; r < 4; ++r)
#pragma unroll
      for (int kt = 0; kt < KT; ++kt)
        st[kt] = __builtin_amdgcn_mfma_f32_16x16x4f32(cq[kt][r], vcur[r], st[kt], 0, 0, 0);
#pragma unroll
    for (int kt = 0; kt < KT; ++kt) st[kt] *= bc[kt];
    __syncthreads();
    p = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int w = 0; w < NW; ++w)
      p += *reinterpret_cast<const f32x4*>(Ps + (w * WAVE_SIZE + lane) * 4);
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const float m = 4 * lg + r <= li ? p[r] : 0.f;  // key token <= query token
      if (r & 1) ob = __builtin_amdgcn_mfma_f32_16x16x4f32(vcur[r], m, ob, 0, 0, 0);
      else oa = __builtin_amdgcn_mfma_f32_16x16x4f32(vcur[r], m, oa, 0, 0, 0);
    }
    oa += ob;
    // the next chunk's loads are waited for ahead of this chunk's stores, so
    // that no wait has to include the stores (the empty asm keeps the compiler
    // from sinking the work behind them)
    convert(tn);
#pragma unroll
    for (int i = 0; i < KT; ++i) asm volatile("" : "+v"(fq[i]), "+v"(fk[i]), "+v"(b[i]));
#pragma unroll
    for (int r = 0; r < 4; ++r) asm volatile("" : "+v"(vv[r]));
    asm volatile("" : "+v"(prod));
    if (li < cnt) {
      float* orow = o + (long)(first + t0 + li) * inner + (long)h * V;
      const int c0 = col + 4 * lg;
      if (V % 4 == 0) {
        if (c0 < V) *reinterpret_cast<f32x4*>(orow + c0) = oa;
      } else {
#pragma unroll
        for (int r = 0; r < 4; ++r)
          if (c0 + r < V) orow[c0 + r] = oa[r];
      }
    }
  }
#pragma unroll
  for (int kt = 0; kt < KT; ++kt) {
    const int m = 16 * kt + 4 * lg;
    if (!vok) continue;
    if (kvec) {
      if (m < K) *reinterpret_cast<f32x4*>(sp + m) = st[kt];
    } else {
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (m + r < K) sp[m + r] = st[kt][r];
    }
  }
}

template <int KT, bool CHAN, typename TQ>
hipError_t launch_decay_chunks(float* o, const TQ* q, long q_stride, const TQ* k,
                               long k_stride, const TQ* v, long v_stride,
                               float q_scale, const float* decay,
                               const float* channel_decay, float* state,
                               const long* positions, const int* cu_seqlens,
                               const int* slots, int num_seqs, int heads,
                               int qk_heads, int V, int K, hipStream_t stream) {
  constexpr int KP = 16 * KT;
  const size_t smem = sizeof(float) * (size_t)(2 * 16 * (KP + 4) + KP * 20 + KP +
                                               NW * WAVE_SIZE * 4 + NW);
  auto fn = decay_chunk_kernel<KT, CHAN, TQ>;
  if (smem > 48 * 1024) {
    hipError_t e = hipFuncSetAttribute(
        (const void*)fn, hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem);
    if (e != hipSuccess) return e;
  }
  hipLaunchKernelGGL(fn, dim3(cdiv(V, 64), heads, num_seqs), dim3(NT), smem,
                     stream, o, q, q_stride, k, k_stride, v, v_stride, q_scale,
                     decay, channel_decay, state, positions, cu_seqlens, slots,
                     heads, qk_heads, V, K);
  return hipGetLastError();
}

}  // namespace

extern "C" hipError_t ks_rope_scale_heads(void* out, const void* in,
                                          long in_stride, const void* positions,
                                          const void* inv_freq, int half,
                                          int tokens, int heads_a,
                                          float scale_a, int heads_b,
                                          float scale_b, int dim, int width,
                                          int is_f32, hipStream_t stream) {
  if (tokens == 0) return hipSuccess;
  if (!inv_freq) half = 0;
  if (2 * half > dim || (long)(heads_a + heads_b) * dim > width)
    return hipErrorInvalidValue;
  const size_t smem = sizeof(float) * 2 * (size_t)half;
  if (is_f32)
    hipLaunchKernelGGL(rope_scale_heads_kernel<float>, dim3(tokens), dim3(NT),
                       smem, stream, (float*)out, (const float*)in, in_stride,
                       (const long*)positions, (const float*)inv_freq, half,
                       heads_a, scale_a, heads_b, scale_b, dim, width);
  else
    hipLaunchKernelGGL(rope_scale_heads_kernel<short>, dim3(tokens), dim3(NT),
                       smem, stream, (float*)out, (const short*)in, in_stride,
                       (const long*)positions, (const float*)inv_freq, half,
                       heads_a, scale_a, heads_b, scale_b, dim, width);
  HIP_CHECK_KERNEL();
  return hipSuccess;
}

extern "C" hipError_t ks_unit_norm_heads(void* x, long stride, int tokens,
                                         int heads_a, float scale_a,
                                         int heads_b, float scale_b, int dim,
                                         float eps, hipStream_t stream) {
  if (tokens == 0 || heads_a + heads_b == 0) return hipSuccess;
  hipLaunchKernelGGL(unit_norm_heads_kernel, dim3(tokens), dim3(NT), 0, stream,
                     (float*)x, stride, heads_a, scale_a, heads_b, scale_b, dim,
                     eps);
  HIP_CHECK_KERNEL();
  return hipSuccess;
}

extern "C" hipError_t ks_delta_unit_decay(
    void* x, long stride, void* g, const void* a_raw, long a_stride,
    const void* a_log, const void* dt_bias, int tokens, int qk_heads, int dim,
    float q_scale, float eps, int decays, int is_f32, hipStream_t stream) {
  if (tokens == 0) return hipSuccess;
  if (dim < 1 || decays % dim != 0) return hipErrorInvalidValue;
  if (is_f32)
    hipLaunchKernelGGL(delta_unit_decay_kernel<float>, dim3(tokens), dim3(NT), 0,
                       stream, (float*)x, stride, (float*)g, (const float*)a_raw,
                       a_stride, (const float*)a_log, (const float*)dt_bias,
                       qk_heads, dim, q_scale, eps, decays);
  else
    hipLaunchKernelGGL(delta_unit_decay_kernel<short>, dim3(tokens), dim3(NT), 0,
                       stream, (float*)x, stride, (float*)g, (const short*)a_raw,
                       a_stride, (const float*)a_log, (const float*)dt_bias,
                       qk_heads, dim, q_scale, eps, decays);
  HIP_CHECK_KERNEL();
  return hipSuccess;
}

extern "C" hipError_t ks_lowrank_channel_decay(
    void* out, const void* low, long low_stride, const void* w2,
    const void* bias, float tau, int tokens, int r, int n, int is_f32,
    hipStream_t stream) {
  if (tokens == 0) return hipSuccess;
  if (r < 1 || n < 1 || r > 768 || !(tau > 0.f)) return hipErrorInvalidValue;
  const dim3 grid(cdiv(tokens, DT), cdiv(n, NT));
  const size_t smem = sizeof(float) * (size_t)DT * r;
  if (is_f32)
    hipLaunchKernelGGL(lowrank_channel_decay_kernel<float>, grid, dim3(NT), smem,
                       stream, (float*)out, (const float*)low, low_stride,
                       (const float*)w2, (const float*)bias, 1.0f / tau, tokens,
                       r, n);
  else
    hipLaunchKernelGGL(lowrank_channel_decay_kernel<short>, grid, dim3(NT), smem,
                       stream, (float*)out, (const short*)low, low_stride,
                       (const float*)w2, (const float*)bias, 1.0f / tau, tokens,
                       r, n);
  HIP_CHECK_KERNEL();
  return hipSuccess;
}

#define LSCAN_LAUNCH(RR, PCC, DD)                                             \
  hipLaunchKernelGGL((linear_scan_kernel<RR, PCC, DD, TQ>), grid, dim3(256),  \
                     smem, stream, (float*)o, (const TQ*)q, q_stride,         \
                     (const TQ*)k, k_stride, (const TQ*)v, v_stride, q_scale, \
                     (const float*)decay,                                     \
                     ab_is_f32 ? (const float*)a_raw : nullptr,               \
                     ab_is_f32 ? nullptr : (const short*)a_raw,               \
                     ab_is_f32 ? (const float*)b_raw : nullptr,               \
                     ab_is_f32 ? nullptr : (const short*)b_raw, ab_stride,    \
                     (const float*)a_log, (const float*)dt_bias,              \
                     (const float*)channel_decay, (float*)state, (const long*)positions,                   \
                     (const int*)cu_seqlens, (const int*)slots, heads,        \
                     qk_heads, V, K)

#define LSCAN_LAUNCH_PC(RR, DD)                                               \
  do {                                                                        \
    if (pc == 1) LSCAN_LAUNCH(RR, 1, DD);                                     \
    else if (pc == 2) LSCAN_LAUNCH(RR, 2, DD);                                \
    else LSCAN_LAUNCH(RR, 4, DD);                                             \
  } while (0)

#define LSCAN_LAUNCH_R(DD)                                                    \
  do {                                                                        \
    if (R <= 1) LSCAN_LAUNCH_PC(1, DD);                                       \
    else if (R <= 2) LSCAN_LAUNCH_PC(2, DD);                                  \
    else if (R <= 4) LSCAN_LAUNCH_PC(4, DD);                                  \
    else if (R <= 8) LSCAN_LAUNCH_PC(8, DD);                                  \
    else if (pc == 1) LSCAN_LAUNCH(16, 1, DD);                                \
    else LSCAN_LAUNCH(16, 2, DD);                                             \
  } while (0)

// decay != null: decay form; channel_decay without b_raw: channel-decay form
// (the only one that takes bf16 q, k, v); otherwise a delta form, which reads
// b_raw [T, heads] and either channel_decay [T, heads*K] or a_raw [T, heads] (a and
// b: two column ranges of rows with one stride), a_log and dt_bias.
extern "C" hipError_t ks_linear_scan(
    void* o, const void* q, long q_stride, const void* k, long k_stride,
    const void* v, long v_stride, int qkv_is_f32, float q_scale,
    const void* decay, const void* a_raw,
    const void* b_raw, long ab_stride, int ab_is_f32, const void* a_log,
    const void* dt_bias, const void* channel_decay, void* state,
    const void* positions, const void* cu_seqlens, const void* slots,
    int tokens, int num_seqs, int heads, int qk_heads, int V, int K,
    hipStream_t stream) {
  if (num_seqs == 0) return hipSuccess;
  if (qk_heads <= 0 || heads % qk_heads != 0 || K < 1 || K > 256 || V < 1)
    return hipErrorInvalidValue;
  const bool chan = !decay && channel_decay && !b_raw;
  if (!decay && !chan &&
      (!b_raw || (!channel_decay && (!a_raw || !a_log || !dt_bias))))
    return hipErrorInvalidValue;
  if (!qkv_is_f32 && !chan) return hipErrorInvalidValue;
  const int R = cdiv(K, 16);
  // more tokens than sequences: prompt portions, in chunks on the matrix cores
  if ((decay || chan) && tokens > num_seqs) {
#define CHUNK_ARGS(TT)                                                        \
  (float*)o, (const TT*)q, q_stride, (const TT*)k, k_stride, (const TT*)v,    \
      v_stride, q_scale, (const float*)decay, (const float*)channel_decay,    \
      (float*)state, (const long*)positions, (const int*)cu_seqlens,          \
      (const int*)slots, num_seqs, heads, qk_heads, V, K, stream
#define CHUNK_LAUNCH(CC, TT)                                                  \
  do {                                                                        \
    if (R <= 1) return launch_decay_chunks<1, CC, TT>(CHUNK_ARGS(TT));        \
    if (R <= 2) return launch_decay_chunks<2, CC, TT>(CHUNK_ARGS(TT));        \
    if (R <= 4) return launch_decay_chunks<4, CC, TT>(CHUNK_ARGS(TT));        \
    if (R <= 8) return launch_decay_chunks<8, CC, TT>(CHUNK_ARGS(TT));        \
    return launch_decay_chunks<16, CC, TT>(CHUNK_ARGS(TT));                   \
  } while (0)
    if (q_stride > (1 << 26) || k_stride > (1 << 26) || v_stride > (1 << 26) ||
        (long)heads * K > (1 << 26))
      return hipErrorInvalidValue;
    if (!qkv_is_f32) CHUNK_LAUNCH(true, short);
    if (chan) CHUNK_LAUNCH(true, float);
    CHUNK_LAUNCH(false, float);
  }
  int pc = V > 32 ? 4 : (V > 16 ? 2 : 1);
  if (R > 8 && pc > 2) pc = 2;
  // a block walks its tokens one after the other, so a launch with few
  // (sequence, head) pairs takes narrower tiles to put more blocks on the chip
  while (pc > 1 && (long)cdiv(V, 16 * pc) * heads * num_seqs < 1024) pc >>= 1;
  const int xs = 16 * pc;
  const size_t smem = sizeof(float) * ((size_t)SCAN_TC * ((channel_decay ? 3 : 2) * K + 2 * xs + 3));
  dim3 grid(cdiv(V, xs), heads, num_seqs);
  if (!qkv_is_f32) {
    using TQ = short;
    LSCAN_LAUNCH_R(CHANNEL_DECAY);
  } else {
    using TQ = float;
    if (decay) LSCAN_LAUNCH_R(DECAY);
    else if (chan) LSCAN_LAUNCH_R(CHANNEL_DECAY);
    else if (channel_decay) LSCAN_LAUNCH_R(CHANNEL_DELTA);
    else LSCAN_LAUNCH_R(HEAD_DELTA);
  }
  HIP_CHECK_KERNEL();
  return hipSuccess;
}
