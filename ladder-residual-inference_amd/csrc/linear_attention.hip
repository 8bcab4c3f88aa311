// Linear attention with decay: S_t = diag(a_t) S_{t-1} + k_t v_t^T, o_t = S_t^T q_t per head, S [dk, dv] in fp32.
// The decay is per key channel and data-dependent (gated linear attention: a = sigmoid(z)^(1/tau), z a low-rank
// projection plus bias) or a constant per head (retention); q and k may be rotated ("rotate half" pairs) and scaled.
// The head's output is divided by its root mean square, multiplied by an optional gain and by silu(g).
//
// Everything here is fp32 arithmetic on bf16 or fp32 inputs.  The products with the state run on the matrix cores in
// fp32 (v_mfma_f32_16x16x4_f32): the state, the decays and what they multiply are never rounded to 16 bits.
//
// Prefill (any number of tokens): one workgroup per (sequence, head, segment) walks its tokens 16 at a time.  With
// b_t the running sum of log-decays inside the chunk,
//     Q_t = q_t e^{b_t},  K_s = k_s e^{-b_s},  A = tril(Q K^T)
//     O   = Q S + A V,    S <- diag(e^{b_last}) (S + K^T V).
// A wave owns 16 value columns of S in its accumulators: registers i of a 16-row tile are rows 4 (lane / 16) + i, which
// is exactly the operand a k-step over those four channels wants, so S is multiplied where it lies.  Where a chunk's
// decay is so steep that e^{-b} would leave the safe range, the chunk is walked in runs of 4 or 1 tokens instead.
// Few (sequence, head) pairs: the tokens are cut into segments that run side by side -- first the state each segment
// would leave from zero, then a scan over segments, then the outputs from the right initial states.
//
// Decode (one token): one workgroup per (sequence, head) reads the state once, updates it in place and finishes the
// head's output, rotation, decay, norm and gate included.
#include "mixer_common.h"

namespace {

constexpr int CH = 16;              // tokens per chunk
constexpr float STEEP = -24.0f;     // a run of tokens whose log-decay sums below this is cut into shorter runs
constexpr int AS = 20;              // row stride of the score partials in LDS

struct LinAttn {
  const void *q, *k, *v, *g;
  int64_t ld;
  const float* log_decay;   // [B * S, H * dk], or NULL
  const float* head_decay;  // [H] log-decays, used when log_decay is NULL
  const float* rope;        // [rope_len, rot / 2, 2], or NULL
  const int32_t* pos;
  float* state;             // [B, H, dk, dv]
  const void* norm;         // [dv] or NULL
  void* y;
  int64_t ldy;
  int B, S, H, dk, dv, rot, rope_len;
  float q_scale, k_scale, eps;
  int32_t* err;
  float* seg_state;         // [B * H, nseg, dk, dv]
  float* seg_decay;         // [B * H, nseg, dk]
  int nseg, seg_len;
  // decode only: the low-rank decay projection
  const void *lowrank, *a2, *a_bias;
  int rank;
  float inv_tau;
};

// Element c of a rotated head: pairs (i, i + rot / 2) for i < rot / 2; the rest passes.
__device__ __forceinline__ float rotated(float own, float partner, float c, float s, bool first) {
  return first ? own * c - partner * s : own * c + partner * s;
}

// ---------------------------------------------------------------------------------------------- prefill
// state_only: no outputs, the segment starts from zero and leaves its state and its total log-decay in scratch.
template <typename T, int DKT>
__global__ __launch_bounds__(1024) void k_linear_attention(const LinAttn a, const int state_only) {
  constexpr int DKP = 16 * DKT, QS = DKP + 4;
  extern __shared__ __attribute__((aligned(16))) float sm[];
  const int NW = blockDim.x >> 6;
  float* Qs = sm;                       // [16][QS]
  float* Ks = Qs + CH * QS;             // [16][QS]
  float* Bs = Ks + CH * QS;             // [16][DKP] running log-decay
  float* eC = Bs + CH * DKP;            // [DKP] decay of the run just prepared
  float* Ap = eC + DKP;                 // [NW][16][AS] partial scores
  float* ssq = Ap + NW * CH * AS;       // [NW][16]
  int* steep = reinterpret_cast<int*>(ssq + NW * CH);  // [2][2]

  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, g4 = lane >> 4, l16 = lane & 15;
  const int bh = blockIdx.x, seg = blockIdx.y;
  const int b = bh / a.H, h = bh - b * a.H;
  const int dk = a.dk, dv = a.dv;
  const int s0 = seg * a.seg_len, s1 = min(a.S, s0 + a.seg_len);
  const int pos0 = a.pos[0];
  if (pos0 < 0 || (a.rope && pos0 + a.S > a.rope_len)) {
    if (a.err && tid == 0) *a.err = LR_DEV_POS_RANGE;
    return;
  }
  const T* q = reinterpret_cast<const T*>(a.q) + (int64_t)b * a.S * a.ld + h * dk;
  const T* k = reinterpret_cast<const T*>(a.k) + (int64_t)b * a.S * a.ld + h * dk;
  const T* v = reinterpret_cast<const T*>(a.v) + (int64_t)b * a.S * a.ld + h * dv;
  const T* g = reinterpret_cast<const T*>(a.g) + (int64_t)b * a.S * a.ld + h * dv;
  const float* ld_ = a.log_decay ? a.log_decay + (int64_t)b * a.S * a.H * dk + h * dk : nullptr;
  const float hd_ = a.log_decay ? 0.0f : fmaxf(a.head_decay[h], LOG_DECAY_FLOOR);
  const int col = wave * 16 + l16;      // this lane's value column
  const bool live = wave * 16 < dv, colv = col < dv;
  const bool vec = (dk & 3) == 0;
  const int half = a.rot >> 1;
  const bool vrot = vec && (half & 3) == 0;
  const float gain = (a.norm && colv) ? ldf(reinterpret_cast<const T*>(a.norm) + col) : 1.0f;

  // ---- the state: tile m, register i is row 16 m + 4 g4 + i of this lane's column
  f32x4_t S[DKT];
  {
    const float* src = nullptr;
    if (!state_only) {
      if (a.nseg > 1) src = a.seg_state + ((int64_t)bh * a.nseg + seg) * dk * dv;
      else if (pos0 > 0) src = a.state + (int64_t)bh * dk * dv;
    }
#pragma unroll
    for (int m = 0; m < DKT; ++m)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int c = 16 * m + 4 * g4 + i;
        S[m][i] = (src && colv && c < dk) ? src[(int64_t)c * dv + col] : 0.0f;
      }
  }

  // ---- what one chunk needs from memory, fetched one chunk ahead
  const int it = tid / (DKP / 4), ic = (tid % (DKP / 4)) * 4;   // item: token it, channels ic .. ic + 3
  const bool item = tid < CH * (DKP / 4);
  Quad<T> rq, rk, pq, pk;
  float la[CH], vr[4], gr[4], cs[8];
  rq.zero(); rk.zero(); pq.zero(); pk.zero();
  auto fetch = [&](int c0) {
    if (tid < dk) {
#pragma unroll
      for (int t = 0; t < CH; ++t) {
        const int s = c0 + t;
        la[t] = s < s1 ? (ld_ ? fmaxf(ld_[(int64_t)s * a.H * dk + tid], LOG_DECAY_FLOOR) : hd_) : 0.0f;
      }
    }
    rq.zero(); rk.zero(); pq.zero(); pk.zero();
    const int s = c0 + it;
    if (item && s < s1 && ic < dk) {
      const T* qr = q + (int64_t)s * a.ld;
      const T* kr = k + (int64_t)s * a.ld;
      if (vec) {
        rk.load(kr + ic);
        if (!state_only) rq.load(qr + ic);
      } else {
#pragma unroll
        for (int j = 0; j < 4; ++j)
          if (ic + j < dk) { rk.put(j, kr + ic + j); rq.put(j, qr + ic + j); }
      }
      if (a.rope && ic < a.rot) {
        const float* tr = a.rope + (int64_t)(pos0 + s) * half * 2;
        if (vrot) {
          const int pc = ic < half ? ic + half : ic - half, fi = ic < half ? ic : ic - half;
          pk.load(kr + pc);
          if (!state_only) pq.load(qr + pc);
#pragma unroll
          for (int j = 0; j < 8; ++j) cs[j] = tr[2 * fi + j];
        } else {
#pragma unroll
          for (int j = 0; j < 4; ++j) {
            const int c = ic + j;
            if (c < a.rot && c < dk) {
              const int pc = c < half ? c + half : c - half, fi = c < half ? c : c - half;
              pk.put(j, kr + pc);
              pq.put(j, qr + pc);
              cs[2 * j] = tr[2 * fi];
              cs[2 * j + 1] = tr[2 * fi + 1];
            }
          }
        }
      }
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int sr = c0 + 4 * g4 + i;
      const bool ok = colv && sr < s1;
      vr[i] = ok ? ldf(v + (int64_t)sr * a.ld + col) : 0.0f;
    }
  };
  // (the gate values are needed at the end of the chunk only)
  auto fetch_gate = [&](int c0) {
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int sr = c0 + 4 * g4 + i;
      gr[i] = (colv && sr < s1) ? ldf(g + (int64_t)sr * a.ld + col) : 0.0f;
    }
  };

  // ---- the finished chunk's outputs: norm over the head, gain, gate (its row sums lie in ssq)
  f32x4_t o;
  auto emit = [&](int c0) {
    if (!colv) return;
    float ss[4] = {0, 0, 0, 0};
    for (int w = 0; w * 16 < dv; ++w) {
      const float4 p = *reinterpret_cast<const float4*>(&ssq[w * CH + 4 * g4]);
      ss[0] += p.x; ss[1] += p.y; ss[2] += p.z; ss[3] += p.w;
    }
    T* yr = reinterpret_cast<T*>(a.y) + (int64_t)b * a.S * a.ldy + h * dv + col;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int sr = c0 + 4 * g4 + i;
      if (sr < s1) stf(yr + (int64_t)sr * a.ldy, o[i] * (1.0f / sqrtf(ss[i] / (float)dv + a.eps)) * gain * silu_f(gr[i]));
    }
  };

  float total = 0.0f;   // log-decay of the whole segment, for channel tid
  if (tid < 4) steep[tid] = 0;
  fetch(s0);
  __syncthreads();
  int par = 0;
  for (int c0 = s0; c0 < s1; c0 += CH, par ^= 1) {
    // ---- running log-decay of every channel
    if (tid < dk) {
      float acc = 0.0f, run4 = 0.0f;
      bool s16 = false, s4 = false;
#pragma unroll
      for (int t = 0; t < CH; ++t) {
        acc += la[t];
        run4 = (t & 3) ? run4 + la[t] : la[t];
        s4 = s4 || run4 < STEEP;
        Bs[t * DKP + tid] = acc;
      }
      s16 = acc < STEEP;
      total += acc;
      if (s16) steep[2 * par] = 1;
      if (s4) steep[2 * par + 1] = 1;
    } else if (tid < DKP) {
#pragma unroll
      for (int t = 0; t < CH; ++t) Bs[t * DKP + tid] = 0.0f;
    }
    if (tid < 2) steep[2 * (par ^ 1) + tid] = 0;
    __syncthreads();
    if (!state_only && c0 > s0) emit(c0 - CH);
    if (!state_only) fetch_gate(c0);
    const int run = steep[2 * par + 1] ? 1 : (steep[2 * par] ? 4 : CH);   // uniform over the workgroup
    if (run < CH) {
      __syncthreads();
      if (tid < dk) {   // sums that start again with every run
        float acc = 0.0f;
#pragma unroll
        for (int t = 0; t < CH; ++t) {
          acc = (t % run) ? acc + la[t] : la[t];
          Bs[t * DKP + tid] = acc;
        }
      }
      __syncthreads();
    }
    // ---- this thread's item, rotated and scaled
    float fq[4], fk[4];
    rq.get(fq);
    rk.get(fk);
    if (a.rope && item && ic < a.rot) {
      float fpq[4], fpk[4];
      pq.get(fpq);
      pk.get(fpk);
#pragma unroll
      for (int j = 0; j < 4; ++j)
        if (ic + j < a.rot) {
          fq[j] = rotated(fq[j], fpq[j], cs[2 * j], cs[2 * j + 1], ic + j < half);
          fk[j] = rotated(fk[j], fpk[j], cs[2 * j], cs[2 * j + 1], ic + j < half);
        }
    }
#pragma unroll
    for (int j = 0; j < 4; ++j) { fq[j] *= a.q_scale; fk[j] *= a.k_scale; }
    float vv[4] = {vr[0], vr[1], vr[2], vr[3]};
    o = f32x4_t{0, 0, 0, 0};

    for (int lo = 0; lo < CH; lo += run) {
      if (lo > 0) __syncthreads();
      if (item) {
        const float4 bb = *reinterpret_cast<const float4*>(&Bs[it * DKP + ic]);
        const float e[4] = {expf(bb.x), expf(bb.y), expf(bb.z), expf(bb.w)};
        const bool in = it >= lo && it < lo + run;
        float4 wq, wk;
        wq.x = in ? fq[0] * e[0] : 0.0f; wk.x = in ? fk[0] / e[0] : 0.0f;
        wq.y = in ? fq[1] * e[1] : 0.0f; wk.y = in ? fk[1] / e[1] : 0.0f;
        wq.z = in ? fq[2] * e[2] : 0.0f; wk.z = in ? fk[2] / e[2] : 0.0f;
        wq.w = in ? fq[3] * e[3] : 0.0f; wk.w = in ? fk[3] / e[3] : 0.0f;
        *reinterpret_cast<float4*>(&Qs[it * QS + ic]) = wq;
        *reinterpret_cast<float4*>(&Ks[it * QS + ic]) = wk;
        if (it == lo + run - 1) *reinterpret_cast<float4*>(&eC[ic]) = make_float4(e[0], e[1], e[2], e[3]);
      }
      __syncthreads();
      if (lo + run >= CH && c0 + CH < s1) fetch(c0 + CH);   // everything of this chunk is in registers or LDS
      if (!state_only) {
        // scores, the channels shared out among the waves; then Q S while the partial scores settle
        f32x4_t pa = {0, 0, 0, 0};
        for (int m = wave; m < DKT; m += NW) {
          const float4 x = *reinterpret_cast<const float4*>(&Qs[l16 * QS + 16 * m + 4 * g4]);
          const float4 y = *reinterpret_cast<const float4*>(&Ks[l16 * QS + 16 * m + 4 * g4]);
          pa = __builtin_amdgcn_mfma_f32_16x16x4f32(x.x, y.x, pa, 0, 0, 0);
          pa = __builtin_amdgcn_mfma_f32_16x16x4f32(x.y, y.y, pa, 0, 0, 0);
          pa = __builtin_amdgcn_mfma_f32_16x16x4f32(x.z, y.z, pa, 0, 0, 0);
          pa = __builtin_amdgcn_mfma_f32_16x16x4f32(x.w, y.w, pa, 0, 0, 0);
        }
        if (wave < DKT) {
#pragma unroll
          for (int i = 0; i < 4; ++i) Ap[(wave * CH + 4 * g4 + i) * AS + l16] = pa[i];
        }
        if (live) {
          f32x4_t o2 = {0, 0, 0, 0};
#pragma unroll
          for (int m = 0; m < DKT; ++m) {
            const float4 x = *reinterpret_cast<const float4*>(&Qs[l16 * QS + 16 * m + 4 * g4]);
            o = __builtin_amdgcn_mfma_f32_16x16x4f32(x.x, S[m][0], o, 0, 0, 0);
            o2 = __builtin_amdgcn_mfma_f32_16x16x4f32(x.y, S[m][1], o2, 0, 0, 0);
            o = __builtin_amdgcn_mfma_f32_16x16x4f32(x.z, S[m][2], o, 0, 0, 0);
            o2 = __builtin_amdgcn_mfma_f32_16x16x4f32(x.w, S[m][3], o2, 0, 0, 0);
          }
          o += o2;
        }
        __syncthreads();
      }
      if (live) {
        if (!state_only) {
          float4 as = make_float4(0, 0, 0, 0);
          const int np = NW < DKT ? NW : DKT;
          for (int w = 0; w < np; ++w) {
            const float4 p = *reinterpret_cast<const float4*>(&Ap[(w * CH + l16) * AS + 4 * g4]);
            as.x += p.x; as.y += p.y; as.z += p.z; as.w += p.w;
          }
          const int sc = 4 * g4;   // key token of the first of the four values; the query token is l16
          o = __builtin_amdgcn_mfma_f32_16x16x4f32(sc <= l16 ? as.x : 0.0f, vv[0], o, 0, 0, 0);
          o = __builtin_amdgcn_mfma_f32_16x16x4f32(sc + 1 <= l16 ? as.y : 0.0f, vv[1], o, 0, 0, 0);
          o = __builtin_amdgcn_mfma_f32_16x16x4f32(sc + 2 <= l16 ? as.z : 0.0f, vv[2], o, 0, 0, 0);
          o = __builtin_amdgcn_mfma_f32_16x16x4f32(sc + 3 <= l16 ? as.w : 0.0f, vv[3], o, 0, 0, 0);
        }
#pragma unroll
        for (int m = 0; m < DKT; ++m) {
          const float4 e = *reinterpret_cast<const float4*>(&eC[16 * m + 4 * g4]);
          f32x4_t s = S[m];
#pragma unroll
          for (int i = 0; i < 4; ++i)
            s = __builtin_amdgcn_mfma_f32_16x16x4f32(Ks[(4 * g4 + i) * QS + 16 * m + l16], vv[i], s, 0, 0, 0);
          s[0] *= e.x; s[1] *= e.y; s[2] *= e.z; s[3] *= e.w;
          S[m] = s;
        }
      }
    }
    if (!state_only && live) {
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const float s = row16_sum(colv ? o[i] * o[i] : 0.0f);
        if (l16 == 0) ssq[wave * CH + 4 * g4 + i] = s;
      }
    }
  }
  if (!state_only) {
    __syncthreads();
    emit(s0 + ((s1 - s0 - 1) / CH) * CH);
  }
  // ---- the state the segment leaves
  float* dst = nullptr;
  if (state_only) dst = a.seg_state + ((int64_t)bh * a.nseg + seg + 1) * dk * dv;
  else if (seg == a.nseg - 1) dst = a.state + (int64_t)bh * dk * dv;
  if (dst && colv) {
#pragma unroll
    for (int m = 0; m < DKT; ++m)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int c = 16 * m + 4 * g4 + i;
        if (c < dk) dst[(int64_t)c * dv + col] = S[m][i];
      }
  }
  if (state_only && tid < dk) a.seg_decay[((int64_t)bh * a.nseg + seg) * dk + tid] = total;
}

// Slot j of seg_state holds the state segment j - 1 leaves from zero (j >= 1); afterwards the one segment j starts from.
__global__ __launch_bounds__(256) void k_linear_attention_scan(const LinAttn a) {
  const int bh = blockIdx.x;
  const int n = a.dk * a.dv;
  const int e = blockIdx.y * 256 + threadIdx.x;
  if (e >= n) return;
  const int c = e / a.dv;
  float* slot = a.seg_state + (int64_t)bh * a.nseg * n + e;
  const float* dec = a.seg_decay + (int64_t)bh * a.nseg * a.dk + c;
  float acc = a.pos[0] > 0 ? a.state[(int64_t)bh * n + e] : 0.0f;
  slot[0] = acc;
  for (int j = 1; j < a.nseg; ++j) {
    acc = acc * expf(dec[(int64_t)(j - 1) * a.dk]) + slot[(int64_t)j * n];
    slot[(int64_t)j * n] = acc;
  }
}

// log-decays of a gated linear attention: out[row, c] = log sigmoid(a2[c, :] . lowrank[row, :] + bias[c]) / tau
template <typename T>
__global__ __launch_bounds__(256) void k_gla_log_decay(const T* __restrict__ lowrank, int64_t ld, const T* __restrict__ a2,
                                                       const T* __restrict__ bias, float* __restrict__ out, int rows,
                                                       int n, int rank, float inv_tau) {
  constexpr int R = 8;
  extern __shared__ __attribute__((aligned(16))) float tl[];   // [R][rank]
  const int r0 = blockIdx.x * R, nr = min(R, rows - r0);
  for (int i = threadIdx.x; i < R * rank; i += 256) {
    const int r = i / rank, j = i - r * rank;
    tl[i] = r < nr ? ldf(lowrank + (int64_t)(r0 + r) * ld + j) : 0.0f;
  }
  __syncthreads();
  for (int c = blockIdx.y * 256 + threadIdx.x; c < n; c += gridDim.y * 256) {
    float z[R];
    const float bz = ldf(bias + c);
#pragma unroll
    for (int r = 0; r < R; ++r) z[r] = bz;
    const T* w = a2 + (int64_t)c * rank;
    for (int j = 0; j < rank; ++j) {
      const float wj = ldf(w + j);
#pragma unroll
      for (int r = 0; r < R; ++r) z[r] = fmaf(wj, tl[r * rank + j], z[r]);
    }
#pragma unroll
    for (int r = 0; r < R; ++r)
      if (r < nr) out[(int64_t)(r0 + r) * n + c] = log_sigmoid_f(z[r]) * inv_tau;
  }
}

// ---------------------------------------------------------------------------------------------- decode
template <typename T, int V>
__global__ __launch_bounds__(1024) void k_linear_attention_step(const LinAttn a) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  const int bh = blockIdx.x, b = bh / a.H, h = bh - b * a.H, tid = threadIdx.x, nt = blockDim.x;
  const int dk = a.dk, dv = a.dv, half = a.rot >> 1;
  float* qs = sm;
  float* ks = qs + dk;
  float* es = ks + dk;
  float* red = es + dk;               // [rows][dv]
  const int p = a.pos[0];
  if (p < 0 || (a.rope && p >= a.rope_len)) {
    if (a.err && tid == 0) *a.err = LR_DEV_POS_RANGE;
    return;
  }
  const int nq = dv / V, nrow = nt / nq;      // threads along dv, state rows side by side
  const int vq = tid % nq, r0 = tid / nq;
  const bool on = r0 < nrow;
  float* st = a.state + (int64_t)bh * dk * dv + vq * V;
  constexpr int U = 4;
  float s[U][V];
  auto load = [&](int r) {
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int c = r + u * nrow;
      const bool ok = on && c < dk && p > 0;
      if constexpr (V == 4) {
        const float4 t = ok ? *reinterpret_cast<const float4*>(st + (int64_t)c * dv) : make_float4(0, 0, 0, 0);
        s[u][0] = t.x; s[u][1] = t.y; s[u][2] = t.z; s[u][3] = t.w;
      } else {
        s[u][0] = ok ? st[(int64_t)c * dv] : 0.0f;
      }
    }
  };
  load(r0);
  const T* q = reinterpret_cast<const T*>(a.q) + (int64_t)b * a.ld + h * dk;
  const T* k = reinterpret_cast<const T*>(a.k) + (int64_t)b * a.ld + h * dk;
  float vv[V];
#pragma unroll
  for (int j = 0; j < V; ++j) vv[j] = ldf(reinterpret_cast<const T*>(a.v) + (int64_t)b * a.ld + h * dv + vq * V + j);
  for (int c = tid; c < dk; c += nt) {
    float fq = ldf(q + c), fk = ldf(k + c);
    if (a.rope && c < a.rot) {
      const int pc = c < half ? c + half : c - half, fi = c < half ? c : c - half;
      const float* tr = a.rope + ((int64_t)p * half + fi) * 2;
      fq = rotated(fq, ldf(q + pc), tr[0], tr[1], c < half);
      fk = rotated(fk, ldf(k + pc), tr[0], tr[1], c < half);
    }
    float la;
    if (a.lowrank) {
      const T* t = reinterpret_cast<const T*>(a.lowrank) + (int64_t)b * a.ld;
      const T* w = reinterpret_cast<const T*>(a.a2) + (int64_t)(h * dk + c) * a.rank;
      float z = ldf(reinterpret_cast<const T*>(a.a_bias) + h * dk + c);
      for (int j = 0; j < a.rank; ++j) z = fmaf(ldf(w + j), ldf(t + j), z);
      la = log_sigmoid_f(z) * a.inv_tau;
    } else {
      la = a.head_decay[h];
    }
    qs[c] = fq * a.q_scale;
    ks[c] = fk * a.k_scale;
    es[c] = expf(la);
  }
  __syncthreads();
  float acc[V];
#pragma unroll
  for (int j = 0; j < V; ++j) acc[j] = 0.0f;
  for (int r = r0; r < dk; r += U * nrow) {
    if (r != r0) load(r);
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int c = r + u * nrow;
      if (on && c < dk) {
        const float e = es[c], kk = ks[c], qq = qs[c];
        float n[V];
#pragma unroll
        for (int j = 0; j < V; ++j) {
          n[j] = fmaf(e, s[u][j], kk * vv[j]);
          acc[j] = fmaf(n[j], qq, acc[j]);
        }
        if constexpr (V == 4) *reinterpret_cast<float4*>(st + (int64_t)c * dv) = make_float4(n[0], n[1], n[2], n[3]);
        else st[(int64_t)c * dv] = n[0];
      }
    }
  }
  if (on) {
#pragma unroll
    for (int j = 0; j < V; ++j) red[r0 * dv + vq * V + j] = acc[j];
  }
  __syncthreads();
  // the head's output, its mean square, gain and gate
  float mine = 0.0f, ss = 0.0f;
  __shared__ float wsum[16];
  for (int d = tid; d < dv; d += nt) {
    float t = 0.0f;
    for (int r = 0; r < nrow; ++r) t += red[r * dv + d];
    red[d] = t;        // (row 0 of column d is read by this thread only)
    ss += t * t;
    mine = t;
  }
  ss = wave_sum(ss);
  if ((tid & 63) == 0) wsum[tid >> 6] = ss;
  __syncthreads();
  float tot = 0.0f;
  for (int w = 0; w < (nt >> 6); ++w) tot += wsum[w];
  const float inv = 1.0f / sqrtf(tot / (float)dv + a.eps);
  (void)mine;
  for (int d = tid; d < dv; d += nt) {
    const float gain = a.norm ? ldf(reinterpret_cast<const T*>(a.norm) + d) : 1.0f;
    const float gate = silu_f(ldf(reinterpret_cast<const T*>(a.g) + (int64_t)b * a.ld + h * dv + d));
    stf(reinterpret_cast<T*>(a.y) + (int64_t)b * a.ldy + h * dv + d, red[d] * inv * gain * gate);
  }
}

// ---------------------------------------------------------------------------------------------- host
constexpr int MAX_DIM = 256;

int fill(const lr_linear_attention_t* d, LinAttn& a) {
  if (d == nullptr || d->q == nullptr || d->k == nullptr || d->v == nullptr || d->g == nullptr || d->pos == nullptr ||
      d->y == nullptr)
    return LR_E_NULL;
  LR_REQUIRE_PTR(d->state);
  if (d->dtype != LR_BF16 && d->dtype != LR_F32) return LR_E_UNSUPPORTED;
  if (d->B <= 0 || d->S <= 0 || d->H <= 0 || d->dk <= 0 || d->dv <= 0) return LR_E_SHAPE;
  if (d->ld < (int64_t)d->H * d->dk || d->ld < (int64_t)d->H * d->dv || d->ldy < (int64_t)d->H * d->dv) return LR_E_SHAPE;
  if ((int64_t)d->B * d->H > 0x7fffffff || (int64_t)d->B * d->S > 0x7fffffff) return LR_E_SHAPE;
  if (d->ld % 8) return LR_E_ALIGN;
  if (d->dk > MAX_DIM || d->dv > MAX_DIM) return LR_E_UNSUPPORTED;
  const bool gated = d->lowrank != nullptr;
  if (gated && (d->a2 == nullptr || d->a_bias == nullptr)) return LR_E_NULL;
  if (gated && (d->rank <= 0 || !(d->tau > 0.0f))) return LR_E_SHAPE;
  if (gated && d->rank > 1024) return LR_E_UNSUPPORTED;
  if (!gated && d->head_decay == nullptr) return LR_E_NULL;
  if (d->rope && (d->rot_dims <= 0 || d->rot_dims % 2 || d->rot_dims > d->dk || d->rope_len <= 0)) return LR_E_SHAPE;
  if (!(d->eps >= 0.0f)) return LR_E_SHAPE;
  a = LinAttn{};
  a.q = d->q; a.k = d->k; a.v = d->v; a.g = d->g; a.ld = d->ld;
  a.head_decay = d->head_decay; a.rope = d->rope; a.pos = d->pos; a.state = d->state; a.norm = d->norm; a.y = d->y;
  a.ldy = d->ldy; a.B = d->B; a.S = d->S; a.H = d->H; a.dk = d->dk; a.dv = d->dv;
  a.rot = d->rope ? d->rot_dims : 0; a.rope_len = d->rope_len; a.q_scale = d->q_scale; a.k_scale = d->k_scale;
  a.eps = d->eps; a.err = d->err; a.lowrank = d->lowrank; a.a2 = d->a2; a.a_bias = d->a_bias; a.rank = d->rank;
  a.inv_tau = gated ? 1.0f / d->tau : 0.0f;
  a.nseg = 1; a.seg_len = d->S;
  return LR_OK;
}

// Segments: enough workgroups to fill the chip, none shorter than 64 tokens.
int segments(int B, int S, int H) {
  const int64_t wgs = (int64_t)B * H;
  int64_t want = (512 + wgs - 1) / wgs;
  const int64_t most = S / 64;
  if (want > most) want = most;
  return want < 1 ? 1 : (int)want;
}

size_t align16(size_t n) { return (n + 15) & ~(size_t)15; }

template <typename T, int DKT>
int launch(const LinAttn& a, int state_only, hipStream_t s) {
  constexpr int DKP = 16 * DKT;
  int nw = (a.dv + 15) / 16;
  if (nw < DKT) nw = DKT;             // one item of the chunk's preparation per thread
  const size_t lds = sizeof(float) * ((size_t)2 * CH * (DKP + 4) + CH * DKP + DKP + (size_t)nw * CH * AS + nw * CH + 4);
  static std::atomic<unsigned long long> raised{0};
  if (!lr_raise_lds_limit(reinterpret_cast<const void*>(&k_linear_attention<T, DKT>), lds, raised)) return LR_E_LAUNCH;
  k_linear_attention<T, DKT><<<dim3(a.B * a.H, state_only ? a.nseg - 1 : a.nseg), dim3(64 * nw), lds, s>>>(a, state_only);
  return lr_launch_status();
}

template <typename T>
int launch_dk(const LinAttn& a, int state_only, hipStream_t s) {
  if (a.dk <= 32) return launch<T, 2>(a, state_only, s);
  if (a.dk <= 64) return launch<T, 4>(a, state_only, s);
  if (a.dk <= 128) return launch<T, 8>(a, state_only, s);
  return launch<T, 16>(a, state_only, s);
}

template <typename T>
int prefill(LinAttn& a, const lr_linear_attention_t* d, hipStream_t s) {
  char* p = reinterpret_cast<char*>(d->scratch);
  if (a.lowrank) {
    a.log_decay = reinterpret_cast<float*>(p);
    p += align16((size_t)a.B * a.S * a.H * a.dk * sizeof(float));
    const int rows = a.B * a.S, n = a.H * a.dk;
    k_gla_log_decay<T><<<dim3((rows + 7) / 8, (n + 2047) / 2048), dim3(256), (size_t)8 * a.rank * sizeof(float), s>>>(
        (const T*)a.lowrank, a.ld, (const T*)a.a2, (const T*)a.a_bias, const_cast<float*>(a.log_decay), rows, n, a.rank,
        a.inv_tau);
  }
  a.nseg = segments(a.B, a.S, a.H);
  if (a.nseg > 1) {
    a.seg_len = ((a.S + a.nseg - 1) / a.nseg + CH - 1) / CH * CH;
    a.nseg = (a.S + a.seg_len - 1) / a.seg_len;
  }
  if (a.nseg > 1) {
    a.seg_state = reinterpret_cast<float*>(p);
    p += align16((size_t)a.B * a.H * a.nseg * a.dk * a.dv * sizeof(float));
    a.seg_decay = reinterpret_cast<float*>(p);
    const int rc = launch_dk<T>(a, 1, s);
    if (rc != LR_OK) return rc;
    k_linear_attention_scan<<<dim3(a.B * a.H, (a.dk * a.dv + 255) / 256), dim3(256), 0, s>>>(a);
  }
  return launch_dk<T>(a, 0, s);
}

template <typename T>
int step(const LinAttn& a, hipStream_t s) {
  const int v = a.dv % 4 == 0 ? 4 : 1;
  const int nq = a.dv / v;
  // about 16 state values per thread, at least one state row side by side
  int nt = (int)(((int64_t)a.dk * a.dv / 16 + 63) / 64 * 64);
  if (nt < nq) nt = (nq + 63) / 64 * 64;
  nt = nt < 64 ? 64 : (nt > 1024 ? 1024 : nt);
  const size_t lds = sizeof(float) * ((size_t)3 * a.dk + (size_t)(nt / nq) * a.dv + 4);
  if (v == 4) {
    k_linear_attention_step<T, 4><<<dim3(a.B * a.H), dim3(nt), lds, s>>>(a);
  } else {
    k_linear_attention_step<T, 1><<<dim3(a.B * a.H), dim3(nt), lds, s>>>(a);
  }
  return lr_launch_status();
}

}  // namespace

extern "C" size_t lr_linear_attention_scratch_bytes(int B, int S, int H, int dk, int dv, int gated) {
  if (B <= 0 || S <= 0 || H <= 0 || dk <= 0 || dv <= 0 || S == 1) return 0;
  size_t n = gated ? align16((size_t)B * S * H * dk * sizeof(float)) : 0;
  const int ns = segments(B, S, H);
  if (ns > 1) n += align16((size_t)B * H * ns * dk * dv * sizeof(float)) + align16((size_t)B * H * ns * dk * sizeof(float));
  return n;
}

extern "C" int lr_linear_attention(const lr_linear_attention_t* d, lr_stream_t stream) {
  LinAttn a;
  const int rc = fill(d, a);
  if (rc != LR_OK) return rc;
  hipStream_t s = (hipStream_t)stream;
  if (d->S == 1) return d->dtype == LR_F32 ? step<float>(a, s) : step<u16>(a, s);
  const size_t need = lr_linear_attention_scratch_bytes(d->B, d->S, d->H, d->dk, d->dv, d->lowrank != nullptr);
  if (need > 0) {
    LR_REQUIRE_PTR(d->scratch);
    if (d->scratch_bytes < need) return LR_E_SHAPE;
  }
  return d->dtype == LR_F32 ? prefill<float>(a, d, s) : prefill<u16>(a, d, s);
}
