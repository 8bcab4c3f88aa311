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
// A wave owns 32 value columns of S in its accumulators: registers i of a 16-row tile are rows 4 (lane / 16) + i, which
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
constexpr float STEEP = -34.0f;     // a run of tokens whose log2-decay sums below this is cut into shorter runs
constexpr int AS = 20;              // row stride of the score partials in LDS

struct LinAttn {
  const void *q, *k, *v, *g;
  int64_t ld;
  const float* log_decay;   // [B * S, H * dk] base-2 logarithms, or NULL
  const float* head_decay;  // [H] natural logarithms, used when log_decay is NULL
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
// Eight consecutive channels as stored.
template <typename T> struct Oct;
template <> struct Oct<u16> {
  uint4 r;
  __device__ __forceinline__ void load(rsrc_t p, int off) {
    const u32x4_t t = __builtin_amdgcn_raw_buffer_load_b128(p, off, 0, 0);
    r = make_uint4(t.x, t.y, t.z, t.w);
  }
  __device__ __forceinline__ void get(float* f) const { unpack8(r, f); }
};
template <> struct Oct<float> {
  u32x4_t a, b;
  __device__ __forceinline__ void load(rsrc_t p, int off) {
    a = __builtin_amdgcn_raw_buffer_load_b128(p, off, 0, 0);
    b = __builtin_amdgcn_raw_buffer_load_b128(p, off + 16, 0, 0);
  }
  __device__ __forceinline__ void get(float* f) const {
#pragma unroll
    for (int j = 0; j < 4; ++j) { f[j] = __uint_as_float(a[j]); f[4 + j] = __uint_as_float(b[j]); }
  }
};

__device__ __forceinline__ void lds_st8(float* p, const float* f) {
  *reinterpret_cast<float4*>(p) = make_float4(f[0], f[1], f[2], f[3]);
  *reinterpret_cast<float4*>(p + 4) = make_float4(f[4], f[5], f[6], f[7]);
}

constexpr int MAX_NW = 8;   // waves per workgroup, 32 value columns each

// state_only: no outputs, the segment starts from zero and leaves its state and its total log-decay in scratch.
// VEC: dk is a multiple of 8, rotation pairs lie a multiple of 8 apart and rows are 16-byte aligned.
template <typename T, int DKT, bool VEC>
__global__ __launch_bounds__(64 * MAX_NW) void k_linear_attention(const LinAttn a, const int state_only) {
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
  const int s0 = seg * a.seg_len, len = min(a.S - s0, a.seg_len);
  const int pos0 = a.pos[0];
  if (pos0 < 0 || (a.rope && pos0 + a.S > a.rope_len)) {
    if (a.err && tid == 0) *a.err = LR_DEV_POS_RANGE;
    return;
  }
  // (uniform pointers to the current chunk's first row, per-lane offsets that stay the same from chunk to chunk)
  const int64_t row0 = (int64_t)b * a.S + s0;
  const T* q = reinterpret_cast<const T*>(a.q) + row0 * a.ld + h * dk;
  const T* k = reinterpret_cast<const T*>(a.k) + row0 * a.ld + h * dk;
  const T* v = reinterpret_cast<const T*>(a.v) + row0 * a.ld + h * dv;
  const T* g = reinterpret_cast<const T*>(a.g) + row0 * a.ld + h * dv;
  T* y = reinterpret_cast<T*>(a.y) + row0 * a.ldy + h * dv;
  const int lstr = a.H * dk;
  const float* lg = a.log_decay ? a.log_decay + row0 * lstr + h * dk : nullptr;
  const float lh = a.log_decay ? 0.0f : fmaxf(a.head_decay[h] * LOG2E, LOG_DECAY_FLOOR);
  const int half = a.rot >> 1;
  const float* tab = a.rope ? a.rope + (int64_t)(pos0 + s0) * half * 2 : nullptr;
  const int c0w = wave * 32;            // the wave's value columns: c0w + l16 and c0w + 16 + l16
  const bool live = c0w < dv;
  const bool cv[2] = {c0w + l16 < dv, c0w + 16 + l16 < dv};
  float gain[2] = {1.0f, 1.0f};
  if (a.norm) {
#pragma unroll
    for (int n = 0; n < 2; ++n)
      if (cv[n]) gain[n] = ldf(reinterpret_cast<const T*>(a.norm) + c0w + 16 * n + l16);
  }

  const int col[2] = {cv[0] ? c0w + l16 : 0, cv[1] ? c0w + 16 + l16 : 0};   // (loads never branch: they go to a valid
                                                                            // place and the value is dropped)
  // ---- the state: tile (m, n), register i is row 16 m + 4 g4 + i of column c0w + 16 n + l16
  f32x4_t S[DKT][2];
  {
    const bool have = !state_only && (a.nseg > 1 || pos0 > 0);
    const float* src = a.nseg > 1 ? a.seg_state + ((int64_t)bh * a.nseg + seg) * dk * dv : a.state + (int64_t)bh * dk * dv;
#pragma unroll
    for (int m = 0; m < DKT; ++m)
#pragma unroll
      for (int n = 0; n < 2; ++n) S[m][n] = f32x4_t{0, 0, 0, 0};
    if (have) {
#pragma unroll
      for (int m = 0; m < DKT; ++m)
#pragma unroll
        for (int n = 0; n < 2; ++n)
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            const int c = 16 * m + 4 * g4 + i;
            const float t = src[(c < dk ? c : 0) * dv + col[n]];
            S[m][n][i] = (cv[n] && c < dk) ? t : 0.0f;
          }
    }
  }

  // ---- what one chunk needs from memory, fetched while the chunk before is worked on
  constexpr int SZ = (int)sizeof(T);
  const int ldb = (int)a.ld * SZ;       // bytes from token to token
  const int it = tid / (DKP / 8), ic = (tid % (DKP / 8)) * 8;   // item: token it, channels ic .. ic + 7
  const bool item = tid < CH * (DKP / 8) && ic < dk;
  const bool turns = a.rope && ic < a.rot;
  const int pc = ic < half ? ic + half : ic - half, fi = ic < half ? ic : ic - half;
  const int o_item = item ? it * ldb + ic * SZ : NOWHERE;
  const int o_pair = item && turns ? it * ldb + pc * SZ : NOWHERE;
  const int o_cs = item && turns ? (it * half + fi) * 8 : NOWHERE;
  const int o_la = tid < dk ? tid * 4 : NOWHERE;
  const int o_col[2] = {cv[0] ? 4 * g4 * ldb + (c0w + l16) * SZ : NOWHERE,
                        cv[1] ? 4 * g4 * ldb + (c0w + 16 + l16) * SZ : NOWHERE};
  const int ldyb = (int)a.ldy * SZ;
  const int o_y[2] = {cv[0] ? 4 * g4 * ldyb + (c0w + l16) * SZ : NOWHERE,
                      cv[1] ? 4 * g4 * ldyb + (c0w + 16 + l16) * SZ : NOWHERE};
  Oct<T> rq, rk, pq, pk;
  float la[CH], cs[16];
  T vr[2][4], gr[2][4];
  // a chunk of nt tokens starting at row c0 of the segment: its rows of q / k / v / g as a buffer that ends with them
  auto rows_of = [&](const T* base, int c0, int cols) {
    const int nt = min(len - c0, CH);
    return buffer_of(base + (int64_t)c0 * a.ld, (nt - 1) * ldb + cols * SZ);
  };
  auto fetch = [&](int c0) {            // c0: chunk start, from the segment's start
    const int nt = min(len - c0, CH);
    if (lg) {
      const rsrc_t r = buffer_of(lg + (int64_t)c0 * lstr, ((nt - 1) * lstr + dk) * 4);
      int off = fresh(o_la);
#pragma unroll
      for (int t = 0; t < CH; ++t, off += lstr * 4) la[t] = buf_ld(r, off, 0.0f);
    }
    if constexpr (VEC) {
      const rsrc_t rk_ = rows_of(k, c0, dk), rq_ = rows_of(q, c0, dk);
      rk.load(rk_, o_item);
      if (!state_only) rq.load(rq_, o_item);
      if (a.rope) {
        pk.load(rk_, o_pair);
        if (!state_only) pq.load(rq_, o_pair);
        const rsrc_t rt = buffer_of(tab + (int64_t)c0 * half * 2, nt * half * 8);
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const u32x4_t t4 = __builtin_amdgcn_raw_buffer_load_b128(rt, o_cs + 16 * j, 0, 0);
#pragma unroll
          for (int e = 0; e < 4; ++e) cs[4 * j + e] = __uint_as_float(t4[e]);
        }
      }
    }
    const rsrc_t rv = rows_of(v, c0, dv);
    int off[2] = {fresh(o_col[0]), fresh(o_col[1])};
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int n = 0; n < 2; ++n) vr[n][i] = buf_ld(rv, off[n] + i * ldb, T());
  };
  // (the gate values are needed at the end of the chunk only)
  auto fetch_gate = [&](int c0) {
    const rsrc_t rg = rows_of(g, c0, dv);
    int off[2] = {fresh(o_col[0]), fresh(o_col[1])};
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int n = 0; n < 2; ++n) gr[n][i] = buf_ld(rg, off[n] + i * ldb, T());
  };
  // this thread's eight channels of q and k, rotated and scaled
  auto item_values = [&](int c0, float* fq, float* fk) {
    if constexpr (VEC) {
      rq.get(fq);
      rk.get(fk);
      if (turns) {
        float xq[8], xk[8];
        pk.get(xk);
        if (!state_only) pq.get(xq);
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          const float sn = ic < half ? -cs[2 * j + 1] : cs[2 * j + 1];
          fk[j] = fk[j] * cs[2 * j] + xk[j] * sn;
          if (!state_only) fq[j] = fq[j] * cs[2 * j] + xq[j] * sn;
        }
      }
    } else {
#pragma unroll
      for (int j = 0; j < 8; ++j) fq[j] = fk[j] = 0.0f;
      if (item && it < len - c0) {
        const T* kr = k + (int64_t)(c0 + it) * a.ld;
        const T* qr = q + (int64_t)(c0 + it) * a.ld;
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          const int c = ic + j;
          if (c < dk) {
            fq[j] = ldf(qr + c);
            fk[j] = ldf(kr + c);
            if (a.rope && c < a.rot) {
              const int p = c < half ? c + half : c - half, f = c < half ? c : c - half;
              const float* tr = tab + ((int64_t)(c0 + it) * half + f) * 2;
              fq[j] = rotated(fq[j], ldf(qr + p), tr[0], tr[1], c < half);
              fk[j] = rotated(fk[j], ldf(kr + p), tr[0], tr[1], c < half);
            }
          }
        }
      }
    }
#pragma unroll
    for (int j = 0; j < 8; ++j) { fq[j] *= a.q_scale; fk[j] *= a.k_scale; }
  };

  // ---- the finished chunk's outputs: norm over the head, gain, gate (its row sums lie in ssq)
  f32x4_t o[2];
  const float inv_dv = 1.0f / (float)dv;
  auto emit = [&](int c0) {
    if (!live) return;
    float ss[4] = {0, 0, 0, 0};
#pragma clang loop unroll(disable)
    for (int w = 0; w * 32 < dv; ++w) {
      const float4 p = *reinterpret_cast<const float4*>(&ssq[w * CH + 4 * g4]);
      ss[0] += p.x; ss[1] += p.y; ss[2] += p.z; ss[3] += p.w;
    }
    const rsrc_t ry = buffer_of(y + (int64_t)c0 * a.ldy, (min(len - c0, CH) - 1) * ldyb + dv * SZ);
    int off[2] = {fresh(o_y[0]), fresh(o_y[1])};
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const float inv = rsq_f(ss[i] * inv_dv + a.eps);
#pragma unroll
      for (int n = 0; n < 2; ++n)
        buf_st(ry, off[n] + i * ldyb, o[n][i] * inv * gain[n] * silu_f(ldf(&gr[n][i])), T());
    }
  };

  float total = 0.0f;   // log2-decay of the whole segment, for channel tid
  if (tid < 4) steep[tid] = 0;
  fetch(0);
  __syncthreads();
  int par = 0;
  for (int c0 = 0; c0 < len; c0 += CH, par ^= 1) {
    // ---- running log-decay of every channel
    if (tid < dk) {
      float acc = 0.0f, run4 = 0.0f;
      bool s4 = false;
#pragma unroll
      for (int t = 0; t < CH; ++t) {
        if (!lg) la[t] = t < len - c0 ? lh : 0.0f;
        la[t] = fmaxf(la[t], LOG_DECAY_FLOOR);
        acc += la[t];
        run4 = (t & 3) ? run4 + la[t] : la[t];
        s4 = s4 || run4 < STEEP;
        Bs[t * DKP + tid] = acc;
      }
      total += acc;
      if (acc < STEEP) steep[2 * par] = 1;
      if (s4) steep[2 * par + 1] = 1;
    }
    if (tid < 2) steep[2 * (par ^ 1) + tid] = 0;
    float fq[8], fk[8];
    item_values(c0, fq, fk);
    __syncthreads();
    if (!state_only) {
      if (c0 > 0) emit(c0 - CH);
      fetch_gate(c0);
    }
    const int run = __builtin_amdgcn_readfirstlane(steep[2 * par + 1] ? 1 : (steep[2 * par] ? 4 : CH));
    if (run < CH) {
      __syncthreads();
      if (tid < dk) {   // sums that start again with every run
        float acc = 0.0f;
#pragma unroll
        for (int t = 0; t < CH; ++t) {
          acc = (t & (run - 1)) ? acc + la[t] : la[t];
          Bs[t * DKP + tid] = acc;
        }
      }
      __syncthreads();
    }
    float vv[2][4];
#pragma unroll
    for (int n = 0; n < 2; ++n) {
#pragma unroll
      for (int i = 0; i < 4; ++i) vv[n][i] = ldf(&vr[n][i]);
      o[n] = f32x4_t{0, 0, 0, 0};
    }

    for (int lo = 0; lo < CH; lo += run) {
      if (lo > 0) __syncthreads();
      if (tid < CH * (DKP / 8)) {
        float e[8], wq[8], wk[8];
        const bool in = it >= lo && it < lo + run;
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          const float bb = ic + j < dk ? Bs[it * DKP + ic + j] : 0.0f;
          e[j] = exp2_f(bb);
          wq[j] = in ? fq[j] * e[j] : 0.0f;
          wk[j] = in ? fk[j] * exp2_f(-bb) : 0.0f;
        }
        lds_st8(&Qs[it * QS + ic], wq);
        lds_st8(&Ks[it * QS + ic], wk);
        if (it == lo + run - 1) lds_st8(&eC[ic], e);
      }
      __syncthreads();
      if (lo + run >= CH && c0 + CH < len) fetch(c0 + CH);   // everything of this chunk is in registers or LDS
      if (!state_only) {
        // scores, the channels shared out among the waves; then Q S while the partial scores settle
        if (wave < DKT) {
          f32x4_t pa = {0, 0, 0, 0};
#pragma clang loop unroll(disable)
          for (int m = wave; m < DKT; m += NW) {
            const float4 x = *reinterpret_cast<const float4*>(&Qs[l16 * QS + 16 * m + 4 * g4]);
            const float4 z = *reinterpret_cast<const float4*>(&Ks[l16 * QS + 16 * m + 4 * g4]);
            pa = __builtin_amdgcn_mfma_f32_16x16x4f32(x.x, z.x, pa, 0, 0, 0);
            pa = __builtin_amdgcn_mfma_f32_16x16x4f32(x.y, z.y, pa, 0, 0, 0);
            pa = __builtin_amdgcn_mfma_f32_16x16x4f32(x.z, z.z, pa, 0, 0, 0);
            pa = __builtin_amdgcn_mfma_f32_16x16x4f32(x.w, z.w, pa, 0, 0, 0);
          }
#pragma unroll
          for (int i = 0; i < 4; ++i) Ap[(wave * CH + 4 * g4 + i) * AS + l16] = pa[i];
        }
        if (live) {
#pragma unroll
          for (int m = 0; m < DKT; ++m) {
            const float4 x = *reinterpret_cast<const float4*>(&Qs[l16 * QS + 16 * m + 4 * g4]);
            const float xe[4] = {x.x, x.y, x.z, x.w};
#pragma unroll
            for (int i = 0; i < 4; ++i) {
              o[0] = __builtin_amdgcn_mfma_f32_16x16x4f32(xe[i], S[m][0][i], o[0], 0, 0, 0);
              o[1] = __builtin_amdgcn_mfma_f32_16x16x4f32(xe[i], S[m][1][i], o[1], 0, 0, 0);
            }
          }
        }
        __syncthreads();
      }
      if (live) {
        if (!state_only) {
          float as[4] = {0, 0, 0, 0};
          const int np = NW < DKT ? NW : DKT;
#pragma clang loop unroll(disable)
          for (int w = 0; w < np; ++w) {
            const float4 p = *reinterpret_cast<const float4*>(&Ap[(w * CH + l16) * AS + 4 * g4]);
            as[0] += p.x; as[1] += p.y; as[2] += p.z; as[3] += p.w;
          }
#pragma unroll
          for (int i = 0; i < 4; ++i) {   // key token 4 g4 + i, query token l16
            const float w = 4 * g4 + i <= l16 ? as[i] : 0.0f;
            o[0] = __builtin_amdgcn_mfma_f32_16x16x4f32(w, vv[0][i], o[0], 0, 0, 0);
            o[1] = __builtin_amdgcn_mfma_f32_16x16x4f32(w, vv[1][i], o[1], 0, 0, 0);
          }
        }
#pragma unroll
        for (int m = 0; m < DKT; ++m) {
          const float4 e = *reinterpret_cast<const float4*>(&eC[16 * m + 4 * g4]);
          f32x4_t x0 = S[m][0], x1 = S[m][1];
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            const float kx = Ks[(4 * g4 + i) * QS + 16 * m + l16];
            x0 = __builtin_amdgcn_mfma_f32_16x16x4f32(kx, vv[0][i], x0, 0, 0, 0);
            x1 = __builtin_amdgcn_mfma_f32_16x16x4f32(kx, vv[1][i], x1, 0, 0, 0);
          }
          const f32x4_t ev = {e.x, e.y, e.z, e.w};
          S[m][0] = x0 * ev;
          S[m][1] = x1 * ev;
        }
      }
    }
    if (!state_only && live) {
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const float s = row16_sum(o[0][i] * o[0][i] + o[1][i] * o[1][i])   /* (columns beyond dv are zero) */;
        if (l16 == 0) ssq[wave * CH + 4 * g4 + i] = s;
      }
    }
  }
  if (!state_only) {
    __syncthreads();
    emit(((len - 1) / CH) * CH);
  }
  // ---- the state the segment leaves
  float* dst = nullptr;
  if (state_only) dst = a.seg_state + ((int64_t)bh * a.nseg + seg + 1) * dk * dv;
  else if (seg == a.nseg - 1) dst = a.state + (int64_t)bh * dk * dv;
  if (dst) {
#pragma unroll
    for (int m = 0; m < DKT; ++m)
#pragma unroll
      for (int n = 0; n < 2; ++n)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int c = 16 * m + 4 * g4 + i;
          if (cv[n] && c < dk) dst[c * dv + c0w + 16 * n + l16] = S[m][n][i];
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
    acc = acc * exp2_f(dec[(int64_t)(j - 1) * a.dk]) + slot[(int64_t)j * n];
    slot[(int64_t)j * n] = acc;
  }
}

// log2-decays of a gated linear attention: out[row, c] = log2 sigmoid(a2[c, :] . lowrank[row, :] + bias[c]) / tau
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
      if (r < nr) out[(int64_t)(r0 + r) * n + c] = log_sigmoid_f(z[r]) * (inv_tau * LOG2E);
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
  const int nq = dv / V, nrow = nt / nq;      // threads along dv, state rows side by side
  const int vq = tid % nq, r0 = tid / nq;
  const bool on = r0 < nrow;
  float* st = a.state + (int64_t)bh * dk * dv + vq * V;
  constexpr int U = V == 4 ? 8 : 4;
  float s[U][V];
  // (loads never branch or wait for the position: a row outside goes to row 0 and is not used)
  auto load = [&](int r) {
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int c = r + u * nrow;
      const float* src = st + (on && c < dk ? c * dv : 0);
      if constexpr (V == 4) {
        const float4 t = *reinterpret_cast<const float4*>(src);
        s[u][0] = t.x; s[u][1] = t.y; s[u][2] = t.z; s[u][3] = t.w;
      } else {
        s[u][0] = *src;
      }
    }
  };
  load(r0);
  const T* q = reinterpret_cast<const T*>(a.q) + (int64_t)b * a.ld + h * dk;
  const T* k = reinterpret_cast<const T*>(a.k) + (int64_t)b * a.ld + h * dk;
  T vraw[V];
#pragma unroll
  for (int j = 0; j < V; ++j) vraw[j] = (reinterpret_cast<const T*>(a.v) + (int64_t)b * a.ld + h * dv)[vq * V + j];
  // (what the last lines need, for the dimension this thread finishes)
  const int dl = tid < dv ? tid : 0;
  const T graw = (reinterpret_cast<const T*>(a.g) + (int64_t)b * a.ld + h * dv)[dl];
  const T nraw = a.norm ? reinterpret_cast<const T*>(a.norm)[dl] : graw;
  const int p = a.pos[0];
  if (p < 0 || (a.rope && p >= a.rope_len)) {
    if (a.err && tid == 0) *a.err = LR_DEV_POS_RANGE;
    return;
  }
  const bool have = p > 0;     // the first token starts from a zero state
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
      if ((a.rank & 7) == 0) {
        for (int j = 0; j < a.rank; j += 8) {
          T x[8];
          __builtin_memcpy(x, __builtin_assume_aligned(w + j, 16), sizeof(x));
#pragma unroll
          for (int e = 0; e < 8; ++e) z = fmaf(ldf(&x[e]), ldf(t + j + e), z);
        }
      } else {
        for (int j = 0; j < a.rank; ++j) z = fmaf(ldf(w + j), ldf(t + j), z);
      }
      la = log_sigmoid_f(z) * a.inv_tau * LOG2E;
    } else {
      la = a.head_decay[h] * LOG2E;
    }
    qs[c] = fq * a.q_scale;
    ks[c] = fk * a.k_scale;
    es[c] = exp2_f(la);
  }
  float vv[V];
#pragma unroll
  for (int j = 0; j < V; ++j) vv[j] = ldf(&vraw[j]);
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
          n[j] = fmaf(e, have ? s[u][j] : 0.0f, kk * vv[j]);
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
  // the head's output, its mean square, gain and gate (at least dv threads: one dimension each)
  float t = 0.0f;
  __shared__ float wsum[16];
  if (tid < dv)
    for (int r = 0; r < nrow; ++r) t += red[r * dv + tid];
  const float ss = wave_sum(t * t);
  if ((tid & 63) == 0) wsum[tid >> 6] = ss;
  __syncthreads();
  float tot = 0.0f;
  for (int w = 0; w * 64 < dv; ++w) tot += wsum[w];
  const float inv = rsq_f(tot / (float)dv + a.eps);
  if (tid < dv)
    stf(reinterpret_cast<T*>(a.y) + (int64_t)b * a.ldy + h * dv + tid,
        t * inv * (a.norm ? ldf(&nraw) : 1.0f) * silu_f(ldf(&graw)));
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
  if (d->ld > (1 << 24) || d->ldy > (1 << 24) || (int64_t)d->H * d->dk > (1 << 24)) return LR_E_UNSUPPORTED;  // 32-bit offsets in a chunk
  if (d->dk > MAX_DIM || d->dv > MAX_DIM) return LR_E_UNSUPPORTED;
  const bool gated = d->lowrank != nullptr;
  LR_OPTIONAL_PTR(d->a2);
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

// Segments: about as many workgroups as the chip holds at once, none shorter than 64 tokens.
int segments(int B, int S, int H, int dv) {
  const int64_t wgs = (int64_t)B * H;
  int64_t want = ((dv <= 128 ? 512 : 256) + wgs - 1) / wgs;
  const int64_t most = S / 64;
  if (want > most) want = most;
  return want < 1 ? 1 : (int)want;
}

size_t align16(size_t n) { return (n + 15) & ~(size_t)15; }

template <typename T, int DKT, bool VEC>
int launch(const LinAttn& a, int state_only, hipStream_t s) {
  constexpr int DKP = 16 * DKT;
  int nw = (a.dv + 31) / 32;
  if (nw < 4) nw = 4;
  if (64 * nw < CH * (DKP / 8)) nw = CH * (DKP / 8) / 64;   // one item of the chunk's preparation per thread
  const size_t lds = sizeof(float) * ((size_t)2 * CH * (DKP + 4) + CH * DKP + DKP + (size_t)nw * CH * AS + nw * CH + 4);
  static std::atomic<unsigned long long> raised{0};
  if (!lr_raise_lds_limit(reinterpret_cast<const void*>(&k_linear_attention<T, DKT, VEC>), lds, raised)) return LR_E_LAUNCH;
  k_linear_attention<T, DKT, VEC><<<dim3(a.B * a.H, state_only ? a.nseg - 1 : a.nseg), dim3(64 * nw), lds, s>>>(a, state_only);
  return lr_launch_status();
}

template <typename T, int DKT>
int launch(const LinAttn& a, int state_only, hipStream_t s) {
  const bool vec = a.dk % 8 == 0 && a.rot % 16 == 0 && !lr_misaligned(a.q) && !lr_misaligned(a.k) && !lr_misaligned(a.rope);
  return vec ? launch<T, DKT, true>(a, state_only, s) : launch<T, DKT, false>(a, state_only, s);
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
  a.nseg = segments(a.B, a.S, a.H, a.dv);
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
  // about 16 state values per thread, at least a thread per value dimension
  int nt = (int)(((int64_t)a.dk * a.dv / 16 + 63) / 64 * 64);
  if (nt < a.dv) nt = (a.dv + 63) / 64 * 64;
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
  const int ns = segments(B, S, H, dv);
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
