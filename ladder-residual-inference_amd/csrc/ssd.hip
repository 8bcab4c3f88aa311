// Selective state space (Mamba-2): per head S_t = e^(a_t) S_(t-1) + dt_t B_t x_t^T, y_t = S_t^T C_t + D x_t, with S [N, P] in
// fp32, dt = softplus(raw + bias), a = -exp(A_log) dt, and B, C shared by the heads of a group.  x, B and C come out of a
// causal convolution per channel and silu; y is multiplied by silu(z) and then normalised in equal parts.
//
// lr_causal_conv: the convolution of a portion; its last inputs live in a ring of `taps` rows per sequence, a token's at
// position % taps: what a token writes is never what the taps - 1 tokens after it do not need any more.
//
// Prompts and portions (bf16): one workgroup per (sequence, head, 64 columns of P, segment) walks 64 tokens at a time.
// With c_t the running sum of log-decays inside the chunk,
//     Y^T = (X^T M + e^(c_t) S^T C^T),  M[s][t] = (B_s . C_t) e^(c_t - c_s) dt_s for s <= t
//     S   <- e^(c_last) S + (B w)^T X,  w_s = dt_s e^(c_last - c_s)
// on the bf16 matrix cores.  Of the two factors of every product one is stored in bf16 and thus exact; the other one (M, S,
// B w: fp32 values) enters as hi + lo, which keeps it to about 2^-17, and S itself stays in fp32 accumulators.  No exponent
// is ever positive.  M is formed transposed, a token per lane, where it is the operand of the next product as it lies.
// Few (sequence, head) pairs: the tokens are cut into segments that run side by side -- first the state each would leave
// from zero, then a scan over segments, then the outputs from the right initial states.
//
// fp32, and sizes the above is not built for: k_ssd_walk, token by token with the state in registers.
//
// One token: k_ssd_step, one workgroup per (sequence, head): convolution, decay, state read once and updated in place, skip
// and gate in one launch.
#include "mixer_common.h"

namespace {

__device__ __forceinline__ float softplus_f(float z) { return fmaxf(z, 0.0f) + log1pf(expf(-fabsf(z))); }

struct Ssd {
  const void *z, *x, *b, *c, *dt;     // columns of row-major buffers: z and dt with stride ld, x, b and c with stride ldu
  int64_t ld, ldu;
  const void *dt_bias, *a_log, *d;    // [H]
  const int32_t* pos;
  float* state;                       // [B, H, N, P]
  void* y;
  int64_t ldy;
  int B, S, H, G, N, P;
  float* seg_state;                   // [B * H, nseg, N, P]
  float* seg_decay;                   // [B * H, nseg], base-2 logarithms
  int nseg, seg_len;
  int32_t* err;
  // one token: x, b and c are what the convolution is still to be applied to
  const void *conv_w, *conv_b;        // [C, taps], [C]
  void* ring;                         // [B, taps, C]
  int taps, C;
};

// ---------------------------------------------------------------------------------------------- convolution
struct Conv {
  const void* u;
  int64_t ldu;
  const void *w, *bias;
  void* ring;
  void* out;
  int64_t ldo;
  const int32_t* pos;
  int S, C, taps;
};
constexpr int CONV_T = 16;    // tokens per workgroup
constexpr int MAX_TAPS = 8;

// a thread: four channels of CONV_T consecutive tokens, the taps' inputs sliding through registers
template <typename T, int TAPS>
__global__ __launch_bounds__(256) void k_causal_conv(const Conv a) {
  const int taps = TAPS ? TAPS : a.taps;
  constexpr int W = TAPS ? TAPS : MAX_TAPS;
  const int b = blockIdx.z, t0 = blockIdx.x * CONV_T, c = (blockIdx.y * 256 + threadIdx.x) * 4;
  if (c >= a.C) return;
  const int p0 = a.pos[0];
  const T* u = reinterpret_cast<const T*>(a.u) + (int64_t)b * a.S * a.ldu + c;
  T* ring = reinterpret_cast<T*>(a.ring) + (int64_t)b * taps * a.C + c;
  T* out = reinterpret_cast<T*>(a.out) + (int64_t)b * a.S * a.ldo + c;
  float w[4][W], bias[4], win[W][4];
  {
    Quad<T> q;
    q.load(reinterpret_cast<const T*>(a.bias) + c);
    q.get(bias);
  }
#pragma unroll
  for (int j = 0; j < W; ++j) {
    if (j >= taps) break;
#pragma unroll
    for (int e = 0; e < 4; ++e) w[e][j] = ldf(reinterpret_cast<const T*>(a.w) + (int64_t)(c + e) * taps + j);
  }
  // win[j]: the input taps - 1 - j tokens before the current one
#pragma unroll
  for (int j = 0; j + 1 < W; ++j) {
    if (j + 1 >= taps) break;
    const int t = t0 - (taps - 1) + j;
    Quad<T> q;
    q.zero();
    if (t >= 0) q.load(u + (int64_t)t * a.ldu);
    else if (p0 + t >= 0) q.load(ring + (int64_t)((p0 + t) % taps) * a.C);
    q.get(win[j]);
  }
  const int n = min(CONV_T, a.S - t0);
  Quad<T> nx;
  nx.load(u + (int64_t)t0 * a.ldu);
  for (int i = 0; i < n; ++i) {
    float cur[4], o[4];
    nx.get(cur);
    if (i + 1 < n) nx.load(u + (int64_t)(t0 + i + 1) * a.ldu);
#pragma unroll
    for (int e = 0; e < 4; ++e) o[e] = bias[e];
#pragma unroll
    for (int j = 0; j < W; ++j) {
      if (j >= taps) break;
      if (j == taps - 1) {
#pragma unroll
        for (int e = 0; e < 4; ++e) o[e] = fmaf(w[e][j], cur[e], o[e]);
      } else {
#pragma unroll
        for (int e = 0; e < 4; ++e) o[e] = fmaf(w[e][j], win[j][e], o[e]);
      }
    }
#pragma unroll
    for (int e = 0; e < 4; ++e) o[e] = silu_f(o[e]);
    st4(out + (int64_t)(t0 + i) * a.ldo, o);
#pragma unroll
    for (int j = 0; j + 1 < W; ++j) {
      if (j + 1 >= taps) break;
#pragma unroll
      for (int e = 0; e < 4; ++e) win[j][e] = j + 2 == taps ? cur[e] : win[j + 1 < W ? j + 1 : j][e];
    }
  }
  // the first workgroup is the only one that reads the ring, so it is the one that fills it: the portion's last inputs
  if (t0 == 0) {
    for (int t = max(0, a.S - (taps - 1)); t < a.S; ++t) {
      Quad<T> q;
      q.load(u + (int64_t)t * a.ldu);
      float f[4];
      q.get(f);
      st4(ring + (int64_t)((p0 + t) % taps) * a.C, f);
    }
  }
}

// ---------------------------------------------------------------------------------------------- token by token
// One workgroup: 16 columns of P of one (sequence, head).  A thread: one column, every 16th of N.
constexpr int WALK_T = 32;          // tokens whose inputs lie in LDS together

template <typename T, int NPT>
__global__ __launch_bounds__(256) void k_ssd_walk(const Ssd a) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  float* bs = sm;                           // [WALK_T][N]
  float* cs = bs + WALK_T * a.N;            // [WALK_T][N]
  float* xs = cs + WALK_T * a.N;            // [WALK_T][16]
  float* es = xs + WALK_T * 16;             // [WALK_T] decays
  float* ds = es + WALK_T;                  // [WALK_T] dt
  float* part = ds + WALK_T;                // [WALK_T][4][16]
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, pl = lane & 15, n0 = (wave * 4 + (lane >> 4)) * NPT;
  const int bh = blockIdx.x, b = bh / a.H, h = bh - b * a.H, g = h / (a.H / a.G), pc = blockIdx.y * 16;
  const bool on = pc + pl < a.P;
  const int p0 = a.pos[0];
  const T* x = reinterpret_cast<const T*>(a.x) + h * a.P + pc;
  const T* B = reinterpret_cast<const T*>(a.b) + g * a.N;
  const T* C = reinterpret_cast<const T*>(a.c) + g * a.N;
  const T* z = reinterpret_cast<const T*>(a.z) + h * a.P + pc;
  const T* dt = reinterpret_cast<const T*>(a.dt) + h;
  T* y = reinterpret_cast<T*>(a.y) + h * a.P + pc;
  const float bias = ldf(reinterpret_cast<const T*>(a.dt_bias) + h), A = expf(ldf(reinterpret_cast<const T*>(a.a_log) + h));
  const float D = ldf(reinterpret_cast<const T*>(a.d) + h);
  float* st = a.state + (int64_t)bh * a.N * a.P + pc + pl;
  float s[NPT];
#pragma unroll
  for (int i = 0; i < NPT; ++i) s[i] = p0 > 0 && on && n0 + i < a.N ? st[(int64_t)(n0 + i) * a.P] : 0.0f;
  for (int t0 = 0; t0 < a.S; t0 += WALK_T) {
    const int nt = min(WALK_T, a.S - t0);
    const int64_t row = (int64_t)b * a.S + t0;
    __syncthreads();
    for (int i = tid; i < nt * a.N; i += 256) {
      const int t = i / a.N, n = i - t * a.N;
      bs[t * a.N + n] = ldf(B + (row + t) * a.ldu + n);
      cs[t * a.N + n] = ldf(C + (row + t) * a.ldu + n);
    }
    for (int i = tid; i < nt * 16; i += 256) {
      const int t = i >> 4, p = i & 15;
      xs[i] = pc + p < a.P ? ldf(x + (row + t) * a.ldu + p) : 0.0f;
    }
    if (tid < nt) {
      const float d = softplus_f(ldf(dt + (row + tid) * a.ld) + bias);
      ds[tid] = d;
      es[tid] = expf(-A * d);
    }
    __syncthreads();
    for (int t = 0; t < nt; ++t) {
      const float e = es[t], dx = ds[t] * xs[t * 16 + pl];
      float acc = 0.0f;
#pragma unroll
      for (int i = 0; i < NPT; ++i) {
        const int n = min(n0 + i, a.N - 1);
        s[i] = fmaf(e, s[i], dx * bs[t * a.N + n]);
        if (n0 + i < a.N) acc = fmaf(s[i], cs[t * a.N + n], acc);
      }
      acc += __shfl_xor(acc, 16, LR_WAVE);
      acc += __shfl_xor(acc, 32, LR_WAVE);
      if (lane < 16) part[(t * 4 + wave) * 16 + pl] = acc;
    }
    __syncthreads();
    for (int i = tid; i < nt * 16; i += 256) {
      const int t = i >> 4, p = i & 15;
      if (pc + p < a.P) {
        const float* q = part + t * 64 + p;
        const float v = ((q[0] + q[16]) + (q[32] + q[48])) + D * xs[i];
        stf(y + (row + t) * a.ldy + p, v * silu_f(ldf(z + (row + t) * a.ld + p)));
      }
    }
  }
  if (on) {
#pragma unroll
    for (int i = 0; i < NPT; ++i)
      if (n0 + i < a.N) st[(int64_t)(n0 + i) * a.P] = s[i];
  }
}

// ---------------------------------------------------------------------------------------------- one token
// 256 threads: four columns each, the rows of S side by side.  Everything from memory is asked for before anything is used.
template <typename T, int TAPS>
__global__ __launch_bounds__(256) void k_ssd_step(const Ssd a) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  const int bh = blockIdx.x, b = bh / a.H, h = bh - b * a.H, hpg = a.H / a.G, g = h / hpg, tid = threadIdx.x;
  const int N = a.N, P = a.P, taps = TAPS ? TAPS : a.taps;
  float* xs = sm;               // [P]
  float* bs = xs + P;           // [N]
  float* cs = bs + N;           // [N]
  float* red = cs + N;          // [rows side by side][P]
  const int nq = P / 4, nrow = 256 / nq, vq = tid % nq, r0 = tid / nq;
  const bool on = r0 < nrow;
  float* st = a.state + (int64_t)bh * N * P + vq * 4;
  constexpr int U = 8;
  float4 s[U];
  auto load = [&](int r) {
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int n = r + u * nrow;
      s[u] = *reinterpret_cast<const float4*>(st + (on && n < N ? (int64_t)n * P : 0));
    }
  };
  load(r0);
  const int p = a.pos[0];
  if (p < 0) {
    if (a.err && tid == 0) *a.err = LR_DEV_POS_RANGE;
    return;
  }
  // the convolution of this head's channels: x, then B and C of its group
  constexpr int W = TAPS ? TAPS : MAX_TAPS, IT = 3;      // (P + 2 N <= 768 channels)
  const int nch = P + 2 * N, slot = p % taps;
  const T* cw = reinterpret_cast<const T*>(a.conv_w);
  const T* cb = reinterpret_cast<const T*>(a.conv_b);
  T* ring = reinterpret_cast<T*>(a.ring) + (int64_t)b * taps * a.C;
  const T* u = reinterpret_cast<const T*>(a.x) + (int64_t)b * a.ldu;       // channel 0 of the convolution
  auto channel = [&](int i) { return i < P ? h * P + i : (i < P + N ? a.H * P + g * N + i - P : a.H * P + (a.G + g) * N + i - P - N); };
  T raw[IT], cbias[IT], past[IT][W], w[IT][W];
#pragma unroll
  for (int k = 0; k < IT; ++k) {
    if (256 * k >= nch) break;
    const int ch = channel(min(tid + 256 * k, nch - 1));
    raw[k] = u[ch];
    cbias[k] = cb[ch];
#pragma unroll
    for (int j = 0; j < W; ++j) {      // j tokens back
      if (j >= taps) break;
      w[k][j] = cw[(int64_t)ch * taps + taps - 1 - j];
      if (j > 0) past[k][j] = ring[(int64_t)((p - j + taps) % taps) * a.C + ch];
    }
  }
  const T* dtp = reinterpret_cast<const T*>(a.dt) + (int64_t)b * a.ld + h;
  const T draw = *dtp, dbias = reinterpret_cast<const T*>(a.dt_bias)[h], araw = reinterpret_cast<const T*>(a.a_log)[h];
  const T Draw = reinterpret_cast<const T*>(a.d)[h];
  const T zraw = reinterpret_cast<const T*>(a.z)[(int64_t)b * a.ld + h * P + (tid < P ? tid : 0)];
  __builtin_amdgcn_sched_barrier(0);
#pragma unroll
  for (int k = 0; k < IT; ++k) {
    if (256 * k >= nch) break;
    const int i = tid + 256 * k;
    float v = fmaf(ldf(&w[k][0]), ldf(&raw[k]), ldf(&cbias[k]));
#pragma unroll
    for (int j = 1; j < W; ++j) {
      if (j >= taps) break;
      v = fmaf(ldf(&w[k][j]), p >= j ? ldf(&past[k][j]) : 0.0f, v);
    }
    if (i < nch) {
      sm[i] = silu_f(v);
      // (into a slot nobody reads in this step)
      if (taps > 1 && (i < P || h % hpg == 0)) ring[(int64_t)slot * a.C + channel(i)] = raw[k];
    }
  }
  const float dt = softplus_f(ldf(&draw) + ldf(&dbias));
  const float e = p > 0 ? expf(-expf(ldf(&araw)) * dt) : 0.0f;
  const float D = ldf(&Draw);
  __syncthreads();
  float4 xv = *reinterpret_cast<const float4*>(xs + vq * 4);
  const float dx[4] = {dt * xv.x, dt * xv.y, dt * xv.z, dt * xv.w};
  float acc[4] = {0, 0, 0, 0};
  for (int r = r0; r < N; r += U * nrow) {
    if (r != r0) load(r);
#pragma unroll
    for (int k = 0; k < U; ++k) {
      const int n = r + k * nrow;
      if (on && n < N) {
        const float bb = bs[n], cc = cs[n];
        const float old[4] = {s[k].x, s[k].y, s[k].z, s[k].w};
        float nw[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          nw[j] = fmaf(e, p > 0 ? old[j] : 0.0f, bb * dx[j]);
          acc[j] = fmaf(nw[j], cc, acc[j]);
        }
        *reinterpret_cast<float4*>(st + (int64_t)n * P) = make_float4(nw[0], nw[1], nw[2], nw[3]);
      }
    }
  }
  if (on) *reinterpret_cast<float4*>(red + r0 * P + vq * 4) = make_float4(acc[0], acc[1], acc[2], acc[3]);
  __syncthreads();
  if (tid < P) {
    float t = D * xs[tid];
    for (int r = 0; r < nrow; ++r) t += red[r * P + tid];
    stf(reinterpret_cast<T*>(a.y) + (int64_t)b * a.ldy + h * P + tid, t * silu_f(ldf(&zraw)));
  }
}

// ---------------------------------------------------------------------------------------------- chunks of 64 tokens
constexpr int CK = 64;              // tokens per chunk
constexpr int TR = CK + 8;          // row length of the transposed tiles, in elements
constexpr float DECAY_FLOOR = -86.0f;   // one token's log2-decay is cut off here: 2^-86 of a state is nothing in fp32

__device__ __forceinline__ u32 pair_of(u32 a, u32 b, bool high) {
  return high ? (a >> 16) | (b & 0xffff0000u) : (a & 0xffffu) | (b << 16);
}

// eight fp32 values as bf16 hi + lo operands
__device__ __forceinline__ void split8(const float* f, bf16x8_t& hi, bf16x8_t& lo) {
  u32x4_t h, l;
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const float x = f[2 * j], y = f[2 * j + 1];
    h[j] = pack_bf2(x, y);
    l[j] = pack_bf2(x - bf_lo(h[j]), y - bf_hi(h[j]));
  }
  hi = __builtin_bit_cast(bf16x8_t, h);
  lo = __builtin_bit_cast(bf16x8_t, l);
}

// NT: N in tiles of 16.  state_only: no outputs; the segment starts from zero and leaves its state and log-decay in scratch.
template <int NT>
__global__ __launch_bounds__(256, NT > 8 ? 1 : 2) void k_ssd_chunk(const Ssd a, const int state_only) {
  constexpr int NR = 16 * NT + 8, KN = NT / 2, NW = NT >= 4 ? NT / 4 : 1;   // NW: tiles of N per wave in the state update
  extern __shared__ __attribute__((aligned(16))) u16 su[];
  u16* Bs = su;                       // [CK][NR]       B by token
  u16* Bt = Bs + CK * NR;             // [16 NT][TR]    B by channel
  u16* Xt = Bt + 16 * NT * TR;        // [64][TR]       x by column
  u16* Sh = Xt + 64 * TR;             // [64][NR]       S^T, high and low parts
  u16* Sl = Sh + 64 * NR;
  float* cum = reinterpret_cast<float*>(Sl + 64 * NR);   // [2][CK] running log2-decay
  float* dts = cum + 2 * CK;                             // [2][CK]
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, g4 = lane >> 4, l16 = lane & 15;
  const int np = (a.P + 63) / 64;
  const int bh = blockIdx.x / np, pc = (blockIdx.x - bh * np) * 64, seg = blockIdx.y;
  const int b = bh / a.H, h = bh - b * a.H, g = h / (a.H / a.G);
  const int N = a.N, P = a.P, pw = min(64, P - pc), pt = pw / 16;      // (N and P are multiples of 16)
  const int s0 = seg * a.seg_len, len = min(a.S - s0, a.seg_len);
  const int p0 = a.pos[0];
  const int64_t row0 = (int64_t)b * a.S + s0;
  const u16* x = reinterpret_cast<const u16*>(a.x) + row0 * a.ldu + h * P + pc;
  const u16* B = reinterpret_cast<const u16*>(a.b) + row0 * a.ldu + g * N;
  const u16* C = reinterpret_cast<const u16*>(a.c) + row0 * a.ldu + g * N;
  const u16* z = reinterpret_cast<const u16*>(a.z) + row0 * a.ld + h * P + pc;
  const u16* dt = reinterpret_cast<const u16*>(a.dt) + row0 * a.ld + h;
  u16* y = reinterpret_cast<u16*>(a.y) + row0 * a.ldy + h * P + pc;
  const float bias = ldf(reinterpret_cast<const u16*>(a.dt_bias) + h);
  const float A2 = -expf(ldf(reinterpret_cast<const u16*>(a.a_log) + h)) * LOG2E;
  const float D = ldf(reinterpret_cast<const u16*>(a.d) + h);
  const int lb = (int)a.ldu * 2, lz = (int)a.ld * 2, lyb = (int)a.ldy * 2;

  // ---- the state: tile (m, n) of this wave, register i is row 16 (NW wave + m) + 4 g4 + i of column 16 n + l16
  f32x4_t S[NW][4];
  const bool mine = wave * NW < NT;
  {
    const bool have = !state_only && (a.nseg > 1 || p0 > 0);
    const float* src = a.nseg > 1 ? a.seg_state + ((int64_t)bh * a.nseg + seg) * N * P : a.state + (int64_t)bh * N * P;
#pragma unroll
    for (int m = 0; m < NW; ++m)
#pragma unroll
      for (int n = 0; n < 4; ++n)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int r = 16 * (NW * wave + m) + 4 * g4 + i;
          const bool ok = have && mine && r < N && n < pt;
          const float t = src[ok ? (int64_t)r * P + pc + 16 * n + l16 : 0];
          S[m][n][i] = ok ? t : 0.0f;
        }
  }
  auto store_state = [&]() {        // S^T, hi and lo, for the outputs of the next chunk
    if (!mine || state_only) return;
#pragma unroll
    for (int m = 0; m < NW; ++m)
#pragma unroll
      for (int n = 0; n < 4; ++n) {
        const int at = (16 * n + l16) * NR + 16 * (NW * wave + m) + 4 * g4;
        const f32x4_t v = S[m][n];
        const uint2 hi = make_uint2(pack_bf2(v[0], v[1]), pack_bf2(v[2], v[3]));
        *reinterpret_cast<uint2*>(&Sh[at]) = hi;
        *reinterpret_cast<uint2*>(&Sl[at]) = make_uint2(pack_bf2(v[0] - bf_lo(hi.x), v[1] - bf_hi(hi.x)),
                                                       pack_bf2(v[2] - bf_lo(hi.y), v[3] - bf_hi(hi.y)));
      }
  };

  // ---- staging: an item is eight columns of two neighbouring tokens, 32 pairs of tokens side by side
  constexpr int BI = NT / 4 > 0 ? NT / 4 : 1;        // items of B per thread (NT * 2 slices of 8, 32 pairs, 256 threads)
  const int kp = tid & 31, sl = tid >> 5;            // pair, slice (8 of them at once)
  u32x4_t br[BI][2], xr[2], cr[KN];
  float draw = 0.0f;
  const int t = 16 * wave + l16;        // this lane's token in the products
  auto fetch = [&](int c0) {
    const int nt = min(len - c0, CK);
    const rsrc_t rb = buffer_of(B + (int64_t)c0 * a.ldu, (nt - 1) * lb + N * 2);
    const rsrc_t rx = buffer_of(x + (int64_t)c0 * a.ldu, (nt - 1) * lb + pw * 2);
#pragma unroll
    for (int e = 0; e < 2; ++e) {
      const int t = 2 * kp + e;
#pragma unroll
      for (int i = 0; i < BI; ++i) {
        const int c = (sl + 8 * i) * 8;
        br[i][e] = __builtin_amdgcn_raw_buffer_load_b128(rb, t < nt && c < N ? t * lb + c * 2 : NOWHERE, 0, 0);
      }
      xr[e] = __builtin_amdgcn_raw_buffer_load_b128(rx, t < nt && sl * 8 < pw ? t * lb + sl * 16 : NOWHERE, 0, 0);
    }
    if (!state_only) {
      const rsrc_t rc = buffer_of(C + (int64_t)c0 * a.ldu, (nt - 1) * lb + N * 2);
#pragma unroll
      for (int k = 0; k < KN; ++k)
        cr[k] = __builtin_amdgcn_raw_buffer_load_b128(rc, t < nt && 32 * k + 8 * g4 < N ? t * lb + (32 * k + 8 * g4) * 2 : NOWHERE, 0, 0);
    }
    if (wave == 0) {
      const u16 r = dt[(int64_t)(c0 + min(lane, nt - 1)) * a.ld];
      draw = bf_to_f(r);
    }
  };
  // Transposed rows hold pairs of tokens in dwords; a slice's rows lie 8 * 36 dwords apart, so the pair index is turned by
  // the slice to spread them over the banks (groups of eight tokens stay whole for the reader).
  auto turn = [](int group, int r) { return group ^ ((r >> 3) & 7); };
  auto stage = [&]() {
    u32* bt32 = reinterpret_cast<u32*>(Bt);
    u32* xt32 = reinterpret_cast<u32*>(Xt);
#pragma unroll
    for (int i = 0; i < BI; ++i) {
      const int c = (sl + 8 * i) * 8;
      if (c < 16 * NT) {
#pragma unroll
        for (int e = 0; e < 2; ++e)
          if (!state_only) *reinterpret_cast<u32x4_t*>(&Bs[(2 * kp + e) * NR + c]) = br[i][e];
        const int at = turn(kp >> 2, c) * 4 + (kp & 3);
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          bt32[(c + 2 * j) * (TR / 2) + at] = pair_of(br[i][0][j], br[i][1][j], false);
          bt32[(c + 2 * j + 1) * (TR / 2) + at] = pair_of(br[i][0][j], br[i][1][j], true);
        }
      }
    }
    const int c = sl * 8, at = turn(kp >> 2, c) * 4 + (kp & 3);
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      xt32[(c + 2 * j) * (TR / 2) + at] = pair_of(xr[0][j], xr[1][j], false);
      xt32[(c + 2 * j + 1) * (TR / 2) + at] = pair_of(xr[0][j], xr[1][j], true);
    }
  };
  // dt and the running log-decay of a chunk, a token per lane of wave 0 (tokens beyond the end: dt 0, no decay)
  auto decays = [&](int c0, int buf) {
    if (wave != 0) return;
    const int nt = min(len - c0, CK);
    const float d = lane < nt ? softplus_f(draw + bias) : 0.0f;
    float v = fmaxf(A2 * d, DECAY_FLOOR);
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const float t = __shfl_up(v, o, LR_WAVE);
      v += lane >= o ? t : 0.0f;
    }
    cum[buf * CK + lane] = v;
    dts[buf * CK + lane] = d;
  };

  float total = 0.0f;
  fetch(0);
  decays(0, 0);
  stage();
  store_state();
  __syncthreads();
  int buf = 0;
  for (int c0 = 0; c0 < len; c0 += CK, buf ^= 1) {
    const int nt = min(len - c0, CK);
    const bool more = c0 + CK < len;
    const float* cm = cum + buf * CK;
    const float* dm = dts + buf * CK;
    bf16x8_t cf[KN];
    uint2 zr[4], xq[4];
    if (!state_only) {
#pragma unroll
      for (int k = 0; k < KN; ++k) cf[k] = __builtin_bit_cast(bf16x8_t, cr[k]);
      const rsrc_t rz = buffer_of(z + (int64_t)c0 * a.ld, (nt - 1) * lz + pw * 2);
      const rsrc_t rx = buffer_of(x + (int64_t)c0 * a.ldu, (nt - 1) * lb + pw * 2);
#pragma unroll
      for (int n = 0; n < 4; ++n) {
        const int o = n < pt && t < nt ? (16 * n + 4 * g4) * 2 : NOWHERE;
        const u32x2_t v = __builtin_amdgcn_raw_buffer_load_b64(rz, o >= 0 ? o + t * lz : NOWHERE, 0, 0);
        const u32x2_t w = __builtin_amdgcn_raw_buffer_load_b64(rx, o >= 0 ? o + t * lb : NOWHERE, 0, 0);
        zr[n] = make_uint2(v.x, v.y);
        xq[n] = make_uint2(w.x, w.y);
      }
    }
    if (more) fetch(c0 + CK);
    const float clast = cm[CK - 1];
    total += clast;

    if (!state_only) {
      // ---- what the state brings: rows are columns of P, columns tokens
      const float ct = cm[t], et = exp2_f(ct);
      f32x4_t o[4];
#pragma unroll
      for (int n = 0; n < 4; ++n) {
        o[n] = f32x4_t{0, 0, 0, 0};
      }
      // (columns beyond P are zeros: computed, not stored)
#pragma unroll
      for (int k = 0; k < KN; ++k) {
#pragma unroll
        for (int n = 0; n < 4; ++n) {
          const bf16x8_t sh = *reinterpret_cast<const bf16x8_t*>(&Sh[(16 * n + l16) * NR + 32 * k + 8 * g4]);
          o[n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(sh, cf[k], o[n], 0, 0, 0);
        }
#pragma unroll
        for (int n = 0; n < 4; ++n) {
          const bf16x8_t sv = *reinterpret_cast<const bf16x8_t*>(&Sl[(16 * n + l16) * NR + 32 * k + 8 * g4]);
          o[n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(sv, cf[k], o[n], 0, 0, 0);
        }
      }
#pragma unroll
      for (int n = 0; n < 4; ++n) o[n] *= et;
      // ---- the chunk's own tokens, 32 keys at a time
#pragma unroll
      for (int j = 0; j < 2; ++j) {
        if (2 * j <= wave) {
          float m[8];
          const int tl = fresh(t) - 4 * g4;       // (compared here: as loop invariants the masks would not fit the scalar registers)
#pragma unroll
          for (int e = 0; e < 2; ++e) {
            const int st = 2 * j + e;
            f32x4_t gt = {0, 0, 0, 0};
            if (st <= wave) {
#pragma unroll
              for (int k = 0; k < KN; ++k) {
                const bf16x8_t bf = *reinterpret_cast<const bf16x8_t*>(&Bs[(16 * st + l16) * NR + 32 * k + 8 * g4]);
                gt = __builtin_amdgcn_mfma_f32_16x16x32_bf16(bf, cf[k], gt, 0, 0, 0);
              }
            }
            const float4 c4 = *reinterpret_cast<const float4*>(&cm[16 * st + 4 * g4]);
            const float4 d4 = *reinterpret_cast<const float4*>(&dm[16 * st + 4 * g4]);
            const float cc[4] = {c4.x, c4.y, c4.z, c4.w}, dd[4] = {d4.x, d4.y, d4.z, d4.w};
#pragma unroll
            for (int i = 0; i < 4; ++i) {
              const float w = exp2_f(ct - cc[i]) * dd[i];
              m[4 * e + i] = 16 * st + i <= tl ? gt[i] * w : 0.0f;
            }
          }
          bf16x8_t mh, ml;
          split8(m, mh, ml);
#pragma unroll
          for (int n = 0; n < 4; ++n) {
            // tokens 32 j + 4 g4 + {0 .. 3} and 16 further
            const int r = 16 * n + l16;
            const uint2 v0 = *reinterpret_cast<const uint2*>(&Xt[r * TR + 8 * turn(4 * j + (g4 >> 1), r) + 4 * (g4 & 1)]);
            const uint2 v1 = *reinterpret_cast<const uint2*>(&Xt[r * TR + 8 * turn(4 * j + 2 + (g4 >> 1), r) + 4 * (g4 & 1)]);
            const bf16x8_t xv = __builtin_bit_cast(bf16x8_t, u32x4_t{v0.x, v0.y, v1.x, v1.y});
            o[n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(xv, mh, o[n], 0, 0, 0);
            o[n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(xv, ml, o[n], 0, 0, 0);
          }
        }
      }
      // ---- skip, gate, store: register i is column 16 n + 4 g4 + i of token t
      const rsrc_t ry = buffer_of(y + (int64_t)c0 * a.ldy, (nt - 1) * lyb + pw * 2);
#pragma unroll
      for (int n = 0; n < 4; ++n) {
        const float xe[4] = {bf_lo(xq[n].x), bf_hi(xq[n].x), bf_lo(xq[n].y), bf_hi(xq[n].y)};
        const float ze[4] = {bf_lo(zr[n].x), bf_hi(zr[n].x), bf_lo(zr[n].y), bf_hi(zr[n].y)};
        float f[4];
#pragma unroll
        for (int i = 0; i < 4; ++i) f[i] = fmaf(D, xe[i], o[n][i]) * silu_f(ze[i]);
        const u32x2_t pk = {pack_bf2(f[0], f[1]), pack_bf2(f[2], f[3])};
        __builtin_amdgcn_raw_buffer_store_b64(pk, ry, n < pt && t < nt ? t * lyb + (16 * n + 4 * g4) * 2 : NOWHERE, 0, 0);
      }
    }

    // ---- the state behind the chunk
    if (mine) {
      const float el = exp2_f(clast);
#pragma unroll
      for (int m = 0; m < NW; ++m)
#pragma unroll
        for (int n = 0; n < 4; ++n) S[m][n] *= el;
#pragma unroll
      for (int k = 0; k < 2; ++k) {
        float w[8];
        {
          const float4 ca = *reinterpret_cast<const float4*>(&cm[32 * k + 8 * g4]), cb = *reinterpret_cast<const float4*>(&cm[32 * k + 8 * g4 + 4]);
          const float4 da = *reinterpret_cast<const float4*>(&dm[32 * k + 8 * g4]), db = *reinterpret_cast<const float4*>(&dm[32 * k + 8 * g4 + 4]);
          const float cc[8] = {ca.x, ca.y, ca.z, ca.w, cb.x, cb.y, cb.z, cb.w}, dd[8] = {da.x, da.y, da.z, da.w, db.x, db.y, db.z, db.w};
#pragma unroll
          for (int i = 0; i < 8; ++i) w[i] = exp2_f(clast - cc[i]) * dd[i];
        }
        bf16x8_t xv[4];
#pragma unroll
        for (int n = 0; n < 4; ++n) {
          const int r = 16 * n + l16;
          xv[n] = *reinterpret_cast<const bf16x8_t*>(&Xt[r * TR + 8 * turn(4 * k + g4, r)]);
        }
#pragma unroll
        for (int m = 0; m < NW; ++m) {
          const int r = 16 * (NW * wave + m) + l16;
          float f[8];
          unpack8(*reinterpret_cast<const uint4*>(&Bt[r * TR + 8 * turn(4 * k + g4, r)]), f);
#pragma unroll
          for (int i = 0; i < 8; ++i) f[i] *= w[i];
          bf16x8_t bh_, bl;
          split8(f, bh_, bl);
#pragma unroll
          for (int n = 0; n < 4; ++n) S[m][n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(bh_, xv[n], S[m][n], 0, 0, 0);
#pragma unroll
          for (int n = 0; n < 4; ++n) S[m][n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(bl, xv[n], S[m][n], 0, 0, 0);
        }
      }
    }
    if (more) {
      decays(c0 + CK, buf ^ 1);
      __syncthreads();
      stage();
      store_state();
      __syncthreads();
    }
  }
  // ---- the state the segment leaves
  float* dst = nullptr;
  if (state_only) dst = a.seg_state + ((int64_t)bh * a.nseg + seg + 1) * N * P;
  else if (seg == a.nseg - 1) dst = a.state + (int64_t)bh * N * P;
  if (dst && mine) {
    const int g4_ = fresh(g4);        // (the masks are formed here, not kept since the state was read)
#pragma unroll
    for (int m = 0; m < NW; ++m)
#pragma unroll
      for (int n = 0; n < 4; ++n)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int r = 16 * (NW * wave + m) + 4 * g4_ + i;
          if (r < N && n < pt) dst[(int64_t)r * P + pc + 16 * n + l16] = S[m][n][i];
        }
  }
  if (state_only && tid == 0 && pc == 0) a.seg_decay[(int64_t)bh * a.nseg + seg] = total;
}

// Slot j of seg_state holds the state segment j - 1 leaves from zero (j >= 1); afterwards the one segment j starts from.
__global__ __launch_bounds__(256) void k_ssd_scan(const Ssd a) {
  const int bh = blockIdx.x, n = a.N * a.P, e = blockIdx.y * 256 + threadIdx.x;
  if (e >= n) return;
  float* slot = a.seg_state + (int64_t)bh * a.nseg * n + e;
  const float* dec = a.seg_decay + (int64_t)bh * a.nseg;
  float acc = a.pos[0] > 0 ? a.state[(int64_t)bh * n + e] : 0.0f;
  slot[0] = acc;
  for (int j = 1; j < a.nseg; ++j) {
    acc = fmaf(acc, exp2_f(dec[j - 1]), slot[(int64_t)j * n]);
    slot[(int64_t)j * n] = acc;
  }
}

// ---------------------------------------------------------------------------------------------- norm in parts
// A workgroup: one part of one row, in place.  Column c of the `cols` that count lies at (c / P) * PP + c % P.
template <typename T>
__global__ __launch_bounds__(256) void k_parts_norm(T* y, int64_t ld, const T* __restrict__ gain, int len, int P, int PP, float eps) {
  __shared__ float red[4];
  T* row = y + (int64_t)blockIdx.x * ld;
  const int c0 = blockIdx.y * len, tid = threadIdx.x;
  float ss = 0.0f;
  if (P == PP && (len & 3) == 0) {
    for (int c = c0 + 4 * tid; c < c0 + len; c += 1024) {
      Quad<T> q;
      q.load(row + c);
      float f[4];
      q.get(f);
      ss += (f[0] * f[0] + f[1] * f[1]) + (f[2] * f[2] + f[3] * f[3]);
    }
  } else {
    for (int c = c0 + tid; c < c0 + len; c += 256) {
      const float f = ldf(row + (c / P) * PP + c % P);
      ss = fmaf(f, f, ss);
    }
  }
  ss = wave_sum(ss);
  if ((tid & 63) == 0) red[tid >> 6] = ss;
  __syncthreads();
  const float inv = 1.0f / sqrtf(((red[0] + red[1]) + (red[2] + red[3])) / (float)len + eps);
  if (P == PP && (len & 3) == 0) {
    for (int c = c0 + 4 * tid; c < c0 + len; c += 1024) {
      Quad<T> q, w;
      q.load(row + c);
      w.load(gain + c);
      float f[4], k[4];
      q.get(f);
      w.get(k);
#pragma unroll
      for (int j = 0; j < 4; ++j) f[j] *= inv * k[j];
      st4(row + c, f);
    }
  } else {
    for (int c = c0 + tid; c < c0 + len; c += 256) {
      const int at = (c / P) * PP + c % P;
      stf(row + at, ldf(row + at) * inv * ldf(gain + at));
    }
  }
}

// ---------------------------------------------------------------------------------------------- host
size_t align16(size_t n) { return (n + 15) & ~(size_t)15; }

// Segments: about two workgroups per CU, none shorter than two chunks.
int segments(int B, int S, int H, int P) {
  const int64_t wgs = (int64_t)B * H * ((P + 63) / 64);
  int64_t want = 512 / wgs;
  const int64_t most = S / (2 * CK);
  if (want > most) want = most;
  return want < 1 ? 1 : (int)want;
}

bool on_matrix_cores(int N, int P, int dtype) { return dtype == LR_BF16 && N % 16 == 0 && P % 16 == 0 && N <= 256; }

template <int NT>
int launch_chunk(const Ssd& a, int state_only, hipStream_t s) {
  constexpr size_t lds = sizeof(u16) * ((size_t)CK * (16 * NT + 8) + 16 * NT * TR + 64 * TR + 2 * 64 * (16 * NT + 8)) + sizeof(float) * 4 * CK;
  static std::atomic<unsigned long long> raised{0};
  if (!lr_raise_lds_limit(reinterpret_cast<const void*>(&k_ssd_chunk<NT>), lds, raised)) return LR_E_LAUNCH;
  k_ssd_chunk<NT><<<dim3(a.B * a.H * ((a.P + 63) / 64), state_only ? a.nseg - 1 : a.nseg), dim3(256), lds, s>>>(a, state_only);
  return lr_launch_status();
}
int launch_chunk(const Ssd& a, int state_only, hipStream_t s) {
  return a.N <= 32 ? launch_chunk<2>(a, state_only, s) : a.N <= 64 ? launch_chunk<4>(a, state_only, s)
         : a.N <= 128 ? launch_chunk<8>(a, state_only, s) : launch_chunk<16>(a, state_only, s);
}

template <typename T, int NPT>
int launch_walk(const Ssd& a, hipStream_t s) {
  const size_t lds = sizeof(float) * WALK_T * (2 * a.N + 16 + 2 + 64);
  static std::atomic<unsigned long long> raised{0};
  if (!lr_raise_lds_limit(reinterpret_cast<const void*>(&k_ssd_walk<T, NPT>), lds, raised)) return LR_E_LAUNCH;
  k_ssd_walk<T, NPT><<<dim3(a.B * a.H, (a.P + 15) / 16), dim3(256), lds, s>>>(a);
  return lr_launch_status();
}
template <typename T>
int walk(const Ssd& a, hipStream_t s) {
  const int npt = (a.N + 15) / 16;
  return npt <= 2 ? launch_walk<T, 2>(a, s) : npt <= 4 ? launch_walk<T, 4>(a, s) : npt <= 8 ? launch_walk<T, 8>(a, s) : launch_walk<T, 16>(a, s);
}

template <typename T, int TAPS>
void launch_conv(const Conv& a, int B, hipStream_t s) {
  k_causal_conv<T, TAPS><<<dim3((a.S + CONV_T - 1) / CONV_T, (a.C + 1023) / 1024, B), dim3(256), 0, s>>>(a);
}
template <typename T>
void conv(const Conv& a, int B, hipStream_t s) {
  if (a.taps == 4) launch_conv<T, 4>(a, B, s);
  else if (a.taps == 3) launch_conv<T, 3>(a, B, s);
  else launch_conv<T, 0>(a, B, s);
}

int fill(const lr_ssd_t* d, Ssd& a) {
  if (d == nullptr || d->z == nullptr || d->x == nullptr || d->b == nullptr || d->c == nullptr || d->dt == nullptr ||
      d->dt_bias == nullptr || d->a_log == nullptr || d->d == nullptr || d->pos == nullptr || d->y == nullptr)
    return LR_E_NULL;
  LR_REQUIRE_PTR(d->state);
  if (d->dtype != LR_BF16 && d->dtype != LR_F32) return LR_E_UNSUPPORTED;
  if (d->B <= 0 || d->S <= 0 || d->H <= 0 || d->G <= 0 || d->N <= 0 || d->P <= 0 || d->H % d->G) return LR_E_SHAPE;
  const int64_t hp = (int64_t)d->H * d->P, gn = (int64_t)d->G * d->N;
  if (d->ld < hp || d->ldy < hp || d->ldu < hp || d->ldu < gn || (int64_t)d->B * d->S > 0x7fffffff) return LR_E_SHAPE;
  if (d->N % 8 || d->P % 8 || d->ld % 8 || d->ldu % 8 || d->ldy % 8 || lr_misaligned(d->z) || lr_misaligned(d->x) ||
      lr_misaligned(d->b) || lr_misaligned(d->c) || lr_misaligned(d->y))
    return LR_E_ALIGN;
  if (d->N > 256 || d->P > 256 || d->ld > (1 << 22) || d->ldu > (1 << 22) || d->ldy > (1 << 22) || (int64_t)d->B * d->H > (1 << 20))
    return LR_E_UNSUPPORTED;
  a = Ssd{};
  a.z = d->z; a.x = d->x; a.b = d->b; a.c = d->c; a.dt = d->dt; a.ld = d->ld; a.ldu = d->ldu;
  a.dt_bias = d->dt_bias; a.a_log = d->a_log; a.d = d->d; a.pos = d->pos; a.state = d->state; a.y = d->y; a.ldy = d->ldy;
  a.B = d->B; a.S = d->S; a.H = d->H; a.G = d->G; a.N = d->N; a.P = d->P; a.nseg = 1; a.seg_len = d->S; a.err = d->err;
  return LR_OK;
}

}  // namespace

extern "C" int lr_causal_conv(const void* u, int64_t ldu, const void* w, const void* bias, void* ring, const int32_t* pos,
                              void* out, int64_t ldo, int B, int S, int C, int taps, int dtype, lr_stream_t stream) {
  LR_REQUIRE_PTR(u);
  LR_REQUIRE_PTR(w);
  LR_REQUIRE_PTR(bias);
  LR_REQUIRE_PTR(ring);
  LR_REQUIRE_PTR(out);
  if (pos == nullptr) return LR_E_NULL;
  if (B <= 0 || S <= 0 || C <= 0 || taps <= 0 || ldu < C || ldo < C) return LR_E_SHAPE;
  if (C % 8 || ldu % 8 || ldo % 8) return LR_E_ALIGN;
  if (taps > MAX_TAPS || B > 65535 || C > 1024 * 65535) return LR_E_UNSUPPORTED;
  const Conv a = {u, ldu, w, bias, ring, out, ldo, pos, S, C, taps};
  if (dtype == LR_BF16) conv<u16>(a, B, (hipStream_t)stream);
  else if (dtype == LR_F32) conv<float>(a, B, (hipStream_t)stream);
  else return LR_E_UNSUPPORTED;
  return lr_launch_status();
}

extern "C" size_t lr_ssd_scratch_bytes(int B, int S, int H, int N, int P, int dtype) {
  if (B <= 0 || S <= 1 || H <= 0 || N <= 0 || P <= 0 || !on_matrix_cores(N, P, dtype)) return 0;
  const int ns = segments(B, S, H, P);
  return ns > 1 ? align16((size_t)B * H * ns * N * P * sizeof(float)) + align16((size_t)B * H * ns * sizeof(float)) : 0;
}

extern "C" int lr_ssd(const lr_ssd_t* d, lr_stream_t stream) {
  Ssd a;
  int rc = fill(d, a);
  if (rc != LR_OK) return rc;
  hipStream_t s = (hipStream_t)stream;
  if (!on_matrix_cores(a.N, a.P, d->dtype)) return d->dtype == LR_F32 ? walk<float>(a, s) : walk<u16>(a, s);
  a.nseg = segments(a.B, a.S, a.H, a.P);
  if (a.nseg > 1) {
    LR_REQUIRE_PTR(d->scratch);
    if (d->scratch_bytes < lr_ssd_scratch_bytes(a.B, a.S, a.H, a.N, a.P, d->dtype)) return LR_E_SHAPE;
    a.seg_len = ((a.S + a.nseg - 1) / a.nseg + CK - 1) / CK * CK;
    a.seg_state = reinterpret_cast<float*>(d->scratch);
    a.seg_decay = a.seg_state + align16((size_t)a.B * a.H * a.nseg * a.N * a.P * sizeof(float)) / sizeof(float);
    a.nseg = (a.S + a.seg_len - 1) / a.seg_len;
  }
  if (a.nseg > 1) {
    rc = launch_chunk(a, 1, s);
    if (rc != LR_OK) return rc;
    k_ssd_scan<<<dim3(a.B * a.H, (a.N * a.P + 255) / 256), dim3(256), 0, s>>>(a);
  }
  return launch_chunk(a, 0, s);
}

extern "C" int lr_ssd_step(const lr_ssd_t* d, const void* conv_w, const void* conv_b, void* ring, int taps, lr_stream_t stream) {
  Ssd a;
  const int rc = fill(d, a);
  if (rc != LR_OK) return rc;
  LR_REQUIRE_PTR(conv_w);
  LR_REQUIRE_PTR(conv_b);
  LR_REQUIRE_PTR(ring);
  if (taps <= 0 || d->S != 1 || d->ldu < (int64_t)d->H * d->P + 2 * (int64_t)d->G * d->N) return LR_E_SHAPE;
  if (taps > MAX_TAPS) return LR_E_UNSUPPORTED;
  a.conv_w = conv_w; a.conv_b = conv_b; a.ring = ring; a.taps = taps; a.C = a.H * a.P + 2 * a.G * a.N;
  const size_t lds = sizeof(float) * ((size_t)a.P + 2 * a.N + (256 / (a.P / 4)) * a.P);
  hipStream_t s = (hipStream_t)stream;
  const dim3 grid(a.B * a.H), blk(256);
  if (d->dtype == LR_F32) k_ssd_step<float, 0><<<grid, blk, lds, s>>>(a);
  else if (taps == 4) k_ssd_step<u16, 4><<<grid, blk, lds, s>>>(a);
  else k_ssd_step<u16, 0><<<grid, blk, lds, s>>>(a);
  return lr_launch_status();
}

extern "C" int lr_parts_norm(void* y, int64_t ld, const void* gain, int rows, int cols, int parts, int P, int PP, float eps, int dtype,
                             lr_stream_t stream) {
  LR_REQUIRE_PTR(y);
  LR_REQUIRE_PTR(gain);
  if (rows <= 0 || cols <= 0 || parts <= 0 || cols % parts || P <= 0 || PP < P || cols % P || ld < (int64_t)(cols / P) * PP ||
      !(eps >= 0.0f))
    return LR_E_SHAPE;
  if (ld % 8) return LR_E_ALIGN;
  if (parts > 65535) return LR_E_UNSUPPORTED;
  const dim3 grid(rows, parts), blk(256);
  if (dtype == LR_BF16)
    k_parts_norm<u16><<<grid, blk, 0, (hipStream_t)stream>>>((u16*)y, ld, (const u16*)gain, cols / parts, P, PP, eps);
  else if (dtype == LR_F32)
    k_parts_norm<float><<<grid, blk, 0, (hipStream_t)stream>>>((float*)y, ld, (const float*)gain, cols / parts, P, PP, eps);
  else
    return LR_E_UNSUPPORTED;
  return lr_launch_status();
}
