// Element access for the kernels that run in bf16 or in fp32 (template parameter: u16 = bf16 storage, float), and the
// fp32 functions they share.  Everything is computed in fp32; the storage type only decides what is read and written.
#pragma once
#include "lr_common.h"

__device__ __forceinline__ float ldf(const u16* p) { return bf_to_f(*p); }
__device__ __forceinline__ float ldf(const float* p) { return *p; }
__device__ __forceinline__ void stf(u16* p, float v) { *p = f_to_bf(v); }
__device__ __forceinline__ void stf(float* p, float v) { *p = v; }

// four consecutive elements as stored (8 or 16 bytes), and their values
template <typename T> struct Quad;
template <> struct Quad<u16> {
  uint2 r;
  __device__ __forceinline__ void zero() { r = make_uint2(0, 0); }
  __device__ __forceinline__ void load(const u16* p) { r = *reinterpret_cast<const uint2*>(p); }
  __device__ __forceinline__ void get(float* f) const {
    f[0] = bf_lo(r.x); f[1] = bf_hi(r.x); f[2] = bf_lo(r.y); f[3] = bf_hi(r.y);
  }
  __device__ __forceinline__ void put(int j, const u16* p) {
    const u32 v = *p;
    u32& w = j < 2 ? r.x : r.y;
    w = (j & 1) ? (w & 0xffffu) | (v << 16) : (w & 0xffff0000u) | v;
  }
};
template <> struct Quad<float> {
  float4 r;
  __device__ __forceinline__ void zero() { r = make_float4(0, 0, 0, 0); }
  __device__ __forceinline__ void load(const float* p) { r = *reinterpret_cast<const float4*>(p); }
  __device__ __forceinline__ void get(float* f) const { f[0] = r.x; f[1] = r.y; f[2] = r.z; f[3] = r.w; }
  __device__ __forceinline__ void put(int j, const float* p) { reinterpret_cast<float*>(&r)[j] = *p; }
};

__device__ __forceinline__ void st4(u16* p, const float* f) {
  *reinterpret_cast<uint2*>(p) = make_uint2(pack_bf2(f[0], f[1]), pack_bf2(f[2], f[3]));
}
__device__ __forceinline__ void st4(float* p, const float* f) {
  *reinterpret_cast<float4*>(p) = make_float4(f[0], f[1], f[2], f[3]);
}

// 2^x, 1 / x and 1 / sqrt(x) by the hardware instructions (1 ulp in fp32)
__device__ __forceinline__ float exp2_f(float x) { return __builtin_amdgcn_exp2f(x); }
__device__ __forceinline__ float rcp_f(float x) { return __builtin_amdgcn_rcpf(x); }
__device__ __forceinline__ float rsq_f(float x) { return __builtin_amdgcn_rsqf(x); }
constexpr float LOG2E = 1.4426950408889634f;

__device__ __forceinline__ float silu_f(float z) { return z * rcp_f(1.0f + exp2_f(-z * LOG2E)); }

// log of sigmoid(z)^(1/tau): -softplus(-z) / tau
__device__ __forceinline__ float log_sigmoid_f(float z) { return fminf(z, 0.0f) - log1pf(expf(-fabsf(z))); }

// A single step's log-decay is cut off here: 2^-86 of a state is nothing in fp32, and 2^86 is still a finite factor
// (decays are carried as base-2 logarithms).
constexpr float LOG_DECAY_FLOOR = -86.0f;

// Sum over the 16 lanes of a row (lanes 16 r .. 16 r + 15), every lane getting the result.
__device__ __forceinline__ float row16_sum(float v) {
  v += lr_dpp<0x128>(v);  // row_ror:8
  v += lr_dpp<0x124>(v);  // row_ror:4
  v += lr_dpp<0x4e>(v);   // quad_perm [2,3,0,1]
  v += lr_dpp<0xb1>(v);   // quad_perm [1,0,3,2]
  return v;
}
__device__ __forceinline__ float row16_max(float v) {
  v = fmaxf(v, lr_dpp<0x128>(v));
  v = fmaxf(v, lr_dpp<0x124>(v));
  v = fmaxf(v, lr_dpp<0x4e>(v));
  return fmaxf(v, lr_dpp<0xb1>(v));
}

// ---- buffer access: a uniform base and size, per-lane 32-bit byte offsets; beyond the size loads give zero and stores
//      are dropped, so a ragged edge needs no branch
typedef __amdgpu_buffer_rsrc_t rsrc_t;
constexpr int NOWHERE = (int)0x80000000;   // an offset outside every buffer
__device__ __forceinline__ rsrc_t buffer_of(const void* p, int bytes) {
  return __builtin_amdgcn_make_buffer_rsrc(const_cast<void*>(p), 0, bytes, 0x00020000);
}
// (the per-lane offset alone takes part in the range check, so a row's offset belongs in it and not in the scalar one)
__device__ __forceinline__ u16 buf_ld(rsrc_t r, int off, u16) { return __builtin_amdgcn_raw_buffer_load_b16(r, off, 0, 0); }
__device__ __forceinline__ float buf_ld(rsrc_t r, int off, float) {
  return __uint_as_float(__builtin_amdgcn_raw_buffer_load_b32(r, off, 0, 0));
}
__device__ __forceinline__ void buf_st(rsrc_t r, int off, float v, u16) {
  __builtin_amdgcn_raw_buffer_store_b16(f_to_bf(v), r, off, 0, 0);
}
__device__ __forceinline__ void buf_st(rsrc_t r, int off, float v, float) {
  __builtin_amdgcn_raw_buffer_store_b32(__float_as_uint(v), r, off, 0, 0);
}
// The same value, unknown to the optimiser: what is computed from it inside a loop stays there instead of being kept in
// registers across it.
__device__ __forceinline__ int fresh(int x) {
  asm volatile("" : "+v"(x));
  return x;
}
