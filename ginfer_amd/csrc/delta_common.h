// What the kernels of delta_scan.hip and delta_chunk.hip share: the parameters' checks, the prepared row, decays and inputs.
#pragma once
#include "common.h"
#include "ginfer_amd.h"

#define DL_THREADS 256
#define DL_WAVES (DL_THREADS / WAVE)
#define DL_COLS 16           // value columns of a workgroup of the scan: four to a wavefront
#define DL_MAX_TAPS 16
#define DL_MAX_VDIM 512
#define DL_PREP_TOKENS 8

__device__ __forceinline__ float dl_silu(float z) { return z / (1.f + expf(-z)); }
__device__ __forceinline__ float dl_softplus(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }

// The input of channel c at `back` tokens before the token at row t (place `local` of its entry's tokens, position pos)
__device__ __forceinline__ float dl_input(const ga_delta_args& a, int64_t t, int local, int pos, int64_t slot, int back, int c) {
  if (local >= back) return a.proj[(t - back) * a.stride + a.conv_at + c];
  if (pos < back) return 0.f;
  return a.ring[(slot * a.taps + (pos - back) % a.taps) * (int64_t)a.channels + c];
}

// the decay's logarithm and the step of a head from its two columns of the projection
__device__ __forceinline__ float2 dl_log_coefficients(bool delta, float za, float zb, float dt_bias, float rate) {
  const float sp = dl_softplus(za + dt_bias);
  return make_float2(-rate * sp, delta ? 1.f / (1.f + expf(-zb)) : sp);
}

// A prepared row: q [groups][pad], k [groups][pad], v [heads * vdim], rounded up to 4; pad = dim rounded up to 64 (what lies between
// dim and pad is not written and not used).
__host__ __device__ __forceinline__ int dl_pad(const ga_delta_args& a) { return (a.dim + 63) / 64 * 64; }
__host__ __device__ __forceinline__ int64_t dl_row(const ga_delta_args& a) {
  return ((int64_t)2 * a.groups * dl_pad(a) + (int64_t)a.heads * a.vdim + 3) / 4 * 4;
}
// where convolved channel c lies in a prepared row
__device__ __forceinline__ int dl_place(const ga_delta_args& a, int c) {
  const int n = a.groups * a.dim, pad = dl_pad(a);
  int i = c - a.q_at;
  if (i >= 0 && i < n) return i / a.dim * pad + i % a.dim;
  i = c - a.k_at;
  if (i >= 0 && i < n) return (a.groups + i / a.dim) * pad + i % a.dim;
  return 2 * a.groups * pad + (c - a.v_at);
}

// The last taps inputs of an entry (n tokens from row `first` on, the first at position start) into the ring, the channels dealt to
// `threads` threads of which this is number `mine`
__device__ __forceinline__ void dl_keep_inputs(const ga_delta_args& a, int first, int n, int start, int64_t slot, int mine, int threads) {
  if (a.taps <= 1) return;
  for (int c = mine; c < a.channels; c += threads)
    for (int i = max(0, n - a.taps); i < n; ++i)
      a.ring[(slot * a.taps + (start + i) % a.taps) * (int64_t)a.channels + c] = a.proj[(int64_t)(first + i) * a.stride + a.conv_at + c];
}

static int dl_check(const ga_delta_args& a) {
  if (a.heads <= 0 || a.groups <= 0 || a.heads % a.groups || a.dim <= 0 || a.dim > 256 || a.vdim <= 0 || a.vdim > DL_MAX_VDIM) return -1;
  if (a.taps < 1 || a.taps > DL_MAX_TAPS || (a.taps > 1 && !a.ring) || !a.conv_w) return -2;
  if (a.heads > 65535) return -3;
  if (!a.proj || !a.state || !a.slots || !a.cu || !a.q_start || !a.rate || !a.dt_bias || (!a.delta && !a.skip)) return -4;
  return 0;
}
