// The recurrences of delta_scan.hip in chunks of 16 tokens on the matrix cores' 32-bit instruction.  Inside a chunk, with L_t the sum
// of the decays' logarithms up to token t (from the chunk's start), A_t = exp(L_t), and S the state in front of the chunk:
//   delta        (I + B) U = diag(b) (V - diag(A) K S),   B_ti = b_t exp(L_t - L_i) k_t.k_i for i < t        (U: the writes u_t)
//   state space  U = diag(b) V
//   both         O = diag(A) Q S + P U,                   P_ti = exp(L_t - L_i) q_t.k_i for i <= t
//                S <- A_15 S + K^T diag(exp(L_15 - L_t)) U
// (no exponent is positive, so nothing grows; a last chunk is filled up with tokens that write nothing and do not decay).
//   plan   a workgroup per chunk and group of heads: K, Q and K^T in the order in which a wavefront takes them as operands, and per head
//          W = (I + B)^-1 diag(b) (by substitution, a lane a column: stable, where the powers of B may be large), P and the decays.
//          All of it for every chunk at once: none of it knows the state
//   scan   a workgroup per (entry, head, 16 value columns) walks the entry's chunks.  The state's rows are dealt to four wavefronts,
//          block 4 j + w of 16 rows to wavefront w, and lie in registers as the matrix cores leave them; their partial K S meet in
//          LDS (one barrier a chunk), every wavefront then makes U for itself, and the partial results O meet a chunk later.
// v_mfma_f32_16x16x4_f32: D[m][n] += sum_k A[m][k] B[k][n]; lane l supplies A[l % 16][k] and B[k][l % 16] of one k and receives D[4 (l /
// 16) + i][l % 16].  Four instructions i = 0 .. 3 cover 16 values of k, lane l supplying k = 4 (l / 16) + i: an operand A is four
// consecutive elements of a row, and a result D is, as it is, an operand B.
#include "delta_common.h"

#define DC_CHUNK 16
typedef __attribute__((ext_vector_type(4))) float f32x4;

__device__ __forceinline__ f32x4 dc_mfma(float a, float b, f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }

// chunks of entry e: numbers dc_first(e) on (never overlapping, some numbers unused)
__device__ __forceinline__ int dc_first(const int32_t* __restrict__ cu, int e) { return cu[e] / DC_CHUNK + e; }
// floats per chunk: operands of a group [3][DP / 16][64][4] (K, Q, K^T); of a head W [64][4], P [64][4], A [16], E [16]
__host__ __device__ __forceinline__ int dc_group_floats(const ga_delta_args& a) { return 3 * DC_CHUNK * dl_pad(a); }
#define DC_HEAD_FLOATS 544

// ---------------------------------------------------------------------------------------------------- plan
template <int R4, bool DELTA>
__global__ __launch_bounds__(DL_THREADS) void delta_chunk_plan_kernel(float* __restrict__ ops, float* __restrict__ heads_out,
                                                                      const float* __restrict__ act, const float2* __restrict__ coef,
                                                                      const ga_delta_args a, int entries) {
  constexpr int DP = 64 * R4, PITCH = DP + 4;
  __shared__ __attribute__((aligned(16))) float ks[DC_CHUNK][PITCH], qs[DC_CHUNK][PITCH];
  __shared__ f32x4 part[DL_WAVES][2][WAVE];
  __shared__ __attribute__((aligned(16))) float bm[DELTA ? DL_WAVES * 4 : 1][DC_CHUNK][20];
  const int id = blockIdx.x, g = blockIdx.y;
  int lo = 0, hi = entries - 1;                            // the last entry whose first chunk is not behind this one
  while (lo < hi) {
    const int m = (lo + hi + 1) / 2;
    if (dc_first(a.cu, m) <= id) lo = m;
    else hi = m - 1;
  }
  const int e = lo, c = id - dc_first(a.cu, e), n = a.cu[e + 1] - a.cu[e];
  if (c < 0 || c * DC_CHUNK >= n) return;                  // the whole workgroup
  const int64_t t0 = a.cu[e] + c * DC_CHUNK;
  const int nt = min(DC_CHUNK, n - c * DC_CHUNK);
  const int tid = threadIdx.x, lane = tid % WAVE, w = tid / WAVE, l16 = lane & 15, lg = lane >> 4;
  const int64_t row = dl_row(a);
  for (int idx = tid; idx < DC_CHUNK * DP / 4; idx += DL_THREADS) {
    const int tt = idx / (DP / 4), i = 4 * (idx % (DP / 4));
    const float* q = act + (t0 + min(tt, nt - 1)) * row + g * DP + i;
    const float* k = q + a.groups * DP;
    const float4 q4 = *reinterpret_cast<const float4*>(q), k4 = *reinterpret_cast<const float4*>(k);
    const float qe[4] = {q4.x, q4.y, q4.z, q4.w}, ke[4] = {k4.x, k4.y, k4.z, k4.w};
#pragma unroll
    for (int x = 0; x < 4; ++x) {
      const bool in = tt < nt && i + x < a.dim;
      qs[tt][i + x] = in ? qe[x] : 0.f;
      ks[tt][i + x] = in ? ke[x] : 0.f;
    }
  }
  __syncthreads();
  f32x4* go = reinterpret_cast<f32x4*>(ops + ((int64_t)id * a.groups + g) * dc_group_floats(a));
  f32x4 kk = f32x4{0.f, 0.f, 0.f, 0.f}, kq = kk;           // k_t.k_i, and q_t.k_i with t = l16, i = 4 lg + x
#pragma unroll
  for (int j = 0; j < R4; ++j) {
    const int blk = 4 * j + w;
    const f32x4 k4 = *reinterpret_cast<const f32x4*>(&ks[l16][16 * blk + 4 * lg]);
    const f32x4 q4 = *reinterpret_cast<const f32x4*>(&qs[l16][16 * blk + 4 * lg]);
    f32x4 kt;
#pragma unroll
    for (int x = 0; x < 4; ++x) kt[x] = ks[4 * lg + x][16 * blk + l16];
    go[blk * WAVE + lane] = k4;
    go[(4 * R4 + blk) * WAVE + lane] = q4;
    go[(8 * R4 + blk) * WAVE + lane] = kt;
#pragma unroll
    for (int x = 0; x < 4; ++x) {
      if (DELTA) kk = dc_mfma(k4[x], k4[x], kk);
      kq = dc_mfma(k4[x], q4[x], kq);
    }
  }
  part[w][0][lane] = kk;
  part[w][1][lane] = kq;
  __syncthreads();
  kk = (part[0][0][lane] + part[1][0][lane]) + (part[2][0][lane] + part[3][0][lane]);
  kq = (part[0][1][lane] + part[1][1][lane]) + (part[2][1][lane] + part[3][1][lane]);
  const int per = a.heads / a.groups;
  // four heads of the group to a wavefront at a time
  for (int h0 = 4 * w; h0 < per; h0 += 4 * DL_WAVES) {
    const int here = min(4, per - h0);
    float b_of_column = 0.f;                               // of head lg of the four, token l16
    for (int x = 0; x < here; ++x) {
      const int h = g * per + h0 + x;
      const float2 c2 = l16 < nt ? coef[(t0 + l16) * a.heads + h] : make_float2(0.f, 0.f);
      float L = c2.x;                                      // summed up over the 16 lanes
#pragma unroll
      for (int o = 1; o < DC_CHUNK; o <<= 1) {
        const float up = __shfl_up(L, o, DC_CHUNK);
        if (l16 >= o) L += up;
      }
      const float last = __shfl(L, DC_CHUNK - 1, DC_CHUNK);
      float* ho = heads_out + ((int64_t)id * a.heads + h) * DC_HEAD_FLOATS;
      f32x4 P, B;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int ti = 4 * lg + i;
        const float decay = expf(fminf(L - __shfl(L, ti, DC_CHUNK), 0.f));
        P[i] = ti <= l16 ? decay * kq[i] : 0.f;
        if (!DELTA) P[i] *= __shfl(c2.y, ti, DC_CHUNK);    // the state space writes b v: b goes with P and with E
        if (DELTA) B[i] = ti < l16 ? c2.y * decay * kk[i] : 0.f;
      }
      reinterpret_cast<f32x4*>(ho)[WAVE + lane] = P;
      if (lane < DC_CHUNK) {
        ho[512 + lane] = expf(L);
        ho[528 + lane] = expf(last - L) * (DELTA ? 1.f : c2.y);
      }
      if (DELTA) {
        *reinterpret_cast<f32x4*>(&bm[w * 4 + x][l16][4 * lg]) = B;
        if (lg == x) b_of_column = c2.y;
      }
    }
    if (DELTA) {
      __builtin_amdgcn_wave_barrier();                     // a wavefront's LDS keeps its order
      if (lg < here) {
        float T[DC_CHUNK];                                 // column l16 of (I + B)^-1 of head lg
#pragma unroll
        for (int t = 0; t < DC_CHUNK; ++t) {
          float acc = t == l16 ? 1.f : 0.f;
#pragma unroll
          for (int i = 0; i < t; ++i) acc = fmaf(-bm[w * 4 + lg][t][i], T[i], acc);
          T[t] = acc;
        }
        float* wo = heads_out + ((int64_t)id * a.heads + g * per + h0 + lg) * DC_HEAD_FLOATS;
#pragma unroll
        for (int t = 0; t < DC_CHUNK; ++t) wo[((l16 >> 2) * DC_CHUNK + t) * 4 + (l16 & 3)] = T[t] * b_of_column;
      }
      __builtin_amdgcn_wave_barrier();
    }
  }
}

// ---------------------------------------------------------------------------------------------------- scan
template <int R4, bool DELTA>
struct ChunkOperands {
  f32x4 k[DELTA ? R4 : 1], q[R4], kt[R4], w, A, E, v;
  float p, last;
  float v_own, z_own;          // the state space's output: of this thread's own place (token tid / 16, column tid % 16)
};

template <int R4, bool DELTA>
__global__ __launch_bounds__(DL_THREADS) __attribute__((amdgpu_waves_per_eu(2, 4))) void delta_chunk_scan_kernel(
    float* __restrict__ out, const float* __restrict__ ops, const float* __restrict__ heads_in, const float* __restrict__ act,
    const ga_delta_args a, int tokens) {
  constexpr int DP = 64 * R4;
  __shared__ f32x4 meet[DELTA ? 2 : 1][DL_WAVES][WAVE], results[2][DL_WAVES][WAVE];
  const int e = blockIdx.x, h = blockIdx.y, v0 = blockIdx.z * 16;
  const int first = a.cu[e], n = a.cu[e + 1] - first;
  if (n <= 0) return;
  const int tid = threadIdx.x, lane = tid % WAVE, w = __builtin_amdgcn_readfirstlane(tid / WAVE), l16 = lane & 15, lg = lane >> 4;
  const int wl = tid / WAVE;                               // the wavefront's number once more, not known to be the same in all lanes
  const int g = h / (a.heads / a.groups), start = a.q_start[e];
  const int64_t slot = a.slots[e], row = dl_row(a);
  const int blocks = (a.vdim + 3) / 4, cb = blockIdx.z * 4 + (l16 >> 2);
  // element i of S[j]: row 64 j + 16 w + 4 lg + i of column v0 + l16
  f32x4* st = reinterpret_cast<f32x4*>(a.state) + ((slot * a.heads + h) * blocks + cb) * (int64_t)(R4 * WAVE) + (l16 & 3) * 16 + 4 * w + lg;
  f32x4 S[R4];
  const f32x4 zero = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int j = 0; j < R4; ++j) S[j] = (start > 0 && cb < blocks) ? st[j * WAVE] : zero;
  const int id0 = dc_first(a.cu, e), chunks = (n + DC_CHUNK - 1) / DC_CHUNK;
  const int own_t = tid / 16, own_c = tid % 16;
  const bool own_ok = v0 + own_c < a.vdim;
  // Where the next chunk to be asked for lies: uniform pointers that move on by a chunk (the last one is asked for again at the end),
  // and byte offsets of the lane's own.
  const char* go = reinterpret_cast<const char*>(ops + ((int64_t)id0 * a.groups + g) * dc_group_floats(a));
  const char* ho = reinterpret_cast<const char*>(heads_in + ((int64_t)id0 * a.heads + h) * DC_HEAD_FLOATS);
  const char* vp = reinterpret_cast<const char*>(act + (int64_t)first * row + 2 * a.groups * DP + h * a.vdim + v0);
  const char* zp = reinterpret_cast<const char*>(a.proj + (int64_t)first * a.stride + a.gate_at + h * a.vdim + v0);
  const int64_t go_step = (int64_t)a.groups * dc_group_floats(a) * 4, ho_step = (int64_t)a.heads * DC_HEAD_FLOATS * 4;
  const int64_t vp_step = DC_CHUNK * row * 4, zp_step = DC_CHUNK * a.stride * 4;
  const uint32_t row_bytes = (uint32_t)row * 4, z_bytes = (uint32_t)a.stride * 4;
  const uint32_t lane16 = (uint32_t)lane * 16, wave16 = (uint32_t)(w * WAVE + lane) * 16, lg16 = (uint32_t)lg * 16;
  const uint32_t p_at = (uint32_t)(1024 + 16 * lane + 4 * w);
  const uint32_t col_bytes = (uint32_t)min(l16, a.vdim - 1 - v0) * 4, own_bytes = (uint32_t)min(own_c, a.vdim - 1 - v0) * 4;
  int left = n;                                            // tokens from the next chunk to be asked for on
  auto load = [](const char* base, uint32_t at) { return *reinterpret_cast<const float*>(base + at); };
  auto load4 = [](const char* base, uint32_t at) { return *reinterpret_cast<const f32x4*>(base + at); };
  auto fetch = [&](ChunkOperands<R4, DELTA>& x) {
#pragma unroll
    for (int j = 0; j < R4; ++j) {
      if (DELTA) x.k[j] = load4(go + j * 4 * WAVE * 16, wave16);
      x.q[j] = load4(go + (4 * R4 + 4 * j) * WAVE * 16, wave16);
      x.kt[j] = load4(go + (8 * R4 + 4 * j) * WAVE * 16, wave16);
    }
    if (DELTA) x.w = load4(ho, lane16);
    x.p = load(ho, p_at);
    x.A = load4(ho + 2048, lg16);
    x.E = load4(ho + 2112, lg16);
    x.last = *reinterpret_cast<const float*>(ho + 2048 + 4 * (DC_CHUNK - 1));
    // tokens behind the last stand for it: their columns of W and P and their E are zero; columns behind the last are not stored
    const uint32_t last_row = (uint32_t)(min(DC_CHUNK, left) - 1);
#pragma unroll
    for (int i = 0; i < 4; ++i) x.v[i] = load(vp, min((uint32_t)(4 * lg + i) * row_bytes, last_row * row_bytes) + col_bytes);
    if (!DELTA) {
      x.v_own = load(vp, min((uint32_t)own_t * row_bytes, last_row * row_bytes) + own_bytes);
      x.z_own = load(zp, min((uint32_t)own_t * z_bytes, last_row * z_bytes) + own_bytes);
    }
    const bool more = left > DC_CHUNK;
    left -= more ? DC_CHUNK : 0;
    go += more ? go_step : 0;
    ho += more ? ho_step : 0;
    vp += more ? vp_step : 0;
    zp += more ? zp_step : 0;
  };
  const float skip = DELTA ? 0.f : a.skip[h];
  // a chunk's results, from the four wavefronts' parts; places that are not the entry's go to the row behind the last token's
  const int read_at = (own_t >> 2) * 16 + own_c, read_i = own_t & 3;
  float* to = out + ((int64_t)(first + own_t) * a.heads + h) * a.vdim + v0 + own_c - 2 * (int64_t)DC_CHUNK * a.heads * a.vdim;   // of chunk -2
  float* const aside = out + ((int64_t)tokens * a.heads + h) * a.vdim;
  const int64_t to_step = (int64_t)DC_CHUNK * a.heads * a.vdim;
  int own_left = own_ok ? n - own_t + 2 * DC_CHUNK : 0;    // > 0: the token of the chunk that is put next is the entry's
  auto put = [&](bool real, int b, float v_own, float z_own) {
    float o = (results[b][0][read_at][read_i] + results[b][1][read_at][read_i]) + (results[b][2][read_at][read_i] + results[b][3][read_at][read_i]);
    if (!DELTA) o = (o + skip * v_own) * dl_silu(z_own);
    *(real && own_left > 0 ? to : aside) = o;
    to += to_step;
    own_left -= DC_CHUNK;
  };
  ChunkOperands<R4, DELTA> x[3];
  fetch(x[0]);
  fetch(x[1]);
  float v_before[2] = {0.f, 0.f}, z_before[2] = {0.f, 0.f};
  results[0][w][lane] = results[1][w][lane] = zero;        // (read, not stored, in the first two chunks)
  __syncthreads();
  // No branch from here to the end of a chunk: what is not a product is issued in the products' shadow, and the compiler's count of
  // the states that a product's reader has to wait for ends at a branch that skips (seen in its assembly, and in results).
  auto chunk = [&](int c, ChunkOperands<R4, DELTA>& y, ChunkOperands<R4, DELTA>& next, int b) {
    f32x4 qs = zero;
    if (DELTA) {
      f32x4 ks[2] = {zero, zero};
#pragma unroll
      for (int j = 0; j < R4; ++j)
#pragma unroll
        for (int i = 0; i < 4; ++i) ks[i & 1] = dc_mfma(y.k[j][i], S[j][i], ks[i & 1]);
      meet[b][w][lane] = ks[0] + ks[1];
    }
    fetch(next);                                           // what is used two chunks on
#pragma unroll
    for (int j = 0; j < R4; ++j)
#pragma unroll
      for (int i = 0; i < 4; ++i) qs = dc_mfma(y.q[j][i], S[j][i], qs);
    put(c >= 2, b, v_before[b], z_before[b]);               // (its parts were in before the barrier of the chunk before)
    if (!DELTA) {
      v_before[b] = y.v_own;
      z_before[b] = y.z_own;
    }
    f32x4 U, R[R4];
#pragma unroll
    for (int j = 0; j < R4; ++j) R[j] = S[j] * y.last;
    // a product, then what fits into its shadow
#pragma unroll
    for (int i = 0; i < (DELTA ? 8 : 4) * R4; ++i) {
      __builtin_amdgcn_sched_group_barrier(0x008, 1, 0);
      __builtin_amdgcn_sched_group_barrier(0x020, DELTA ? 2 : 3, 0);
      __builtin_amdgcn_sched_group_barrier(0x002, DELTA ? 5 : 8, 0);
    }
    __syncthreads();
    if (DELTA) {
      const f32x4 all = (meet[b][0][lane] + meet[b][1][lane]) + (meet[b][2][lane] + meet[b][3][lane]);
      const f32x4 X = y.v - y.A * all;
      f32x4 u1 = zero;
      U = zero;
      U = dc_mfma(y.w[0], X[0], U);
      u1 = dc_mfma(y.w[1], X[1], u1);
      U = dc_mfma(y.w[2], X[2], U);
      u1 = dc_mfma(y.w[3], X[3], u1);
      U += u1;
    } else {
      U = y.v;
    }
    const f32x4 V = U * y.E;
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int j = 0; j < R4; ++j) R[j] = dc_mfma(y.kt[j][i], V[i], R[j]);
    float u_w = U[0];                                      // this wavefront's share of P U
    u_w = wl == 1 ? U[1] : u_w;
    u_w = wl == 2 ? U[2] : u_w;
    u_w = wl == 3 ? U[3] : u_w;
    results[b][w][lane] = dc_mfma(y.p, u_w, y.A * qs);
#pragma unroll
    for (int j = 0; j < R4; ++j) {
      S[j] = R[j];
      asm volatile("" : "+v"(S[j]));
    }
    asm volatile("s_nop 15");                              // the next chunk, behind a branch, may read S in its first instruction
  };
  for (int c = 0; c < chunks; c += 6) {
    chunk(c, x[0], x[2], 0);
    if (c + 1 < chunks) chunk(c + 1, x[1], x[0], 1);
    if (c + 2 < chunks) chunk(c + 2, x[2], x[1], 0);
    if (c + 3 < chunks) chunk(c + 3, x[0], x[2], 1);
    if (c + 4 < chunks) chunk(c + 4, x[1], x[0], 0);
    if (c + 5 < chunks) chunk(c + 5, x[2], x[1], 1);
  }
  __syncthreads();
  const int last = chunks - 1;
  const bool odd = last & 1;
  put(last >= 1, odd ? 0 : 1, odd ? v_before[0] : v_before[1], odd ? z_before[0] : z_before[1]);
  put(true, odd ? 1 : 0, odd ? v_before[1] : v_before[0], odd ? z_before[1] : z_before[0]);
  if (cb < blocks) {
#pragma unroll
    for (int j = 0; j < R4; ++j) st[j * WAVE] = S[j];
  }
  dl_keep_inputs(a, first, n, start, slot, (h * gridDim.z + blockIdx.z) * DL_THREADS + tid, gridDim.y * gridDim.z * DL_THREADS);
}

static int64_t dc_chunks(int tokens, int entries) { return (int64_t)tokens / DC_CHUNK + entries; }

extern "C" int64_t ga_delta_chunk_floats(const ga_delta_args* args, int tokens, int entries, int what) {
  const ga_delta_args& a = *args;
  return dc_chunks(tokens, entries) * (what == 0 ? (int64_t)a.groups * dc_group_floats(a) : (int64_t)a.heads * DC_HEAD_FLOATS);
}

#define DC_GO(D) do { const int r = (a.dim + 63) / 64; if (r == 1) GO(1, D); else if (r == 2) GO(2, D); else if (r == 3) GO(3, D); else GO(4, D); } while (0)

extern "C" int ga_delta_chunk_plan(void* ops, void* heads, const void* act, const void* coef, const ga_delta_args* args, int tokens, int entries,
                                   hipStream_t stream) {
  if (tokens <= 0 || entries <= 0) return 0;
  const ga_delta_args& a = *args;
  const int rc = dl_check(a);
  if (rc) return rc;
  if ((((uintptr_t)ops | (uintptr_t)heads | (uintptr_t)act) & 15) || a.groups > 65535) return -5;
  dim3 grid((unsigned)dc_chunks(tokens, entries), a.groups), block(DL_THREADS);
#define GO(R4, D) hipLaunchKernelGGL((delta_chunk_plan_kernel<R4, D>), grid, block, 0, stream, (float*)ops, (float*)heads, (const float*)act, \
                                     (const float2*)coef, a, entries)
  if (a.delta) DC_GO(true); else DC_GO(false);
#undef GO
  return GA_CHECK_LAUNCH();
}

extern "C" int ga_delta_chunk_scan(void* out, const void* ops, const void* heads, const void* act, const ga_delta_args* args, int tokens,
                                   int entries, hipStream_t stream) {
  if (entries <= 0 || tokens <= 0) return 0;
  const ga_delta_args& a = *args;
  const int rc = dl_check(a);
  if (rc) return rc;
  if (((uintptr_t)ops | (uintptr_t)heads | (uintptr_t)act | (uintptr_t)a.state) & 15) return -5;
  dim3 grid(entries, a.heads, (a.vdim + 15) / 16), block(DL_THREADS);
#define GO(R4, D) hipLaunchKernelGGL((delta_chunk_scan_kernel<R4, D>), grid, block, 0, stream, (float*)out, (const float*)ops, (const float*)heads, \
                                     (const float*)act, a, tokens)
  if (a.delta) DC_GO(true); else DC_GO(false);
#undef GO
  return GA_CHECK_LAUNCH();
}
