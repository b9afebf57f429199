// Recurrences with a 32-bit state per request whose decay is one number per token and head: the gated delta rule and the
// state-space recurrence of Mamba-2.  Per head, S is [dim, vdim] (its group's q and k, its own v):
//   delta        S <- a S;  u = b (v - S^T k);  S <- S + k u^T;  o = S^T q          b = sigmoid(zb), q and k unit vectors
//   state space  S <- a S + k (b v)^T;          o = S^T q + D v                     b = softplus(zb + bias)
//   both         a = exp(-rate * softplus(za + bias))
// q, k and v are columns of one 32-bit projection that have passed a short causal convolution over time (per channel) and silu;
// za, zb and the gate z of the output are columns of the same projection.
//   prepare   a step's convolved channels (float): a thread a channel and 8 tokens, unit vectors made in LDS; and the decays and
//             steps of its tokens.  A row holds q and k, 64-aligned heads (`pad` wide), then v: what a tile of the scan loads
//   scan      any entries: a workgroup owns (entry, head, 16 or 32 value columns) and walks the entry's tokens 16 at a time,
//             their q, k and v in LDS, asked for from memory two tiles ahead and stored one ahead, one barrier a tile.  16 lanes of a wavefront share a column: lane s keeps rows 64 j + 4 s .. + 3
//             of it in registers, and their sums meet in four rotations inside the 16 lanes
//             (delta_chunk.hip does the same in chunks on the matrix cores, where results may differ by rounding with the cut)
//   step      single tokens, all in one launch: a workgroup owns (entry, head), makes its channels, moves the state (all of
//             its loads under way before the channels are made) and, for the delta rule, norms and gates the head's result
// The sums of a token are taken in the same order in scan and step, so results do not depend on how the tokens were cut.
// State layouts.  S: [slot][head][vdim / 4][dim / 64][lane][4], the order in which a wavefront reads it (rows beyond dim hold
// zeros).  The convolution's inputs: a ring [slot][taps][channels], the row p % taps being position p's: a step's own row is
// none of the taps - 1 rows it reads, so a workgroup may write it while another one still reads.
#include "delta_common.h"

// the sum over the 16 lanes of a row, the same bits in every lane: rotations by 8, 4, 2 and 1
template <int CTRL>
__device__ __forceinline__ float dl_rotated(float v) {
  return __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), CTRL, 0xf, 0xf, false));
}
__device__ __forceinline__ float dl_row_sum(float v) {
  v += dl_rotated<0x128>(v);
  v += dl_rotated<0x124>(v);
  v += dl_rotated<0x122>(v);
  v += dl_rotated<0x121>(v);
  return v;
}

// 1 / the length of x[0 .. n) (n elements in LDS), by one wavefront
__device__ __forceinline__ float dl_inverse_length(const float* x, int n, float eps, int lane) {
  float ss = 0.f;
  for (int i = lane; i < n; i += WAVE) ss = fmaf(x[i], x[i], ss);
  return 1.f / sqrtf(wave_sum(ss) + eps);
}

// A token's share of one column in a lane: rows 64 j + 4 s .. + 3.  Returns the lane's part of o, for dl_row_sum
template <int R4, bool DELTA>
__device__ __forceinline__ float dl_advance(float4 (&S)[R4], const float4 (&k)[R4], const float4 (&q)[R4], float v, float a, float b) {
  float u;
  if (DELTA) {
    float d0 = 0.f, d1 = 0.f;
#pragma unroll
    for (int j = 0; j < R4; ++j) {
      d0 = fmaf(S[j].x, k[j].x, d0);
      d1 = fmaf(S[j].y, k[j].y, d1);
      d0 = fmaf(S[j].z, k[j].z, d0);
      d1 = fmaf(S[j].w, k[j].w, d1);
    }
    u = b * (v - a * dl_row_sum(d0 + d1));
  } else {
    u = b * v;
  }
  float o0 = 0.f, o1 = 0.f;
#pragma unroll
  for (int j = 0; j < R4; ++j) {
    S[j].x = fmaf(k[j].x, u, a * S[j].x);
    S[j].y = fmaf(k[j].y, u, a * S[j].y);
    S[j].z = fmaf(k[j].z, u, a * S[j].z);
    S[j].w = fmaf(k[j].w, u, a * S[j].w);
    o0 = fmaf(S[j].x, q[j].x, o0);
    o1 = fmaf(S[j].y, q[j].y, o1);
    o0 = fmaf(S[j].z, q[j].z, o0);
    o1 = fmaf(S[j].w, q[j].w, o1);
  }
  return o0 + o1;
}

// ---------------------------------------------------------------------------------------------------- prepare
// grid (token tiles, channel blocks): first the blocks of whole q and k heads (DL_THREADS / dim heads each), then the others, and
// the last for the decays (logs: their logarithms) and steps: coef float2 [tokens][heads]
template <int TAPS, int TB>      // TAPS 0: any number
__global__ __launch_bounds__(DL_THREADS) void delta_prepare_kernel(float* __restrict__ out, float2* __restrict__ coef,
                                                                   const ga_delta_args a,
                                                                   const int32_t* __restrict__ token_entry, int tokens, int logs) {
  __shared__ float ys[TB][DL_THREADS];
  __shared__ float factor[TB][DL_THREADS];
  const int tid = threadIdx.x;
  const int unit_channels = a.delta ? 2 * a.groups * a.dim : 0;
  const int heads_here = a.delta ? DL_THREADS / a.dim : 1, block_channels = heads_here * a.dim;
  const int unit_blocks = a.delta ? (2 * a.groups + heads_here - 1) / heads_here : 0;
  const bool unit = (int)blockIdx.y < unit_blocks;
  int c, last;
  if (unit) {
    c = blockIdx.y * block_channels + tid;
    last = min(unit_channels, (int)(blockIdx.y + 1) * block_channels);
  } else {
    c = unit_channels + (blockIdx.y - unit_blocks) * DL_THREADS + tid;
    last = a.channels;
  }
  const bool live = c < last;
  const int64_t t0 = (int64_t)blockIdx.x * TB;
  const int nt = min((int64_t)TB, tokens - t0);
  if (blockIdx.y == gridDim.y - 1) {
    for (int i = tid; i < nt * a.heads; i += DL_THREADS) {
      const int64_t t = t0 + i / a.heads;
      const int h = i % a.heads;
      const float* row = a.proj + t * a.stride;
      float2 c2 = dl_log_coefficients(a.delta, row[a.a_at + h], row[a.b_at + h], a.dt_bias[h], a.rate[h]);
      if (!logs) c2.x = expf(c2.x);
      coef[t * a.heads + h] = c2;
    }
    return;
  }
  float* to = out + t0 * dl_row(a) + (live ? dl_place(a, c) : 0);
  const int64_t to_row = dl_row(a);
  float y[TB];
#pragma unroll
  for (int i = 0; i < TB; ++i) y[i] = 0.f;
  if (live) {
    const int taps = TAPS ? TAPS : a.taps;
    const float bias = a.conv_bias ? a.conv_bias[c] : 0.f;
    const float* w = a.conv_w + (int64_t)c * taps;
    if (TAPS) {
      float wr[TAPS ? TAPS : 1], x[TB + (TAPS ? TAPS : 1)];      // x[TAPS - 1 + i]: the input of token t0 + i
#pragma unroll
      for (int j = 0; j < TAPS; ++j) wr[j] = w[j];
      const float* col = a.proj + a.conv_at + c;
#pragma unroll
      for (int i = 1 - TAPS; i < TB; ++i) {
        const int64_t t = t0 + i;
        x[TAPS - 1 + i] = (t >= 0 && i < nt) ? col[t * a.stride] : 0.f;
      }
#pragma unroll
      for (int i = 0; i < TB; ++i) {
        if (i >= nt) break;
        const int64_t t = t0 + i;
        const int e = token_entry[t], local = (int)(t - a.cu[e]);
        float acc = bias;
        if (local >= TAPS - 1) {
#pragma unroll
          for (int j = 0; j < TAPS; ++j) acc = fmaf(wr[j], x[i + j], acc);
        } else {
          const int pos = a.q_start[e] + local;
          const int64_t slot = a.slots[e];
#pragma unroll
          for (int j = 0; j < TAPS; ++j)
            acc = fmaf(wr[j], local >= TAPS - 1 - j ? x[i + j] : dl_input(a, t, local, pos, slot, TAPS - 1 - j, c), acc);
        }
        y[i] = dl_silu(acc);
      }
    } else {
      for (int i = 0; i < nt; ++i) {
        const int64_t t = t0 + i;
        const int e = token_entry[t], local = (int)(t - a.cu[e]), pos = a.q_start[e] + local;
        const int64_t slot = taps > 1 ? a.slots[e] : 0;
        float acc = bias;
        for (int j = 0; j < taps; ++j) acc = fmaf(w[j], dl_input(a, t, local, pos, slot, taps - 1 - j, c), acc);
        y[i] = dl_silu(acc);
      }
    }
  }
  if (!unit) {
    if (live) {
#pragma unroll
      for (int i = 0; i < TB; ++i)
        if (i < nt) to[i * to_row] = y[i];
    }
    return;
  }
#pragma unroll
  for (int i = 0; i < TB; ++i) ys[i][tid] = y[i];
  __syncthreads();
  for (int r = tid / WAVE; r < nt * heads_here; r += DL_WAVES) {
    const int i = r / heads_here, hh = r % heads_here;
    const float f = dl_inverse_length(&ys[i][hh * a.dim], a.dim, a.unit_eps, tid % WAVE);
    if (tid % WAVE == 0) factor[i][hh] = f;
  }
  __syncthreads();
  if (live) {
    const float scale = c < a.groups * a.dim ? a.q_scale : 1.f;
    const int hh = tid / a.dim;
#pragma unroll
    for (int i = 0; i < TB; ++i)
      if (i < nt) to[i * to_row] = y[i] * factor[i][hh] * scale;
  }
}

// ---------------------------------------------------------------------------------------------------- scan
// grid (entries, heads, blocks of 16 C value columns): C blocks of four columns to a wavefront; TILE tokens (8 or 16) per trip
// through LDS.  act, coef: as prepare leaves them.  out float [tokens, heads, vdim]: o, or for the state space (o + D v) silu(z).
template <int R4, bool DELTA, int C, int TILE>
__global__ __launch_bounds__(DL_THREADS) __attribute__((amdgpu_waves_per_eu(1, 4))) void delta_scan_kernel(
    float* __restrict__ out, const float* __restrict__ act, const float2* __restrict__ coef, const ga_delta_args a) {
  constexpr int DP = 64 * R4, COLS = DL_COLS * C;
  constexpr int QUADS = TILE * DP / 4 / DL_THREADS;          // 16-byte pieces of a tile's q (and of its k) that a thread brings
  constexpr int VALS = TILE * COLS / DL_THREADS > 0 ? TILE * COLS / DL_THREADS : 1;
  static_assert(TILE * DP % (4 * DL_THREADS) == 0, "whole pieces");
  __shared__ __attribute__((aligned(16))) float ks[2][TILE][DP], qs[2][TILE][DP];
  __shared__ float vs[2][TILE][COLS];
  __shared__ float2 cf[2][TILE];
  const int e = blockIdx.x, h = blockIdx.y, v0 = blockIdx.z * COLS;
  const int first = a.cu[e], n = a.cu[e + 1] - first;
  if (n <= 0) return;
  const int tid = threadIdx.x, lane = tid % WAVE, wave = tid / WAVE, s = lane & 15, col = wave * 4 * C + (lane >> 4);
  const int g = h / (a.heads / a.groups);
  const int start = a.q_start[e];
  const int64_t slot = a.slots[e];
  const int blocks = (a.vdim + 3) / 4, cb = (blockIdx.z * DL_WAVES + wave) * C;
  float4* st = reinterpret_cast<float4*>(a.state) + ((slot * a.heads + h) * blocks + cb) * (int64_t)(R4 * WAVE) + lane;
  float4 S[C][R4];
#pragma unroll
  for (int c = 0; c < C; ++c)
#pragma unroll
    for (int j = 0; j < R4; ++j)
      S[c][j] = (start > 0 && cb + c < blocks) ? st[(c * R4 + j) * WAVE] : make_float4(0.f, 0.f, 0.f, 0.f);
  const int row = (int)dl_row(a);
  const float* qp = act + (int64_t)first * row + g * DP;
  const float* kp = qp + a.groups * DP;
  const float* vp = act + (int64_t)first * row + 2 * a.groups * DP + h * a.vdim + v0;
  const float* zp = a.proj + (int64_t)first * a.stride + a.gate_at + h * a.vdim + v0;
  const float2* cp = coef + (int64_t)first * a.heads + h;
  float* op = out + ((int64_t)first * a.heads + h) * a.vdim + v0;
  float4 rq[QUADS], rk[QUADS];
  float rv[VALS];
  float2 rc;
  // a tile's operands: only asked for here.  Rows behind the entry's last are read as the last and never used; so are columns.
  auto fetch = [&](int t0) {
    const int nt = min(TILE, n - t0);
    const float* q = qp + (int64_t)t0 * row;
    const float* k = kp + (int64_t)t0 * row;
    const float* v = vp + (int64_t)t0 * row;
#pragma unroll
    for (int x = 0; x < QUADS; ++x) {
      const int idx = tid + x * DL_THREADS;
      const int at = min(idx / (DP / 4), nt - 1) * row + 4 * (idx % (DP / 4));
      rq[x] = *reinterpret_cast<const float4*>(q + at);
      rk[x] = *reinterpret_cast<const float4*>(k + at);
    }
#pragma unroll
    for (int x = 0; x < VALS; ++x) {
      const int idx = tid + x * DL_THREADS;
      rv[x] = v[min(idx / COLS, nt - 1) * row + min(idx % COLS, a.vdim - 1 - v0)];
    }
    rc = cp[(int64_t)(t0 + min(tid, nt - 1)) * a.heads];
  };
  const bool ragged = a.dim != DP;                           // the rows beyond dim are zeros
  auto store = [&](int b) {
#pragma unroll
    for (int x = 0; x < QUADS; ++x) {
      const int idx = tid + x * DL_THREADS, tt = idx / (DP / 4), i = 4 * (idx % (DP / 4));
      float4 q = rq[x], k = rk[x];
      if (ragged) {
        q = make_float4(i < a.dim ? q.x : 0.f, i + 1 < a.dim ? q.y : 0.f, i + 2 < a.dim ? q.z : 0.f, i + 3 < a.dim ? q.w : 0.f);
        k = make_float4(i < a.dim ? k.x : 0.f, i + 1 < a.dim ? k.y : 0.f, i + 2 < a.dim ? k.z : 0.f, i + 3 < a.dim ? k.w : 0.f);
      }
      *reinterpret_cast<float4*>(&qs[b][tt][i]) = q;
      *reinterpret_cast<float4*>(&ks[b][tt][i]) = k;
    }
#pragma unroll
    for (int x = 0; x < VALS; ++x) {
      const int idx = tid + x * DL_THREADS;
      if (idx < TILE * COLS) vs[b][idx / COLS][idx % COLS] = rv[x];
    }
    if (tid < TILE) cf[b][tid] = rc;
  };
  const float skip = DELTA ? 0.f : a.skip[h];
  fetch(0);
  store(0);
  if (TILE < n) fetch(TILE);
  __syncthreads();
  int b = 0;
  for (int t0 = 0; t0 < n; t0 += TILE, b ^= 1) {
    const int nt = min(TILE, n - t0);
    // lane s of a column keeps token s's result (and its gate): no branch stands between the tokens
    float mine[C], z[C];
#pragma unroll
    for (int c = 0; c < C; ++c) {
      mine[c] = 0.f;
      z[c] = (!DELTA && s < nt && col + 4 * c < a.vdim - v0) ? zp[(int64_t)(t0 + s) * a.stride + col + 4 * c] : 0.f;
    }
    struct Token { float4 k[R4], q[R4]; float2 ab; float v[C]; };
    auto read = [&](int tt, Token& x) {
#pragma unroll
      for (int j = 0; j < R4; ++j) {
        x.k[j] = *reinterpret_cast<const float4*>(&ks[b][tt][64 * j + 4 * s]);
        x.q[j] = *reinterpret_cast<const float4*>(&qs[b][tt][64 * j + 4 * s]);
      }
      x.ab = cf[b][tt];
#pragma unroll
      for (int c = 0; c < C; ++c) x.v[c] = vs[b][tt][col + 4 * c];
    };
    auto keep = [&](int tt, const float (&part)[C]) {
#pragma unroll
      for (int c = 0; c < C; ++c) {
        const float o = dl_row_sum(part[c]);
        mine[c] = s == tt ? o : mine[c];
      }
    };
    if (nt == TILE) {
      // a token's operands are read while the one before is worked on (its reads may not sink below this line), and the sum of a
      // result fills the waits of the next token's chain
      Token x[2];
      float part[2][C];
      read(0, x[0]);
#pragma unroll
      for (int tt = 0; tt < TILE; ++tt) {
        if (tt + 1 < TILE) read(tt + 1, x[(tt + 1) & 1]);
        __builtin_amdgcn_sched_barrier(0);
        const Token& y = x[tt & 1];
#pragma unroll
        for (int c = 0; c < C; ++c) part[tt & 1][c] = dl_advance<R4, DELTA>(S[c], y.k, y.q, y.v[c], y.ab.x, y.ab.y);
        if (tt > 0) keep(tt - 1, part[(tt - 1) & 1]);
      }
      keep(TILE - 1, part[(TILE - 1) & 1]);
    } else {
      for (int tt = 0; tt < nt; ++tt) {
        Token y;
        read(tt, y);
        float part[C];
#pragma unroll
        for (int c = 0; c < C; ++c) part[c] = dl_advance<R4, DELTA>(S[c], y.k, y.q, y.v[c], y.ab.x, y.ab.y);
        keep(tt, part);
      }
    }
    if (s < nt) {
#pragma unroll
      for (int c = 0; c < C; ++c)
        if (col + 4 * c < a.vdim - v0) {
          float o = mine[c];
          if (!DELTA) o = (o + skip * vs[b][s][col + 4 * c]) * dl_silu(z[c]);
          op[(int64_t)(t0 + s) * a.heads * a.vdim + col + 4 * c] = o;
        }
    }
    if (t0 + TILE < n) {
      store(b ^ 1);
      if (t0 + 2 * TILE < n) fetch(t0 + 2 * TILE);
    }
    __syncthreads();
  }
#pragma unroll
  for (int c = 0; c < C; ++c)
    if (cb + c < blocks) {
#pragma unroll
      for (int j = 0; j < R4; ++j) st[(c * R4 + j) * WAVE] = S[c][j];
    }
  dl_keep_inputs(a, first, n, start, slot, (h * gridDim.z + blockIdx.z) * DL_THREADS + tid, gridDim.y * gridDim.z * DL_THREADS);
}

// ---------------------------------------------------------------------------------------------------- step
// grid (entries, heads): every entry brings one token.  DELTA: out T [tokens, ..] (row stride out_stride), the head's columns
// from h * vdim on, out_scale * weight * silu(gate) * o / rms(o) (the sum of squares in the order of the head norm's kernel);
// else float, (o + D v) silu(gate).  TAPS 0: any number.
template <int R4, bool DELTA, typename T, int TAPS>
__global__ __launch_bounds__(DL_THREADS) void delta_step_kernel(T* __restrict__ out, int64_t out_stride, const ga_delta_args a,
                                                                const float* __restrict__ weight, float eps, float out_scale) {
  constexpr int NB = 16 / R4;                              // column blocks that a wavefront has in registers at a time
  constexpr int RD = 2;                                    // channels of a thread that are under way at a time
  __shared__ __attribute__((aligned(16))) float ks[64 * R4], qs[64 * R4];
  __shared__ float vs[DL_MAX_VDIM], os[DL_MAX_VDIM];
  __shared__ float lengths[2];
  const int e = blockIdx.x, h = blockIdx.y;
  const int tid = threadIdx.x, lane = tid % WAVE, wave = tid / WAVE, s = lane & 15;
  const int64_t t = a.cu[e];
  const int pos = a.q_start[e];
  const int64_t slot = a.slots[e];
  if (a.cu[e + 1] - (int)t <= 0) return;
  const int per_group = a.heads / a.groups, g = h / per_group;
  const int blocks = (a.vdim + 3) / 4;
  const float* row = a.proj + t * a.stride;
  // the channels first: they are what the rest waits for
  const int total = 2 * a.dim + a.vdim;
  auto channel = [&](int i) { return i < a.dim ? a.q_at + g * a.dim + i : i < 2 * a.dim ? a.k_at + g * a.dim + (i - a.dim) : a.v_at + h * a.vdim + (i - 2 * a.dim); };
  constexpr int TP = TAPS ? TAPS : 1;
  float own[RD], back[RD][TP], w[RD][TP], bias[RD];
  auto ask = [&](int i0) {
#pragma unroll
    for (int r = 0; r < RD; ++r) {
      const int i = i0 + r * DL_THREADS;
      const int c = channel(i < total ? i : 0);
      own[r] = row[a.conv_at + c];
      bias[r] = a.conv_bias ? a.conv_bias[c] : 0.f;
      if (TAPS) {
#pragma unroll
        for (int j = 0; j < TAPS; ++j) w[r][j] = a.conv_w[(int64_t)c * TAPS + j];
#pragma unroll
        for (int j = 0; j < TAPS - 1; ++j) {
          const int p = pos - (TAPS - 1 - j);
          back[r][j] = p >= 0 ? a.ring[(slot * TAPS + p % TP) * (int64_t)a.channels + c] : 0.f;
        }
      }
    }
  };
  ask(tid);
  const float za = row[a.a_at + h], zb = row[a.b_at + h], dt_bias = a.dt_bias[h], rate = a.rate[h];
  float gate[2], wt[2];                                    // of the value columns tid and tid + DL_THREADS
#pragma unroll
  for (int r = 0; r < 2; ++r) {
    const int i = tid + r * DL_THREADS;
    gate[r] = i < a.vdim ? row[a.gate_at + h * a.vdim + i] : 0.f;
    wt[r] = (DELTA && i < a.vdim) ? weight[i] : 0.f;
  }
  float4* st = reinterpret_cast<float4*>(a.state) + (slot * a.heads + h) * blocks * (int64_t)(R4 * WAVE) + lane;
  float4 S[NB][R4];
  auto load = [&](int first) {
#pragma unroll
    for (int b = 0; b < NB; ++b) {
      const int cb = first + b * DL_WAVES + wave;
#pragma unroll
      for (int j = 0; j < R4; ++j)
        S[b][j] = (pos > 0 && cb < blocks) ? st[(int64_t)cb * (R4 * WAVE) + j * WAVE] : make_float4(0.f, 0.f, 0.f, 0.f);
    }
  };
  load(0);
  for (int i = tid; i < 64 * R4; i += DL_THREADS)
    if (i >= a.dim) ks[i] = qs[i] = 0.f;
  for (int i0 = tid; i0 < total; i0 += RD * DL_THREADS) {
    if (i0 != tid) ask(i0);
#pragma unroll
    for (int r = 0; r < RD; ++r) {
      const int i = i0 + r * DL_THREADS;
      if (i >= total) continue;
      const int c = channel(i);
      float acc = bias[r];
      if (TAPS) {
#pragma unroll
        for (int j = 0; j < TAPS - 1; ++j) acc = fmaf(w[r][j], back[r][j], acc);
        acc = fmaf(w[r][TP - 1], own[r], acc);
      } else {
        const float* wc = a.conv_w + (int64_t)c * a.taps;
        for (int j = 0; j < a.taps - 1; ++j) acc = fmaf(wc[j], dl_input(a, t, 0, pos, slot, a.taps - 1 - j, c), acc);
        acc = fmaf(wc[a.taps - 1], own[r], acc);
      }
      const float y = dl_silu(acc);
      // the token's own row of the ring (the heads of a group share q and k: the first of them writes)
      if (a.taps > 1 && (i >= 2 * a.dim || h == g * per_group)) a.ring[(slot * a.taps + pos % a.taps) * (int64_t)a.channels + c] = own[r];
      if (i < a.dim) qs[i] = y;
      else if (i < 2 * a.dim) ks[i - a.dim] = y;
      else vs[i - 2 * a.dim] = y;
    }
  }
  float2 c2 = dl_log_coefficients(DELTA, za, zb, dt_bias, rate);
  c2.x = expf(c2.x);
  __syncthreads();
  if (DELTA) {
    if (wave < 2) {
      const float f = dl_inverse_length(wave ? ks : qs, a.dim, a.unit_eps, lane);
      if (lane == 0) lengths[wave] = f;
    }
    __syncthreads();
  }
  float4 k[R4], q[R4];
  const float fq = DELTA ? lengths[0] : 1.f, fk = DELTA ? lengths[1] : 1.f, sq = DELTA ? a.q_scale : 1.f;
#pragma unroll
  for (int j = 0; j < R4; ++j) {
    k[j] = *reinterpret_cast<const float4*>(&ks[64 * j + 4 * s]);
    q[j] = *reinterpret_cast<const float4*>(&qs[64 * j + 4 * s]);
    if (DELTA) {
      k[j].x *= fk; k[j].y *= fk; k[j].z *= fk; k[j].w *= fk;
      q[j].x = q[j].x * fq * sq; q[j].y = q[j].y * fq * sq; q[j].z = q[j].z * fq * sq; q[j].w = q[j].w * fq * sq;
    }
  }
  for (int first = 0; first < blocks; first += NB * DL_WAVES) {
    if (first > 0) load(first);
#pragma unroll
    for (int b = 0; b < NB; ++b) {
      const int cb = first + b * DL_WAVES + wave;
      if (cb < blocks) {
        const int col = cb * 4 + (lane >> 4);
        const float o = dl_row_sum(dl_advance<R4, DELTA>(S[b], k, q, col < a.vdim ? vs[col] : 0.f, c2.x, c2.y));
#pragma unroll
        for (int j = 0; j < R4; ++j) st[(int64_t)cb * (R4 * WAVE) + j * WAVE] = S[b][j];
        if (s == 0 && col < a.vdim) os[col] = o;
      }
    }
  }
  __syncthreads();
  T* op = out + t * out_stride + (int64_t)h * a.vdim;
  float rms = 1.f;
  if (DELTA) {
    float ss = 0.f;                                        // by every wavefront for itself
    for (int i = 4 * lane; i < a.vdim; i += 4 * WAVE)
#pragma unroll
      for (int x = 0; x < 4; ++x)
        if (i + x < a.vdim) ss = fmaf(os[i + x], os[i + x], ss);
    rms = sqrtf(wave_sum(ss) / (float)a.vdim + eps);
  }
  const float skip = DELTA ? 0.f : a.skip[h];
#pragma unroll
  for (int r = 0; r < 2; ++r) {
    const int i = tid + r * DL_THREADS;
    if (i >= a.vdim) continue;
    if (DELTA) Num<T>::st(op + i, os[i] / rms * wt[r] * dl_silu(gate[r]) * out_scale);
    else Num<T>::st(op + i, (os[i] + skip * vs[i]) * dl_silu(gate[r]));
  }
}

extern "C" int64_t ga_delta_row(const ga_delta_args* args) { return dl_row(*args); }

extern "C" int ga_delta_prepare(void* act, void* coef, const ga_delta_args* args, const void* token_entry, int tokens, int logs,
                                hipStream_t stream) {
  if (tokens <= 0) return 0;
  const ga_delta_args& a = *args;
  const int rc = dl_check(a);
  if (rc) return rc;
  const int units = a.delta ? 2 * a.groups : 0, heads_here = a.delta ? DL_THREADS / a.dim : 1;
  const int plain = a.channels - units * a.dim;
  const int64_t blocks = (units + heads_here - 1) / heads_here + (plain + DL_THREADS - 1) / DL_THREADS + 1;
  if (plain < 0 || blocks > 65535 || dl_row(a) > (1 << 26)) return -5;
#define GO(TAPS, TB) hipLaunchKernelGGL((delta_prepare_kernel<TAPS, TB>), dim3((tokens + TB - 1) / TB, (unsigned)blocks), dim3(DL_THREADS), 0, \
                                        stream, (float*)act, (float2*)coef, a, (const int32_t*)token_entry, tokens, logs)
  const bool few = (int64_t)tokens * blocks <= 2048;         // a token to a workgroup while that does not fill the chip
  if (a.taps == 4) { if (few) GO(4, 1); else GO(4, DL_PREP_TOKENS); }
  else { if (few) GO(0, 1); else GO(0, DL_PREP_TOKENS); }
#undef GO
  return GA_CHECK_LAUNCH();
}

extern "C" int ga_delta_scan(void* out, const void* act, const void* coef, const ga_delta_args* args, int entries, hipStream_t stream) {
  if (entries <= 0) return 0;
  const ga_delta_args& a = *args;
  const int rc = dl_check(a);
  if (rc) return rc;
  // two column blocks to a wavefront, which read q and k from LDS once for both, where that still fills the chip
  const int64_t wide = (int64_t)entries * a.heads * ((a.vdim + 2 * DL_COLS - 1) / (2 * DL_COLS));
  const int cols = wide >= 384 ? 2 * DL_COLS : DL_COLS;
  dim3 grid(entries, a.heads, (a.vdim + cols - 1) / cols), block(DL_THREADS);
  if (((uintptr_t)act & 15) || dl_row(a) > (1 << 26)) return -5;
#define GO(R4, D, C, TILE) hipLaunchKernelGGL((delta_scan_kernel<R4, D, C, TILE>), grid, block, 0, stream, (float*)out, (const float*)act, (const float2*)coef, a)
  // (the widest keys take half the tokens a trip: two buffers of 16 would not fit the LDS)
#define GR(D, C) do { const int r = (a.dim + 63) / 64; if (r == 1) GO(1, D, C, 16); else if (r == 2) GO(2, D, C, 16); else if (r == 3) GO(3, D, C, 16); else GO(4, D, C, 8); } while (0)
  if (cols > DL_COLS) { if (a.delta) GR(true, 2); else GR(false, 2); }
  else { if (a.delta) GR(true, 1); else GR(false, 1); }
#undef GR
#undef GO
  return GA_CHECK_LAUNCH();
}

extern "C" int ga_delta_step(void* out, int64_t out_stride, const ga_delta_args* args, const void* weight, float eps, float out_scale,
                             int out_bf16, int entries, hipStream_t stream) {
  if (entries <= 0) return 0;
  const ga_delta_args& a = *args;
  const int rc = dl_check(a);
  if (rc) return rc;
  if (a.delta ? !weight : out_bf16) return -6;
  dim3 grid(entries, a.heads), block(DL_THREADS);
#define GT(R4, D, T, N) hipLaunchKernelGGL((delta_step_kernel<R4, D, T, N>), grid, block, 0, stream, (T*)out, out_stride, a, (const float*)weight, eps, out_scale)
#define GO(R4, D, T) do { if (a.taps == 4) GT(R4, D, T, 4); else GT(R4, D, T, 0); } while (0)
#define GR(D, T) do { const int r = (a.dim + 63) / 64; if (r == 1) GO(1, D, T); else if (r == 2) GO(2, D, T); else if (r == 3) GO(3, D, T); else GO(4, D, T); } while (0)
  if (!a.delta) GR(false, float);
  else if (out_bf16) GR(true, bf16_t);
  else GR(true, float);
#undef GR
#undef GO
#undef GT
  return GA_CHECK_LAUNCH();
}
