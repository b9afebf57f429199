// The experts of a routed feed-forward over their OWN rows (bfloat16), without the host knowing how many rows each has:
//   plan     the token-expert pairs (pair p = token p / top, its choice p % top) grouped by expert, every expert's group cut into
//            tiles of up to TM rows; the tile list lies on the device, (expert, first row, rows) each, and the launches below
//            are as large as the list can get: workgroups beyond its end leave at once.  A step of up
//            to 64 pairs needs no plan: the kernel for few rows finds its tile in the ids themselves.
//   gate-up  act[r, c] = silu(w g) * (w u) (weight_inside) or w * silu(g) * u, g = x[token of r] . Wg_e[c], u = ... Wu_e[c],
//            w the pair's weight; r is the place in the grouped order
//   down     parts[k][t][:] = Wd_e act[r], r the place of pair t * top + k: every choice's result by itself, in 32-bit, for the
//            consumer to add in the order of the choice.  Choices that name no expert here (experts without weights) are left out of
//            everything
// Weights lie as the dense product over all experts has them: expert e's ff gate rows and then its ff up rows in one matrix
// [experts * 2 ff, hidden], the down matrices side by side in one [hidden, experts * ff].
//
// On v_mfma_f32_16x16x32_bf16 (D[m][n] += sum_k A[m][k] B[n][k]; lane l supplies row l % 16 and k-slots (l / 16) * 8 .. + 7 of
// both operands and receives D[(l / 16) * 4 + i][l % 16]), A = 16 rows of a weight matrix, B = 16 of the tile's tokens.
// Two shapes of the same product:
//   few rows   a workgroup takes 16 columns of the result (gate-up: 16 gate and 16 up rows), its wavefronts deal K among
//              themselves in chunks of 128 and stream the weights from memory straight into operands, once for up to 64 rows
//   many rows  a workgroup takes 256 rows of the weight matrix by 64, 128 or 256 of the tile's rows, both brought into LDS in
//              slabs of K, a slab ahead
// A row's result does not depend on the rows beside it, and every sum has an order that depends on K alone.
#include "common.h"
#include "ginfer_amd.h"

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;
typedef __attribute__((ext_vector_type(4))) float f32x4;

__device__ __forceinline__ bf16x8 eg_zero8() {
  const uint4 z = make_uint4(0u, 0u, 0u, 0u);
  return __builtin_bit_cast(bf16x8, z);
}
__device__ __forceinline__ bf16x8 eg_load8(const bf16_t* p) { return __builtin_bit_cast(bf16x8, *reinterpret_cast<const uint4*>(p)); }

__device__ __forceinline__ float eg_act(float g, float u, float w, int inside) {
  if (inside) {
    g *= w;
    u *= w;
    return g / (1.f + expf(-g)) * u;
  }
  return w * (g / (1.f + expf(-g)) * u);
}
__device__ __forceinline__ uint2 eg_pack4(float a, float b, float c, float d) {
  return make_uint2((uint32_t)f32_to_bf16(a) | ((uint32_t)f32_to_bf16(b) << 16), (uint32_t)f32_to_bf16(c) | ((uint32_t)f32_to_bf16(d) << 16));
}

// ---------------------------------------------------------------------------------------------------- plan
#define EP_THREADS 1024
#define EP_MAX_EXPERTS 256

// One workgroup.  tiles int32 [max_tiles][4] = (expert, first row, rows, -), count[0] = tiles in use.
__global__ __launch_bounds__(EP_THREADS) void expert_plan_kernel(const int32_t* __restrict__ ids, int32_t* __restrict__ pair_of_row,
                                                                  int32_t* __restrict__ tiles, int32_t* __restrict__ count, int pairs,
                                                                  int experts, int tile_rows, int max_tiles) {
  __shared__ int n[EP_MAX_EXPERTS], next[EP_MAX_EXPERTS], first_tile[EP_MAX_EXPERTS + 1], first_row[EP_MAX_EXPERTS + 1];
  const int tid = threadIdx.x;
  for (int e = tid; e < EP_MAX_EXPERTS; e += EP_THREADS) n[e] = next[e] = 0;
  __syncthreads();
  for (int p = tid; p < pairs; p += EP_THREADS) {
    const int e = ids[p];
    if (e >= 0 && e < experts) atomicAdd(&n[e], 1);
  }
  __syncthreads();
  if (tid < WAVE) {                       // one wavefront adds up rows and tiles, four experts a lane
    int rows[4], tl[4], r = 0, t = 0;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      rows[j] = n[4 * tid + j];
      tl[j] = (rows[j] + tile_rows - 1) / tile_rows;
      r += rows[j];
      t += tl[j];
    }
    int ri = r, ti = t;
#pragma unroll
    for (int o = 1; o < WAVE; o <<= 1) {
      const int a = __shfl_up(ri, o, WAVE), b = __shfl_up(ti, o, WAVE);
      if (tid >= o) { ri += a; ti += b; }
    }
    r = ri - r;
    t = ti - t;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      first_row[4 * tid + j] = r;
      first_tile[4 * tid + j] = t;
      r += rows[j];
      t += tl[j];
    }
    if (tid == WAVE - 1) count[0] = t < max_tiles ? t : max_tiles;
  }
  __syncthreads();
  for (int e = tid; e < experts; e += EP_THREADS)
    for (int k = 0, t = first_tile[e]; k < n[e]; k += tile_rows, ++t)
      if (t < max_tiles) {
        tiles[4 * t] = e;
        tiles[4 * t + 1] = first_row[e] + k;
        tiles[4 * t + 2] = n[e] - k < tile_rows ? n[e] - k : tile_rows;
        tiles[4 * t + 3] = 0;
      }
  for (int p = tid; p < pairs; p += EP_THREADS) {
    const int e = ids[p];
    if (e >= 0 && e < experts) pair_of_row[first_row[e] + atomicAdd(&next[e], 1)] = p;
  }
}

extern "C" int ga_expert_plan(const void* ids, void* pair_of_row, void* tiles, void* count, int pairs, int experts, int tile_rows,
                              int max_tiles, hipStream_t stream) {
  if (pairs <= 0) return 0;
  if (experts <= 0 || experts > EP_MAX_EXPERTS || tile_rows <= 0 || max_tiles <= 0) return -1;
  hipLaunchKernelGGL(expert_plan_kernel, dim3(1), dim3(EP_THREADS), 0, stream, (const int32_t*)ids, (int32_t*)pair_of_row,
                     (int32_t*)tiles, (int32_t*)count, pairs, experts, tile_rows, max_tiles);
  return GA_CHECK_LAUNCH();
}

// ---------------------------------------------------------------------------------------------------- few rows
// MATS = 2: gate-up (A rows: MB x 16 gate and the same up rows of the expert), MATS = 1: down.  NT groups of 16 rows to a tile, so
// that the weights are read once for all of them, MB groups of 16 columns to a workgroup, so that the rows are read less often
// where there are many; KW wavefronts deal K.  grid (column groups, tiles); K a multiple of 8.
#define ES_CHUNK 128

// The plan of a step of up to 64 pairs, worked out by every wavefront for itself (lane p holds pair p): experts in the order of
// their first pair.  false: there is no tile of this number.  Writes the tile's pairs (every wavefront the same ones).
__device__ __forceinline__ bool es_plan_tile(const int32_t* __restrict__ ids, int pairs, int experts, int tile, int tile_rows, int& e,
                                             int& r0, int& rows, int32_t* tile_pairs, int lane) {
  const int id = lane < pairs ? ids[lane] : -1;
  uint64_t left = __ballot(id >= 0 && id < experts);         // choices beyond the experts that have weights are not ours
  int first = 0;
  while (left) {
    e = __builtin_amdgcn_readlane(id, __builtin_ctzll(left));
    const uint64_t mine = __ballot(id == e);
    const int n = __popcll(mine), tiles = (n + tile_rows - 1) / tile_rows;
    if (tile < tiles) {
      const int from = tile * tile_rows;
      r0 = first + from;
      rows = n - from < tile_rows ? n - from : tile_rows;
      const int at = __popcll(mine & ((1ull << lane) - 1)) - from;
      if (id == e && at >= 0 && at < rows) tile_pairs[at] = lane;
      return true;
    }
    tile -= tiles;
    first += n;
    left &= ~mine;
  }
  return false;
}

template <int MATS, int NT, int MB, int KW>
__global__ __launch_bounds__(KW * WAVE) void expert_few_kernel(void* __restrict__ out, const bf16_t* __restrict__ in,
                                                               const bf16_t* __restrict__ w, int64_t w_expert, int64_t w_row,
                                                               const float* __restrict__ weights, const int32_t* __restrict__ pair_of_row,
                                                               const int32_t* __restrict__ tiles, const int32_t* __restrict__ count,
                                                               const int32_t* __restrict__ ids, int experts, int K, int cols, int top,
                                                               int tokens, int inside) {
  constexpr int MM = MATS * MB;                              // operands of the weights: block mb of matrix m at m * MB + mb
  __shared__ float red[KW][MM * NT][4][WAVE];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, c = lane & 15, g = lane >> 4;
  __shared__ int32_t tile_pairs[16 * NT];                    // the tile's token-expert pairs
  int e, r0, rows;
  if (ids == nullptr) {
    const int tile = blockIdx.y;
    if (tile >= count[0]) return;                            // the whole workgroup
    e = tiles[4 * tile];
    r0 = tiles[4 * tile + 1];
    rows = tiles[4 * tile + 2];
    for (int i = threadIdx.x; i < rows; i += KW * WAVE) tile_pairs[i] = pair_of_row[r0 + i];
  } else if (!es_plan_tile(ids, top * tokens, experts, blockIdx.y, 16 * NT, e, r0, rows, tile_pairs, lane)) {
    return;                                                  // the whole workgroup: every wavefront comes to the same tile
  }
  __syncthreads();
  const int c0 = blockIdx.x * 16 * MB;
  const bf16_t* wp[MM];
#pragma unroll
  for (int m = 0; m < MM; ++m) {
    int col = c0 + (m % MB) * 16 + c;
    if (col >= cols) col = cols - 1;                         // columns beyond the last are computed and not stored
    wp[m] = w + (int64_t)e * w_expert + ((int64_t)(m / MB) * cols + col) * w_row + 8 * g;
  }
  const bf16_t* xp[NT];
#pragma unroll
  for (int n = 0; n < NT; ++n) {
    const int i = 16 * n + c < rows ? 16 * n + c : 0;        // rows beyond the last likewise
    xp[n] = in + (int64_t)(MATS == 2 ? tile_pairs[i] / top : r0 + i) * K + 8 * g;
  }
  f32x4 acc[MM][NT];
#pragma unroll
  for (int m = 0; m < MM; ++m)
#pragma unroll
    for (int n = 0; n < NT; ++n) acc[m][n] = f32x4{0.f, 0.f, 0.f, 0.f};
  for (int k0 = wave * ES_CHUNK; k0 < K; k0 += KW * ES_CHUNK) {
    bf16x8 a[ES_CHUNK / 32][MM], b[ES_CHUNK / 32][NT];
#pragma unroll
    for (int s = 0; s < ES_CHUNK / 32; ++s) {
      const int k = k0 + 32 * s;
      const bool in_k = k + 8 * g < K;
#pragma unroll
      for (int m = 0; m < MM; ++m) a[s][m] = in_k ? eg_load8(wp[m] + k) : eg_zero8();
#pragma unroll
      for (int n = 0; n < NT; ++n) b[s][n] = in_k ? eg_load8(xp[n] + k) : eg_zero8();
    }
#pragma unroll
    for (int s = 0; s < ES_CHUNK / 32; ++s)
#pragma unroll
      for (int m = 0; m < MM; ++m)
#pragma unroll
        for (int n = 0; n < NT; ++n) acc[m][n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a[s][m], b[s][n], acc[m][n], 0, 0, 0);
  }
#pragma unroll
  for (int m = 0; m < MM; ++m)
#pragma unroll
    for (int n = 0; n < NT; ++n)
#pragma unroll
      for (int i = 0; i < 4; ++i) red[wave][m * NT + n][i][lane] = acc[m][n][i];
  __syncthreads();
  for (int task = wave; task < NT * MB; task += KW) {
    const int n = task % NT, mb = task / NT;
    float v[MATS][4];
#pragma unroll
    for (int m = 0; m < MATS; ++m)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        float s = 0.f;
#pragma unroll
        for (int q = 0; q < KW; ++q) s += red[q][(m * MB + mb) * NT + n][i][lane];
        v[m][i] = s;
      }
    const int r = 16 * n + c;
    if (r >= rows) continue;
    const int pair = tile_pairs[r], col = c0 + mb * 16 + 4 * g;
    if (col >= cols) continue;                               // cols is a multiple of 8
    if (MATS == 2) {
      const float wt = weights[pair];
      float y[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) y[i] = eg_act(v[0][i], v[MATS - 1][i], wt, inside);
      *reinterpret_cast<uint2*>((bf16_t*)out + (int64_t)(r0 + r) * cols + col) = eg_pack4(y[0], y[1], y[2], y[3]);
    } else {
      const int t = pair / top;
      *reinterpret_cast<float4*>((float*)out + ((int64_t)(pair - t * top) * tokens + t) * cols + col) =
          make_float4(v[0][0], v[0][1], v[0][2], v[0][3]);
    }
  }
}

// ---------------------------------------------------------------------------------------------------- many rows
// 256 rows of the weight matrix (gate-up: 128 gate and the same 128 up rows) by TM = 64 WN rows of the tile; 2 by WN wavefronts,
// each 128 by 64: 8 operands of the weights against 4 of the rows for every 32 of K.  K in slabs of 64 that go straight from
// memory into LDS, the next one on its way while one is multiplied.  A slab's rows are 128 bytes, eight 16-byte pieces; piece q
// of row r lies at place q ^ (r & 7), so that the rows an operand reads lie in different banks.  K a multiple of 32 (the last slab may
// be half a slab).
typedef __attribute__((address_space(3))) unsigned char lds_byte_t;

// 1 KB from memory into LDS, 16 bytes a lane from the lane's own address; the place is the same for all lanes.  Written out
// because the compiler makes every LDS read wait for loads of this kind that are under way, also where they fill another
// buffer; the loop below waits for them itself.  (s_nop: the place register must rest a cycle before it is read.)
__device__ __forceinline__ void et_bring(uint32_t place, const bf16_t* src) {
  asm volatile("s_mov_b32 m0, %0\n\ts_nop 0\n\tglobal_load_lds_dwordx4 %1, off" ::"s"(place), "v"(src) : "memory");
}
// the wavefront's own loads are in, its LDS reads are through; then all meet
__device__ __forceinline__ void et_wait_and_meet() { asm volatile("s_waitcnt vmcnt(0) lgkmcnt(0)\n\ts_barrier" ::: "memory"); }

#define ET_SLAB 64
template <int MATS, int WN>
__global__ __launch_bounds__(128 * WN, (WN == 1 ? 1 : 2)) void expert_many_kernel(
    void* __restrict__ out, const bf16_t* __restrict__ in, const bf16_t* __restrict__ w, int64_t w_expert, int64_t w_row,
    const float* __restrict__ weights, const int32_t* __restrict__ pair_of_row, const int32_t* __restrict__ tiles,
    const int32_t* __restrict__ count, int K, int cols, int top, int tokens, int inside) {
  constexpr int WR = 256, TM = 64 * WN, WAVES = 2 * WN;
  constexpr int LOADS = (WR + TM) / 8 / WAVES;               // kilobytes (8 rows) of a slab that a wavefront brings
  constexpr int SLAB_BYTES = (WR + TM) * 128;
  constexpr int COLS = WR / MATS;                            // result columns of the workgroup
  extern __shared__ __attribute__((aligned(16))) unsigned char lds[];
  // The workgroups in use dealt to the 8 XCDs in runs (workgroup b lands on XCD b % 8), so that neighbours, which share
  // weights or rows, share an L2; inside a run four tiles by all columns, tiles fastest.
  const int col_groups = (cols + COLS - 1) / COLS, n_tiles = count[0], total = n_tiles * col_groups;
  const int run = (total + 7) / 8, at = blockIdx.x / 8;
  const int id = (blockIdx.x % 8) * run + at;
  if (at >= run || id >= total) return;                      // the whole workgroup
  const int per_group = 4 * col_groups, grp = id / per_group, left = id - grp * per_group;
  const int tiles_here = min(4, n_tiles - 4 * grp);
  const int tile = 4 * grp + left % tiles_here, c0 = left / tiles_here * COLS;
  const int e = tiles[4 * tile], r0 = tiles[4 * tile + 1], rows = tiles[4 * tile + 2];
  const int tid = threadIdx.x, lane = tid & 63, c = lane & 15, g = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6), wm = wave & 1, wn = wave >> 1;
  const uint32_t base = (uint32_t)(uintptr_t)(lds_byte_t*)lds;
  const int piece = (lane & 7) ^ (lane >> 3);                // of the lane's row, in every load
  const bf16_t* src[LOADS];
#pragma unroll
  for (int j = 0; j < LOADS; ++j) {
    const int r = (wave * LOADS + j) * 8 + (lane >> 3);
    if (r < WR) {
      const int m = MATS == 2 ? r / COLS : 0;
      int col = c0 + r - m * COLS;
      if (col >= cols) col = cols - 1;                       // computed and not stored
      src[j] = w + (int64_t)e * w_expert + ((int64_t)m * cols + col) * w_row + 8 * piece;
    } else {
      const int x = r - WR < rows ? r0 + r - WR : r0;
      src[j] = in + (int64_t)(MATS == 2 ? pair_of_row[x] / top : x) * K + 8 * piece;
    }
  }
  f32x4 acc[8][4];
#pragma unroll
  for (int m = 0; m < 8; ++m)
#pragma unroll
    for (int n = 0; n < 4; ++n) acc[m][n] = f32x4{0.f, 0.f, 0.f, 0.f};
  // the lane's place in a slab of its rows' pieces: row r at 128 r, piece 4 kb + g of it at 16 ((4 kb + g) ^ (r & 7)); the
  // operands' rows are 16 apart, so r & 7 is c & 7 for all of them
  const int lane_row = c * 128;
  const int slabs = (K + ET_SLAB - 1) / ET_SLAB;
  const bool half = K % ET_SLAB != 0;
  auto bring = [&](int s) {
    const uint32_t place = base + (uint32_t)((s & 1) * SLAB_BYTES + wave * LOADS * 1024);
    // in a last slab of 32 the pieces behind K stand in for nothing: the ones before are brought twice
    const int back = (half && s == slabs - 1 && piece >= 4) ? 32 : 0;
#pragma unroll
    for (int j = 0; j < LOADS; ++j) et_bring(place + j * 1024, src[j] + (int64_t)s * ET_SLAB - back);
  };
  bring(0);
  for (int s = 0; s < slabs; ++s) {
    et_wait_and_meet();                   // slab s is in, and nobody reads the other buffer any more
    if (s + 1 < slabs) bring(s + 1);
    const unsigned char* cur = lds + (s & 1) * SLAB_BYTES;
    // a wavefront whose rows lie behind the tile's last has nothing to multiply: a group's last tile is often a short one
    const int blocks = wn * 64 >= rows ? 0 : (half && s == slabs - 1) ? 1 : 2;
    for (int kb = 0; kb < blocks; ++kb) {
      const int at16 = ((4 * kb + g) ^ (c & 7)) * 16 + lane_row;
      bf16x8 b[4];
#pragma unroll
      for (int n = 0; n < 4; ++n)
        b[n] = __builtin_bit_cast(bf16x8, *reinterpret_cast<const uint4*>(cur + (WR + wn * 64 + n * 16) * 128 + at16));
#pragma unroll
      for (int m = 0; m < 8; ++m) {
        // gate-up: operands 0 .. 3 are gate rows, 4 .. 7 the up rows of the same columns
        const int r = MATS == 2 ? (m >> 2) * COLS + wm * 64 + (m & 3) * 16 : wm * 128 + m * 16;
        const bf16x8 a = __builtin_bit_cast(bf16x8, *reinterpret_cast<const uint4*>(cur + r * 128 + at16));
#pragma unroll
        for (int n = 0; n < 4; ++n) acc[m][n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b[n], acc[m][n], 0, 0, 0);
      }
    }
  }
#pragma unroll
  for (int n = 0; n < 4; ++n) {
    const int r = wn * 64 + n * 16 + c;
    if (r >= rows) continue;
    const int pair = pair_of_row[r0 + r];
    if (MATS == 2) {
      const float wt = weights[pair];
      bf16_t* o = (bf16_t*)out + (int64_t)(r0 + r) * cols;
#pragma unroll
      for (int m = 0; m < 4; ++m) {
        const int col = c0 + wm * 64 + m * 16 + 4 * g;
        float y[4];
#pragma unroll
        for (int i = 0; i < 4; ++i) y[i] = eg_act(acc[m][n][i], acc[m + 4][n][i], wt, inside);
        if (col < cols) *reinterpret_cast<uint2*>(o + col) = eg_pack4(y[0], y[1], y[2], y[3]);  // cols is a multiple of 8
      }
    } else {
      const int t = pair / top;
      float* o = (float*)out + ((int64_t)(pair - t * top) * tokens + t) * cols;
#pragma unroll
      for (int m = 0; m < 8; ++m) {
        const int col = c0 + wm * 128 + m * 16 + 4 * g;
        if (col < cols) *reinterpret_cast<float4*>(o + col) = make_float4(acc[m][n][0], acc[m][n][1], acc[m][n][2], acc[m][n][3]);
      }
    }
  }
}

// tile_rows (as given to the plan): 16, 32 or 64 the kernel for few rows; -64, 128 or 256 the one for many (64 rows a tile where
// -64; needs K in steps of 32).  Operands bfloat16 at 16-byte addresses, K and cols multiples of 8.
template <int MATS>
static int eg_launch(void* out, const void* in, const void* w, int64_t w_expert, int64_t w_row, const void* weights,
                     const void* pair_of_row, const void* tiles, const void* count, const void* ids, int experts, int max_tiles, int K,
                     int cols, int top, int tokens, int inside, int tile_rows, hipStream_t stream) {
  if (tokens <= 0 || max_tiles <= 0) return 0;
  if (K <= 0 || K % 8 || cols <= 0 || cols % 8 || top <= 0 || w_row % 8 || w_expert % 8 ||
      (((uintptr_t)out | (uintptr_t)in | (uintptr_t)w) & 15))
    return -1;
  // ids instead of a plan: the kernel for few rows plans a step of up to 64 pairs itself
  if (ids ? ((int64_t)top * tokens > 64 || tile_rows < 0 || tile_rows > 64) : (!pair_of_row || !tiles || !count)) return -4;
#define OPERANDS out, (const bf16_t*)in, (const bf16_t*)w, w_expert, w_row, (const float*)weights, (const int32_t*)pair_of_row,  \
                 (const int32_t*)tiles, (const int32_t*)count
#define SIZES K, cols, top, tokens, inside
#define FEW(NT, MB, KW)                                                                                                       \
  hipLaunchKernelGGL((expert_few_kernel<MATS, NT, MB, KW>), dim3((cols + 16 * MB - 1) / (16 * MB), max_tiles), dim3(KW * WAVE), \
                     0, stream, OPERANDS, (const int32_t*)ids, experts, SIZES)
#define MANY(WN)                                                                                                              \
  do {                                                                                                                        \
    const int64_t n = (int64_t)((cols + 256 / MATS - 1) / (256 / MATS)) * max_tiles;                                          \
    constexpr int bytes = (256 + 64 * WN) * 128 * 2;                                                                          \
    static const hipError_t raised = hipFuncSetAttribute(reinterpret_cast<const void*>(expert_many_kernel<MATS, WN>),         \
                                                         hipFuncAttributeMaxDynamicSharedMemorySize, bytes);                  \
    if (raised != hipSuccess) return (int)raised;                                                                             \
    if (K % 32 || n > 0x7ffffff0) return -2;                                                                                  \
    hipLaunchKernelGGL((expert_many_kernel<MATS, WN>), dim3((unsigned)((n + 7) / 8 * 8)), dim3(128 * WN), bytes, stream, OPERANDS, SIZES); \
  } while (0)
  if (max_tiles > 65535) return -2;
  if (tile_rows == 16) FEW(1, 1, 8);
  else if (tile_rows == 32) FEW(2, 2, 4);
  else if (tile_rows == 64) FEW(4, 2, 4);
  else if (tile_rows == 256) MANY(4);
  else if (tile_rows == 128) MANY(2);
  else if (tile_rows == -64) MANY(1);
  else return -3;
#undef MANY
#undef FEW
#undef SIZES
#undef OPERANDS
  return GA_CHECK_LAUNCH();
}

extern "C" int ga_expert_gate_up(void* act, const void* x, const void* w_gate_up, const void* weights, const void* pair_of_row,
                                 const void* tiles, const void* count, const void* ids, int experts, int max_tiles, int hidden, int ff, int top,
                                 int tokens, int weight_inside, int tile_rows, hipStream_t stream) {
  return eg_launch<2>(act, x, w_gate_up, (int64_t)2 * ff * hidden, hidden, weights, pair_of_row, tiles, count, ids, experts, max_tiles, hidden, ff,
                      top, tokens, weight_inside, tile_rows, stream);
}

extern "C" int ga_expert_down(void* parts, const void* act, const void* w_down, int64_t w_row, const void* pair_of_row,
                              const void* tiles, const void* count, const void* ids, int experts, int max_tiles, int hidden, int ff, int top,
                              int tokens, int tile_rows, hipStream_t stream) {
  return eg_launch<1>(parts, act, w_down, ff, w_row, nullptr, pair_of_row, tiles, count, ids, experts, max_tiles, ff, hidden, top, tokens, 0,
                      tile_rows, stream);
}
