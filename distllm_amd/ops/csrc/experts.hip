// Routed experts, gated units or squared ReLU.
//
//   route:   softmax scores of a row over all experts, the best groups, the
//            best experts in them                    -> ids, weights [M, top]
//            or sigmoid scores, the best with a correction added
//   plan:    (row, choice) pairs sorted by expert, cut into tiles of rows
//   product: one grouped product per tile; the first one gathers the rows
//            and applies silu(gate) * up or relu(up)^2, the second scatters
//            its rows to row * top + choice
//
// Gated units, [E, 2F, K]: gate and up rows alternate in groups of 16, so
// that a tile of columns holds both halves of the unit. The number of tiles is
// known on the device only: grids have the most there can be and surplus
// workgroups leave at once.
#include "common.h"

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;

extern __shared__ __attribute__((aligned(16))) char smem[];

// ---- routing ----------------------------------------------------------------
// Softmax scores, or (correction not null) sigmoid scores whose sum with the
// correction [E] makes the choice; weights are the scores times `scale`.
// With `gate`, one more logit is the gate of an expert that serves every row;
// its sigmoid is a weight behind those of the chosen experts, or (shards > 0)
// the weight of `shards` further choices, experts E, E + 1, ..
struct RouteArgs {
  int E, groups, keep, top;
  const float* correction;
  float scale;
  bool gate;
  int shards;

  __host__ __device__ __forceinline__ int logits() const { return E + gate; }
  __host__ __device__ __forceinline__ int ids() const { return top + shards; }
  __host__ __device__ __forceinline__ int cols() const {
    return shards > 0 ? top + shards : top + gate;
  }
};

// the largest number of a wave, by lane shifts within and between rows of 16
__device__ __forceinline__ float wave_max(float v) {
#define WM(ctrl, rows)                                                     \
  v = fmaxf(v, __int_as_float(__builtin_amdgcn_update_dpp(                 \
                   __float_as_int(v), __float_as_int(v), ctrl, rows, 0xf,  \
                   false)))
  WM(0x111, 0xf);  // row_shr:1, :2, :4, :8
  WM(0x112, 0xf);
  WM(0x114, 0xf);
  WM(0x118, 0xf);
  WM(0x142, 0xa);  // row_bcast:15 to rows 1 and 3
  WM(0x143, 0xc);  // row_bcast:31 to rows 2 and 3
#undef WM
  return __int_as_float(__builtin_amdgcn_readlane(__float_as_int(v), 63));
}

// One wave chooses for one row. z: logits, overwritten; gm, ok
// [groups]. A lane holds the scores of experts lane + 64 i, i < PER.
template <int PER>
__device__ void select_row(float* z, float* gm, int* ok, const RouteArgs& a,
                           int* __restrict__ ids, float* __restrict__ weights,
                           int lane) {
  const int E = a.E, groups = a.groups;
  float s[PER], w[PER];  // what is compared, what it weighs
  float scale = a.scale;
  if (a.correction != nullptr) {
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      const int e = lane + 64 * i;
      w[i] = e < E ? sigmoid_exact(z[e]) : 0.f;
      s[i] = e < E ? w[i] + a.correction[e] : 0.f;
    }
    for (int j = a.top + lane; j < a.cols(); j += 64) {
      weights[j] = sigmoid_exact(z[E]);
      if (j < a.ids()) ids[j] = E + j - a.top;
    }
  } else {
    float mx = -INFINITY;
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      const int e = lane + 64 * i;
      s[i] = e < E ? z[e] : -INFINITY;
      mx = fmaxf(mx, s[i]);
    }
    mx = wave_reduce_max(mx);
    float sum = 0.f;
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      w[i] = s[i] = expf(s[i] - mx);
      sum += s[i];
    }
    scale /= wave_reduce_sum(sum);
  }
  if (groups > 1) {
#pragma unroll
    for (int i = 0; i < PER; ++i)
      if (lane + 64 * i < E) z[lane + 64 * i] = s[i];
    wave_sync();
    const int per = E / groups;
    for (int c = lane; c < groups; c += 64) {
      float b = -INFINITY;
      for (int i = 0; i < per; ++i) b = fmaxf(b, z[c * per + i]);
      gm[c] = b;
    }
    wave_sync();
    for (int c = lane; c < groups; c += 64) {
      int rank = 0;
      for (int i = 0; i < groups; ++i)
        rank += gm[i] > gm[c] || (gm[i] == gm[c] && i < c);
      ok[c] = rank < a.keep;
    }
    wave_sync();
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      const int e = lane + 64 * i;
      if (e < E && !ok[e / per]) s[i] = -INFINITY;
    }
  }
#pragma unroll
  for (int i = 0; i < PER; ++i)
    if (lane + 64 * i >= E) s[i] = -INFINITY;
  float own = -INFINITY, weight = 0.f;  // the lane's best, and which it is
  int at = 0;
  auto best = [&]() {
    own = -INFINITY;
#pragma unroll
    for (int i = 0; i < PER; ++i)
      if (s[i] > own) {
        own = s[i];
        weight = w[i];
        at = i;
      }
  };
  best();
  int id = -1;  // lane t keeps choice t until 64 are stored together
  float wt = 0.f;
  for (int t = 0; t < a.top; ++t) {
    const float m = wave_max(own);
    int e = -1;  // not a number: no expert
    float we = 0.f;
    if (m > -INFINITY) {
      const int who = __builtin_ctzll(__ballot(own == m));
      e = who + 64 * __builtin_amdgcn_readlane(at, who);
      we = __int_as_float(
          __builtin_amdgcn_readlane(__float_as_int(weight), who));
      const bool mine = lane == who;
#pragma unroll
      for (int i = 0; i < PER; ++i)
        if (mine && i == at) s[i] = -INFINITY;
      best();
    }
    if ((t & 63) == lane) {
      id = e;
      wt = we * scale;
    }
    if ((t & 63) == 63 || t + 1 == a.top) {
      const int place = (t & ~63) + lane;
      if (place <= t) {
        ids[place] = id;
        weights[place] = wt;
      }
    }
  }
}

__device__ __forceinline__ void no_choice(const RouteArgs& a, int* ids,
                                          float* weights, int lane) {
  for (int t = lane; t < a.ids(); t += 64) ids[t] = -1;
  for (int t = lane; t < a.cols(); t += 64) weights[t] = 0.f;
}

// from given logits; one wave per row
__global__ void __launch_bounds__(256)
select_kernel(const float* __restrict__ logits, const int* __restrict__ ctx,
              int M, const RouteArgs a, int* __restrict__ ids,
              float* __restrict__ weights) {
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  const int n = a.logits();
  float* z = reinterpret_cast<float*>(smem) + wid * (n + 2 * a.groups);
  float* gm = z + n;
  int* ok = reinterpret_cast<int*>(gm + a.groups);
  const int row = blockIdx.x * 4 + wid;
  if (row >= M) return;
  int* id = ids + (long)row * a.ids();
  float* w = weights + (long)row * a.cols();
  if (ctx[row] <= 0) {
    no_choice(a, id, w, lane);
    return;
  }
  for (int e = lane; e < n; e += 64) z[e] = logits[(long)row * n + e];
  wave_sync();
  select_row<16>(z, gm, ok, a, id, w, lane);
}

// bf16 rows against the router's weights [logits, K], fp32 sums, then the
// choice: 16 rows per workgroup, its NW waves split K and then the rows. NE
// tiles of 16 logits.
template <int NE, int NW>
__global__ void __launch_bounds__(NW * 64)
route_kernel(const unsigned short* __restrict__ h,
             const unsigned short* __restrict__ W,
             const int* __restrict__ ctx, int M, int K, const RouteArgs args,
             int* __restrict__ ids, float* __restrict__ weights) {
  constexpr int EP = NE * 16;
  constexpr int WS = 16 * (EP + 4);  // sums of a wave
  const int E = args.logits(), groups = args.groups;
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  const int i16 = lane & 15, g = lane >> 4;
  const int m0 = blockIdx.x * 16;
  // An operand's 16 rows of 64 bytes are loaded with four lanes to a row,
  // whole pieces of memory, and pass LDS to get where the product wants them.
  const int lrow = lane >> 2, lcol = (lane & 3) * 8;
  const unsigned short* src[NE + 1];
#pragma unroll
  for (int j = 0; j < NE; ++j)
    src[j] = W + (long)min(j * 16 + lrow, E - 1) * K + lcol;
  src[NE] = h + (long)min(m0 + lrow, M - 1) * K + lcol;
  char* own = smem + wid * (NE + 1) * 1024;
  const int put = lrow * 64 + (((lane & 3) ^ ((lrow >> 2) & 3)) * 16);
  const int get = i16 * 64 + ((g ^ ((i16 >> 2) & 3)) * 16);
  f32x4 acc[NE];
#pragma unroll
  for (int j = 0; j < NE; ++j) acc[j] = {0.f, 0.f, 0.f, 0.f};
  // U steps of loads are in flight together
  constexpr int U = NE <= 9 ? 2 : 1;
  for (int k0 = wid * 32; k0 < K; k0 += U * NW * 32) {
    i32x4 x[U][NE + 1];
#pragma unroll
    for (int s = 0; s < U; ++s)
#pragma unroll
      for (int j = 0; j <= NE; ++j)
        x[s][j] = *reinterpret_cast<const i32x4*>(
            src[j] + min(k0 + s * NW * 32, K - 32));
    __builtin_amdgcn_sched_barrier(0);
#pragma unroll
    for (int s = 0; s < U; ++s) {
      if (k0 + s * NW * 32 >= K) x[s][NE] = (i32x4)0;
      wave_sync();
#pragma unroll
      for (int j = 0; j <= NE; ++j)
        *reinterpret_cast<i32x4*>(own + j * 1024 + put) = x[s][j];
      wave_sync();
      const bf16x8 a = *reinterpret_cast<const bf16x8*>(own + NE * 1024 + get);
#pragma unroll
      for (int j = 0; j < NE; ++j)
        acc[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
            *reinterpret_cast<const bf16x8*>(own + j * 1024 + get), a, acc[j],
            0, 0, 0);
    }
  }
  __syncthreads();
  // rows of the sum: experts (g * 4 + r); columns: rows of h (i16)
  float* part = reinterpret_cast<float*>(smem);  // [NW][16][EP + 4]
#pragma unroll
  for (int j = 0; j < NE; ++j)
    *reinterpret_cast<f32x4*>(part + wid * WS + i16 * (EP + 4) + j * 16 +
                              g * 4) = acc[j];
  __syncthreads();
  float* gm = part + NW * WS + wid * 2 * groups;
  int* ok = reinterpret_cast<int*>(gm + groups);
  for (int i = wid; i < 16; i += NW) {
    const int row = m0 + i;
    if (row >= M) break;
    int* id = ids + (long)row * args.ids();
    float* w = weights + (long)row * args.cols();
    if (ctx[row] <= 0) {
      no_choice(args, id, w, lane);
      continue;
    }
    float* z = part + i * (EP + 4);
    for (int e = lane; e < E; e += 64) {
      float v = z[e];
#pragma unroll
      for (int p = 1; p < NW; ++p) v += z[e + p * WS];
      z[e] = v;
    }
    wave_sync();
    select_row<(EP + 63) / 64>(z, gm, ok, args, id, w, lane);
    wave_sync();
  }
}

extern "C" bool route_covers(int logits) { return logits <= 256; }

extern "C" void launch_select(const float* logits, const int* ctx, int M,
                              int E, int groups, int keep, int top,
                              const float* correction, float scale, bool gate,
                              int shards, int* ids, float* weights,
                              hipStream_t stream) {
  const RouteArgs a{E, groups, keep, top, correction, scale, gate, shards};
  hipLaunchKernelGGL(select_kernel, dim3((M + 3) / 4), dim3(256),
                     4 * (a.logits() + 2 * groups) * 4, stream, logits, ctx, M,
                     a, ids, weights);
}

extern "C" void launch_route(const void* h, const void* W, const int* ctx,
                             int M, int E, int K, int groups, int keep,
                             int top, const float* correction, float scale,
                             bool gate, int shards, int* ids, float* weights,
                             hipStream_t stream) {
  const RouteArgs a{E, groups, keep, top, correction, scale, gate, shards};
  const int n = a.logits();
#define RT(NE, NW)                                                           \
  hipLaunchKernelGGL((route_kernel<NE, NW>), dim3((M + 15) / 16),            \
                     dim3(NW * 64),                                          \
                     max(NW * (16 * (NE * 16 + 4) + 2 * groups) * 4,         \
                         NW * (NE + 1) * 1024),                              \
                     stream,                                                 \
                     (const unsigned short*)h, (const unsigned short*)W, ctx, \
                     M, K, a, ids, weights)
  if (n <= 16) RT(1, 16);
  else if (n <= 32) RT(2, 16);
  else if (n <= 48) RT(3, 16);
  else if (n <= 64) RT(4, 16);
  else if (n <= 80) RT(5, 16);
  else if (n <= 128) RT(8, 8);
  else if (n <= 144) RT(9, 8);
  else RT(16, 4);
#undef RT
}

// ---- plan ---------------------------------------------------------------------
// perm [A]: pair (row * top + choice) of each sorted place; tiles
// [max_tiles, 4]: expert, first place, places; ntiles. One workgroup.
__global__ void __launch_bounds__(1024)
expert_plan_kernel(const int* __restrict__ ids, int A, int E, int TM,
                   int max_tiles, int* __restrict__ perm,
                   int* __restrict__ tiles, int* __restrict__ ntiles) {
  constexpr int PU = 8;
  __shared__ int count[1024], first[1024], tile0[1024];
  const int tid = threadIdx.x;
  count[tid] = 0;
  __syncthreads();
  // several at a time: their round trips to memory and LDS overlap
  for (int a0 = tid; a0 < A; a0 += 1024 * PU) {
    int e[PU];
#pragma unroll
    for (int i = 0; i < PU; ++i)
      e[i] = a0 + i * 1024 < A ? ids[a0 + i * 1024] : -1;
#pragma unroll
    for (int i = 0; i < PU; ++i)
      if (e[i] >= 0 && e[i] < E) atomicAdd(&count[e[i]], 1);
  }
  __syncthreads();
  const int c = count[tid], nt = (c + TM - 1) / TM;
  first[tid] = c;
  tile0[tid] = nt;
  __syncthreads();
  for (int off = 1; off < 1024; off <<= 1) {  // inclusive sums
    const int x = tid >= off ? first[tid - off] : 0;
    const int y = tid >= off ? tile0[tid - off] : 0;
    __syncthreads();
    first[tid] += x;
    tile0[tid] += y;
    __syncthreads();
  }
  const int f = first[tid] - c, t0 = tile0[tid] - nt;
  if (tid == 1023) *ntiles = min(tile0[tid], max_tiles);
  for (int i = 0; i < nt; ++i)
    if (t0 + i < max_tiles) {
      int* t = tiles + (long)(t0 + i) * 4;
      t[0] = tid;
      t[1] = f + i * TM;
      t[2] = min(TM, c - i * TM);
    }
  __syncthreads();
  count[tid] = f;
  __syncthreads();
  for (int a0 = tid; a0 < A; a0 += 1024 * PU) {
    int e[PU], at[PU];
#pragma unroll
    for (int i = 0; i < PU; ++i)
      e[i] = a0 + i * 1024 < A ? ids[a0 + i * 1024] : -1;
#pragma unroll
    for (int i = 0; i < PU; ++i)
      at[i] = e[i] >= 0 && e[i] < E ? atomicAdd(&count[e[i]], 1) : -1;
#pragma unroll
    for (int i = 0; i < PU; ++i)
      if (at[i] >= 0) perm[at[i]] = a0 + i * 1024;
  }
}

// The same for many pairs, in blocks of PB pairs: counts of every block
// [blocks, E], then their sums and the tiles (one workgroup), then the places.
#define PB 2048

__global__ void __launch_bounds__(256)
expert_count_kernel(const int* __restrict__ ids, int A, int E,
                    int* __restrict__ counts) {
  __shared__ int count[1024];
  for (int e = threadIdx.x; e < E; e += 256) count[e] = 0;
  __syncthreads();
  const int a0 = blockIdx.x * PB;
#pragma unroll
  for (int i = 0; i < PB / 256; ++i) {
    const int a = a0 + i * 256 + threadIdx.x;
    const int e = a < A ? ids[a] : -1;
    if (e >= 0 && e < E) atomicAdd(&count[e], 1);
  }
  __syncthreads();
  for (int e = threadIdx.x; e < E; e += 256)
    counts[(long)blockIdx.x * E + e] = count[e];
}

// counts become the first place of every block's pairs of an expert
__global__ void __launch_bounds__(1024)
expert_offset_kernel(int* __restrict__ counts, int blocks, int E, int TM,
                     int max_tiles, int* __restrict__ tiles,
                     int* __restrict__ ntiles) {
  __shared__ int first[1024], tile0[1024], part[1024];
  const int tid = threadIdx.x;
  // S threads share an expert's blocks
  const int S = E <= 64 ? 16 : E <= 128 ? 8 : E <= 256 ? 4 : E <= 512 ? 2 : 1;
  const int e = tid / S, sub = tid % S;
  const int per = (blocks + S - 1) / S;
  const int b0 = sub * per, b1 = min(blocks, b0 + per);
  int c = 0;
  if (e < E) {
#pragma unroll 4
    for (int b = b0; b < b1; ++b) c += counts[(long)b * E + e];
  }
  part[tid] = c;
  __syncthreads();
  int before = 0, total = 0;  // of my expert: in blocks before mine, in all
  for (int i = 0; i < S; ++i) {
    const int x = part[tid / S * S + i];
    before += i < sub ? x : 0;
    total += x;
  }
  const bool lead = sub == 0 && e < E;
  const int nt = lead ? (total + TM - 1) / TM : 0;
  first[tid] = lead ? total : 0;
  tile0[tid] = nt;
  __syncthreads();
  for (int off = 1; off < 1024; off <<= 1) {  // inclusive sums
    const int x = tid >= off ? first[tid - off] : 0;
    const int y = tid >= off ? tile0[tid - off] : 0;
    __syncthreads();
    first[tid] += x;
    tile0[tid] += y;
    __syncthreads();
  }
  const int f = first[tid] - total, t0 = tile0[tid] - nt;
  if (tid == 1023) *ntiles = min(tile0[tid], max_tiles);
  for (int i = 0; i < nt; ++i)
    if (t0 + i < max_tiles) {
      int* t = tiles + (long)(t0 + i) * 4;
      t[0] = e;
      t[1] = f + i * TM;
      t[2] = min(TM, total - i * TM);
    }
  if (e < E) {  // first[] is the same for the threads of an expert
    int at = first[tid] - total + before;
    for (int b = b0; b < b1; ++b) {
      int* p = counts + (long)b * E + e;
      const int x = *p;
      *p = at;
      at += x;
    }
  }
}

__global__ void __launch_bounds__(256)
expert_place_kernel(const int* __restrict__ ids, int A, int E,
                    const int* __restrict__ counts, int* __restrict__ perm) {
  __shared__ int at[1024];
  for (int e = threadIdx.x; e < E; e += 256)
    at[e] = counts[(long)blockIdx.x * E + e];
  __syncthreads();
  const int a0 = blockIdx.x * PB;
#pragma unroll
  for (int i = 0; i < PB / 256; ++i) {
    const int a = a0 + i * 256 + threadIdx.x;
    const int e = a < A ? ids[a] : -1;
    if (e >= 0 && e < E) perm[atomicAdd(&at[e], 1)] = a;
  }
}

// ints of scratch that the plan of A pairs needs
extern "C" long expert_plan_scratch(long A, int E) {
  return A >= 16 * PB ? (A + PB - 1) / PB * E : 0;
}

extern "C" void launch_expert_plan(const int* ids, int A, int E, int TM,
                                   int max_tiles, int* perm, int* tiles,
                                   int* ntiles, int* scratch,
                                   hipStream_t stream) {
  if (expert_plan_scratch(A, E) > 0) {
    const int blocks = (A + PB - 1) / PB;
    hipLaunchKernelGGL(expert_count_kernel, dim3(blocks), dim3(256), 0,
                       stream, ids, A, E, scratch);
    hipLaunchKernelGGL(expert_offset_kernel, dim3(1), dim3(1024), 0, stream,
                       scratch, blocks, E, TM, max_tiles, tiles, ntiles);
    hipLaunchKernelGGL(expert_place_kernel, dim3(blocks), dim3(256), 0,
                       stream, ids, A, E, scratch, perm);
    return;
  }
  hipLaunchKernelGGL(expert_plan_kernel, dim3(1), dim3(1024), 0, stream, ids,
                     A, E, TM, max_tiles, perm, tiles, ntiles);
}

// ---- product, few rows per expert ----------------------------------------------
// Weight-streaming bound: a workgroup takes 64 weight rows and up to 16 MT
// places; its waves split K, 64 numbers at a time. Eight lanes load a row's 128
// bytes together (a wave that loaded the product's operands directly would
// ask for 16 rows at once, a line per lane, and be bound by that); the
// wave's own part of LDS brings them into operand order, the next step's are
// on their way in registers meanwhile.
// UNIT: 1, 2: rows are gathered (place -> perm / top), a gated unit halves
// the columns, or each is relu(.)^2; 0: rows are places and the output row is
// perm[place].
template <int MT, int UNIT>
__global__ void __launch_bounds__(256)
expert_rows_kernel(const unsigned short* __restrict__ x,
                   const unsigned short* __restrict__ W,
                   unsigned short* __restrict__ out,
                   const int* __restrict__ perm,
                   const int* __restrict__ tiles,
                   const int* __restrict__ ntiles, int N, int K, int top) {
  constexpr bool GLU = UNIT == 1, UP = UNIT != 0;
  constexpr int RROW = 68;  // padded row of 64 sums
  constexpr int NL = 8 + 2 * MT;  // loads of 8 rows: weights, places
  if ((int)blockIdx.y >= *ntiles) return;
  const int* tile = tiles + (long)blockIdx.y * 4;
  const int e = tile[0], s0 = tile[1], cnt = tile[2];
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  const int i16 = lane & 15, g = lane >> 4;
  const int n0 = blockIdx.x * 64;
  const int r8 = lane >> 3, c8 = (lane & 7) * 8;
  const unsigned short* wr = W + ((long)e * N + n0 + r8) * K + c8;
  const unsigned short* xr[2 * MT];
#pragma unroll
  for (int t = 0; t < 2 * MT; ++t) {
    const int s = s0 + min(t * 8 + r8, cnt - 1);
    xr[t] = x + (long)(UP ? perm[s] / top : s) * K + c8;
  }
  char* own = smem + wid * NL * 1024;
  const int put = r8 * 128 + (((lane & 7) ^ r8) * 16);
  f32x4 acc[MT][4];
#pragma unroll
  for (int t = 0; t < MT; ++t)
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[t][j] = {0.f, 0.f, 0.f, 0.f};
  i32x4 next[NL];
  auto load = [&](int k) {
#pragma unroll
    for (int q = 0; q < 8; ++q)
      next[q] = *reinterpret_cast<const i32x4*>(wr + (long)q * 8 * K + k);
#pragma unroll
    for (int t = 0; t < 2 * MT; ++t)
      next[8 + t] = *reinterpret_cast<const i32x4*>(xr[t] + k);
  };
  auto frag = [&](int row16, int kk) {
    return *reinterpret_cast<const bf16x8*>(
        own + (row16 * 16 + i16) * 128 +
        (((kk * 4 + g) ^ (i16 & 7)) * 16));
  };
  if (wid * 64 < K) load(wid * 64);
  for (int k = wid * 64; k < K; k += 256) {
    wave_sync();  // the step before is consumed
#pragma unroll
    for (int q = 0; q < NL; ++q)
      *reinterpret_cast<i32x4*>(own + q * 1024 + put) = next[q];
    load(min(k + 256, K - 64));
    wave_sync();
#pragma unroll
    for (int kk = 0; kk < 2; ++kk) {
      bf16x8 wf[4], xf[MT];
#pragma unroll
      for (int j = 0; j < 4; ++j) wf[j] = frag(j, kk);
#pragma unroll
      for (int t = 0; t < MT; ++t) xf[t] = frag(4 + t, kk);
#pragma unroll
      for (int t = 0; t < MT; ++t)
#pragma unroll
        for (int j = 0; j < 4; ++j)
          acc[t][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
              wf[j], xf[t], acc[t][j], 0, 0, 0);
    }
  }
  __syncthreads();
  // sums: rows are weight rows, columns places -> [wave][place][column]
  float* part = reinterpret_cast<float*>(smem);
#pragma unroll
  for (int t = 0; t < MT; ++t)
#pragma unroll
    for (int j = 0; j < 4; ++j)
      *reinterpret_cast<f32x4*>(
          part + ((wid * MT + t) * 16 + i16) * RROW + j * 16 + g * 4) =
          acc[t][j];
  __syncthreads();
  constexpr int WS = MT * 16 * RROW;  // per wave
  constexpr int OC = GLU ? 32 : 64;   // output columns
  for (int i = threadIdx.x; i < cnt * (OC / 4); i += 256) {
    const int m = i / (OC / 4), c = i % (OC / 4) * 4;
    const float* p = part + m * RROW + (GLU ? c / 16 * 32 + c % 16 : c);
    s16x4 o;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      float v = (p[r] + p[WS + r]) + (p[2 * WS + r] + p[3 * WS + r]);
      if (GLU) {
        const float* u = p + 16;
        v = silu(v) *
            ((u[r] + u[WS + r]) + (u[2 * WS + r] + u[3 * WS + r]));
      }
      if (UNIT == 2) v = relu2(v);
      o[r] = (short)f2bf(v);
    }
    const long row = UP ? s0 + m : perm[s0 + m];
    *reinterpret_cast<s16x4*>(out + row * (GLU ? N / 2 : N) +
                              blockIdx.x * OC + c) = o;
  }
}

// ---- product, many rows per expert ----------------------------------------------
// 128 x 128 x 64 tiles, four waves of 64 x 64, both operands through LDS in
// two buffers by global_load_lds with the bank swizzle on the source address
// (the structure of gemm.hip, with gathered and scattered rows).
#define ET_M 128
#define ET_N 128
#define ET_K 64
#define ET_TILE (128 * ET_K * 2)
#define ET_LDS (68 * 1024)

template <int UNIT>
__global__ void __launch_bounds__(256, 2)
expert_tile_kernel(const unsigned short* __restrict__ x,
                   const unsigned short* __restrict__ W,
                   unsigned short* __restrict__ out,
                   const int* __restrict__ perm,
                   const int* __restrict__ tiles,
                   const int* __restrict__ ntiles, int N, int K, int top) {
  constexpr bool GLU = UNIT == 1, UP = UNIT != 0;
  const int nt_all = *ntiles;
  const int ncol = (N + ET_N - 1) / ET_N;
  // contiguous runs of (tile, column block) per XCD, columns fastest: they
  // share the rows of x
  const int total = nt_all * ncol;
  const int per = (total + 7) / 8;
  const int xcd = blockIdx.x % 8, j8 = blockIdx.x / 8;
  const int bid = xcd * per + j8;
  if (j8 >= per || bid >= total) return;
  const int* tile = tiles + (long)(bid / ncol) * 4;
  const int e = tile[0], s0 = tile[1], cnt = tile[2];
  const int n0 = bid % ncol * ET_N;
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;

  // rows of this thread's four pieces of each operand
  const int r_in = lane >> 3, c_src = ((lane & 7) ^ r_in) * 8;
  const unsigned short *xs[4], *ws[4];
#pragma unroll
  for (int p = 0; p < 4; ++p) {
    const int r = wid * 32 + p * 8 + r_in;
    const int s = s0 + min(r, cnt - 1);
    xs[p] = x + (long)(UP ? perm[s] / top : s) * K + c_src;
    ws[p] = W + ((long)e * N + min(n0 + r, N - 1)) * K + c_src;
  }
  auto stage = [&](int k0, int buf) {
#pragma unroll
    for (int p = 0; p < 4; ++p) {
      char* dst = smem + buf * 2 * ET_TILE + (wid * 32 + p * 8) * 128 +
                  lane * 16;
      __builtin_amdgcn_global_load_lds(
          (const __attribute__((address_space(1))) unsigned int*)(xs[p] + k0),
          (__attribute__((address_space(3))) unsigned int*)dst, 16, 0, 0);
      __builtin_amdgcn_global_load_lds(
          (const __attribute__((address_space(1))) unsigned int*)(ws[p] + k0),
          (__attribute__((address_space(3))) unsigned int*)(dst + ET_TILE),
          16, 0, 0);
    }
  };
  auto frag = [&](int off, int row, int chunk) {
    return *reinterpret_cast<const bf16x8*>(
        smem + off + row * 128 + ((chunk ^ (row & 7)) * 16));
  };

  f32x4 acc[4][4];
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[i][j] = {0.f, 0.f, 0.f, 0.f};
  const int wrow = (wid >> 1) * 64, wcol = (wid & 1) * 64;

  stage(0, 0);
  asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
  __syncthreads();
  const int nk = K / ET_K;
  for (int t = 0; t < nk; ++t) {
    const int buf = t & 1;
    if (t + 1 < nk) stage((t + 1) * ET_K, buf ^ 1);
    const int offX = buf * 2 * ET_TILE, offW = offX + ET_TILE;
#pragma unroll
    for (int kk = 0; kk < 2; ++kk) {
      bf16x8 af[4], bf[4];
      const int chunk = kk * 4 + (lane >> 4);
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        af[i] = frag(offX, wrow + i * 16 + (lane & 15), chunk);
        bf[i] = frag(offW, wcol + i * 16 + (lane & 15), chunk);
      }
      __builtin_amdgcn_s_setprio(1);
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j)
          acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
              af[i], bf[j], acc[i][j], 0, 0, 0);
      __builtin_amdgcn_s_setprio(0);
    }
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();
  }

  // sums -> padded LDS (a wave's own 64 x 64) -> rows
  float* ep = reinterpret_cast<float*>(smem) + wid * 64 * 68;
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j)
#pragma unroll
      for (int r = 0; r < 4; ++r)
        ep[(i * 16 + (lane >> 4) * 4 + r) * 68 + j * 16 + (lane & 15)] =
            acc[i][j][r];
  __syncthreads();
  if (GLU) {
    const int F = N / 2;
    const int c8 = lane & 3, col = (n0 + wcol) / 2 + c8 * 8;
    for (int r = lane >> 2; r < 64; r += 16) {
      if (wrow + r >= cnt || col >= F) break;
      const float* p = ep + r * 68 + (c8 >> 1) * 32 + (c8 & 1) * 8;
      float o[8];
#pragma unroll
      for (int i = 0; i < 8; ++i) o[i] = silu(p[i]) * p[16 + i];
      store8(out + (long)(s0 + wrow + r) * F + col, o);
    }
  } else {
    const int c8 = lane & 7, col = n0 + wcol + c8 * 8;
    for (int r = lane >> 3; r < 64; r += 8) {
      if (wrow + r >= cnt || col >= N) break;
      float o[8];
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        o[i] = ep[r * 68 + c8 * 8 + i];
        if (UNIT == 2) o[i] = relu2(o[i]);
      }
      const long row = UP ? s0 + wrow + r : perm[s0 + wrow + r];
      store8(out + row * N + col, o);
    }
  }
}

// ---- product in 32-bit: 16 places x 64 columns, one sum in four per thread ---
template <int UNIT>
__global__ void __launch_bounds__(256)
expert_f32_kernel(const float* __restrict__ x, const float* __restrict__ W,
                  float* __restrict__ out, const int* __restrict__ perm,
                  const int* __restrict__ tiles,
                  const int* __restrict__ ntiles, int N, int K, int top) {
  constexpr bool GLU = UNIT == 1, UP = UNIT != 0;
  __shared__ float xl[16][33], wl[64][33], sum[16][65];
  if ((int)blockIdx.y >= *ntiles) return;
  const int* tile = tiles + (long)blockIdx.y * 4;
  const int e = tile[0], s0 = tile[1], cnt = tile[2];
  const int n0 = blockIdx.x * 64, tid = threadIdx.x;
  const int m = tid / 16, c = tid % 16;
  float acc[4] = {0.f, 0.f, 0.f, 0.f};
  for (int k0 = 0; k0 < K; k0 += 32) {
    __syncthreads();
    for (int i = tid; i < 16 * 32; i += 256) {
      const int s = s0 + min(i / 32, cnt - 1);
      xl[i / 32][i % 32] =
          x[(long)(UP ? perm[s] / top : s) * K + k0 + i % 32];
    }
    for (int i = tid; i < 64 * 32; i += 256)
      wl[i / 32][i % 32] = W[((long)e * N + n0 + i / 32) * K + k0 + i % 32];
    __syncthreads();
    for (int k = 0; k < 32; ++k)
#pragma unroll
      for (int j = 0; j < 4; ++j) acc[j] += xl[m][k] * wl[c + j * 16][k];
  }
#pragma unroll
  for (int j = 0; j < 4; ++j) sum[m][c + j * 16] = acc[j];
  __syncthreads();
  constexpr int OC = GLU ? 32 : 64;
  for (int i = tid; i < cnt * OC; i += 256) {
    const int r = i / OC, o = i % OC;
    float v = sum[r][GLU ? o / 16 * 32 + o % 16 : o];
    if (GLU) v = v * sigmoid_exact(v) * sum[r][o / 16 * 32 + o % 16 + 16];
    if (UNIT == 2) v = relu2(v);
    const long row = UP ? s0 + r : perm[s0 + r];
    out[row * (GLU ? N / 2 : N) + blockIdx.x * OC + o] = v;
  }
}

// TM: rows per tile of the plan (16, 32, 64, 128, or 256 for the tiles of
// expert_gemm16.hip)
extern "C" void launch_expert_gemm16(const void*, const void*, void*,
                                     const int*, const int*, const int*, int,
                                     int, int, int, int, hipStream_t);

// unit: 0 second product, 1 gated units, 2 squared ReLU
extern "C" void launch_expert_gemm(const void* x, const void* W, void* out,
                                   const int* perm, const int* tiles,
                                   const int* ntiles, int max_tiles, int N,
                                   int K, int top, int TM, int unit,
                                   bool fp32, hipStream_t stream) {
  typedef unsigned short u16;
  const dim3 grid(N / 64, max_tiles);
  if (fp32) {
#define EF(GL)                                                              \
  hipLaunchKernelGGL((expert_f32_kernel<GL>), grid, dim3(256), 0, stream,   \
                     (const float*)x, (const float*)W, (float*)out, perm,   \
                     tiles, ntiles, N, K, top)
    if (unit == 1) EF(1);
    else if (unit == 2) EF(2);
    else EF(0);
#undef EF
    return;
  }
  if (TM == 256) {
    launch_expert_gemm16(x, W, out, perm, tiles, ntiles, max_tiles, N, K, top,
                         unit, stream);
    return;
  }
#define ER(MT, GL)                                                          \
  hipLaunchKernelGGL((expert_rows_kernel<MT, GL>), grid, dim3(256),         \
                     max(4 * MT * 16 * 68 * 4, 4 * (8 + 2 * MT) * 1024),    \
                     stream, (const u16*)x,                                 \
                     (const u16*)W, (u16*)out, perm, tiles, ntiles, N, K, top)
#define ET(GL)                                                              \
  hipLaunchKernelGGL((expert_tile_kernel<GL>),                              \
                     dim3(((long)max_tiles * ((N + ET_N - 1) / ET_N) + 7) /  \
                          8 * 8),                                           \
                     dim3(256), ET_LDS, stream, (const u16*)x,              \
                     (const u16*)W, (u16*)out, perm, tiles, ntiles, N, K, top)
#define EX(GL)                   \
  do {                           \
    if (TM == 16) ER(1, GL);     \
    else if (TM == 32) ER(2, GL); \
    else if (TM == 64) ER(4, GL); \
    else ET(GL);                 \
  } while (0)
  if (unit == 1) EX(1);
  else if (unit == 2) EX(2);
  else EX(0);
#undef EX
#undef ET
#undef ER
}
