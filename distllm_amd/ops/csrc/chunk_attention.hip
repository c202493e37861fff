// What precedes attention over pages (see chunk_attention.h): norm and
// rotation of query and key heads, cache write.
#include "chunk_attention.h"

// Eight numbers x of a normed head from number c on, rotated with their
// partners y (normed, too). cs: cos, sin of the row's pairs.
__device__ __forceinline__ void rotate8(float* x, const float* y, int c,
                                        int half, const float* cs) {
  float t[16];
  const bool low = c < half;
  load8<float>(cs + (low ? c : c - half) * 2, t);
  load8<float>(cs + (low ? c : c - half) * 2 + 8, t + 8);
#pragma unroll
  for (int i = 0; i < 8; ++i)
    x[i] = x[i] * t[2 * i] + (low ? -y[i] : y[i]) * t[2 * i + 1];
}

// ---- norm of query and key heads, cache write -----------------------------
// ab row: H query heads of dp, then (own keys) G key heads of dp and G value
// heads of vp, from column v_at on. With a table, the first 2 * half numbers
// of a normed head are rotated. LPH lanes share a query or key head, a
// workgroup norms UN times 256 / LPH of them. Values: the first row of a run
// of consecutive positions in one page writes the run, whole 32-byte page
// rows where the run covers the page; a wave looks at VR rows of one head.
// ROT 1: half is a multiple of 8, so that partners are eight in a row, too;
// 2: any half.
template <typename T, int LPH, int UN, int ROT>
__global__ void __launch_bounds__(256)
attn_prep_kernel(const T* __restrict__ ab, int ld, int M, int H, int G,
                 int dp, int vp, int n, const float* __restrict__ wq,
                 const float* __restrict__ wk, float eps, T* __restrict__ q,
                 T* __restrict__ kpages, T* __restrict__ vpages,
                 const int* __restrict__ block_table, int max_blocks,
                 int num_blocks, const int* __restrict__ row_seq,
                 const int* __restrict__ ctx, int norm_wgs, int VR, int v_at,
                 const float* __restrict__ table, int half) {
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  // page of a position, or -1
  auto page_of = [&](int row, int pos) {
    if (pos < 0 || pos / PBLK >= max_blocks) return -1;
    const int b = block_table[(long)row_seq[row] * max_blocks + pos / PBLK];
    return b >= 0 && b < num_blocks ? b : -1;
  };
  if ((int)blockIdx.x < norm_wgs) {
    constexpr int UPI = 256 / LPH;
    const int units = H + (kpages != nullptr ? G : 0);
    const int total = M * units;  // the host checks that it fits
    const int c0 = threadIdx.x % LPH * 8;
    const int u0 = blockIdx.x * UPI * UN + threadIdx.x / LPH;
    // a unit's head starts at (row, hd); its lanes' first eight columns
    // stay in registers, heads of more than 512 read the others twice
    float v[UN][8], y[ROT == 1 ? UN : 1][8];
    // where the partners of eight columns start
    auto partner = [&](int c) {
      return c < half ? c + half : c < 2 * half ? c - half : c;
    };
#pragma unroll
    for (int k = 0; k < UN; ++k) {
      const int u = min(u0 + k * UPI, total - 1);
#pragma unroll
      for (int i = 0; i < 8; ++i) v[k][i] = 0.f;
      if (c0 < dp) {
        const T* src =
            ab + (long)(u / units) * ld + (long)(u % units) * dp;
        load8<T>(src + c0, v[k]);
        if (ROT == 1) load8<T>(src + partner(c0), y[k]);
      }
    }
#pragma unroll
    for (int k = 0; k < UN; ++k) {
      const int u = u0 + k * UPI;
      if (u >= total) return;  // whole LPH groups
      const int row = u / units, hd = u % units;
      const T* src = ab + (long)row * ld + (long)hd * dp;
      const float* w = hd >= H ? wk : wq;
      float ss = 0.f;
#pragma unroll
      for (int i = 0; i < 8; ++i) ss += v[k][i] * v[k][i];
      for (int c = c0 + LPH * 8; c < dp; c += LPH * 8) {
        float x[8];
        load8<T>(src + c, x);
#pragma unroll
        for (int i = 0; i < 8; ++i) ss += x[i] * x[i];
      }
#pragma unroll
      for (int off = LPH / 2; off > 0; off >>= 1)
        ss += __shfl_xor(ss, off, 64);
      const float inv = 1.f / sqrtf(ss / n + eps);
      T* dst = q + ((long)row * H + hd) * dp;
      if (hd >= H) {
        const int pos = ctx[row] - 1, page = page_of(row, pos);
        if (page < 0) continue;
        dst = kpages +
              (((long)page * G + hd - H) * PBLK + pos % PBLK) * dp;
      }
      for (int c = c0; c < dp; c += LPH * 8) {
        float x[8], wv[8];
        if (c != c0) load8<T>(src + c, v[k]);
        load8<float>(w + c, wv);
#pragma unroll
        for (int i = 0; i < 8; ++i) x[i] = v[k][i] * inv * wv[i];
        const float* cs = table + (long)row * 2 * half;
        if (ROT == 1 && c < 2 * half) {
          if (c != c0) load8<T>(src + partner(c), y[k]);
          load8<float>(w + partner(c), wv);
#pragma unroll
          for (int i = 0; i < 8; ++i) y[k][i] *= inv * wv[i];
          rotate8(x, y[k], c, half, cs);
        }
        if (ROT == 2) {
#pragma unroll
          for (int i = 0; i < 8; ++i) {
            const int o = partner(c + i);
            const bool low = c + i < half, in = c + i < 2 * half;
            const int pair = in ? min(o, c + i) : 0;
            const float z = to_f(src[o]) * inv * w[o];
            const float r = x[i] * cs[pair * 2] +
                            (low ? -z : z) * cs[pair * 2 + 1];
            x[i] = in ? r : x[i];
          }
        }
        store8(dst + c, x);
      }
    }
    return;
  }
  const long u = ((long)blockIdx.x - norm_wgs) * 4 + wid;
  const int r0 = (int)(u / G) * VR, g = (int)(u % G);
  if (r0 >= M) return;
  bool first = false;
  if (lane < VR && r0 + lane < M) {
    const int row = r0 + lane, pos = ctx[row] - 1;
    first = pos >= 0 && (pos % PBLK == 0 || row == 0 ||
                         row_seq[row - 1] != row_seq[row] ||
                         ctx[row - 1] != pos);
  }
  for (unsigned long long todo = __ballot(first); todo != 0;
       todo &= todo - 1) {
    const int row = r0 + __builtin_ctzll(todo);
    const int pos = ctx[row] - 1, seq = row_seq[row];
    const int page = page_of(row, pos);
    if (page < 0) continue;
    int run = 1;
    while (pos % PBLK + run < PBLK && row + run < M &&
           row_seq[row + run] == seq && ctx[row + run] == ctx[row] + run)
      ++run;
    const T* src = ab + (long)row * ld + v_at + (long)g * vp;
    T* dst = vpages + ((long)page * G + g) * vp * PBLK;
    for (int c = lane * 2; c < vp; c += 128) {
      typedef __attribute__((ext_vector_type(2))) T pair;
      if (run == PBLK) {
        pair v[PBLK];
#pragma unroll
        for (int j = 0; j < PBLK; ++j)
          v[j] = *reinterpret_cast<const pair*>(src + (long)j * ld + c);
#pragma unroll
        for (int h = 0; h < 2; ++h) {
          T t[PBLK];
#pragma unroll
          for (int j = 0; j < PBLK; ++j) t[j] = v[j][h];
          T* d = dst + (long)(c + h) * PBLK;
#pragma unroll
          for (int j = 0; j < PBLK * (int)sizeof(T) / 16; ++j)
            reinterpret_cast<i32x4*>(d)[j] =
                reinterpret_cast<const i32x4*>(t)[j];
        }
      } else {
        for (int j = 0; j < run; ++j) {
          const pair v =
              *reinterpret_cast<const pair*>(src + (long)j * ld + c);
          T* d = dst + (long)c * PBLK + pos % PBLK + j;
          d[0] = v[0];
          d[PBLK] = v[1];
        }
      }
    }
  }
}

// table [M, half, 2] or null
extern "C" void launch_attn_prep(
    const void* ab, int ld, int M, int H, int G, int dp, int vp, int n,
    const float* wq, const float* wk, float eps, void* q, void* kpages,
    void* vpages, const int* block_table, int max_blocks, int num_blocks,
    const int* row_seq, const int* ctx, int v_at, const float* table,
    int half, bool fp32, hipStream_t stream) {
  const int lph = dp <= 64 ? 8 : dp <= 128 ? 16 : dp <= 256 ? 32 : 64;
  const bool own = kpages != nullptr;
  const long units = (long)M * (H + (own ? G : 0));
  const int un = units >= 65536 ? 4 : 1, vr = M >= 2048 ? 16 : 1;
  const int per = 256 / lph * un;
  const int norm_wgs = (int)((units + per - 1) / per);
  const int v_wgs = own ? (int)(((long)(M + vr - 1) / vr * G + 3) / 4) : 0;
#define APK_R(T, L, U, R)                                                     \
  hipLaunchKernelGGL((attn_prep_kernel<T, L, U, R>), dim3(norm_wgs + v_wgs),  \
                     dim3(256), 0, stream, (const T*)ab, ld, M, H, G, dp, vp, \
                     n, wq, wk, eps, (T*)q, (T*)kpages, (T*)vpages,           \
                     block_table, max_blocks, num_blocks, row_seq, ctx,       \
                     norm_wgs, vr, v_at, table, half)
#define APK(T, L, U)                          \
  do {                                        \
    if (table == nullptr) APK_R(T, L, U, 0);  \
    else if (half % 8 == 0) APK_R(T, L, U, 1); \
    else APK_R(T, L, U, 2);                   \
  } while (0)
#define APK_U(T, L)           \
  do {                        \
    if (un == 1) APK(T, L, 1); \
    else APK(T, L, 4);        \
  } while (0)
#define APK_L(T)                 \
  do {                           \
    if (lph == 8) APK_U(T, 8);   \
    else if (lph == 16) APK_U(T, 16); \
    else if (lph == 32) APK_U(T, 32); \
    else APK_U(T, 64);           \
  } while (0)
  if (fp32) APK_L(float);
  else APK_L(unsigned short);
#undef APK_L
#undef APK_U
#undef APK
#undef APK_R
}
