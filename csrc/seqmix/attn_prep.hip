// Input passes of grouped-query attention behind short convolutions, and the pooled blocks of
// its key/value pool.
//
// conv_rope_norm_store_k: one projection buffer holds q (H heads x D) | k (G x D) | v (GV x V) of
// every row (differential attention has two q / k heads, its maps, per value head; a layer that
// reads another layer's keys and values has queries only, G = GV = 0).  Each channel goes through a
// causal convolution over the sequence's last K projected values (those before the portion come from the slot's saved tail, or are zero before
// position 0); nrot channel pairs (i, i + nrot) of every q / k head are turned by the angle
// pos * inv_freq[i] (cos and sin times rm); q and k heads are divided by their root mean square,
// sqrt(mean x^2 + eps) (`norm`);
// q also takes a factor per head (`temp`), which stands for a factor on that head's scores.  q
// goes to its own buffer, k | v to the row of the paged pool that the token owns.  Convolution,
// angles, rotation and norm are fp32.  One wavefront per (row, head).
//
// Pooled blocks: block b of a sequence is the P tokens bP .. bP + P - 1; its key and value are the
// means of theirs as the pool holds them.  A second pool keeps them in the activation type: the
// page that holds a block's last token t has ceil(page / P) rows in it, row (t % page) / P is the
// block's.  A block is formed in the step that brings its last token, from the first pool:
// pool_blocks_k, after every row of the step is stored.  A portion of one token (decode) needs
// no second pass: its wavefronts read back the block's other tokens, which earlier steps
// stored, and add their own; they move the convolution's tail forward as well.
#include "common.h"
using namespace sm;

template <typename T>
__global__ void __launch_bounds__(256)
conv_rope_norm_store_k(const T* __restrict__ proj, int ldp, int H, int G, int GV, int D, int V,
                       int norm, float rm,
                       const float* __restrict__ cw, int K, float* tail,
                       const int* __restrict__ ent, const int* __restrict__ row_ent,
                       const float* __restrict__ inv_freq, int nrot, const float* __restrict__ temp,
                       float eps, const int* __restrict__ pos, const int* __restrict__ cache_rows,
                       T* pool, T* __restrict__ q_out, int ldq, T* __restrict__ blk, int P,
                       const int* __restrict__ bt, int max_pages, int page, int LDS) {
  extern __shared__ float smem[];
  const int r = blockIdx.x, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int hh = blockIdx.y * 4 + wave;                 // q heads, then k heads, then v heads
  const bool on = hh < H + G + GV;
  const int kind = hh < H ? 0 : hh < H + G ? 1 : 2;
  const int hd = kind == 0 ? hh : kind == 1 ? hh - H : hh - H - G;
  const int n = kind == 2 ? V : D;
  const int c0 = kind == 0 ? hd * D : kind == 1 ? (H + hd) * D : (H + G) * D + hd * V;
  const int C = (H + G) * D + GV * V, W = G * D + GV * V;
  float* s = smem + wave * LDS;
  const int e = row_ent[r];
  const Entry en = load_entry(ent, e);
  const int t = r - en.row0;
  const bool single = en.n == 1;
  if (on)
    for (int i = lane; i < n; i += 64) {
      const int c = c0 + i;
      const float* w = cw + (size_t)c * K;
      float* tl = tail + (size_t)en.slot * (K - 1) * C + c;
      float acc = 0.0f;
      for (int kk = 0; kk < K; kk++) {
        const int q = t - (K - 1) + kk;
        float v = 0.0f;
        if (q >= 0) v = ldf(proj, (size_t)(en.row0 + q) * ldp + c);
        else if (en.start > 0) v = tl[(size_t)(K - 1 + q) * C];
        acc += w[kk] * v;
        // the tail after this token is its window without the oldest value (a slot is written
        // after the value it held has been used)
        if (single && kk > 0) tl[(size_t)(kk - 1) * C] = v;
      }
      s[i] = acc;
    }
  __syncthreads();
  if (!on) return;
  const int p = pos[r];
  T* crow = pool + (size_t)cache_rows[r] * W;
  T* dst = kind == 0 ? q_out + (size_t)r * ldq + hd * D : kind == 1 ? crow + hd * D
                                                                    : crow + G * D + hd * V;
  float rs = 1.0f;
  if (kind < 2) {
    float ss = 0.0f;
    for (int j = lane; j < nrot; j += 64) {   // a pair stays with one lane
      const float a = s[j], b = s[j + nrot];
      float sn, cs;
      sincosf((float)p * inv_freq[j], &sn, &cs);
      sn *= rm;
      cs *= rm;
      const float x = a * cs - b * sn, y = b * cs + a * sn;
      s[j] = x;
      s[j + nrot] = y;
      ss += x * x + y * y;
    }
    if (norm) {
      for (int i = 2 * nrot + lane; i < n; i += 64) ss += s[i] * s[i];
      ss = wave_sum(ss);
      rs = 1.0f / sqrtf(ss / (float)n + eps);
    }
    if (kind == 0 && temp) rs *= temp[hd];
  }
  // another lane may have turned the value this lane stores
  __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
  const bool ends = blk && single && kind > 0 && (p + 1) % P == 0;
  const int wo = kind == 1 ? hd * D : G * D + hd * V;      // place in a pool row
  const int* pages = bt + (size_t)e * max_pages;
  T* brow = ends ? blk + ((size_t)pages[p / page] * ((page + P - 1) / P) + (p % page) / P) * W + wo
                 : nullptr;
  for (int i = lane; i < n; i += 64) {
    T own;
    stf(&own, 0, s[i] * rs);
    dst[i] = own;
    if (ends) {
      float sum = 0.0f;
      for (int j = p - P + 1; j < p; j++)
        sum += ldf(pool, ((size_t)pages[j / page] * page + j % page) * W + wo + i);
      stf(brow, i, (sum + ldf(&own, 0)) / (float)P);
    }
  }
}

// The same for prompts, RT consecutive rows of four heads per workgroup: the angles of the rows are
// formed once for its heads (sincos in LDS), every wavefront walks the rows of one head with the
// taps and the window of its channels in registers.  Head sizes up to 256, KT taps.  It
// neither moves tails nor forms blocks.
#define RT 8
template <typename T, int KT>
__global__ void __launch_bounds__(256)
conv_rope_norm_rows_k(const T* __restrict__ proj, int ldp, int H, int G, int GV, int D, int V,
                      int norm, float rm,
                      const float* __restrict__ cw, const float* __restrict__ tail,
                      const int* __restrict__ ent, const int* __restrict__ row_ent,
                      const float* __restrict__ inv_freq, int nrot, const float* __restrict__ temp,
                      float eps, const int* __restrict__ pos, const int* __restrict__ cache_rows,
                      T* __restrict__ pool, T* __restrict__ q_out, int ldq, int R, int LDS) {
  constexpr int NM = 4;               // channels of a lane at most
  extern __shared__ float smem[];     // [RT][nrot][2] cos | sin, then a head per wavefront
  const int r0 = blockIdx.x * RT, nr = min(RT, R - r0);
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  float* s = smem + RT * nrot * 2 + wave * LDS;
  for (int idx = threadIdx.x; idx < nr * nrot; idx += 256) {
    float sn, cs;
    sincosf((float)pos[r0 + idx / nrot] * inv_freq[idx % nrot], &sn, &cs);
    smem[2 * idx] = cs * rm;
    smem[2 * idx + 1] = sn * rm;
  }
  __syncthreads();
  const int C = (H + G) * D + GV * V, W = G * D + GV * V;
  const int hh = blockIdx.y * 4 + wave;
  if (hh < H + G + GV) {
    const int kind = hh < H ? 0 : hh < H + G ? 1 : 2;
    const int hd = kind == 0 ? hh : kind == 1 ? hh - H : hh - H - G;
    const int n = kind == 2 ? V : D;
    const int c0 = kind == 0 ? hd * D : kind == 1 ? (H + hd) * D : (H + G) * D + hd * V;
    const float tq = kind == 0 && temp ? temp[hd] : 1.0f;
    float w[NM][KT], u[NM][KT - 1];
#pragma unroll
    for (int m = 0; m < NM; m++) {
      const int c = c0 + min(lane + 64 * m, n - 1);
      if (64 * m < n) {
#pragma unroll
        for (int kk = 0; kk < KT; kk++) w[m][kk] = cw[(size_t)c * KT + kk];
#pragma unroll
        for (int kk = 0; kk < KT - 1; kk++)
          u[m][kk] = ldf(proj, (size_t)max(r0 - (KT - 1) + kk, 0) * ldp + c);
      }
    }
    float nx[NM];
#pragma unroll
    for (int m = 0; m < NM; m++)
      nx[m] = 64 * m < n ? ldf(proj, (size_t)r0 * ldp + c0 + min(lane + 64 * m, n - 1)) : 0.0f;
    for (int i = 0; i < nr; i++) {
      const int r = r0 + i;
      const Entry en = load_entry(ent, row_ent[r]);
      const int t = r - en.row0;
      float cur[NM];
#pragma unroll
      for (int m = 0; m < NM; m++) cur[m] = nx[m];
      if (i + 1 < nr) {
#pragma unroll
        for (int m = 0; m < NM; m++)
          if (64 * m < n) nx[m] = ldf(proj, (size_t)(r + 1) * ldp + c0 + min(lane + 64 * m, n - 1));
      }
#pragma unroll
      for (int m = 0; m < NM; m++) {
        if (64 * m >= n) break;
        const int ch = lane + 64 * m, c = c0 + min(ch, n - 1);
        float acc = 0.0f;
#pragma unroll
        for (int kk = 0; kk < KT - 1; kk++) {
          const int q = t - (KT - 1) + kk;
          float v = u[m][kk];
          if (q < 0) v = en.start > 0 ? tail[((size_t)en.slot * (KT - 1) + (KT - 1 + q)) * C + c] : 0.0f;
          acc += w[m][kk] * v;
        }
        acc += w[m][KT - 1] * cur[m];
#pragma unroll
        for (int kk = 0; kk + 1 < KT - 1; kk++) u[m][kk] = u[m][kk + 1];
        u[m][KT - 2] = cur[m];
        if (ch < n) s[ch] = acc;
      }
      __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
      T* crow = pool + (size_t)cache_rows[r] * W;
      T* dst = kind == 0 ? q_out + (size_t)r * ldq + hd * D : kind == 1 ? crow + hd * D
                                                                        : crow + G * D + hd * V;
      float rs = 1.0f;
      if (kind < 2) {
        float ss = 0.0f;
        for (int j = lane; j < nrot; j += 64) {
          const float a = s[j], b = s[j + nrot];
          const float cs = smem[2 * (i * nrot + j)], sn = smem[2 * (i * nrot + j) + 1];
          const float x = a * cs - b * sn, y = b * cs + a * sn;
          s[j] = x;
          s[j + nrot] = y;
          ss += x * x + y * y;
        }
        rs = tq;
        if (norm) {
          for (int k = 2 * nrot + lane; k < n; k += 64) ss += s[k] * s[k];
          ss = wave_sum(ss);
          rs = 1.0f / sqrtf(ss / (float)n + eps) * tq;
        }
      }
      __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
      for (int k = lane; k < n; k += 64) stf(dst, k, s[k] * rs);
      __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");   // before the next row overwrites s
    }
  }
}

// blocks that the step's portions of at least min_n tokens complete; one workgroup per (block,
// entry), grid.x covers the entry with most of them
template <typename T>
__global__ void __launch_bounds__(256)
pool_blocks_k(const T* __restrict__ pool, int W, T* __restrict__ blk, int P,
              const int* __restrict__ ent, const int* __restrict__ bt, int max_pages, int page,
              int min_n) {
  const int e = blockIdx.y;
  const Entry en = load_entry(ent, e);
  const int last = (en.start / P + blockIdx.x) * P + P - 1;
  if (en.n < min_n || last >= en.start + en.n) return;
  const int* pages = bt + (size_t)e * max_pages;
  T* brow = blk + ((size_t)pages[last / page] * ((page + P - 1) / P) + (last % page) / P) * W;
  for (int c = threadIdx.x; c < W; c += blockDim.x) {
    float sum = 0.0f;
    int j = last - P + 1;
    for (; j + 4 <= last + 1; j += 4) {   // four loads in flight, added in order
      float v[4];
#pragma unroll
      for (int u = 0; u < 4; u++)
        v[u] = ldf(pool, ((size_t)pages[(j + u) / page] * page + (j + u) % page) * W + c);
#pragma unroll
      for (int u = 0; u < 4; u++) sum += v[u];
    }
    for (; j <= last; j++) sum += ldf(pool, ((size_t)pages[j / page] * page + j % page) * W + c);
    stf(brow, c, sum / (float)P);
  }
}

extern "C" {

// rows: several rows per workgroup (3 or 4 taps, head sizes up to 256); the tails and blocks of
// every portion, also of single tokens, are then left to other kernels
int p2p_sm_conv_rope_norm_store(const void* proj, int ldp, int H, int G, int GV, int D, int V,
                                int norm, float rm, const float* cw, int K, float* tail, const int* ent,
                                const int* row_ent, const float* inv_freq, int nrot,
                                const float* temp, float eps, const int* pos,
                                const int* cache_rows, void* pool, void* q_out, int ldq, void* blk,
                                int P, const int* bt, int max_pages, int page, int R, int rows,
                                int f32, hipStream_t st) {
  if (R <= 0) return 0;
  if (H < 1 || G < 0 || GV < 0 || (G + GV > 0 && !pool) || D < 1 || V < 1 || K < 1 || nrot < 0 ||
      2 * nrot > D || page < 1 || (blk && P < 1))
    return (int)hipErrorInvalidValue;
  const int LDS = D > V ? D : V;
  if ((size_t)4 * LDS * 4 > 64 * 1024) return (int)hipErrorInvalidValue;
  const size_t shm = ((size_t)RT * nrot * 2 + 4 * LDS) * 4;
  if (rows) {
    if ((K != 4 && K != 3) || LDS > 256 || shm > 64 * 1024) return (int)hipErrorInvalidValue;
    dim3 gr((R + RT - 1) / RT, (H + G + GV + 3) / 4);
#define CRN(KT)                                                                                   \
  SM_DISPATCH_T(f32, hipLaunchKernelGGL((conv_rope_norm_rows_k<T, KT>), gr, dim3(256), shm, st,   \
                                         (const T*)proj, ldp, H, G, GV, D, V, norm, rm, cw, tail, ent, \
                                         row_ent,                                                 \
                                         inv_freq, nrot, temp, eps, pos, cache_rows, (T*)pool,    \
                                         (T*)q_out, ldq, R, LDS))
    if (K == 4) CRN(4);
    else CRN(3);
#undef CRN
    return (int)hipGetLastError();
  }
  dim3 grid(R, (H + G + GV + 3) / 4);
  SM_DISPATCH_T(f32, hipLaunchKernelGGL(conv_rope_norm_store_k<T>, grid, dim3(256),
                                         (size_t)4 * LDS * 4, st, (const T*)proj, ldp, H, G, GV, D, V, norm, rm,
                                         cw, K, tail, ent, row_ent, inv_freq, nrot, temp, eps, pos,
                                         cache_rows, (T*)pool, (T*)q_out, ldq, (T*)blk, P, bt,
                                         max_pages, page, LDS));
  return (int)hipGetLastError();
}

// max_blocks: the most blocks a portion of the step completes
int p2p_sm_pool_blocks(const void* pool, int W, void* blk, int P, const int* ent, int E,
                       int max_blocks, const int* bt, int max_pages, int page, int min_n, int f32,
                       hipStream_t st) {
  if (E <= 0 || max_blocks <= 0) return 0;
  if (P < 1 || W < 1 || page < 1) return (int)hipErrorInvalidValue;
  dim3 grid(max_blocks, E);
  SM_DISPATCH_T(f32, hipLaunchKernelGGL(pool_blocks_k<T>, grid, dim3(256), 0, st, (const T*)pool,
                                         W, (T*)blk, P, ent, bt, max_pages, page, min_n));
  return (int)hipGetLastError();
}

}  // extern "C"
