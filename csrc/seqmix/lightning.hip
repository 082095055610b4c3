// Lightning attention over long portions: per head S_t = lam S_(t-1) + k_t v_t^T, o_t = S_t^T q_t
// with a constant decay lam, in chunks of up to 64 tokens on the fp32 matrix instructions
// (v_mfma_f32_16x16x4_f32: products and sums in fp32).  q, k, v = silu of the projections, applied
// while they are staged in LDS.  With t, s counted inside a chunk of n tokens and S the state
// before it,
//   local pass   L = sum_t lam^(n-1-t) k_t v_t^T                                   [D x V]
//   chain        S_next = lam^n S + L over each portion's chunks, from the slot's state (or zero
//                at position 0); the last one is the slot's new state
//   output pass  o_t = lam^(t+1) S^T q_t + sum_{s <= t} lam^(t-s) (q_t . k_s) v_s
// `pw` [H, 65] holds the powers lam^0 .. lam^64 of every head, so no power is formed here.
// One workgroup of four wavefronts per (chunk, head).  Sizes are padded to multiples of 16 with
// zeros in LDS; rows are laid out so that the lanes of a fragment read hit different banks.
#include "common.h"
using namespace sm;

typedef float f32x4 __attribute__((ext_vector_type(4)));

#define LC 64   // tokens of a chunk

__device__ __forceinline__ float lsilu(float x) {
  return x * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-1.4426950408889634f * x));
}

// row lengths in LDS: fragments that take 16 rows x 4 neighbours want ld = 4 mod 64, fragments
// that take 4 rows x 16 neighbours ld = 16 mod 64
static __host__ __device__ __forceinline__ int ld_rows(int n) { return n + ((4 - n) & 63); }
static __host__ __device__ __forceinline__ int ld_cols(int n) { return n + ((16 - n) & 63); }

// n rows of `width` numbers of src (row stride ld) -> dst [LC][ldd] through silu, times scale(t);
// zeros up to `pad` columns and in rows n .. LC-1
template <typename T, typename F>
__device__ __forceinline__ void stage(const T* __restrict__ src, size_t ld, int n, int width, int pad,
                                      float* dst, int ldd, bool vec, F scale) {
  if (vec) {   // four numbers per load
    const int w4 = pad / 4;
    for (int idx = threadIdx.x; idx < LC * w4; idx += 256) {
      const int t = idx / w4, c = (idx % w4) * 4;
      float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
      if (t < n && c < width) {
        const T* p = src + (size_t)t * ld + c;
        if constexpr (sizeof(T) == 2) {
          const uint2 u = *(const uint2*)p;
          v.x = __uint_as_float(u.x << 16); v.y = __uint_as_float(u.x & 0xffff0000u);
          v.z = __uint_as_float(u.y << 16); v.w = __uint_as_float(u.y & 0xffff0000u);
        } else {
          v = *(const float4*)p;
        }
        const float m = scale(t);
        v.x = lsilu(v.x) * m; v.y = lsilu(v.y) * m; v.z = lsilu(v.z) * m; v.w = lsilu(v.w) * m;
      }
      *(float4*)(dst + t * ldd + c) = v;
    }
    return;
  }
  for (int idx = threadIdx.x; idx < LC * pad; idx += 256) {
    const int t = idx / pad, c = idx % pad;
    dst[t * ldd + c] = (t < n && c < width) ? lsilu(ldf(src, (size_t)t * ld + c)) * scale(t) : 0.0f;
  }
}

template <typename T, int NVT>   // value size padded to NVT * 16
__global__ void __launch_bounds__(256)
lightning_local_k(const T* __restrict__ proj, int ldp, const float* __restrict__ pw,
                  const int* __restrict__ vent, float* __restrict__ cs, int H, int D, int V,
                  int vec) {
  extern __shared__ __align__(16) float smem[];
  const int c = blockIdx.x, h = blockIdx.y;
  const Entry en = load_entry(vent, c);
  const int DP = (D + 15) & ~15, VP = NVT * 16, LDK = ld_cols(DP), LDV = ld_cols(VP);
  float* sK = smem;
  float* sV = smem + LC * LDK;
  const T* row = proj + (size_t)en.row0 * ldp;
  const float* p = pw + (size_t)h * (LC + 1);
  const int n = en.n;
  stage(row + (size_t)H * D + h * D, (size_t)ldp, n, D, DP, sK, LDK, vec, [&](int t) { return p[n - 1 - t]; });
  stage(row + (size_t)2 * H * D + h * V, (size_t)ldp, n, V, VP, sV, LDV, vec, [](int) { return 1.0f; });
  __syncthreads();
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, i16 = lane & 15, k4 = lane >> 4;
  const int steps = (n + 3) / 4;
  float* out = cs + ((size_t)c * H + h) * D * V;
  for (int dt = wave; dt * 16 < DP; dt += 4) {
    f32x4 acc[NVT];
#pragma unroll
    for (int j = 0; j < NVT; j++) acc[j] = f32x4{0.f, 0.f, 0.f, 0.f};
    for (int s = 0; s < steps; s++) {
      const float a = sK[(4 * s + k4) * LDK + dt * 16 + i16];
#pragma unroll
      for (int j = 0; j < NVT; j++)
        acc[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(a, sV[(4 * s + k4) * LDV + j * 16 + i16], acc[j], 0, 0, 0);
    }
#pragma unroll
    for (int j = 0; j < NVT; j++)
#pragma unroll
      for (int r = 0; r < 4; r++) {
        const int d = dt * 16 + k4 * 4 + r, v = j * 16 + i16;
        if (d < D && v < V) out[(size_t)d * V + v] = acc[j][r];
      }
  }
}

// init_c replaces the local state of chunk c; cent: per portion (first chunk, chunks, first
// position, slot)
__global__ void __launch_bounds__(256)
lightning_chain_k(float* __restrict__ cs, const float* __restrict__ pw, const int* __restrict__ vent,
                  float* __restrict__ state, const int* __restrict__ cent, int H, int DV) {
  const int idx = blockIdx.x * 256 + threadIdx.x, h = blockIdx.y, e = blockIdx.z;
  if (idx >= DV) return;
  const int c0 = cent[4 * e], nc = cent[4 * e + 1], start = cent[4 * e + 2], slot = cent[4 * e + 3];
  const float* p = pw + (size_t)h * (LC + 1);
  float* sg = state + ((size_t)slot * H + h) * DV + idx;
  const size_t step = (size_t)H * DV;
  float* q = cs + (size_t)c0 * step + (size_t)h * DV + idx;
  float cur = start > 0 ? *sg : 0.0f;
  for (int k = 0; k < nc; k += 8) {
    float loc[8], dec[8];   // eight chunks' loads in flight
#pragma unroll
    for (int u = 0; u < 8; u++) {
      const int kk = min(k + u, nc - 1);
      loc[u] = q[(size_t)kk * step];
      dec[u] = p[vent[4 * (c0 + kk) + 1]];
    }
#pragma unroll
    for (int u = 0; u < 8; u++)
      if (k + u < nc) {
        q[(size_t)(k + u) * step] = cur;
        cur = fmaf(dec[u], cur, loc[u]);
      }
  }
  *sg = cur;
}

template <typename T, int NVT>
__global__ void __launch_bounds__(256)
lightning_out_k(const T* __restrict__ proj, int ldp, const float* __restrict__ pw,
                const int* __restrict__ vent, const float* __restrict__ cs, float* __restrict__ out,
                int ldo, int H, int D, int V, int vec) {
  extern __shared__ __align__(16) float smem[];
  const int c = blockIdx.x, h = blockIdx.y;
  const Entry en = load_entry(vent, c);
  const int n = en.n;
  const int DP = (D + 15) & ~15, VP = NVT * 16, LDQ = ld_rows(DP), LDV = ld_cols(VP), LDP = LC + 4;
  float* sQ = smem;                                          // later the weights of the second product
  float* sK = smem + LC * max(LDQ, LDP);                     // later the values
  float* sV = sK;
  float* sP = smem;                                          // [LC][LDP]
  const T* row = proj + (size_t)en.row0 * ldp;
  const float* p = pw + (size_t)h * (LC + 1);
  auto one = [](int) { return 1.0f; };
  stage(row + (size_t)h * D, (size_t)ldp, n, D, DP, sQ, LDQ, vec, one);
  stage(row + (size_t)H * D + h * D, (size_t)ldp, n, D, DP, sK, LDQ, vec, one);
  __syncthreads();
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, i16 = lane & 15, k4 = lane >> 4;
  const int r0 = wave * 16;                                  // this wavefront's 16 tokens
  // weights lam^(t-s) q_t . k_s, s <= t
  f32x4 w[LC / 16];
#pragma unroll
  for (int j = 0; j < LC / 16; j++) w[j] = f32x4{0.f, 0.f, 0.f, 0.f};
  // from the state before the chunk: S^T q, lam^(t+1) comes after the sum
  f32x4 acc[NVT];
#pragma unroll
  for (int j = 0; j < NVT; j++) acc[j] = f32x4{0.f, 0.f, 0.f, 0.f};
  if (r0 < n) {
    for (int s = 0; s < DP / 4; s++) {
      const float a = sQ[(r0 + i16) * LDQ + 4 * s + k4];
#pragma unroll
      for (int j = 0; j < LC / 16; j++)
        if (j <= wave)
          w[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(a, sK[(j * 16 + i16) * LDQ + 4 * s + k4], w[j], 0, 0, 0);
    }
    const float* S = cs + ((size_t)c * H + h) * D * V;
#pragma unroll 2
    for (int s = 0; s < DP / 4; s++) {
      const float a = sQ[(r0 + i16) * LDQ + 4 * s + k4];     // zero beyond D
      const float* Sr = S + (size_t)min(4 * s + k4, D - 1) * V;
      float b[NVT];
#pragma unroll
      for (int j = 0; j < NVT; j++) b[j] = Sr[min(j * 16 + i16, V - 1)];
#pragma unroll
      for (int j = 0; j < NVT; j++)
        acc[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(a, b[j], acc[j], 0, 0, 0);
    }
#pragma unroll
    for (int r = 0; r < 4; r++) {
      const float m = p[r0 + k4 * 4 + r + 1];
#pragma unroll
      for (int j = 0; j < NVT; j++) acc[j][r] *= m;
    }
  }
  __syncthreads();   // queries and keys have been read
  stage(row + (size_t)2 * H * D + h * V, (size_t)ldp, n, V, VP, sV, LDV, vec, one);
#pragma unroll
  for (int j = 0; j < LC / 16; j++)
#pragma unroll
    for (int r = 0; r < 4; r++) {
      const int t = r0 + k4 * 4 + r, s = j * 16 + i16;
      sP[t * LDP + s] = s <= t ? w[j][r] * p[t - s] : 0.0f;
    }
  __syncthreads();
  if (r0 >= n) return;
  for (int s = 0; s < (wave + 1) * 4; s++) {
    const float a = sP[(r0 + i16) * LDP + 4 * s + k4];
#pragma unroll
    for (int j = 0; j < NVT; j++)
      acc[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(a, sV[(4 * s + k4) * LDV + j * 16 + i16], acc[j], 0, 0, 0);
  }
#pragma unroll
  for (int r = 0; r < 4; r++) {
    const int t = r0 + k4 * 4 + r;
    if (t >= n) continue;
    float* o = out + (size_t)(en.row0 + t) * ldo + (size_t)h * V;
#pragma unroll
    for (int j = 0; j < NVT; j++) {
      const int v = j * 16 + i16;
      if (v < V) o[v] = acc[j][r];
    }
  }
}

template <typename T, int NVT>
static int launch_light(const T* proj, int ldp, const float* pw, float* state, const int* vent,
                        int NV, const int* cent, int E, float* cs, float* out, int ldo, int H, int D,
                        int V, hipStream_t st) {
  const int DP = (D + 15) & ~15, VP = NVT * 16;
  const int vec = D % 4 == 0 && V % 4 == 0 && ldp % 4 == 0 && (size_t)proj % (4 * sizeof(T)) == 0;
  const size_t shm1 = (size_t)LC * (ld_cols(DP) + ld_cols(VP)) * 4;
  const int lq = ld_rows(DP), lv = ld_cols(VP);
  const size_t shm2 = (size_t)LC * ((lq > LC + 4 ? lq : LC + 4) + (lq > lv ? lq : lv)) * 4;
  if (shm1 > 160 * 1024 || shm2 > 160 * 1024) return (int)hipErrorInvalidValue;
  static const hipError_t attr = [] {
    hipError_t e = hipFuncSetAttribute((const void*)lightning_local_k<T, NVT>,
                                       hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
    return e != hipSuccess ? e
                           : hipFuncSetAttribute((const void*)lightning_out_k<T, NVT>,
                                                 hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
  }();
  if (attr != hipSuccess) return (int)attr;
  dim3 grid(NV, H);
  hipLaunchKernelGGL((lightning_local_k<T, NVT>), grid, dim3(256), shm1, st, proj, ldp, pw, vent, cs, H,
                     D, V, vec);
  hipLaunchKernelGGL(lightning_chain_k, dim3((D * V + 255) / 256, H, E), dim3(256), 0, st, cs, pw, vent,
                     state, cent, H, D * V);
  hipLaunchKernelGGL((lightning_out_k<T, NVT>), grid, dim3(256), shm2, st, proj, ldp, pw, vent, cs, out,
                     ldo, H, D, V, vec);
  return (int)hipGetLastError();
}

extern "C" {

// vent [NV]: the portions' chunks of at most 64 tokens as entries (row0, n, 1, chunk index); cs fp32
// [NV, H, D, V] scratch; pw fp32 [H, 65]; out fp32 [R, H*V]
int p2p_sm_lightning_chunked(const void* proj, int ldp, const float* pw, float* state,
                             const int* vent, int NV, const int* cent, int E, float* cs, float* out,
                             int ldo, int H, int D, int V, int f32, hipStream_t st) {
  if (E <= 0 || NV <= 0) return 0;
  if (H < 1 || D < 1 || V < 1 || D > 256 || V > 256) return (int)hipErrorInvalidValue;
#define LG(NVT)                                                                                   \
  SM_DISPATCH_T(f32, return (launch_light<T, NVT>((const T*)proj, ldp, pw, state, vent, NV, cent, E, \
                                                  cs, out, ldo, H, D, V, st)))
  if (V <= 32) LG(2);
  else if (V <= 64) LG(4);
  else if (V <= 128) LG(8);
  else LG(16);
#undef LG
  return 0;
}

}  // extern "C"
