// Gated linear attention over long portions: per head S_t = diag(a_t) S_(t-1) + k_t v_t^T,
// o_t = S_t^T q_t with a decay a_t[i] = sigmoid(z_t[i])^(1/tau) per key channel, in chunks of up to 64
// tokens on the fp32 matrix instructions (v_mfma_f32_16x16x4_f32: products and sums in fp32).  `z`
// arrives as a product of its low rank (activation type), its bias is added here; q takes D^-1/2.
//
// Between tokens s < t lies the product of the decays a_(s+1) .. a_t, per channel.  Split as a quotient of
// two running products it would overflow; every factor used here is a product of decays and at
// most 1.  A chunk is cut into four runs of 16 tokens.  With G_J the product over run J,
//   Q'_t = q_t * (a up to and with t inside its run),   K'_s = k_s * (a after s inside its run),
// the weight of s (run J) for t (run I > J) is sum_i Q'_t K'_s G_(J+1) .. G_(I-1), a matrix product with
// the G's folded into one operand; the state before the chunk is read with Q'_t G_0 .. G_(I-1).
// Inside a run the weights are formed directly, walking back from t with a running product of
// decays per channel.
//   local pass   L = sum_s (k_s * decays after s) v_s^T, and the product of all decays     [D x V], [D]
//   chain        S_next = diag(product) S + L (chain.h)
//   output pass  as above; then the head's RMS norm over V, its weight and the silu gate
// One workgroup of eight wavefronts per (chunk, head).  Key and value sizes up to 128 (padded with
// zeros in LDS); rows are laid out so that the lanes of a fragment read hit different banks.
#include "chain.h"
using namespace sm;

typedef float f32x4 __attribute__((ext_vector_type(4)));

#define GC 64        // tokens of a chunk
#define GT 512       // threads

static __host__ __device__ constexpr int ld_rows(int n) { return n + ((4 - n) & 63); }
static __host__ __device__ constexpr int ld_cols(int n) { return n + ((16 - n) & 63); }

__device__ __forceinline__ f32x4 mfma4(float a, float b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0);
}

struct GlaArgs {
  const void* proj; int ldp;      // q (H*D) | k (H*D) | v (H*V) | gate (H*V) | ..
  const void* z; int ldz;         // decay logits before their bias [rows, H*D]
  const float* za; float inv_tau;
  const float* normw; float eps, out_scale;
  const int* vent; float* cs; float* cd;
  void* out; int ldo;
  int H, D, V, vec;
};

// A [GC][PAD] tile in two steps, so that the loads of several tiles are in flight together: `load` takes
// n rows of `width` numbers into registers (four numbers per load; nothing without `vec`), `put` writes
// them to dst [GC][ldd] through f(value, channel), with `fill` in columns from `width` and rows from n on.
template <typename T, int PAD> struct Tile {
  static constexpr int W4 = PAD / 4, N = GC * W4 / GT;
  static_assert(N * GT == GC * W4, "tile size");
  struct alignas(4 * sizeof(T)) V4 { T v[4]; };
  V4 r[N];
  const T* src; size_t ld; int n, width; bool vec;
  __device__ __forceinline__ void load(const T* s, size_t ld_, int n_, int width_, bool vec_) {
    src = s; ld = ld_; n = n_; width = width_; vec = vec_;
    if (!vec) return;
#pragma unroll
    for (int u = 0; u < N; u++) {
      const int idx = threadIdx.x + u * GT, t = idx / W4, c = (idx % W4) * 4;
      r[u] = *(const V4*)(src + (size_t)min(t, n - 1) * ld + (c < width ? c : 0));
    }
  }
  template <typename F>
  __device__ __forceinline__ void put(float* dst, int ldd, float fill, F f) const {
    if (vec) {
#pragma unroll
      for (int u = 0; u < N; u++) {
        const int idx = threadIdx.x + u * GT, t = idx / W4, c = (idx % W4) * 4;
        const bool in = t < n && c < width;
        float4 v;
        v.x = in ? f(ldf(r[u].v, 0), c) : fill;
        v.y = in ? f(ldf(r[u].v, 1), c + 1) : fill;
        v.z = in ? f(ldf(r[u].v, 2), c + 2) : fill;
        v.w = in ? f(ldf(r[u].v, 3), c + 3) : fill;
        *(float4*)(dst + t * ldd + c) = v;
      }
      return;
    }
    for (int idx = threadIdx.x; idx < GC * PAD; idx += GT) {
      const int t = idx / PAD, c = idx % PAD;
      dst[t * ldd + c] = (t < n && c < width) ? f(ldf(src, (size_t)t * ld + c), c) : fill;
    }
  }
};

template <typename T, int DP, int VT>   // key size padded to DP, value size to VT * 64
__global__ void __launch_bounds__(GT) gla_local_k(GlaArgs g) {
  constexpr int LDK = ld_cols(DP), LDV = ld_cols(VT * 64);
  extern __shared__ __align__(16) float smem[];
  float* sK = smem;
  float* sA = smem + GC * LDK;                     // later the values
  float* sV = sA;
  float* sG = sA + GC * (LDK > LDV ? LDK : LDV);   // [4][DP]
  const int c = blockIdx.x, h = blockIdx.y, H = g.H, D = g.D, V = g.V;
  const Entry en = load_entry(g.vent, c);
  const int n = en.n;
  const T* row = (const T*)g.proj + (size_t)en.row0 * g.ldp;
  const float* za = g.za + (size_t)h * D;
  const float inv_tau = g.inv_tau;
  auto same = [](float x, int) { return x; };
  Tile<T, DP> tk, tz;
  Tile<T, VT * 64> tv;
  tz.load((const T*)g.z + (size_t)en.row0 * g.ldz + (size_t)h * D, (size_t)g.ldz, n, D, g.vec);
  tk.load(row + (size_t)(H + h) * D, (size_t)g.ldp, n, D, g.vec);
  tv.load(row + (size_t)2 * H * D + (size_t)h * V, (size_t)g.ldp, n, V, g.vec);
  tz.put(sA, LDK, 1.0f, [&](float x, int i) { return sigmoid_root(x + za[i], inv_tau); });
  tk.put(sK, LDK, 0.0f, same);
  __syncthreads();
  for (int it = threadIdx.x; it < 4 * DP; it += GT) {
    const int J = it / DP, i = it % DP;
    float p = 1.0f;
#pragma unroll
    for (int t = 15; t >= 0; t--) {
      const int o = (16 * J + t) * LDK + i;
      const float a = sA[o];
      sK[o] *= p;
      p *= a;
    }
    sG[J * DP + i] = p;
  }
  __syncthreads();
  tv.put(sV, LDV, 0.0f, same);
  for (int i = threadIdx.x; i < D; i += GT)
    g.cd[((size_t)c * H + h) * D + i] = sG[i] * sG[DP + i] * sG[2 * DP + i] * sG[3 * DP + i];
  __syncthreads();
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, i16 = lane & 15, k4 = lane >> 4;
  const int steps = (n + 3) / 4;
  float* out = g.cs + ((size_t)c * H + h) * D * V;
  for (int it = wave; it < DP / 4; it += 8) {      // (16 key channels, a quarter of the value columns)
    const int dt = it >> 2, v0 = (it & 3) * VT * 16, d0 = dt * 16 + i16;
    if (v0 >= V || dt * 16 >= D) continue;
    float tf[4];                                   // decays of the runs after a token's own
    tf[3] = 1.0f;
#pragma unroll
    for (int J = 2; J >= 0; J--) tf[J] = tf[J + 1] * sG[(J + 1) * DP + d0];
    f32x4 acc[VT];
#pragma unroll
    for (int j = 0; j < VT; j++) acc[j] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int J = 0; J < 4; J++)
#pragma unroll
      for (int s = 4 * J; s < 4 * J + 4; s++) {
        if (s < steps) {
          const float a = sK[(4 * s + k4) * LDK + d0] * tf[J];
#pragma unroll
          for (int j = 0; j < VT; j++) acc[j] = mfma4(a, sV[(4 * s + k4) * LDV + v0 + j * 16 + i16], acc[j]);
        }
      }
#pragma unroll
    for (int j = 0; j < VT; j++)
#pragma unroll
      for (int r = 0; r < 4; r++) {
        const int d = dt * 16 + k4 * 4 + r, v = v0 + j * 16 + i16;
        if (d < D && v < V) out[(size_t)d * V + v] = acc[j][r];
      }
  }
}

template <typename T, int DP, int VT>
__global__ void __launch_bounds__(GT) gla_out_k(GlaArgs g) {
  constexpr int LDQ = ld_rows(DP), LDV = ld_cols(VT * 64), LDP = GC + 4, DQ = DP / 4;
  extern __shared__ __align__(16) float smem[];
  float* sQ = smem;
  float* sK = sQ + GC * LDQ;
  float* sA = sK + GC * LDQ;                       // later the values
  float* sV = sA;
  float* sP = sA + GC * (LDQ > LDV ? LDQ : LDV);   // [GC][LDP] weights of the chunk's own tokens
  float* sG = sP + GC * LDP;                       // [4][DP]
  float* sF = sG + 4 * DP;                         // [4][DP] decays of the runs before
  float* sN = sF + 4 * DP;                         // [GC][4] shares of the heads' sums of squares
  const int c = blockIdx.x, h = blockIdx.y, H = g.H, D = g.D, V = g.V;
  const Entry en = load_entry(g.vent, c);
  const int n = en.n;
  const T* row = (const T*)g.proj + (size_t)en.row0 * g.ldp;
  const float* za = g.za + (size_t)h * D;
  const float inv_tau = g.inv_tau, qs = 1.0f / sqrtf((float)D);
  auto same = [](float x, int) { return x; };
  Tile<T, DP> tq, tk, tz;
  Tile<T, VT * 64> tv;
  tz.load((const T*)g.z + (size_t)en.row0 * g.ldz + (size_t)h * D, (size_t)g.ldz, n, D, g.vec);
  tq.load(row + (size_t)h * D, (size_t)g.ldp, n, D, g.vec);
  tk.load(row + (size_t)(H + h) * D, (size_t)g.ldp, n, D, g.vec);
  tv.load(row + (size_t)2 * H * D + (size_t)h * V, (size_t)g.ldp, n, V, g.vec);
  tz.put(sA, LDQ, 1.0f, [&](float x, int i) { return sigmoid_root(x + za[i], inv_tau); });
  tq.put(sQ, LDQ, 0.0f, [&](float x, int) { return x * qs; });
  tk.put(sK, LDQ, 0.0f, same);
  __syncthreads();
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, i16 = lane & 15, k4 = lane >> 4;
  // this wavefront's last products cover row runs {0, 3} or {1, 2} and a quarter of the value columns;
  // its part of the state before the chunk is read now and used then
  const int v0 = (wave & 3) * VT * 16;
  const int I0 = wave >> 2, I1 = 3 - I0;
  float S[DP / 4][VT];
  if (v0 < V && 16 * I0 < n) {
    const float* Sg = g.cs + ((size_t)c * H + h) * D * V;
#pragma unroll
    for (int s = 0; s < DP / 4; s++)
#pragma unroll
      for (int j = 0; j < VT; j++)
        S[s][j] = Sg[(size_t)min(4 * s + k4, D - 1) * V + min(v0 + j * 16 + i16, V - 1)];
  }
  {
    // weights inside a run: wavefronts I and I + 4 take run I, one the 8 nearest tokens, the other
    // the 8 before; lane (token, quarter of the channels)
    const int I = wave & 3, half = wave >> 2;
    if (16 * I < n) {
      float prod[DQ];
      const float* qr = sQ + (16 * I + i16) * LDQ + k4 * DQ;
#pragma unroll
      for (int i = 0; i < DQ; i += 4) {
        const float4 q = *(const float4*)(qr + i);
        prod[i] = q.x; prod[i + 1] = q.y; prod[i + 2] = q.z; prod[i + 3] = q.w;
      }
      for (int d = 0; d < 8 + 8 * half; d++) {
        const int s = (i16 - d) & 15;              // a token after t by wrapping: its weight is 0
        const float* kr = sK + (16 * I + s) * LDQ + k4 * DQ;
        const float* ar = sA + (16 * I + s) * LDQ + k4 * DQ;
        float w0 = 0.0f, w1 = 0.0f;
        const bool mine = d >= 8 * half;
#pragma unroll
        for (int i = 0; i < DQ; i += 4) {
          const float4 a = *(const float4*)(ar + i);
          if (mine) {
            const float4 k = *(const float4*)(kr + i);
            w0 += prod[i] * k.x + prod[i + 2] * k.z;
            w1 += prod[i + 1] * k.y + prod[i + 3] * k.w;
          }
          prod[i] *= a.x; prod[i + 1] *= a.y; prod[i + 2] *= a.z; prod[i + 3] *= a.w;
        }
        if (mine) {
          float w = w0 + w1;
          w += __shfl_xor(w, 16, 64);
          w += __shfl_xor(w, 32, 64);
          if (k4 == 0) sP[(16 * I + i16) * LDP + 16 * I + s] = d <= i16 ? w : 0.0f;
        }
      }
    }
  }
  __syncthreads();
  for (int it = threadIdx.x; it < 4 * DP; it += GT) {
    const int J = it / DP, i = it % DP;
    const int o = 16 * J * LDQ + i;
    float a[16];
#pragma unroll
    for (int t = 0; t < 16; t++) a[t] = sA[o + t * LDQ];
    float p = 1.0f;
#pragma unroll
    for (int t = 15; t >= 0; t--) {
      sK[o + t * LDQ] *= p;
      p *= a[t];
    }
    sG[J * DP + i] = p;
    p = 1.0f;
#pragma unroll
    for (int t = 0; t < 16; t++) {
      p *= a[t];
      sQ[o + t * LDQ] *= p;
    }
  }
  __syncthreads();
  tv.put(sV, LDV, 0.0f, same);
  for (int i = threadIdx.x; i < DP; i += GT) {
    float p = 1.0f;
#pragma unroll
    for (int I = 0; I < 4; I++) {
      sF[I * DP + i] = p;
      p *= sG[I * DP + i];
    }
  }
  if (wave < 6) {   // weights between runs (I, J): (1,0) (2,0) (2,1) (3,0) (3,1) (3,2)
    const int I = wave < 1 ? 1 : wave < 3 ? 2 : 3, J = wave - (I * (I - 1)) / 2;
    if (16 * I < n) {
      const float* qr = sQ + (16 * I + i16) * LDQ + k4;
      const float* kr = sK + (16 * J + i16) * LDQ + k4;
      const float* g0 = sG + (J + 1) * DP + k4;    // decays of the runs in between, if any
      const float* g1 = sG + (J + 2) * DP + k4;
      f32x4 w = f32x4{0.f, 0.f, 0.f, 0.f};
      if (I == J + 1) {
#pragma unroll
        for (int s = 0; s < DP / 4; s++) w = mfma4(qr[4 * s], kr[4 * s], w);
      } else if (I == J + 2) {
#pragma unroll
        for (int s = 0; s < DP / 4; s++) w = mfma4(qr[4 * s] * g0[4 * s], kr[4 * s], w);
      } else {
#pragma unroll
        for (int s = 0; s < DP / 4; s++) w = mfma4(qr[4 * s] * g0[4 * s] * g1[4 * s], kr[4 * s], w);
      }
#pragma unroll
      for (int r = 0; r < 4; r++) sP[(16 * I + k4 * 4 + r) * LDP + 16 * J + i16] = w[r];
    }
  }
  __syncthreads();
  f32x4 acc[2][VT];
#pragma unroll
  for (int u = 0; u < 2; u++)
#pragma unroll
    for (int j = 0; j < VT; j++) acc[u][j] = f32x4{0.f, 0.f, 0.f, 0.f};
  if (v0 < V && 16 * I0 < n) {
#pragma unroll
    for (int s = 0; s < DP / 4; s++) {
      const int d = 4 * s + k4;                    // queries are zero beyond D
      const float a0 = sQ[(16 * I0 + i16) * LDQ + d] * sF[I0 * DP + d];
      const float a1 = sQ[(16 * I1 + i16) * LDQ + d] * sF[I1 * DP + d];
#pragma unroll
      for (int j = 0; j < VT; j++) {
        acc[0][j] = mfma4(a0, S[s][j], acc[0][j]);
        acc[1][j] = mfma4(a1, S[s][j], acc[1][j]);
      }
    }
#pragma unroll
    for (int u = 0; u < 2; u++) {
      const int I = u ? I1 : I0;
      if (16 * I >= n) continue;
      for (int s = 0; s < 4 * (I + 1); s++) {
        const float a = sP[(16 * I + i16) * LDP + 4 * s + k4];
#pragma unroll
        for (int j = 0; j < VT; j++) acc[u][j] = mfma4(a, sV[(4 * s + k4) * LDV + v0 + j * 16 + i16], acc[u][j]);
      }
    }
  }
  // head norm: the rows' sums of squares over this wavefront's columns, then over the four quarters
#pragma unroll
  for (int u = 0; u < 2; u++)
#pragma unroll
    for (int r = 0; r < 4; r++) {
      float ss = 0.0f;
#pragma unroll
      for (int j = 0; j < VT; j++)
        if (v0 + j * 16 + i16 < V) ss += acc[u][j][r] * acc[u][j][r];
#pragma unroll
      for (int o = 8; o > 0; o >>= 1) ss += __shfl_xor(ss, o, 64);
      if (i16 == 0) sN[(16 * (u ? I1 : I0) + k4 * 4 + r) * 4 + (wave & 3)] = ss;
    }
  __syncthreads();
#pragma unroll
  for (int u = 0; u < 2; u++)
#pragma unroll
    for (int r = 0; r < 4; r++) {
      const int t = 16 * (u ? I1 : I0) + k4 * 4 + r;
      if (t >= n) continue;
      const float4 q = *(const float4*)(sN + 4 * t);
      const float rs = g.out_scale / sqrtf((q.x + q.y + q.z + q.w) / (float)V + g.eps);
      const T* gt = row + (size_t)t * g.ldp + (size_t)2 * H * D + (size_t)(H + h) * V;
      T* o = (T*)g.out + (size_t)(en.row0 + t) * g.ldo + (size_t)h * V;
#pragma unroll
      for (int j = 0; j < VT; j++) {
        const int v = v0 + j * 16 + i16;
        if (v < V) stf(o, v, acc[u][j][r] * rs * g.normw[v] * silu_(ldf(gt, v)));
      }
    }
}

template <typename T, int DP, int VT>
static int launch_gla(GlaArgs g, float* state, int NV, const int* cent, int E, hipStream_t st) {
  constexpr int LDK = ld_cols(DP), LDQ = ld_rows(DP), LDV = ld_cols(VT * 64);
  const size_t shm1 = (size_t)(GC * (LDK + (LDK > LDV ? LDK : LDV)) + 4 * DP) * 4;
  const size_t shm2 = (size_t)(GC * (2 * LDQ + (LDQ > LDV ? LDQ : LDV) + GC + 4) + 8 * DP + 4 * GC) * 4;
  static_assert(GC * (2 * LDQ + (LDQ > LDV ? LDQ : LDV) + GC + 4) + 8 * DP + 4 * GC <= 40 * 1024, "LDS");
  static const hipError_t attr = [] {
    hipError_t e = hipFuncSetAttribute((const void*)gla_local_k<T, DP, VT>,
                                       hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
    return e != hipSuccess ? e
                           : hipFuncSetAttribute((const void*)gla_out_k<T, DP, VT>,
                                                 hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
  }();
  if (attr != hipSuccess) return (int)attr;
  g.vec = g.D % 4 == 0 && g.V % 4 == 0 && g.ldp % 4 == 0 && g.ldz % 4 == 0 &&
          (size_t)g.proj % (4 * sizeof(T)) == 0 && (size_t)g.z % (4 * sizeof(T)) == 0;
  dim3 grid(NV, g.H);
  hipLaunchKernelGGL((gla_local_k<T, DP, VT>), grid, dim3(GT), shm1, st, g);
  hipLaunchKernelGGL(diag_chain_k, dim3((g.D * g.V + 255) / 256, E * g.H), dim3(256), 0, st, g.cs, g.cd, state,
                     cent, g.H, g.D, g.V);
  hipLaunchKernelGGL((gla_out_k<T, DP, VT>), grid, dim3(GT), shm2, st, g);
  return (int)hipGetLastError();
}

extern "C" {

// vent [NV]: the portions' chunks of at most 64 tokens as entries (row0, n, 1, chunk index); cs fp32
// [NV, H, D, V] and cd fp32 [NV, H, D] scratch; out [R, H*V] in the activation type
int p2p_sm_gla_chunked(const void* proj, int ldp, const void* z, int ldz, const float* za, float inv_tau,
                       const float* normw, float* state, const int* vent, int NV, const int* cent, int E,
                       float* cs, float* cd, void* out, int ldo, int H, int D, int V, float eps,
                       float out_scale, int f32, hipStream_t st) {
  if (E <= 0 || NV <= 0) return 0;
  if (H < 1 || D < 1 || V < 1 || D > 128 || V > 128) return (int)hipErrorInvalidValue;
  GlaArgs g = {proj, ldp, z, ldz, za, inv_tau, normw, eps, out_scale, vent, cs, cd, out, ldo, H, D, V, 0};
#define GL(DP, VT) SM_DISPATCH_T(f32, return (launch_gla<T, DP, VT>(g, state, NV, cent, E, st)))
#define GLV(DP)             \
  do {                      \
    if (V <= 64) GL(DP, 1); \
    else GL(DP, 2);         \
  } while (0)
  if (D <= 32) GLV(32);
  else if (D <= 64) GLV(64);
  else GLV(128);
#undef GLV
#undef GL
  return 0;
}

}  // extern "C"
