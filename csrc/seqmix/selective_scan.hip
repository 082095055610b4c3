// Selective scan of the first Mamba: every channel c carries N state numbers of its own,
//   S[n] <- exp(dt A[n]) S[n] + dt x B[n],   y = sum_n S[n] C[n] + D x,   y * silu(z),
// with one step size dt = softplus(raw + bias) per channel and token, A = -exp(A_log) per channel
// and state, B and C shared by the channels.  Everything here is fp32; x, B, C, z and the raw step
// sizes arrive in the activation type.  The state of a slot is stored [N][I] (channels
// contiguous), so is A, premultiplied by log2(e): the decay is exp2(dt A).
//
// selective_scan_k: lane = channel, a wavefront keeps NS states of 64 channels in registers; N > NS
// splits over SN wavefronts whose shares of y meet in LDS.  B and C of a stretch of tokens are
// staged in LDS (read back as broadcasts), x / raw dt / z are read straight from their rows, a few
// tokens ahead.  Long portions run as chunks side by side: local pass from zero states (end
// state and sum of dt per channel), a chain over the chunks (the decay over a chunk is
// exp2(A sum dt)), output pass from the true initial states.
//
// selective_step_k: portions of one token.  The states of 64 channels spread over as many
// wavefronts as give each few of them; the wavefronts also share the projection of the step
// sizes from their low rank (weights stored [rank][I]), which saves a matrix product.
#include "common.h"
using namespace sm;

struct SelArgs {
  const void* x; int ldx;      // [R, I] convolved inputs
  const void* bc; int ldbc;    // B at column 0, C at column N
  const void* dt; int lddt;    // raw step sizes [R, I] (scan) or their low-rank rows [R, rank] (step)
  const void* wdt; int rank;   // [rank][I] (step)
  const float* dtb; const float* A2; const float* Dp;
  const void* z; int ldz;
  float* state; const int* ent;
  void* y; int ldy;
  int I, N, CT, mode;
  float* dtsum;                // [chunks, I] (mode 1)
};

#define SEL_U 4   // tokens whose inputs are loaded together

// mode 0: portions from their slots' states, states written back; 1: a chunk from zero, end state to
// `state[slot]`, sum of dt to dtsum; 2: a chunk from state[slot], outputs only
template <typename T, int NS>
__global__ void __launch_bounds__(1024)
selective_scan_k(SelArgs a, int SN, int CW) {
  extern __shared__ __align__(16) float smem[];
  const int I = a.I, N = a.N, CT = a.CT, mode = a.mode;
  const Entry en = load_entry(a.ent, blockIdx.y);
  if (en.n <= 0) return;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int sn = wave % SN, cw = wave / SN;
  const int c = (blockIdx.x * CW + cw) * 64 + lane, n0 = sn * NS;
  const bool act = c < I;
  const int cc = act ? c : I - 1;
  const int NP = SN * NS;
  float* sB = smem;                  // [CT][NP]
  float* sC = sB + CT * NP;          // [CT][NP]
  float* sy = sC + CT * NP;          // [CT][SN][CW * 64], only when SN > 1
  const T* x = (const T*)a.x; const T* bc = (const T*)a.bc; const T* dt = (const T*)a.dt;
  const T* z = (const T*)a.z; T* y = (T*)a.y;
  float S[NS], A[NS];
  float* Sg = a.state + (size_t)en.slot * N * I + cc;
  const bool from_state = mode == 2 || (mode == 0 && en.start > 0);
#pragma unroll
  for (int q = 0; q < NS; q++) {
    const int n = min(n0 + q, N - 1);   // states beyond N ride along with B = C = 0
    A[q] = a.A2[(size_t)n * I + cc];
    S[q] = from_state ? Sg[(size_t)n * I] : 0.0f;
  }
#pragma unroll
  for (int q = 0; q < NS; q++) if (n0 + q >= N) S[q] = 0.0f;
  const float bias = a.dtb[cc], Dc = a.Dp[cc];
  float dts = 0.0f;
  for (int t0 = 0; t0 < en.n; t0 += CT) {
    const int ct = min(CT, en.n - t0);
    __syncthreads();
    for (int idx = threadIdx.x; idx < ct * NP; idx += blockDim.x) {
      const int t = idx / NP, n = idx % NP;
      const size_t row = (size_t)(en.row0 + t0 + t) * a.ldbc;
      sB[idx] = n < N ? ldf(bc, row + n) : 0.0f;
      sC[idx] = n < N ? ldf(bc, row + N + n) : 0.0f;
    }
    __syncthreads();
    for (int t1 = 0; t1 < ct; t1 += SEL_U) {
      float xv[SEL_U], dv[SEL_U], zv[SEL_U];
#pragma unroll
      for (int u = 0; u < SEL_U; u++) {
        const size_t row = (size_t)(en.row0 + t0 + min(t1 + u, ct - 1));
        xv[u] = ldf(x, row * a.ldx + cc);
        dv[u] = ldf(dt, row * a.lddt + cc);
        zv[u] = mode != 1 && sn == 0 ? ldf(z, row * a.ldz + cc) : 0.0f;
      }
#pragma unroll
      for (int u = 0; u < SEL_U; u++) {
        const int t = t1 + u;
        if (t >= ct) break;
        const float d = softplus_(dv[u] + bias), dx = d * xv[u];
        dts += d;
        const float4* B4 = (const float4*)(sB + t * NP + n0);
        const float4* C4 = (const float4*)(sC + t * NP + n0);
        float acc = 0.0f, acc1 = 0.0f;
#pragma unroll
        for (int q = 0; q < NS / 4; q++) {
          const float4 b = B4[q];
          S[4 * q] = fmaf(exp2_(d * A[4 * q]), S[4 * q], dx * b.x);
          S[4 * q + 1] = fmaf(exp2_(d * A[4 * q + 1]), S[4 * q + 1], dx * b.y);
          S[4 * q + 2] = fmaf(exp2_(d * A[4 * q + 2]), S[4 * q + 2], dx * b.z);
          S[4 * q + 3] = fmaf(exp2_(d * A[4 * q + 3]), S[4 * q + 3], dx * b.w);
          if (mode != 1) {
            const float4 k = C4[q];
            acc = fmaf(S[4 * q], k.x, acc);
            acc1 = fmaf(S[4 * q + 1], k.y, acc1);
            acc = fmaf(S[4 * q + 2], k.z, acc);
            acc1 = fmaf(S[4 * q + 3], k.w, acc1);
          }
        }
        if (mode != 1) {
          acc += acc1;
          if (sn == 0) acc = (acc + Dc * xv[u]) * (SN == 1 ? silu_(zv[u]) : 1.0f);
          if (SN > 1) sy[(t * SN + sn) * CW * 64 + cw * 64 + lane] = acc;
          else if (act) stf(y, (size_t)(en.row0 + t0 + t) * a.ldy + c, acc);
        }
      }
    }
    if (SN > 1 && mode != 1) {
      __syncthreads();
      const int W = CW * 64;
      for (int idx = threadIdx.x; idx < ct * W; idx += blockDim.x) {
        const int t = idx / W, l = idx % W, ch = blockIdx.x * W + l;
        if (ch >= I) continue;
        float acc = 0.0f;
        for (int k = 0; k < SN; k++) acc += sy[(t * SN + k) * W + l];
        const size_t row = (size_t)(en.row0 + t0 + t);
        stf(y, row * a.ldy + ch, acc * silu_(ldf(z, row * a.ldz + ch)));
      }
    }
  }
  if (mode != 2 && act) {
#pragma unroll
    for (int q = 0; q < NS; q++)
      if (n0 + q < N) Sg[(size_t)(n0 + q) * I] = S[q];
    if (mode == 1 && sn == 0) a.dtsum[(size_t)blockIdx.y * I + c] = dts;
  }
}

// Chains the chunks of each portion: init_c replaces the local end state of chunk c in `tmp`,
// init_{c+1} = exp2(A dtsum_c) init_c + local_c; the end goes to the portion's slot.
// cent: per portion (first chunk, chunks, first position, slot).
__global__ void __launch_bounds__(256)
selective_chain_k(float* __restrict__ tmp, const float* __restrict__ dtsum,
                  const float* __restrict__ A2, float* __restrict__ state,
                  const int* __restrict__ cent, int I, int N) {
  const int c = blockIdx.x * 256 + threadIdx.x, n = blockIdx.y, e = blockIdx.z;
  if (c >= I) return;
  const int c0 = cent[4 * e], nc = cent[4 * e + 1], start = cent[4 * e + 2], slot = cent[4 * e + 3];
  const float A = A2[(size_t)n * I + c];
  float* sg = state + ((size_t)slot * N + n) * I + c;
  const size_t step = (size_t)N * I;
  float* p = tmp + (size_t)c0 * step + (size_t)n * I + c;
  const float* d = dtsum + (size_t)c0 * I + c;
  float cur = start > 0 ? *sg : 0.0f;
  for (int k = 0; k < nc; k += 8) {
    float loc[8], dec[8];   // eight chunks' loads in flight
#pragma unroll
    for (int u = 0; u < 8; u++) {
      const int kk = min(k + u, nc - 1);
      loc[u] = p[(size_t)kk * step];
      dec[u] = exp2_(A * d[(size_t)kk * I]);
    }
#pragma unroll
    for (int u = 0; u < 8; u++) {
      if (k + u < nc) {
        p[(size_t)(k + u) * step] = cur;
        cur = fmaf(dec[u], cur, loc[u]);
      }
    }
  }
  *sg = cur;
}

// one token per portion: 64 channels per workgroup, wavefront sn holds states sn*NS .. of them
template <typename T, int NS>
__global__ void __launch_bounds__(1024) selective_step_k(SelArgs a, int SN) {
  extern __shared__ float smem[];    // [SN][64] shares of dt, then of y
  const int I = a.I, N = a.N;
  const Entry en = load_entry(a.ent, blockIdx.y);
  if (en.n != 1) return;
  const int lane = threadIdx.x & 63, sn = threadIdx.x >> 6;
  const int c = blockIdx.x * 64 + lane, n0 = sn * NS;
  const bool act = c < I;
  const int cc = act ? c : I - 1;
  const size_t row = (size_t)en.row0;
  const T* bc = (const T*)a.bc + row * a.ldbc;
  const T* lr = (const T*)a.dt + row * a.lddt;
  const T* w = (const T*)a.wdt + cc;
  float* Sg = a.state + (size_t)en.slot * N * I + cc;
  float S[NS], A[NS], B[NS], C[NS];
#pragma unroll
  for (int q = 0; q < NS; q++) {
    const int n = min(n0 + q, N - 1);
    A[q] = a.A2[(size_t)n * I + cc];
    S[q] = en.start > 0 ? Sg[(size_t)n * I] : 0.0f;
    B[q] = ldf(bc, n);
    C[q] = n0 + q < N ? ldf(bc, N + n) : 0.0f;
  }
  const float xv = ldf((const T*)a.x, row * a.ldx + cc), zv = ldf((const T*)a.z, row * a.ldz + cc);
  const float Dc = a.Dp[cc];
  float part = 0.0f;
  int k = sn;
  for (; k + 7 * SN < a.rank; k += 8 * SN) {   // eight weights in flight
    float wv[8], lv[8];
#pragma unroll
    for (int u = 0; u < 8; u++) {
      wv[u] = ldf(w, (size_t)(k + u * SN) * I);
      lv[u] = ldf(lr, k + u * SN);
    }
#pragma unroll
    for (int u = 0; u < 8; u++) part = fmaf(wv[u], lv[u], part);
  }
  for (; k < a.rank; k += SN) part = fmaf(ldf(w, (size_t)k * I), ldf(lr, k), part);
  smem[sn * 64 + lane] = part;
  __syncthreads();
  float raw = a.dtb[cc];
  for (int i = 0; i < SN; i++) raw += smem[i * 64 + lane];
  const float d = softplus_(raw), dx = d * xv;
  float acc = sn == 0 ? Dc * xv : 0.0f;
#pragma unroll
  for (int q = 0; q < NS; q++) {
    S[q] = fmaf(exp2_(d * A[q]), S[q], dx * B[q]);
    acc = fmaf(S[q], C[q], acc);
    if (act && n0 + q < N) Sg[(size_t)(n0 + q) * I] = S[q];
  }
  __syncthreads();   // every wavefront has read the shares of dt
  smem[sn * 64 + lane] = acc;
  __syncthreads();
  if (sn == 0 && act) {
    float s = 0.0f;
    for (int i = 0; i < SN; i++) s += smem[i * 64 + lane];
    stf((T*)a.y, row * a.ldy + c, s * silu_(zv));
  }
}

static int launch_sel(SelArgs a, int E, int f32, hipStream_t st) {
  if (E <= 0) return 0;
  const int N = a.N;
  const int ns = N <= 4 ? 4 : N <= 8 ? 8 : N <= 16 ? 16 : N <= 24 ? 24 : 32;
  const int SN = (N + ns - 1) / ns;
  if (N < 1 || SN > 16 || a.I < 1) return (int)hipErrorInvalidValue;
  const int CW = SN >= 4 ? 1 : 4 / SN;
  const int NP = SN * ns;
  int CT = 32;
  auto lds = [&](int ct) { return (size_t)ct * (2 * NP + (SN > 1 ? SN * CW * 64 : 0)) * 4; };
  while (CT > SEL_U && lds(CT) > 32 * 1024) CT /= 2;
  if (lds(CT) > 64 * 1024) return (int)hipErrorInvalidValue;
  a.CT = CT;
  dim3 grid((a.I + CW * 64 - 1) / (CW * 64), E), block(64 * SN * CW);
#define SEL(NS) \
  SM_DISPATCH_T(f32, hipLaunchKernelGGL((selective_scan_k<T, NS>), grid, block, lds(CT), st, a, SN, CW))
  if (ns == 4) SEL(4);
  else if (ns == 8) SEL(8);
  else if (ns == 16) SEL(16);
  else if (ns == 24) SEL(24);
  else SEL(32);
#undef SEL
  return (int)hipGetLastError();
}

extern "C" {

// NV == 0: the portions of `ent` in one pass; else their chunks vent [NV] side by side (cent: see
// selective_chain_k; tmp fp32 [NV, N, I], dtsum fp32 [NV, I])
int p2p_sm_selective_scan(const void* x, int ldx, const void* bc, int ldbc, const void* dt,
                          int lddt, const float* dtb, const float* A2, const float* Dp,
                          const void* z, int ldz, float* state, const int* ent, int E, void* y,
                          int ldy, int I, int N, const int* vent, int NV, const int* cent,
                          float* tmp, float* dtsum, int f32, hipStream_t st) {
  SelArgs a = {};
  a.x = x; a.ldx = ldx; a.bc = bc; a.ldbc = ldbc; a.dt = dt; a.lddt = lddt; a.dtb = dtb; a.A2 = A2;
  a.Dp = Dp; a.z = z; a.ldz = ldz; a.state = state; a.ent = ent; a.y = y; a.ldy = ldy; a.I = I;
  a.N = N;
  if (E <= 0) return 0;
  if (NV <= 0) return launch_sel(a, E, f32, st);
  a.state = tmp; a.ent = vent; a.dtsum = dtsum; a.mode = 1;
  int err = launch_sel(a, NV, f32, st);
  if (err) return err;
  hipLaunchKernelGGL(selective_chain_k, dim3((I + 255) / 256, N, E), dim3(256), 0, st, tmp, dtsum,
                     A2, state, cent, I, N);
  if ((err = (int)hipGetLastError())) return err;
  a.mode = 2;
  return launch_sel(a, NV, f32, st);
}

int p2p_sm_selective_step(const void* x, int ldx, const void* bc, int ldbc, const void* lr,
                          int ldlr, const void* wdt, int rank, const float* dtb, const float* A2,
                          const float* Dp, const void* z, int ldz, float* state, const int* ent,
                          int E, void* y, int ldy, int I, int N, int f32, hipStream_t st) {
  if (E <= 0) return 0;
  SelArgs a = {};
  a.x = x; a.ldx = ldx; a.bc = bc; a.ldbc = ldbc; a.dt = lr; a.lddt = ldlr; a.wdt = wdt;
  a.rank = rank; a.dtb = dtb; a.A2 = A2; a.Dp = Dp; a.z = z; a.ldz = ldz; a.state = state;
  a.ent = ent; a.y = y; a.ldy = ldy; a.I = I; a.N = N;
  const int ns = N <= 32 ? 4 : N <= 128 ? 8 : 32;
  const int SN = (N + ns - 1) / ns;
  if (N < 1 || SN > 16 || I < 1 || rank < 1) return (int)hipErrorInvalidValue;
  dim3 grid((I + 63) / 64, E), block(64 * SN);
#define STEP(NS) \
  SM_DISPATCH_T(f32, hipLaunchKernelGGL((selective_step_k<T, NS>), grid, block, SN * 64 * 4, st, a, SN))
  if (ns == 4) STEP(4);
  else if (ns == 8) STEP(8);
  else STEP(32);
#undef STEP
  return (int)hipGetLastError();
}

}  // extern "C"
