// Hyper-connections: the residual of a row is a bundle of NS fp32 streams, x [rows, NS, n].  A
// sublayer reads a weighted sum of them and its result y is written back to all of them at once
// while they exchange,
//   u = sum_s in[s] x_s,      x_t <- sum_s mix[s * NS + t] x_s + out[t] y.
// The norm between u and the sublayer is a dynamic tanh, h = tanh(alpha u) w + b, which has no
// mean or variance: the whole pass is pointwise, so the update after one sublayer and the input of
// the next one are formed together and every stream is read and written once.
//
// y = a + b + sum_k cw[r, k] cy[r * top + k], each part optional (a, b: products in the activation
// type; cy: the token's routed expert outputs), summed in fp32.
#include "common.h"
using namespace sm;

// tanh by e^(-2|x|), near 0 by its Taylor series (through x^9: below 1e-8 of the value there)
__device__ __forceinline__ float tanhf_(float x) {
  const float a = fabsf(x), q = x * x;
  const float e = __builtin_amdgcn_exp2f(-2.8853900817779268f * a);
  const float far = copysignf((1.0f - e) * __builtin_amdgcn_rcpf(1.0f + e), x);
  const float near =
      x * (1.0f + q * (-1.0f / 3.0f + q * (2.0f / 15.0f + q * (-17.0f / 315.0f + q * (62.0f / 2835.0f)))));
  return a < 0.25f ? near : far;
}

template <typename T, int VEC> struct alignas(VEC * sizeof(T)) Pack { T v[VEC]; };

template <typename T, int VEC>
__device__ __forceinline__ void ldv(const T* p, float* o) {
  const Pack<T, VEC> k = *(const Pack<T, VEC>*)p;
#pragma unroll
  for (int i = 0; i < VEC; i++) o[i] = ldf(k.v, i);
}
template <typename T, int VEC>
__device__ __forceinline__ void stv(T* p, const float* o) {
  Pack<T, VEC> k;
#pragma unroll
  for (int i = 0; i < VEC; i++) stf(k.v, i, o[i]);
  *(Pack<T, VEC>*)p = k;
}

struct StreamArgs {
  float* x; int n;
  const int* rows;                                  // rows of x to take (output row i = x row rows[i])
  const void* a; int lda; const void* b; int ldb;   // addends of y
  const void* cy; int ldcy; const float* cw; int top;
  const float* mix; const float* out;               // exchange and write (mix null: x as it is)
  const float* in;                                  // read coefficients (null: all 1)
  const float* w; const float* bias; float alpha;   // dynamic tanh (w null: h = u)
  void* h; int ldh;
  const void* embed; const int* ids; float scale;   // start of a step: every stream is embed[ids] * scale
  int write;                                        // store the updated streams
};

template <typename T, int NS, int VEC>
__global__ void stream_mix_k(StreamArgs g) {
  const int i = blockIdx.x, c = (blockIdx.y * blockDim.x + threadIdx.x) * VEC, n = g.n;
  if (c >= n) return;
  const int r = g.rows ? g.rows[i] : i;
  float* xr = g.x + (size_t)r * NS * n + c;
  float x[NS][VEC];
  if (g.embed) {
    float e[VEC];
    ldv<T, VEC>((const T*)g.embed + (size_t)g.ids[r] * n + c, e);
#pragma unroll
    for (int s = 0; s < NS; s++)
#pragma unroll
      for (int k = 0; k < VEC; k++) x[s][k] = e[k] * g.scale;
  } else {
#pragma unroll
    for (int s = 0; s < NS; s++) ldv<float, VEC>(xr + (size_t)s * n, x[s]);
  }
  if (g.mix) {
    float y[VEC], t[VEC];
#pragma unroll
    for (int k = 0; k < VEC; k++) y[k] = 0.0f;
    if (g.a) ldv<T, VEC>((const T*)g.a + (size_t)r * g.lda + c, y);
    if (g.b) {
      ldv<T, VEC>((const T*)g.b + (size_t)r * g.ldb + c, t);
#pragma unroll
      for (int k = 0; k < VEC; k++) y[k] += t[k];
    }
    if (g.cy) {
      const T* cy = (const T*)g.cy + (size_t)r * g.top * g.ldcy + c;
      const float* cw = g.cw + (size_t)r * g.top;
      for (int q = 0; q < g.top; q += 2) {   // two experts' loads in flight
        const bool two = q + 1 < g.top;
        float t2[VEC];
        ldv<T, VEC>(cy + (size_t)q * g.ldcy, t);
        ldv<T, VEC>(cy + (size_t)(two ? q + 1 : q) * g.ldcy, t2);
        const float wa = cw[q], wb = two ? cw[q + 1] : 0.0f;
#pragma unroll
        for (int k = 0; k < VEC; k++) y[k] += wa * t[k] + wb * t2[k];
      }
    }
    float z[NS][VEC];
#pragma unroll
    for (int to = 0; to < NS; to++) {
      const float o = g.out[to];
#pragma unroll
      for (int k = 0; k < VEC; k++) z[to][k] = o * y[k];
#pragma unroll
      for (int s = 0; s < NS; s++) {
        const float m = g.mix[s * NS + to];
#pragma unroll
        for (int k = 0; k < VEC; k++) z[to][k] += m * x[s][k];
      }
    }
#pragma unroll
    for (int s = 0; s < NS; s++)
#pragma unroll
      for (int k = 0; k < VEC; k++) x[s][k] = z[s][k];
  }
  if (g.write) {
#pragma unroll
    for (int s = 0; s < NS; s++) stv<float, VEC>(xr + (size_t)s * n, x[s]);
  }
  if (!g.h) return;
  float u[VEC];
#pragma unroll
  for (int k = 0; k < VEC; k++) u[k] = 0.0f;
#pragma unroll
  for (int s = 0; s < NS; s++) {
    const float m = g.in ? g.in[s] : 1.0f;
#pragma unroll
    for (int k = 0; k < VEC; k++) u[k] += m * x[s][k];
  }
  if (g.w) {
    float w[VEC], bb[VEC];
    ldv<float, VEC>(g.w + c, w);
    ldv<float, VEC>(g.bias + c, bb);
#pragma unroll
    for (int k = 0; k < VEC; k++) u[k] = tanhf_(g.alpha * u[k]) * w[k] + bb[k];
  }
  stv<T, VEC>((T*)g.h + (size_t)i * g.ldh + c, u);
}

template <int VEC>
static int launch_streams(const StreamArgs& g, int R, int ns, int f32, hipStream_t st) {
  // prompts fill the chip with whole rows; a decode step's few rows are cut finer
  const int per = (g.n + VEC - 1) / VEC;
  const int threads = R >= 256 && per > 64 ? 256 : 64;
  dim3 grid(R, (per + threads - 1) / threads), block(threads);
#define SL(N)                                                                           \
  case N:                                                                               \
    SM_DISPATCH_T(f32, hipLaunchKernelGGL((stream_mix_k<T, N, VEC>), grid, block, 0, st, g)); \
    break
  switch (ns) {
    SL(1); SL(2); SL(3); SL(4); SL(5); SL(6); SL(7); SL(8);
    default: return (int)hipErrorInvalidValue;
  }
#undef SL
  return (int)hipGetLastError();
}

extern "C" {

// R: rows of the output (and of the update: with `rows`, only those rows of x are taken)
int p2p_sm_stream_mix(float* x, int R, int ns, int n, const int* rows, const void* a, int lda,
                      const void* b, int ldb, const void* cy, int ldcy, const float* cw, int top,
                      const float* mix, const float* out, const float* in, const float* w,
                      const float* bias, float alpha, void* h, int ldh, const void* embed,
                      const int* ids, float scale, int write, int f32, hipStream_t st) {
  if (R <= 0 || n <= 0) return 0;
  if ((mix && !out) || (w && !bias) || (cy && (!cw || top < 1)) || (embed && (!ids || mix)) ||
      (!mix && (a || b || cy)) || (rows && write))
    return (int)hipErrorInvalidValue;
  StreamArgs g = {x, n, rows, a, lda, b, ldb, cy, ldcy, cw, top, mix, out, in, w, bias, alpha, h, ldh,
                  embed, ids, scale, write};
  const size_t al = f32 ? 15 : 7;
  auto ok = [&](const void* p, int ld) { return !p || (((size_t)p & al) == 0 && ld % 4 == 0); };
  const bool v4 = n % 4 == 0 && ((size_t)x & 15) == 0 && ok(a, lda) && ok(b, ldb) && ok(cy, ldcy) &&
                  ok(h, ldh) && ok(embed, n) && ((size_t)w & 15) == 0 && ((size_t)bias & 15) == 0;
  return v4 ? launch_streams<4>(g, R, ns, f32, st) : launch_streams<1>(g, R, ns, f32, st);
}

}  // extern "C"
