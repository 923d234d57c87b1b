// Parallel residual streams of a hyper-connected decoder: the pass between two sublayers.
//
//   X_t <- sum_s mix[s, t] X_s + out_w[t] * y        (all streams at once, from the old ones; y: the closing sublayer's output)
//   u    = sum_s in_w[s] X_s                          (what the opening sublayer reads)
//   out  = (u - mean(u)) / sqrt(mean((u - mean)^2) + eps) * norm_w
//
// Streams X fp32 [T, s, D], statistics fp32 (two-pass variance from registers). One workgroup per token row: the streams are
// read and written once, u stays in registers between the passes. x0: the old streams are all equal to x0 [T, D] (the embedding
// output), so the first pass of a step only writes X. y null: no closing sublayer; in_w null: no opening one.
#include "gai_common.h"
#include "gai_kernels.h"

using namespace gai;

namespace {

struct HyperArgs {
  float* X;
  const float* x0;
  const void* y;
  int ldy;
  const float *mix, *out_w, *in_w, *norm_w;
  void* out;
  int T, ns, D;
  float eps;
};

template <int V>
__device__ __forceinline__ void ldv(const float* p, float (&x)[V]) {
  if constexpr (V == 4) {
    const float4 f = *reinterpret_cast<const float4*>(p);
    x[0] = f.x; x[1] = f.y; x[2] = f.z; x[3] = f.w;
  } else {
    x[0] = *p;
  }
}
template <int V>
__device__ __forceinline__ void ldv(const bf16* p, float (&x)[V]) {
  if constexpr (V == 4) {
    const bf16x4 f = *reinterpret_cast<const bf16x4*>(p);
#pragma unroll
    for (int e = 0; e < 4; ++e) x[e] = (float)f[e];
  } else {
    x[0] = (float)*p;
  }
}
template <int V>
__device__ __forceinline__ void stv(float* p, const float (&x)[V]) {
  if constexpr (V == 4) *reinterpret_cast<float4*>(p) = float4{x[0], x[1], x[2], x[3]};
  else *p = x[0];
}
template <int V>
__device__ __forceinline__ void stv(bf16* p, const float (&x)[V]) {
  if constexpr (V == 4) *reinterpret_cast<bf16x4*>(p) = bf16x4{(bf16)x[0], (bf16)x[1], (bf16)x[2], (bf16)x[3]};
  else *p = (bf16)x[0];
}

constexpr int kRegs = 4;  // V-element groups of u per thread that stay in registers (wider rows re-read the streams)

// NS: number of streams, or (EXACT false) an upper bound of it
template <typename TY, typename TA, int NS, bool EXACT, int V>
__global__ __launch_bounds__(1024) void hyper_connect_kernel(HyperArgs a) {
  __shared__ float scratch[16];
  const int row = blockIdx.x, tid = threadIdx.x, NT = blockDim.x, D = a.D;
  const int ns = EXACT ? NS : a.ns;
  float* X = a.X + (size_t)row * ns * D;
  const float* x0 = a.x0 ? a.x0 + (size_t)row * D : nullptr;
  const TY* y = a.y ? (const TY*)a.y + (size_t)row * a.ldy : nullptr;
  float u[kRegs][V];
  float sum = 0.f;
  const int G = D / V, steps = (G + NT - 1) / NT;

  auto pass = [&](int i, float (&uu)[V]) {  // group i: new streams stored, u returned
    float o[NS][V];
#pragma unroll
    for (int s = 0; s < NS; ++s)
      if (EXACT || s < ns) {
        if (x0) {
          if (s == 0) ldv<V>(x0 + (size_t)i * V, o[0]);
          else
#pragma unroll
            for (int e = 0; e < V; ++e) o[s][e] = o[0][e];
        } else {
          ldv<V>(X + (size_t)s * D + (size_t)i * V, o[s]);
        }
      }
#pragma unroll
    for (int e = 0; e < V; ++e) uu[e] = 0.f;
    float yv[V];
    if (y) ldv<V>(y + (size_t)i * V, yv);
#pragma unroll
    for (int t = 0; t < NS; ++t)
      if (EXACT || t < ns) {
        float n[V];
        if (y) {
          const float ow = a.out_w[t];
#pragma unroll
          for (int e = 0; e < V; ++e) n[e] = ow * yv[e];
#pragma unroll
          for (int s = 0; s < NS; ++s)
            if (EXACT || s < ns) {
              const float m = a.mix[s * ns + t];
#pragma unroll
              for (int e = 0; e < V; ++e) n[e] = fmaf(m, o[s][e], n[e]);
            }
        } else {
#pragma unroll
          for (int e = 0; e < V; ++e) n[e] = o[t][e];
        }
        if (y || x0) stv<V>(X + (size_t)t * D + (size_t)i * V, n);
        if (a.in_w) {
          const float iw = a.in_w[t];
#pragma unroll
          for (int e = 0; e < V; ++e) uu[e] = fmaf(iw, n[e], uu[e]);
        }
      }
  };
  auto read_u = [&](int i, float (&uu)[V]) {
#pragma unroll
    for (int e = 0; e < V; ++e) uu[e] = 0.f;
    for (int t = 0; t < ns; ++t) {
      float n[V];
      ldv<V>(X + (size_t)t * D + (size_t)i * V, n);
#pragma unroll
      for (int e = 0; e < V; ++e) uu[e] = fmaf(a.in_w[t], n[e], uu[e]);
    }
  };
#pragma unroll
  for (int b = 0; b < kRegs; ++b) {
    const int i = tid + b * NT;
    if (i < G) {
      pass(i, u[b]);
#pragma unroll
      for (int e = 0; e < V; ++e) sum += u[b][e];
    } else {
#pragma unroll
      for (int e = 0; e < V; ++e) u[b][e] = 0.f;
    }
  }
  for (int b = kRegs; b < steps; ++b) {
    const int i = tid + b * NT;
    if (i < G) {
      float uu[V];
      pass(i, uu);
#pragma unroll
      for (int e = 0; e < V; ++e) sum += uu[e];
    }
  }
  if (!a.in_w) return;
  const float mean = block_sum(sum, scratch) / D;
  float sq = 0.f;
#pragma unroll
  for (int b = 0; b < kRegs; ++b)
    if (tid + b * NT < G)
#pragma unroll
      for (int e = 0; e < V; ++e) {
        const float d = u[b][e] - mean;
        sq = fmaf(d, d, sq);
      }
  for (int b = kRegs; b < steps; ++b) {
    const int i = tid + b * NT;
    if (i < G) {
      float uu[V];
      read_u(i, uu);
#pragma unroll
      for (int e = 0; e < V; ++e) sq = fmaf(uu[e] - mean, uu[e] - mean, sq);
    }
  }
  const float inv = 1.0f / sqrtf(block_sum(sq, scratch) / D + a.eps);
  TA* out = (TA*)a.out + (size_t)row * D;
#pragma unroll
  for (int b = 0; b < kRegs; ++b) {
    const int i = tid + b * NT;
    if (i < G) {
      float w[V];
      ldv<V>(a.norm_w + (size_t)i * V, w);
#pragma unroll
      for (int e = 0; e < V; ++e) w[e] *= (u[b][e] - mean) * inv;
      stv<V>(out + (size_t)i * V, w);
    }
  }
  for (int b = kRegs; b < steps; ++b) {
    const int i = tid + b * NT;
    if (i < G) {
      float w[V], uu[V];
      ldv<V>(a.norm_w + (size_t)i * V, w);
      read_u(i, uu);
#pragma unroll
      for (int e = 0; e < V; ++e) w[e] *= (uu[e] - mean) * inv;
      stv<V>(out + (size_t)i * V, w);
    }
  }
}

template <typename TY, typename TA>
void launch(const HyperArgs& a, hipStream_t st) {
  const bool vec = a.D % 4 == 0 && a.ldy % 4 == 0 && ((size_t)a.y & 15) == 0;
  const int G = vec ? a.D / 4 : a.D;
  // decode steps: one group per thread; prompts: two, so that a CU holds several rows
  int NT = (a.T < 512 ? G : (G + 1) / 2);
  NT = (NT + 63) / 64 * 64;
  if (NT > 1024) NT = 1024;
#define GAI_HC(NS, EX)                                                       \
  do {                                                                       \
    if (vec) hyper_connect_kernel<TY, TA, NS, EX, 4><<<a.T, NT, 0, st>>>(a); \
    else hyper_connect_kernel<TY, TA, NS, EX, 1><<<a.T, NT, 0, st>>>(a);     \
  } while (0)
  switch (a.ns) {
    case 1: GAI_HC(1, true); break;
    case 2: GAI_HC(2, true); break;
    case 3: GAI_HC(3, true); break;
    case 4: GAI_HC(4, true); break;
    default:
      if (a.ns <= 8) GAI_HC(8, false); else GAI_HC(16, false);
  }
#undef GAI_HC
}

}  // namespace

void gai_hyper_connect(float* X, const float* x0, const void* y, int ldy, const float* mix, const float* out_w,
                       const float* in_w, const float* norm_w, void* out, int T, int ns, int D, float eps, int dt_y,
                       int dt_out, hipStream_t st) {
  if (T == 0) return;
  if (ns < 1 || ns > 16) gai_launch_error(__FILE__, __LINE__, "hyper_connect: 1 .. 16 streams");
  const HyperArgs a{X, x0, y, y ? ldy : 0, mix, out_w, in_w, norm_w, out, T, ns, D, eps};
  if (dt_y) {
    if (dt_out) launch<float, float>(a, st); else launch<float, bf16>(a, st);
  } else {
    if (dt_out) launch<bf16, float>(a, st); else launch<bf16, bf16>(a, st);
  }
  GAI_LAUNCH_CHECK();
}
