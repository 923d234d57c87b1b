// Per-head products y[t, h, :] = W[h] x[t, h, :], x [T, H * K], W [H, N, K], y [T, H * N], optionally times sigmoid(gate)
// element by element: the two folds of latent attention (queries through the key expansion; weighted latents through the
// value expansion, with the output gate) on token-major rows, so nothing is transposed in memory.
//
// bf16: v_mfma_f32_32x32x16_bf16 with rows = output channels and columns = tokens, so a lane ends up with four consecutive
// channels of one token. Prompts: a workgroup of four waves takes 128 tokens x 64 channels of a head, the weight slice
// in LDS, token rows straight from memory. Decode steps (few tokens): one wave per 32 tokens x 32 channels, everything
// straight from memory. fp32 (and bf16 off the 8-element grid): a tiled fp32 FMA kernel.
#include "gai_common.h"
#include "gai_kernels.h"

using namespace gai;

namespace {

struct HeadArgs {
  const void *x, *W, *gate;
  int ldx, ldg;
  void* y;
  int T, H, N, K;
};

__device__ __forceinline__ bf16x8 zero8() {
  bf16x8 z;
#pragma unroll
  for (int e = 0; e < 8; ++e) z[e] = (bf16)0.f;
  return z;
}

// one 32 (channels) x 32 (tokens) accumulator tile -> y, times the gate
__device__ __forceinline__ void store_tile(const HeadArgs& a, const f32x16& acc, int h, int n0, int t, int hb) {
  if (t >= a.T) return;
  bf16* y = (bf16*)a.y + ((size_t)t * a.H + h) * a.N;
  const bf16* gr = a.gate ? (const bf16*)a.gate + (size_t)t * a.ldg + (size_t)h * a.N : nullptr;
#pragma unroll
  for (int r4 = 0; r4 < 4; ++r4) {
    const int n = n0 + 8 * r4 + 4 * hb;
    if (n >= a.N) continue;  // N is a multiple of 4
    float gv[4] = {1.f, 1.f, 1.f, 1.f};
    if (gr) {
      const bf16x4 g4 = *reinterpret_cast<const bf16x4*>(gr + n);
#pragma unroll
      for (int e = 0; e < 4; ++e) gv[e] = 1.0f / (1.0f + __expf(-(float)g4[e]));
    }
    bf16x4 o;
#pragma unroll
    for (int e = 0; e < 4; ++e) o[e] = (bf16)(acc[4 * r4 + e] * gv[e]);
    *reinterpret_cast<bf16x4*>(y + n) = o;
  }
}

// K is a multiple of 8: a lane's 8-channel fragment is inside or past the row
template <int UNROLL>
__global__ __launch_bounds__(64) void head_linear_decode_kernel(HeadArgs a) {
  const int lane = threadIdx.x, ri = lane & 31, hb = lane >> 5;
  const int n0 = blockIdx.x * 32, t0 = blockIdx.y * 32, h = blockIdx.z;
  const int n = min(n0 + ri, a.N - 1), t = min(t0 + ri, a.T - 1);
  const bf16* w = (const bf16*)a.W + ((size_t)h * a.N + n) * a.K;
  const bf16* x = (const bf16*)a.x + (size_t)t * a.ldx + (size_t)h * a.K;
  f32x16 acc = f32x16{};
  const int steps = (a.K + 15) / 16;
#pragma unroll UNROLL
  for (int i = 0; i < steps; ++i) {
    const int k = 16 * i + 8 * hb;
    const bool in = k < a.K;
    const bf16x8 wf = in ? load8(w + k) : zero8(), xf = in ? load8(x + k) : zero8();
    acc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(wf, xf, acc, 0, 0, 0);
  }
  store_tile(a, acc, h, n0, t0 + ri, hb);
}

constexpr int kHT = 128, kHN = 64;

__global__ __launch_bounds__(256) void head_linear_kernel(HeadArgs a) {
  extern __shared__ __attribute__((aligned(16))) char smem[];
  bf16* ws = reinterpret_cast<bf16*>(smem);  // [64][K16 + 8]
  const int tid = threadIdx.x, wv = tid >> 6, lane = tid & 63, ri = lane & 31, hb = lane >> 5;
  const int n0 = blockIdx.x * kHN, h = blockIdx.z;
  const int K16 = (a.K + 15) / 16 * 16, ld = K16 + 8, K8 = K16 / 8;
  for (int i = tid; i < kHN * K8; i += 256) {
    const int r = i / K8, k = (i - r * K8) * 8;
    bf16x8 v = zero8();
    if (n0 + r < a.N && k < a.K) v = load8((const bf16*)a.W + ((size_t)h * a.N + n0 + r) * a.K + k);
    store8(ws + r * ld + k, v);
  }
  __syncthreads();
  const int t = blockIdx.y * kHT + wv * 32 + ri;
  const bf16* x = (const bf16*)a.x + (size_t)min(t, a.T - 1) * a.ldx + (size_t)h * a.K;
  f32x16 acc[2] = {f32x16{}, f32x16{}};
  const bf16* w0 = ws + ri * ld + 8 * hb;
#pragma unroll 4
  for (int i = 0; i < K16 / 16; ++i) {
    const int k = 16 * i + 8 * hb;
    const bf16x8 xf = k < a.K ? load8(x + k) : zero8();
    acc[0] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(load8(w0 + 16 * i), xf, acc[0], 0, 0, 0);
    acc[1] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(load8(w0 + 32 * ld + 16 * i), xf, acc[1], 0, 0, 0);
  }
  store_tile(a, acc[0], h, n0, t, hb);
  store_tile(a, acc[1], h, n0 + 32, t, hb);
}

// any sizes, fp32 arithmetic: 64 tokens x 64 channels per workgroup, 4 x 4 per thread
template <typename TA>
__global__ __launch_bounds__(256) void head_linear_fma_kernel(HeadArgs a) {
  __shared__ float xs[16][68], ws[16][68];
  const int tid = threadIdx.x, tx = tid & 15, ty = tid >> 4;
  const int n0 = blockIdx.x * 64, t0 = blockIdx.y * 64, h = blockIdx.z;
  float acc[4][4] = {};
  for (int k0 = 0; k0 < a.K; k0 += 16) {
#pragma unroll
    for (int i = tid; i < 1024; i += 256) {
      const int r = i >> 4, k = k0 + (i & 15);
      xs[i & 15][r] = (t0 + r < a.T && k < a.K) ? (float)((const TA*)a.x)[(size_t)(t0 + r) * a.ldx + (size_t)h * a.K + k] : 0.f;
      ws[i & 15][r] = (n0 + r < a.N && k < a.K) ? (float)((const TA*)a.W)[((size_t)h * a.N + n0 + r) * a.K + k] : 0.f;
    }
    __syncthreads();
#pragma unroll
    for (int k = 0; k < 16; ++k) {
      float xv[4], wv[4];
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        xv[e] = xs[k][4 * ty + e];
        wv[e] = ws[k][4 * tx + e];
      }
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[i][j] = fmaf(xv[i], wv[j], acc[i][j]);
    }
    __syncthreads();
  }
  for (int i = 0; i < 4; ++i)
    for (int j = 0; j < 4; ++j) {
      const int t = t0 + 4 * ty + i, n = n0 + 4 * tx + j;
      if (t >= a.T || n >= a.N) continue;
      float v = acc[i][j];
      if (a.gate) v /= 1.0f + expf(-(float)((const TA*)a.gate)[(size_t)t * a.ldg + (size_t)h * a.N + n]);
      ((TA*)a.y)[((size_t)t * a.H + h) * a.N + n] = (TA)v;
    }
}

}  // namespace

void gai_head_linear(const void* x, int ldx, const void* W, const void* gate, int ldg, void* y, int T, int H, int N, int K,
                     int dt, hipStream_t st) {
  if (T == 0) return;
  const HeadArgs a{x, W, gate, ldx, ldg, y, T, H, N, K};
  const bool mfma = !dt && K % 8 == 0 && N % 4 == 0 && ldx % 8 == 0 && ((size_t)x & 15) == 0 && ((size_t)W & 15) == 0 &&
                    (!gate || (ldg % 4 == 0 && ((size_t)gate & 7) == 0)) && K <= 1024;
  if (mfma && T <= 64) {
    head_linear_decode_kernel<8><<<dim3((N + 31) / 32, (T + 31) / 32, H), 64, 0, st>>>(a);
  } else if (mfma) {
    const size_t lds = (size_t)kHN * ((K + 15) / 16 * 16 + 8) * sizeof(bf16);
    if (lds > 64 * 1024)
      (void)hipFuncSetAttribute(reinterpret_cast<const void*>(head_linear_kernel),
                                hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
    head_linear_kernel<<<dim3((N + kHN - 1) / kHN, (T + kHT - 1) / kHT, H), 256, lds, st>>>(a);
  } else {
    const dim3 grid((N + 63) / 64, (T + 63) / 64, H);
    if (dt) head_linear_fma_kernel<float><<<grid, 256, 0, st>>>(a);
    else head_linear_fma_kernel<bf16><<<grid, 256, 0, st>>>(a);
  }
  GAI_LAUNCH_CHECK();
}
