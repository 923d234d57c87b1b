// Per-head products y[t, h, :] = W[h] x[t, h, :], x [T, H * K], W [H, N, K], y [T, H * N], optionally times sigmoid(gate)
// element by element: the two folds of latent attention (queries through the key expansion; weighted latents through the
// value expansion, with the output gate) on token-major rows, so nothing is transposed in memory.
//
// bf16: v_mfma_f32_32x32x16_bf16 with rows = output channels and columns = tokens, so a lane ends up with four consecutive
// channels of one token. Prompts: a workgroup of four waves takes 64 tokens of a head, stages their rows once, walks the
// weight in slices of 64 channels and stores through LDS, so that every global access is a coalesced row. Decode steps (few
// tokens), and heads wider than 256: one wave per 32 tokens x 32 channels, everything straight from memory. fp32 (and bf16 off the 8-element grid): a tiled fp32 FMA kernel.
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

constexpr int kHT = 64, kHN = 64, kHY = kHN + 8;

// LDS: x [64][K16 + 8], one weight slice [64][K16 + 8], one output tile [64][72]; all with coalesced 16-byte rows. The next
// weight slice is on its way while this one is multiplied. K <= 256.
__global__ __launch_bounds__(256) void head_linear_kernel(HeadArgs a) {
  extern __shared__ __attribute__((aligned(16))) char smem[];
  const int K16 = (a.K + 15) / 16 * 16, ld = K16 + 8, K8 = K16 / 8;
  bf16* xs = reinterpret_cast<bf16*>(smem);
  bf16* ws = xs + kHT * ld;
  bf16* ys = ws + kHN * ld;
  const int tid = threadIdx.x, wv = tid >> 6, lane = tid & 63, ri = lane & 31, hb = lane >> 5;
  const int t0 = blockIdx.x * kHT, h = blockIdx.y;
  const int r_n = tid >> 2, k_n = (tid & 3) * 8;  // four threads per weight row, 8 channels each, every 32 channels
  const bf16* Wh = (const bf16*)a.W + (size_t)h * a.N * a.K;
  bf16x8 wn[8];
  auto fetch = [&](int n0) {
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      const int k = k_n + 32 * i;
      wn[i] = zero8();
      if (n0 + r_n < a.N && k < a.K) wn[i] = load8(Wh + (size_t)(n0 + r_n) * a.K + k);
    }
  };
  fetch(0);
  for (int i = tid; i < kHT * K8; i += 256) {
    const int r = i / K8, k = (i - r * K8) * 8;
    bf16x8 v = zero8();
    if (t0 + r < a.T && k < a.K) v = load8((const bf16*)a.x + (size_t)(t0 + r) * a.ldx + (size_t)h * a.K + k);
    store8(xs + r * ld + k, v);
  }
  const int tw = (wv & 1) * 32, nw = (wv >> 1) * 32;
  const bf16* xw = xs + (tw + ri) * ld + 8 * hb;
  const bf16* w0 = ws + (nw + ri) * ld + 8 * hb;
  for (int n0 = 0; n0 < a.N; n0 += kHN) {
#pragma unroll
    for (int i = 0; i < 8; ++i)
      if (k_n + 32 * i < K16) store8(ws + r_n * ld + k_n + 32 * i, wn[i]);
    __syncthreads();
    if (n0 + kHN < a.N) fetch(n0 + kHN);
    f32x16 acc = f32x16{};
#pragma unroll 4
    for (int i = 0; i < K16 / 16; ++i)
      acc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(load8(w0 + 16 * i), load8(xw + 16 * i), acc, 0, 0, 0);
    bf16* yw = ys + (tw + ri) * kHY + nw + 4 * hb;
#pragma unroll
    for (int r4 = 0; r4 < 4; ++r4) {
      bf16x4 o;
#pragma unroll
      for (int e = 0; e < 4; ++e) o[e] = (bf16)acc[4 * r4 + e];
      *reinterpret_cast<bf16x4*>(yw + 8 * r4) = o;
    }
    __syncthreads();  // the output tile is there; the weight slice may be overwritten
#pragma unroll
    for (int q = 0; q < kHT * kHN / 4 / 256; ++q) {
      const int i = tid + 256 * q, r = i / (kHN / 4), c = (i % (kHN / 4)) * 4, t = t0 + r, n = n0 + c;
      if (t >= a.T || n >= a.N) continue;
      bf16x4 o = *reinterpret_cast<const bf16x4*>(ys + r * kHY + c);
      if (a.gate) {
        const bf16x4 g4 = *reinterpret_cast<const bf16x4*>((const bf16*)a.gate + (size_t)t * a.ldg + (size_t)h * a.N + n);
#pragma unroll
        for (int e = 0; e < 4; ++e) o[e] = (bf16)((float)o[e] / (1.0f + __expf(-(float)g4[e])));
      }
      *reinterpret_cast<bf16x4*>((bf16*)a.y + ((size_t)t * a.H + h) * a.N + n) = o;
    }
  }
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
                    (!gate || (ldg % 4 == 0 && ((size_t)gate & 7) == 0)) ;
  if (mfma && (T <= 64 || K > 256)) {
    head_linear_decode_kernel<8><<<dim3((N + 31) / 32, (T + 31) / 32, H), 64, 0, st>>>(a);
  } else if (mfma) {
    const size_t lds = ((size_t)(kHT + kHN) * ((K + 15) / 16 * 16 + 8) + (size_t)kHT * kHY) * sizeof(bf16);
    if (lds > 64 * 1024)
      (void)hipFuncSetAttribute(reinterpret_cast<const void*>(head_linear_kernel),
                                hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
    head_linear_kernel<<<dim3((T + kHT - 1) / kHT, H), 256, lds, st>>>(a);
  } else {
    const dim3 grid((N + 63) / 64, (T + 63) / 64, H);
    if (dt) head_linear_fma_kernel<float><<<grid, 256, 0, st>>>(a);
    else head_linear_fma_kernel<bf16><<<grid, 256, 0, st>>>(a);
  }
  GAI_LAUNCH_CHECK();
}
