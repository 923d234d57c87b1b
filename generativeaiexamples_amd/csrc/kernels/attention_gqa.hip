// Paged softmax attention whose query heads share kv heads (grouped-query, multi-query, latent attention over the cached
// latent), bf16 pages, fp32 scores, weights and sums:
//
//   s_ij = scale * (q_i . k_j),  j <= i (and i - j < window when window > 0)
//   o_i  = sigmoid(gate_ih) sum_j e^(s_ij) v_j / (sum_j e^(s_ij) + e^(sink_h))      (gate, sink: optional, one per head)
//
// The R = H / G query heads of one kv head see the same keys, so a "row" here is a (token, head of the group) pair and the
// matrix-core tile is 32 such rows (eight tokens of four heads, say) against 32 keys of that kv head (blockIdx.z). S^T = K.Q^T on v_mfma_f32_32x32x16_bf16 leaves one row per
// lane; the softmax is in-register fp32; P.V runs on the same MFMA with the fp32 weights split into two bf16 terms. K row
// pi(i) feeds accumulator row i with pi = swap of bits 2 and 3, so that the eight weights a lane holds for a 16-key step are
// eight consecutive keys: the V^T fragment is one 16-byte load. The running maximum is allowed to lag by 2^8 before the
// accumulators are rescaled (the weights stay within fp32 and the final division cancels the factor), so rescaling is rare.
//
// gqa_prefill_kernel: NW waves of a workgroup (32 NW consecutive rows of a sequence) share 32-key blocks staged in LDS by
// direct global -> LDS loads, double buffered; both images are XOR-swizzled through the per-lane source address so that
// fragment reads are conflict-free. Long tiles are launched first (causal rows differ in length).
// gqa_split_kernel: sequences with few rows (decoded tokens, short portions): one wave per (32 rows, share of the key blocks),
// fragments straight from memory; partial sums, maxima and denominators are merged by gqa_merge_kernel.
#include "gai_common.h"
#include "gai_kernels.h"

using namespace gai;

namespace {

constexpr float kL2e = 1.4426950408889634f;
constexpr float kOut = -1e30f;     // a masked score
constexpr float kLag = 8.f;        // how far (powers of two) the running maximum may lag
constexpr int kShortRows = 128;    // sequences of fewer rows go to the key-split kernel
constexpr int kMaxSplit = 32;

struct GqaArgs {
  const bf16 *q, *kc, *vc;
  const int *bt, *cu, *ctx;
  int maxb, S, T, H, G, R;         // R = H / G query heads per kv head
  float scale2;                    // scale * log2(e)
  int window;
  const float* sink;               // [H] or null
  const bf16* gate;                // [T, >= H] or null
  int ldg;
  bf16* out;
  int ldo;
  float* part;                     // [nsplit][S * G * prow][DV + 4]: sums, maximum (log2 units), denominator
  int nsplit;
  int tps;                         // tiles of 32 rows per sequence in the key-split launch
  int prow;                        // rows per (sequence, kv head) in part
};

__device__ __forceinline__ int key_perm(int i) { return (i & 0x13) | ((i & 4) << 1) | ((i & 8) >> 1); }

// swizzle of a K row's 16-byte chunks: 16 consecutive rows at one chunk land on the 16 slots of a 256-byte bank row
template <int DK>
__device__ __forceinline__ int k_swz(int row) {
  constexpr int n = DK / 8, low = n & -n, p = low > 16 ? 16 : low;
  return (row / (16 / p)) & (p - 1);
}

__device__ __forceinline__ float half_max(float x) {
  const auto r = __builtin_amdgcn_permlane32_swap(__float_as_uint(x), __float_as_uint(x), false, false);
  return fmaxf(__uint_as_float(r[0]), __uint_as_float(r[1]));
}
__device__ __forceinline__ float half_sum(float x) {
  const auto r = __builtin_amdgcn_permlane32_swap(__float_as_uint(x), __float_as_uint(x), false, false);
  return __uint_as_float(r[0]) + __uint_as_float(r[1]);
}

// scores of one 32-key block (sc: K.Q^T) -> weights in place; m lags, l and acc are rescaled when it moves
template <int NV>
__device__ __forceinline__ void soft_block(f32x16& sc, float scale2, bool masked, int kb, int pos, int lo, int hb, float& m,
                                           float& l, f32x16 (&acc)[NV]) {
  float mt = kOut;
  if (masked) {
#pragma unroll
    for (int r = 0; r < 16; ++r) {
      const int key = kb + (r & 7) + 8 * hb + 16 * (r >> 3);
      sc[r] = key <= pos && key >= lo ? sc[r] * scale2 : kOut;
      mt = fmaxf(mt, sc[r]);
    }
  } else {
#pragma unroll
    for (int r = 0; r < 16; ++r) {
      sc[r] *= scale2;
      mt = fmaxf(mt, sc[r]);
    }
  }
  mt = half_max(mt);
  if (__any(mt > m + kLag)) {
    const float mn = fmaxf(m, mt), al = __builtin_amdgcn_exp2f(m - mn);
    m = mn;
    l *= al;
#pragma unroll
    for (int i = 0; i < NV; ++i) acc[i] *= al;
  }
  float rs = 0.f;
#pragma unroll
  for (int r = 0; r < 16; ++r) {
    const float p = masked && sc[r] < 0.5f * kOut ? 0.f : __builtin_amdgcn_exp2f(sc[r] - m);
    sc[r] = p;
    rs += p;
  }
  l += rs;
}

__device__ __forceinline__ float head_gate(const GqaArgs& a, int t, int head) {
  return 1.0f / (1.0f + __expf(-(float)a.gate[(size_t)t * a.ldg + head]));
}

__device__ __forceinline__ void split_weights(const f32x16& sc, int ks, bf16x8& hi, bf16x8& lo) {
#pragma unroll
  for (int e = 0; e < 8; ++e) {
    const float p = sc[8 * ks + e];
    hi[e] = (bf16)p;
    lo[e] = (bf16)(p - (float)hi[e]);
  }
}

template <int DK, int DV, int NW>
__global__ __launch_bounds__(64 * NW) void gqa_prefill_kernel(GqaArgs a) {
  constexpr int KB = 32 * DK * 2, VB = 32 * DV * 2, KI = KB / 1024, VI = VB / 1024;  // staged bytes / 1-KiB loads per block
  extern __shared__ __attribute__((aligned(16))) char smem[];                          // [2][K | V]
  const int tid = threadIdx.x, wv = tid >> 6, lane = tid & 63, qi = lane & 31, hb = lane >> 5;
  // ---- tile -> (sequence, first row); the last tiles of the launch first
  int total = 0;
  for (int s = 0; s < a.S; ++s) {
    const int rows = (a.cu[s + 1] - a.cu[s]) * a.R;
    total += rows >= kShortRows ? (rows + 32 * NW - 1) / (32 * NW) : 0;
  }
  if ((int)blockIdx.x >= total) return;
  int tile = total - 1 - (int)blockIdx.x, s = 0, rows = 0;
  for (; s < a.S; ++s) {
    rows = (a.cu[s + 1] - a.cu[s]) * a.R;
    const int n = rows >= kShortRows ? (rows + 32 * NW - 1) / (32 * NW) : 0;
    if (tile < n) break;
    tile -= n;
  }
  const int len = a.cu[s + 1] - a.cu[s], c0 = a.ctx[s] - len;   // position of the portion's first token
  const int r_wg = tile * 32 * NW, r_wv = r_wg + 32 * wv, row = min(r_wv + qi, rows - 1);
  const int pos = c0 + row / a.R;
  const int p_first = c0 + min(r_wv, rows - 1) / a.R, p_last = c0 + min(r_wv + 31, rows - 1) / a.R;  // of this wave
  const int wg_first = c0 + r_wg / a.R, wg_last = c0 + min(r_wg + 32 * NW - 1, rows - 1) / a.R;
  const int kb0 = (a.window > 0 ? max(0, wg_first - a.window + 1) : 0) & ~31;
  const int lo = a.window > 0 ? pos - a.window + 1 : 0;
  const int lo_first = a.window > 0 ? p_first - a.window + 1 : 0, lo_last = a.window > 0 ? p_last - a.window + 1 : 0;
  const bool live = r_wv < rows;
  const int* bt = a.bt + (size_t)s * a.maxb;
  const int g = blockIdx.z, t = a.cu[s] + row / a.R, head = g * a.R + row % a.R;
  const bf16* qr = a.q + ((size_t)t * a.H + head) * DK + 8 * hb;
  bf16x8 qf[DK / 16];
#pragma unroll
  for (int i = 0; i < DK / 16; ++i) qf[i] = load8(qr + 16 * i);

  auto stage = [&](int buf, int kb) {
    char* kd = smem + buf * (KB + VB);
    char* vd = kd + KB;
    const int lp = wg_last >> 4, pg0 = bt[min(kb >> 4, lp)], pg1 = bt[min((kb >> 4) + 1, lp)];
#pragma unroll
    for (int i = wv; i < KI; i += NW) {
      const int slot = 64 * i + lane, r = slot / (DK / 8), ch = (slot % (DK / 8)) ^ k_swz<DK>(r);
      const bf16* src = a.kc + (((size_t)(r < 16 ? pg0 : pg1) * a.G + g) * 16 + (r & 15)) * DK + 8 * ch;
      __builtin_amdgcn_global_load_lds(src, GAI_LDS(kd + i * 1024), 16, 0, 0);
    }
#pragma unroll
    for (int i = wv; i < VI; i += NW) {
      const int slot = 64 * i + lane, pg = slot / (2 * DV), c = (slot % (2 * DV)) >> 1, hf = (slot & 1) ^ ((c >> 3) & 1);
      const bf16* src = a.vc + (((size_t)(pg ? pg1 : pg0) * a.G + g) * DV + c) * 16 + 8 * hf;
      __builtin_amdgcn_global_load_lds(src, GAI_LDS(vd + i * 1024), 16, 0, 0);
    }
  };
  f32x16 acc[DV / 32];
#pragma unroll
  for (int i = 0; i < DV / 32; ++i) acc[i] = f32x16{};
  float m = kOut, l = 0.f;
  const int kr = key_perm(qi), ksw = k_swz<DK>(kr);
  stage(0, kb0);
  asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
  __syncthreads();
  int buf = 0;
  for (int kb = kb0; kb <= wg_last; kb += 32, buf ^= 1) {
    if (kb + 32 <= wg_last) stage(buf ^ 1, kb + 32);
    if (live && kb <= p_last && kb + 31 >= lo_first) {
      const char* ks = smem + buf * (KB + VB) + kr * (DK * 2);
      const char* vs = smem + buf * (KB + VB) + KB;
      f32x16 sc = f32x16{};
#pragma unroll
      for (int i = 0; i < DK / 16; ++i)
        sc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(*reinterpret_cast<const bf16x8*>(ks + (((2 * i + hb) ^ ksw) << 4)), qf[i],
                                                     sc, 0, 0, 0);
      soft_block(sc, a.scale2, kb + 31 > p_first || kb < lo_last, kb, pos, lo, hb, m, l, acc);
#pragma unroll
      for (int k2 = 0; k2 < 2; ++k2) {
        bf16x8 ph, pl;
        split_weights(sc, k2, ph, pl);
#pragma unroll
        for (int i = 0; i < DV / 32; ++i) {
          const int c = 32 * i + qi;
          const bf16x8 vf = *reinterpret_cast<const bf16x8*>(vs + ((k2 * 2 * DV + 2 * c + (hb ^ ((c >> 3) & 1))) << 4));
          acc[i] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf, ph, acc[i], 0, 0, 0);
          acc[i] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf, pl, acc[i], 0, 0, 0);
        }
      }
    }
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();
  }
  l = half_sum(l);
  if (r_wv + qi >= rows) return;
  float f = 1.0f;
  if (a.sink) {
    const float sk = a.sink[head] * kL2e, mf = fmaxf(m, sk);
    f = __builtin_amdgcn_exp2f(m - mf);
    l = l * f + __builtin_amdgcn_exp2f(sk - mf);
  }
  f /= l;
  if (a.gate) f *= head_gate(a, t, head);
  bf16* o = a.out + (size_t)t * a.ldo + (size_t)head * DV;
#pragma unroll
  for (int i = 0; i < DV / 32; ++i)
#pragma unroll
    for (int r4 = 0; r4 < 4; ++r4) {
      bf16x4 y;
#pragma unroll
      for (int e = 0; e < 4; ++e) y[e] = (bf16)(acc[i][4 * r4 + e] * f);
      *reinterpret_cast<bf16x4*>(o + 32 * i + 8 * r4 + 4 * hb) = y;
    }
}

// blockIdx.z = kv head, blockIdx.x = sequence * tps + tile of 32 rows, blockIdx.y = share of the key blocks
template <int DK, int DV>
__global__ __launch_bounds__(64) void gqa_split_kernel(GqaArgs a) {
  const int lane = threadIdx.x, qi = lane & 31, hb = lane >> 5;
  const int s = blockIdx.x / a.tps, r0 = (blockIdx.x % a.tps) * 32;
  const int len = a.cu[s + 1] - a.cu[s], rows = len * a.R;
  if (rows >= kShortRows || rows > a.prow || r0 >= rows) return;
  const int c0 = a.ctx[s] - len, row = min(r0 + qi, rows - 1);
  const int pos = c0 + row / a.R, p_first = c0 + r0 / a.R, p_last = c0 + min(r0 + 31, rows - 1) / a.R;
  const int lo = a.window > 0 ? pos - a.window + 1 : 0, lo_last = a.window > 0 ? p_last - a.window + 1 : 0;
  int kb0 = (a.window > 0 ? max(0, p_first - a.window + 1) : 0) & ~31;
  const int nblk = (p_last - kb0) / 32 + 1, per = (nblk + a.nsplit - 1) / a.nsplit;
  kb0 += (int)blockIdx.y * per * 32;
  const int kb1 = min(p_last, kb0 + per * 32 - 1);
  const int* bt = a.bt + (size_t)s * a.maxb;
  const int g = blockIdx.z;
  float* po = a.part + (((size_t)blockIdx.y * a.S + s) * a.G + g) * a.prow * (DV + 4) + (size_t)row * (DV + 4);
  const bool mine = r0 + qi < rows;
  float m = kOut, l = 0.f;
  if (kb0 > kb1) return;  // no key block left for this share: the merge does not read it
  const bf16* qr = a.q + ((size_t)(a.cu[s] + row / a.R) * a.H + g * a.R + row % a.R) * DK + 8 * hb;
  bf16x8 qf[DK / 16];
#pragma unroll
  for (int i = 0; i < DK / 16; ++i) qf[i] = load8(qr + 16 * i);
  f32x16 acc[DV / 32];
#pragma unroll
  for (int i = 0; i < DV / 32; ++i) acc[i] = f32x16{};
  const int kr = key_perm(qi), lp = p_last >> 4;
  for (int kb = kb0; kb <= kb1; kb += 32) {
    const int pg[2] = {bt[kb >> 4], bt[min((kb >> 4) + 1, lp)]};
    const bf16* kp = a.kc + (((size_t)(kr < 16 ? pg[0] : pg[1]) * a.G + g) * 16 + (kr & 15)) * DK + 8 * hb;
    bf16x8 kf[DK / 16], vf[2][DV / 32];  // the values of the block are on their way while it is scored
#pragma unroll
    for (int i = 0; i < DK / 16; ++i) kf[i] = load8(kp + 16 * i);
#pragma unroll
    for (int k2 = 0; k2 < 2; ++k2)
#pragma unroll
      for (int i = 0; i < DV / 32; ++i) vf[k2][i] = load8(a.vc + (((size_t)pg[k2] * a.G + g) * DV + qi) * 16 + 8 * hb + 32 * i * 16);
    f32x16 sc = f32x16{};
#pragma unroll
    for (int i = 0; i < DK / 16; ++i) sc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(kf[i], qf[i], sc, 0, 0, 0);
    soft_block(sc, a.scale2, kb + 31 > p_first || kb < lo_last, kb, pos, lo, hb, m, l, acc);
#pragma unroll
    for (int k2 = 0; k2 < 2; ++k2) {
      bf16x8 ph, pl;
      split_weights(sc, k2, ph, pl);
#pragma unroll
      for (int i = 0; i < DV / 32; ++i) {
        acc[i] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf[k2][i], ph, acc[i], 0, 0, 0);
        acc[i] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf[k2][i], pl, acc[i], 0, 0, 0);
      }
    }
  }
  l = half_sum(l);
  if (!mine) return;
#pragma unroll
  for (int i = 0; i < DV / 32; ++i)
#pragma unroll
    for (int r4 = 0; r4 < 4; ++r4)
      *reinterpret_cast<float4*>(po + 32 * i + 8 * r4 + 4 * hb) =
          float4{acc[i][4 * r4], acc[i][4 * r4 + 1], acc[i][4 * r4 + 2], acc[i][4 * r4 + 3]};
  if (hb == 0) {
    po[DV] = m;
    po[DV + 1] = l;
  }
}

// one wave per row (blockIdx.x) of every short sequence (blockIdx.y), blockIdx.z = kv head
template <int DV>
__global__ __launch_bounds__(64) void gqa_merge_kernel(GqaArgs a) {
  __shared__ float wgt[kMaxSplit];
  const int s = blockIdx.y, row = blockIdx.x, lane = threadIdx.x;
  const int rows = (a.cu[s + 1] - a.cu[s]) * a.R;
  if (rows >= kShortRows || rows > a.prow || row >= rows) return;
  const int g = blockIdx.z, t = a.cu[s] + row / a.R, head = g * a.R + row % a.R;
  const float* p0 = a.part + (((size_t)s * a.G + g) * a.prow + row) * (DV + 4);
  const size_t step = (size_t)a.S * a.G * a.prow * (DV + 4);
  // the shares that held key blocks of this row's tile, as the key-split kernel dealt them out
  const int len = a.cu[s + 1] - a.cu[s], c0 = a.ctx[s] - len, r0 = row & ~31;
  const int k_lo = (a.window > 0 ? max(0, c0 + r0 / a.R - a.window + 1) : 0) & ~31;
  const int nblk = (c0 + min(r0 + 31, rows - 1) / a.R - k_lo) / 32 + 1, per = (nblk + a.nsplit - 1) / a.nsplit;
  const int used = (nblk + per - 1) / per;
  float m = kOut, l = 0.f;
  if (lane < used) {
    m = p0[lane * step + DV];
    l = p0[lane * step + DV + 1];
  }
  const float sk = a.sink ? a.sink[head] * kL2e : kOut;
  const float M = fmaxf(wave_max(m), sk);
  const float w = l > 0.f ? __builtin_amdgcn_exp2f(m - M) : 0.f;
  const float den = wave_sum(l * w) + (a.sink ? __builtin_amdgcn_exp2f(sk - M) : 0.f);
  if (lane < used) wgt[lane] = w / den * (a.gate ? head_gate(a, t, head) : 1.0f);
  __syncthreads();
  bf16* o = a.out + (size_t)t * a.ldo + (size_t)head * DV;
  for (int c = 4 * lane; c < DV; c += 256) {
    f32x4 y = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll 8
    for (int j = 0; j < used; ++j) y += wgt[j] * *reinterpret_cast<const f32x4*>(p0 + j * step + c);
    *reinterpret_cast<bf16x4*>(o + c) = bf16x4{(bf16)y[0], (bf16)y[1], (bf16)y[2], (bf16)y[3]};
  }
}

int tiles_per_seq(int T, int S, int R) { return T == S ? (R + 31) / 32 : kShortRows / 32; }

int split_count(int T, int S, int R, int G) {
  const long tiles = (long)S * G * ((T == S ? R + 31 : (T / S < 4 ? T / S * R + 31 : kShortRows)) / 32);
  const long n = 1024 / (tiles < 1 ? 1 : tiles);
  return n < 4 ? 4 : (n > kMaxSplit ? kMaxSplit : (int)n);
}

int part_rows(int T, int S, int R) { return T == S ? R : kShortRows; }

template <int DK, int DV>
void launch(const GqaArgs& a, hipStream_t st) {
  const long rows = (long)a.T * a.R;   // of one kv head
  if (a.T > a.S || a.R >= kShortRows) {
    constexpr size_t lds = 2 * 32 * (DK + DV) * 2;
    if (rows * a.G >= 256 * 256) {
      if (lds > 64 * 1024)
        (void)hipFuncSetAttribute(reinterpret_cast<const void*>(gqa_prefill_kernel<DK, DV, 8>),
                                  hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
      gqa_prefill_kernel<DK, DV, 8><<<dim3((int)(rows / 256) + a.S, 1, a.G), 512, lds, st>>>(a);
    } else {
      if (lds > 64 * 1024)
        (void)hipFuncSetAttribute(reinterpret_cast<const void*>(gqa_prefill_kernel<DK, DV, 4>),
                                  hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
      gqa_prefill_kernel<DK, DV, 4><<<dim3((int)(rows / 128) + a.S, 1, a.G), 256, lds, st>>>(a);
    }
  }
  if (a.R < kShortRows) {
    gqa_split_kernel<DK, DV><<<dim3(a.tps * a.S, a.nsplit, a.G), 64, 0, st>>>(a);
    gqa_merge_kernel<DV><<<dim3(a.prow, a.S, a.G), 64, 0, st>>>(a);
  }
}

}  // namespace

// 1: the key / value sizes have matrix-core kernels here
int gai_gqa_attention_ok(int DK, int DV) {
  return (DK == DV && (DK == 32 || DK == 64 || DK == 96 || DK == 128 || DK == 160 || DK == 192 || DK == 256)) ||
         (DK == 96 && DV == 64) || (DK == 192 && DV == 128) || (DK == 64 && DV == 128) || (DK == 128 && DV == 64);
}

size_t gai_gqa_attention_ws_floats(int T, int S, int H, int G, int DV) {
  const int R = H / G;
  return R < kShortRows && T > 0 && S > 0 ? (size_t)split_count(T, S, R, G) * S * G * part_rows(T, S, R) * (DV + 4) : 0;
}

void gai_gqa_attention(const void* q, const void* k_cache, const void* v_cache, const int* block_tables, int maxb,
                       const int* cu_q, const int* ctx, int S, void* out, int ldo, int T, int H, int G, int DK, int DV,
                       float scale, int window, const float* sink, const void* gate, int ldg, float* ws, hipStream_t st) {
  if (T == 0 || S == 0) return;
  if (G < 1 || H % G) gai_launch_error(__FILE__, __LINE__, "gqa_attention: heads must be a multiple of kv heads");
  if (ldo % 4) gai_launch_error(__FILE__, __LINE__, "gqa_attention: output rows on a grid of four elements");
  const int R = H / G;
  const GqaArgs a{(const bf16*)q, (const bf16*)k_cache, (const bf16*)v_cache, block_tables, cu_q, ctx, maxb, S, T, H, G, R,
                  scale * kL2e, window, sink, (const bf16*)gate, ldg, (bf16*)out, ldo, ws, split_count(T, S, R, G),
                  tiles_per_seq(T, S, R), part_rows(T, S, R)};
  if (R < kShortRows && !ws) gai_launch_error(__FILE__, __LINE__, "gqa_attention: scratch missing");
#define GAI_GQA(K_, V_) if (DK == K_ && DV == V_) { launch<K_, V_>(a, st); GAI_LAUNCH_CHECK(); return; }
  GAI_GQA(32, 32) GAI_GQA(64, 64) GAI_GQA(96, 96) GAI_GQA(128, 128) GAI_GQA(160, 160) GAI_GQA(192, 192) GAI_GQA(256, 256)
  GAI_GQA(96, 64) GAI_GQA(192, 128) GAI_GQA(64, 128) GAI_GQA(128, 64)
#undef GAI_GQA
  gai_launch_error(__FILE__, __LINE__, "gqa_attention: no kernel for these key / value sizes");
}
