// Matrix-memory LSTM (mLSTM) with exponential gates, fp32 states and gates.
//
//   i = cap tanh((ig + ib) / cap),  f = logsigmoid(cap tanh((fg + fb) / cap))            per head
//   m_t = max(f + m_(t-1), i)
//   S_t = e^(f + m_(t-1) - m_t) S_(t-1) + e^(i - m_t) k v^T,   n_t likewise with k alone
//   o   = S_t^T q / (max(|n_t . q|, e^(-m_t)) + den_eps),  q already times its scale
//   y   = o / rms_head(o) * norm_w * sigmoid(gate)
//
// mlstm_step_kernel: one workgroup per (sequence, head) for steps of single tokens: streams the state once, and the gates,
// the normaliser, the head norm and the output gate ride along.
//
// mlstm_chunk_kernel: portions. With F_t the sum of f over a chunk of 64 tokens up to t, m_0 the entry maximum and
// x_t = max(m_0, max_(s<=t)(i_s - F_s)), m_t = F_t + x_t, so the weight of token s in token t's sum is
// e^((i_s - F_s) - x_t) and that of the entry state e^(m_0 - x_t): F drops out of every exponent, and all exponents are <= 0.
// F, i - F and x are summed in fp64 and carried as pairs of floats. A workgroup owns one head (and up to 128 value
// columns) and walks its chunks: wave w owns 16 state columns for all key channels in accumulator registers of
// v_mfma_f32_16x16x4_f32 (exact fp32 products). An accumulator register holds row 4 (lane / 16) + r of its tile, which is
// the operand order of the next product with the contraction index permuted the same way on both sides, so the state, the
// values and the weighted scores go from one product to the next without shuffles:
//   scores  A[t, s] = (q_t . k_s) e^(...)  -> LDS (tiles on and below the diagonal),
//   outputs O = e^(m_0 - x) Q S + A V,   state S = e^(m_0 - x_63) S + K^T (w V).
// n is one more state column whose value is 1 for every token: the wave that owns it delivers n . q.
//
// Long portions of few sequences are cut into spans of a few chunks that run side by side: every span's own contribution
// (state from zero, entry maximum -inf), a carry pass over the spans of a sequence, then the outputs from each span's entry state.
#include "gai_common.h"
#include "gai_kernels.h"

using namespace gai;

namespace {

constexpr int kC = 64;            // tokens per chunk
constexpr int kMaxTiles = 9;      // 16-column tiles of a workgroup: 128 value columns + the normaliser's column
constexpr int kValCols = 128;
constexpr int kLdA = kC + 4;

struct MlstmArgs {
  const void *q, *k, *v, *gate;
  int ldq, ldk, ldv, ldgate;
  const float *ig, *fg;
  int ldi, ldf;
  const float *ib, *fb, *norm_w;
  float cap, q_scale, eps, den_eps;
  float *S, *n, *m;
  const int *cu, *slots;
  int nseq, H, DK, DV;
  void* y;            // [T, H * DV] activation dtype
  float* o;           // [T, H, DV] fp32: set when a head spans several workgroups (norm and gate run afterwards)
  float* ws_state;    // [spans, H, DK, DV + 1]
  float* ws_scal;     // [spans, H, 4]: own maximum, sum of f (high, low part), entry maximum
  int L;              // tokens per span (0: one workgroup walks a whole sequence)
};

__device__ __forceinline__ float soft_cap(float x, float cap) { return cap * tanhf(x / cap); }
__device__ __forceinline__ float log_sigmoid(float x) { return fminf(x, 0.f) - log1pf(expf(-fabsf(x))); }

// spans of a sequence / first span index: spans of all sequences are numbered one after the other
__device__ __forceinline__ int n_spans(int len, int L) { return (len + L - 1) / L; }

// ---------------------------------------------------------------------------------------------- single tokens
template <typename TA, int VEC>
__global__ __launch_bounds__(1024) void mlstm_step_kernel(MlstmArgs a) {
  extern __shared__ float sh[];  // q [DK] | k [DK] | red [RG][DV] | o [DV]
  __shared__ float scratch[16];
  const int h = blockIdx.x, s = blockIdx.y, tid = threadIdx.x, NT = blockDim.x;
  const int t = a.cu[s], DK = a.DK, DV = a.DV, H = a.H;
  if (a.cu[s + 1] <= t) return;
  const int slot = a.slots[s];
  const int CW = DV / VEC, RG = NT / CW;
  float* qs = sh;
  float* ks = qs + DK;
  float* red = ks + DK;
  float* os = red + RG * DV;
  const float mi = a.m[(size_t)slot * H + h];
  const float li = soft_cap(a.ig[(size_t)t * a.ldi + h] + a.ib[h], a.cap);
  const float lf = log_sigmoid(soft_cap(a.fg[(size_t)t * a.ldf + h] + a.fb[h], a.cap));
  const float mn = fmaxf(lf + mi, li);
  const float wf = expf(lf + mi - mn), wi = expf(li - mn);
  const TA* qr = (const TA*)a.q + (size_t)t * a.ldq + (size_t)h * DK;
  const TA* kr = (const TA*)a.k + (size_t)t * a.ldk + (size_t)h * DK;
  const TA* vr = (const TA*)a.v + (size_t)t * a.ldv + (size_t)h * DV;
  float* nr = a.n + ((size_t)slot * H + h) * DK;
  float nq = 0.f;
  for (int i = tid; i < DK; i += NT) {
    const float qv = (float)qr[i] * a.q_scale, kv = (float)kr[i] * wi;
    const float nv = fmaf(wf, nr[i], kv);
    qs[i] = qv;
    ks[i] = kv;
    nr[i] = nv;
    nq = fmaf(nv, qv, nq);
  }
  nq = block_sum(nq, scratch);  // its barriers also publish qs / ks
  float* Sr = a.S + ((size_t)slot * H + h) * DK * DV;
  const int cg = tid % CW, rg = tid / CW;
  float acc[VEC], vv[VEC];
#pragma unroll
  for (int e = 0; e < VEC; ++e) acc[e] = 0.f;
  if (rg < RG) {
#pragma unroll
    for (int e = 0; e < VEC; ++e) vv[e] = (float)vr[cg * VEC + e];
#pragma unroll 4
    for (int r = rg; r < DK; r += RG) {
      float* p = Sr + (size_t)r * DV + cg * VEC;
      const float kv = ks[r], qv = qs[r];
      if constexpr (VEC == 4) {
        float4 x = *reinterpret_cast<const float4*>(p);
        x.x = fmaf(wf, x.x, kv * vv[0]);
        x.y = fmaf(wf, x.y, kv * vv[1]);
        x.z = fmaf(wf, x.z, kv * vv[2]);
        x.w = fmaf(wf, x.w, kv * vv[3]);
        acc[0] = fmaf(qv, x.x, acc[0]);
        acc[1] = fmaf(qv, x.y, acc[1]);
        acc[2] = fmaf(qv, x.z, acc[2]);
        acc[3] = fmaf(qv, x.w, acc[3]);
        *reinterpret_cast<float4*>(p) = x;
      } else {
        const float x = fmaf(wf, *p, kv * vv[0]);
        acc[0] = fmaf(qv, x, acc[0]);
        *p = x;
      }
    }
#pragma unroll
    for (int e = 0; e < VEC; ++e) red[rg * DV + cg * VEC + e] = acc[e];
  }
  __syncthreads();
  const float inv_den = 1.0f / (fmaxf(fabsf(nq), expf(-mn)) + a.den_eps);
  float ss = 0.f;
  for (int c = tid; c < DV; c += NT) {
    float x = 0.f;
    for (int r = 0; r < RG; ++r) x += red[r * DV + c];
    x *= inv_den;
    os[c] = x;
    ss += x * x;
  }
  ss = block_sum(ss, scratch);
  const float inv = 1.0f / sqrtf(ss / DV + a.eps);
  const TA* gr = (const TA*)a.gate + (size_t)t * a.ldgate + (size_t)h * DV;
  TA* yr = (TA*)a.y + ((size_t)t * H + h) * DV;
  for (int c = tid; c < DV; c += NT) {
    const float g = 1.0f / (1.0f + expf(-(float)gr[c]));
    yr[c] = (TA)(os[c] * inv * a.norm_w[(size_t)h * DV + c] * g);
  }
  if (tid == 0) a.m[(size_t)slot * H + h] = mn;  // every thread read the old value before the barriers above
}

// ---------------------------------------------------------------------------------------------- portions
template <typename TA>
struct RowPad { static constexpr int v = 16 / sizeof(TA); };  // 16 bytes: rows shift by four LDS banks

template <typename TA>
__device__ __forceinline__ f32x4 lds4(const TA* p);
template <>
__device__ __forceinline__ f32x4 lds4<float>(const float* p) { return *reinterpret_cast<const f32x4*>(p); }
template <>
__device__ __forceinline__ f32x4 lds4<bf16>(const bf16* p) {
  const bf16x4 x = *reinterpret_cast<const bf16x4*>(p);
  return f32x4{(float)x[0], (float)x[1], (float)x[2], (float)x[3]};
}

// rows [0, kC) x DKP of a chunk into LDS, zeros past the valid rows and channels
template <typename TA, int DKP>
__device__ __forceinline__ void stage_rows(TA* __restrict__ dst, const TA* __restrict__ src, int ld, int nvalid, int DK,
                                           bool vec, int tid, int NT) {
  constexpr int LD = DKP + RowPad<TA>::v, E = 16 / sizeof(TA);
  if (vec) {
    for (int i = tid; i < kC * (DKP / E); i += NT) {
      const int row = i / (DKP / E), c = (i % (DKP / E)) * E;
      uint4 x = uint4{0, 0, 0, 0};
      if (row < nvalid && c < DK) x = *reinterpret_cast<const uint4*>(src + (size_t)row * ld + c);
      *reinterpret_cast<uint4*>(dst + row * LD + c) = x;
    }
  } else {
    for (int i = tid; i < kC * DKP; i += NT) {
      const int row = i / DKP, c = i % DKP;
      dst[row * LD + c] = (row < nvalid && c < DK) ? src[(size_t)row * ld + c] : (TA)0.f;
    }
  }
}

template <typename TA, int DT, bool OUT>
__global__ __launch_bounds__(64 * kMaxTiles) void mlstm_chunk_kernel(MlstmArgs a) {
  constexpr int DKP = (DT * 16 + 31) / 32 * 32, LD = DKP + RowPad<TA>::v;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  TA* Ks = reinterpret_cast<TA*>(smem);
  TA* Qs = Ks + kC * LD;                                        // (OUT only)
  float* As = reinterpret_cast<float*>(Qs + (OUT ? kC * LD : 0));  // weighted scores [kC][kLdA] (OUT only)
  float* gh = As + (OUT ? kC * kLdA : 0);                       // i - F as a float pair
  float* gl = gh + kC;
  float* xh = gl + kC;                                          // x_t as a float pair
  float* xl = xh + kC;
  float* gam = xl + kC;                                         // e^(m_0 - x_t) * q_scale
  float* wst = gam + kC;                                        // e^(i_s - F_s - x_63)
  float* emm = wst + kC;                                        // e^(-m_t)
  float* nqs = emm + kC;                                        // n_t . q_t
  float* scal = nqs + kC;                                       // [0] decay of the state, [1] m after the chunk
  float* ssq = scal + 4;                                        // [tiles][kC] partial sums of o^2
  const int tid = threadIdx.x, NT = blockDim.x, wv = tid >> 6, lane = tid & 63, col = lane & 15, g = lane >> 4;
  const int h = blockIdx.y, H = a.H, DK = a.DK, DV = a.DV;
  const int NW = NT >> 6;
  // ---- which (sequence, token range)?
  int s = 0, len = 0, j = 0, nsp = 1;
  if (a.L == 0) {
    s = blockIdx.x;
    len = a.cu[s + 1] - a.cu[s];
  } else {
    int seen = 0;
    for (; s < a.nseq; ++s) {
      len = a.cu[s + 1] - a.cu[s];
      nsp = n_spans(len, a.L);
      if ((int)blockIdx.x < seen + nsp) break;
      seen += nsp;
    }
    if (s == a.nseq) return;
    j = (int)blockIdx.x - seen;
  }
  if (len <= 0) return;
  const int t0 = a.cu[s] + j * a.L, cnt = a.L ? min(a.L, len - j * a.L) : len;
  const bool last_span = j == nsp - 1;
  const int slot = a.slots[s];
  const int vc0 = (int)blockIdx.z * kValCols, nv = min(kValCols, DV - vc0);
  const int c = 16 * wv + col;                                   // column within the workgroup; c == nv: the normaliser
  const bool is_val = c < nv, is_n = c == nv;
  const TA* q = (const TA*)a.q + (size_t)t0 * a.ldq + (size_t)h * DK;
  const TA* k = (const TA*)a.k + (size_t)t0 * a.ldk + (size_t)h * DK;
  // row 16 b + 4 g + r of a per-token array: a uniform row pointer plus one 32-bit lane offset per array
  const TA* v = (const TA*)a.v + (size_t)t0 * a.ldv + (size_t)h * DV + vc0;
  const unsigned v_off = (unsigned)(4 * g * a.ldv + c);
  constexpr int E = 16 / sizeof(TA);
  const bool vec = DK % E == 0 && a.ldq % E == 0 && a.ldk % E == 0 && ((size_t)a.q & 15) == 0 && ((size_t)a.k & 15) == 0;
  // ---- entry state: the pool's (whole sequence), the span's from the carry pass, or nothing (a span's own part)
  f32x4 S[DT];
  float m0 = -INFINITY;
  double Fsum = 0.0;
  float* wsS = a.ws_state + ((size_t)blockIdx.x * H + h) * DK * (DV + 1);
  float* wsc = a.ws_scal + ((size_t)blockIdx.x * H + h) * 4;
  float* poolS = a.S + ((size_t)slot * H + h) * DK * DV;
  float* pooln = a.n + ((size_t)slot * H + h) * DK;
#pragma unroll
  for (int b = 0; b < DT; ++b) {
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int kk = 16 * b + 4 * g + r;
      float x = 0.f;
      if (OUT && kk < DK) {
        if (a.L) {
          if (is_val) x = wsS[(size_t)kk * (DV + 1) + vc0 + c];
          else if (is_n) x = wsS[(size_t)kk * (DV + 1) + DV];
        } else {
          if (is_val) x = poolS[(size_t)kk * DV + vc0 + c];
          else if (is_n) x = pooln[kk];
        }
      }
      S[b][r] = x;
    }
  }
  if (OUT) m0 = a.L ? wsc[3] : a.m[(size_t)slot * H + h];

  for (int cb = 0; cb < cnt; cb += kC) {
    const int nvalid = min(kC, cnt - cb);  // rows past it: zero q, k, v and weights
    // ---- stage q, k; the values of this wave's column straight into operand registers; gates by wave 0
    if (OUT) stage_rows<TA, DKP>(Qs, q + (size_t)cb * a.ldq, a.ldq, nvalid, DK, vec, tid, NT);
    stage_rows<TA, DKP>(Ks, k + (size_t)cb * a.ldk, a.ldk, nvalid, DK, vec, tid, NT);
    f32x4 V[4];
#pragma unroll
    for (int b = 0; b < 4; ++b)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int tt = 16 * b + 4 * g + r;
        float x = 0.f;
        if (tt < nvalid) {
          if (is_val) x = (float)(v + (size_t)(cb + 16 * b + r) * a.ldv)[v_off];
          else if (is_n) x = 1.f;
        }
        V[b][r] = x;
      }
    if (wv == 0) {
      const bool ok = lane < nvalid;
      const size_t t = (size_t)t0 + cb + (ok ? lane : 0);
      const float li = soft_cap(a.ig[t * a.ldi + h] + a.ib[h], a.cap);
      const float lf = log_sigmoid(soft_cap(a.fg[t * a.ldf + h] + a.fb[h], a.cap));
      double F = ok ? (double)lf : 0.0;
#pragma unroll
      for (int o = 1; o < 64; o <<= 1) {
        const double y = __shfl_up(F, o, 64);
        if (lane >= o) F += y;
      }
      const double gs = ok ? (double)li - F : -INFINITY;
      double x = fmax(gs, (double)m0);
#pragma unroll
      for (int o = 1; o < 64; o <<= 1) {
        const double y = __shfl_up(x, o, 64);
        if (lane >= o) x = fmax(x, y);
      }
      const double xe = __shfl(x, 63, 64), Fe = __shfl(F, 63, 64);
      const float g_hi = (float)gs, x_hi = (float)x;
      gh[lane] = g_hi;
      gl[lane] = ok ? (float)(gs - (double)g_hi) : 0.f;
      xh[lane] = x_hi;
      xl[lane] = (float)(x - (double)x_hi);
      gam[lane] = expf((float)((double)m0 - x)) * a.q_scale;
      wst[lane] = ok ? expf((float)(gs - xe)) : 0.f;
      emm[lane] = expf(-(float)(F + x));
      if (lane == 0) {
        scal[0] = expf((float)((double)m0 - xe));
        scal[1] = (float)(Fe + xe);
      }
      Fsum += Fe;
    }
    __syncthreads();
    f32x4 acc[4];
    if (OUT) {
      // ---- weighted scores: 16 x 16 tiles on and below the diagonal, dealt out to the waves
      for (int id = wv; id < 10; id += NW) {
        int rt = 0;
        while ((rt + 1) * (rt + 2) / 2 <= id) ++rt;
        const int ct = id - rt * (rt + 1) / 2;
        f32x4 d = f32x4{0.f, 0.f, 0.f, 0.f};
        if constexpr (sizeof(TA) == 2) {  // bf16 products are exact in the fp32 accumulator
          const bf16* qa = (const bf16*)Qs + (16 * rt + col) * LD + 8 * g;
          const bf16* kb = (const bf16*)Ks + (16 * ct + col) * LD + 8 * g;
#pragma unroll
          for (int b = 0; b < DKP / 32; ++b)
            d = __builtin_amdgcn_mfma_f32_16x16x32_bf16(load8(qa + 32 * b), load8(kb + 32 * b), d, 0, 0, 0);
        } else {
          const TA* qa = Qs + (16 * rt + col) * LD + 4 * g;
          const TA* kb = Ks + (16 * ct + col) * LD + 4 * g;
#pragma unroll
          for (int b = 0; b < DT; ++b) {
            const f32x4 x = lds4<TA>(qa + 16 * b), y = lds4<TA>(kb + 16 * b);
#pragma unroll
            for (int r = 0; r < 4; ++r) d = __builtin_amdgcn_mfma_f32_16x16x4f32(x[r], y[r], d, 0, 0, 0);
          }
        }
        const int sk = 16 * ct + col;
        const float kh = gh[sk], kl = gl[sk];
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int tq = 16 * rt + 4 * g + r;
          const float e = expf(fminf((kh - xh[tq]) + (kl - xl[tq]), 0.f));
          As[tq * kLdA + sk] = sk <= tq ? d[r] * a.q_scale * e : 0.f;
        }
      }
      // ---- the entry state's part of the outputs
#pragma unroll
      for (int rt = 0; rt < 4; ++rt) acc[rt] = f32x4{0.f, 0.f, 0.f, 0.f};
      const TA* qa = Qs + col * LD + 4 * g;
#pragma unroll
      for (int b = 0; b < DT; ++b) {
        f32x4 x[4];
#pragma unroll
        for (int rt = 0; rt < 4; ++rt)
          x[rt] = lds4<TA>(qa + 16 * rt * LD + 16 * b);
#pragma unroll
        for (int r = 0; r < 4; ++r)
#pragma unroll
          for (int rt = 0; rt < 4; ++rt)
            acc[rt] = __builtin_amdgcn_mfma_f32_16x16x4f32(x[rt][r], S[b][r], acc[rt], 0, 0, 0);
      }
#pragma unroll
      for (int rt = 0; rt < 4; ++rt) acc[rt] *= *reinterpret_cast<const f32x4*>(gam + 16 * rt + 4 * g);
      __syncthreads();
      // ---- the chunk's own part
#pragma unroll
      for (int b = 0; b < 4; ++b) {
        f32x4 x[4];
#pragma unroll
        for (int rt = b; rt < 4; ++rt) x[rt] = *reinterpret_cast<const f32x4*>(As + (16 * rt + col) * kLdA + 16 * b + 4 * g);
#pragma unroll
        for (int r = 0; r < 4; ++r)
#pragma unroll
          for (int rt = b; rt < 4; ++rt) acc[rt] = __builtin_amdgcn_mfma_f32_16x16x4f32(x[rt][r], V[b][r], acc[rt], 0, 0, 0);
      }
      if (is_n) {
#pragma unroll
        for (int rt = 0; rt < 4; ++rt)
          *reinterpret_cast<f32x4*>(nqs + 16 * rt + 4 * g) = acc[rt];
      }
    }
    // ---- state after the chunk
    const float dec = scal[0];
    m0 = scal[1];
#pragma unroll
    for (int b = 0; b < DT; ++b) S[b] *= dec;
    const TA* ka = Ks + 4 * g * LD + col;
#pragma unroll
    for (int b = 0; b < 4; ++b) {
      const f32x4 wvv = V[b] * *reinterpret_cast<const f32x4*>(wst + 16 * b + 4 * g);
#pragma unroll
      for (int r = 0; r < 4; ++r)
#pragma unroll
        for (int d = 0; d < DT; ++d)
          S[d] = __builtin_amdgcn_mfma_f32_16x16x4f32((float)ka[(16 * b + r) * LD + 16 * d], wvv[r], S[d], 0, 0, 0);
    }
    __syncthreads();  // n . q is there; q, k, scores and gates may be overwritten
    if (OUT) {
#pragma unroll
      for (int rt = 0; rt < 4; ++rt) {
        const f32x4 nq = *reinterpret_cast<const f32x4*>(nqs + 16 * rt + 4 * g);
        const f32x4 em = *reinterpret_cast<const f32x4*>(emm + 16 * rt + 4 * g);
#pragma unroll
        for (int r = 0; r < 4; ++r) acc[rt][r] = is_val ? acc[rt][r] / (fmaxf(fabsf(nq[r]), em[r]) + a.den_eps) : 0.f;
      }
      if (a.o) {
        float* o = a.o + ((size_t)(t0 + cb) * H + h) * DV + vc0;
        const unsigned o_off = (unsigned)(4 * g * H * DV + c);
        if (is_val) {
#pragma unroll
          for (int rt = 0; rt < 4; ++rt)
#pragma unroll
            for (int r = 0; r < 4; ++r)
              if (16 * rt + 4 * g + r < nvalid) (o + (size_t)(16 * rt + r) * H * DV)[o_off] = acc[rt][r];
        }
        __syncthreads();  // emm / nqs are rewritten by the next chunk
      } else {
        // head norm over the workgroup's columns, weight, output gate
#pragma unroll
        for (int rt = 0; rt < 4; ++rt) {
          f32x4 p = acc[rt] * acc[rt];
#pragma unroll
          for (int r = 0; r < 4; ++r) p[r] = group_sum<16>(p[r]);
          if (col == 0) *reinterpret_cast<f32x4*>(ssq + wv * kC + 16 * rt + 4 * g) = p;
        }
        __syncthreads();
        for (int i = tid; i < kC; i += NT) {
          float x = 0.f;
          for (int w = 0; w < NW; ++w) x += ssq[w * kC + i];
          emm[i] = 1.0f / sqrtf(x / DV + a.eps);
        }
        __syncthreads();
        if (is_val) {
          const float nw = a.norm_w[(size_t)h * DV + c];
          const TA* gr = (const TA*)a.gate + (size_t)(t0 + cb) * a.ldgate + (size_t)h * DV;
          TA* y = (TA*)a.y + ((size_t)(t0 + cb) * H + h) * DV;
          const unsigned g_off = (unsigned)(4 * g * a.ldgate + c), y_off = (unsigned)(4 * g * H * DV + c);
#pragma unroll
          for (int rt = 0; rt < 4; ++rt) {
            const f32x4 inv = *reinterpret_cast<const f32x4*>(emm + 16 * rt + 4 * g);
#pragma unroll
            for (int r = 0; r < 4; ++r) {
              if (16 * rt + 4 * g + r < nvalid) {
                const float gv = (float)(gr + (size_t)(16 * rt + r) * a.ldgate)[g_off];
                (y + (size_t)(16 * rt + r) * H * DV)[y_off] = (TA)(acc[rt][r] * inv[r] * nw / (1.0f + expf(-gv)));
              }
            }
          }
        }
        __syncthreads();  // emm is rewritten by the next chunk
      }
    }
  }
  // ---- final state: a span's own part -> scratch; a whole sequence's or its last span's -> the pool
  if (!OUT || last_span) {
#pragma unroll
    for (int b = 0; b < DT; ++b) {
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int kk = 16 * b + 4 * g + r;
        if (kk < DK) {
          if (!OUT) {
            if (is_val) wsS[(size_t)kk * (DV + 1) + vc0 + c] = S[b][r];
            else if (is_n && blockIdx.z == 0) wsS[(size_t)kk * (DV + 1) + DV] = S[b][r];
          } else {
            if (is_val) poolS[(size_t)kk * DV + vc0 + c] = S[b][r];
            else if (is_n && blockIdx.z == 0) pooln[kk] = S[b][r];
          }
        }
      }
    }
    if (tid == 0 && blockIdx.z == 0) {
      if (OUT) {
        a.m[(size_t)slot * H + h] = m0;
      } else {
        wsc[0] = m0;
        wsc[1] = (float)Fsum;
        wsc[2] = (float)(Fsum - (double)(float)Fsum);
      }
    }
  }
}

// Walk the spans of a sequence: replace every span's own part by its entry state (and leave its entry maximum)
__global__ __launch_bounds__(256) void mlstm_carry_kernel(MlstmArgs a) {
  const int s = blockIdx.z, h = blockIdx.y, H = a.H, DK = a.DK, DV = a.DV, W = DV + 1;
  const int e = blockIdx.x * 256 + threadIdx.x;
  if (e >= DK * W) return;
  int first = 0;
  for (int i = 0; i < s; ++i) first += n_spans(a.cu[i + 1] - a.cu[i], a.L);
  const int nsp = n_spans(a.cu[s + 1] - a.cu[s], a.L);
  const int slot = a.slots[s], kk = e / W, c = e - kk * W;
  float x = c < DV ? a.S[(((size_t)slot * H + h) * DK + kk) * DV + c] : a.n[((size_t)slot * H + h) * DK + kk];
  float m = a.m[(size_t)slot * H + h];
  for (int j = 0; j < nsp; ++j) {
    const size_t b = (size_t)(first + j) * H + h;
    float* p = a.ws_state + b * DK * W + e;
    float* sc = a.ws_scal + b * 4;
    const float own = *p;
    *p = x;
    if (e == 0) sc[3] = m;
    const double in = (double)sc[1] + (double)sc[2] + (double)m;
    const double mn = fmax(in, (double)sc[0]);
    x = x * expf((float)(in - mn)) + own * expf((float)((double)sc[0] - mn));
    m = (float)mn;
  }
}

template <typename F>
void big_lds(F f, size_t bytes) {
  if (bytes > 64 * 1024)
    (void)hipFuncSetAttribute(reinterpret_cast<const void*>(f), hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
}

template <typename TA, int DT, bool OUT>
void launch_chunk(const MlstmArgs& a, dim3 grid, int tiles, hipStream_t st) {
  constexpr int DKP = (DT * 16 + 31) / 32 * 32, LD = DKP + RowPad<TA>::v;
  const size_t lds = (size_t)kC * LD * sizeof(TA) * (OUT ? 2 : 1) +
                     ((OUT ? kC * kLdA : 0) + 8 * kC + 4 + (OUT ? tiles * kC : 0)) * sizeof(float);
  big_lds(mlstm_chunk_kernel<TA, DT, OUT>, lds);
  mlstm_chunk_kernel<TA, DT, OUT><<<grid, 64 * tiles, lds, st>>>(a);
}

template <typename TA, int DT>
void launch_portions(const MlstmArgs& a, int spans, hipStream_t st) {
  const int zb = (a.DV + kValCols - 1) / kValCols, nv = a.DV < kValCols ? a.DV : kValCols;
  const int tiles = nv / 16 + 1;  // value columns + the normaliser's
  if (!a.L) {
    launch_chunk<TA, DT, true>(a, dim3(a.nseq, a.H, zb), tiles, st);
    return;
  }
  const dim3 grid(spans, a.H, zb);
  launch_chunk<TA, DT, false>(a, grid, tiles, st);
  mlstm_carry_kernel<<<dim3((a.DK * (a.DV + 1) + 255) / 256, a.H, a.nseq), 256, 0, st>>>(a);
  launch_chunk<TA, DT, true>(a, grid, tiles, st);
}

// tokens per span of a step with portions; 0: every sequence is walked by one workgroup per head
int span_tokens(int T, int S, int H, int DV) {
  const int zb = (DV + kValCols - 1) / kValCols;
  if (zb == 1 && ((long)S * H >= 512 || T / S < 2 * kC)) return 0;
  long L = (long)T * H * zb / 512 / kC * kC;
  return (int)(L < kC ? kC : (L > 4 * kC ? 4 * kC : L));
}

}  // namespace

size_t gai_mlstm_ws_floats(int T, int S, int H, int DK, int DV) {
  if (T <= S || S < 1) return 0;
  const int L = span_tokens(T, S, H, DV);
  const size_t spans = L ? (size_t)T / L + S : 0;
  return spans * H * ((size_t)DK * (DV + 1) + 4) + (DV > kValCols ? (size_t)T * H * DV : 0);
}

void gai_mlstm(const void* q, int ldq, const void* k, int ldk, const void* v, int ldv, const float* ig, int ldi,
               const float* fg, int ldf, const float* ib, const float* fb, float cap, const void* gate, int ldgate,
               const float* norm_w, float* S, float* n, float* m, const int* cu, const int* slots, int nseq, int T, int H,
               int DK, int DV, float q_scale, float eps, float den_eps, void* y, float* ws, int dt, hipStream_t st) {
  if (T == 0 || nseq == 0) return;
  if (DK < 1 || DK > 256 || DV < 1) gai_launch_error(__FILE__, __LINE__, "mlstm: key sizes 1 .. 256");
  if (!(cap > 0.f)) gai_launch_error(__FILE__, __LINE__, "mlstm: the gate cap must be positive");
  MlstmArgs a{q, k, v, gate, ldq, ldk, ldv, ldgate, ig, fg, ldi, ldf, ib, fb, norm_w, cap, q_scale, eps, den_eps,
              S, n, m, cu, slots, nseq, H, DK, DV, y, nullptr, nullptr, nullptr, 0};
  if (T <= nseq) {  // single tokens
    const int vec = DV % 4 == 0 ? 4 : 1, CW = DV / vec;
    if (CW > 1024) gai_launch_error(__FILE__, __LINE__, "mlstm: value size above 4096 (1024 off the grid of four)");
    int NT = (long)nseq * H >= 512 ? 256 : 1024;
    while (NT < CW) NT *= 2;
    const size_t lds = ((size_t)2 * DK + (size_t)(NT / CW) * DV + DV) * sizeof(float);
    const dim3 grid(H, nseq);
#define GAI_STEP(TA)                                                             \
  if (vec == 4) mlstm_step_kernel<TA, 4><<<grid, NT, lds, st>>>(a);              \
  else mlstm_step_kernel<TA, 1><<<grid, NT, lds, st>>>(a)
    if (dt) { GAI_STEP(float); } else { GAI_STEP(bf16); }
#undef GAI_STEP
    GAI_LAUNCH_CHECK();
    return;
  }
  a.L = span_tokens(T, nseq, H, DV);
  const int spans = a.L ? T / a.L + nseq : 0;
  if (gai_mlstm_ws_floats(T, nseq, H, DK, DV) && !ws) gai_launch_error(__FILE__, __LINE__, "mlstm: scratch missing");
  if (a.L) {
    a.ws_state = ws;
    a.ws_scal = ws + (size_t)spans * H * DK * (DV + 1);
  }
  if (DV > kValCols) a.o = ws + (size_t)spans * H * ((size_t)DK * (DV + 1) + 4);
#define GAI_PORTIONS(TA)                                      \
  do {                                                        \
    if (DK <= 16) launch_portions<TA, 1>(a, spans, st);       \
    else if (DK <= 32) launch_portions<TA, 2>(a, spans, st);  \
    else if (DK <= 64) launch_portions<TA, 4>(a, spans, st);  \
    else if (DK <= 128) launch_portions<TA, 8>(a, spans, st); \
    else launch_portions<TA, 16>(a, spans, st);               \
  } while (0)
  if (dt) GAI_PORTIONS(float); else GAI_PORTIONS(bf16);
#undef GAI_PORTIONS
  GAI_LAUNCH_CHECK();
  if (a.o) gai_head_norm_gate(a.o, gate, ldgate, norm_w, 1, 1, y, H * DV, T, H, DV, eps, dt, st);
}
