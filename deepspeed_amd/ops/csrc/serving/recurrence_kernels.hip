// Recurrences over ragged batches for MI355X (gfx950): the block-diagonal
// gates of a real-gated linear recurrent unit, the scan of a recurrence with
// one state per channel, and the chunked form of a matrix-state recurrence
// with one fixed decay per head.
//
// Plain C ABI (raw device pointers + a hipStream_t) so the library builds in
// seconds with hipcc alone and is loaded through ctypes. dtype codes:
// 0 = float, 1 = bfloat16. Gates, decays, step factors and the state are float
// whatever the storage type.

#include "serving_common.h"

namespace {

typedef __attribute__((ext_vector_type(8))) short short8;
typedef __attribute__((ext_vector_type(4))) float floatx4;

constexpr float LOG2E = 1.4426950408889634f;

// EXACT: libm exponentials (32-bit serving); otherwise the hardware's exp2 and
// reciprocal (relative error below 1e-6 over the range that matters)
template <bool EXACT>
__device__ __forceinline__ float exp_(float x) {
  return EXACT ? expf(x) : __builtin_amdgcn_exp2f(x * LOG2E);
}
template <bool EXACT>
__device__ __forceinline__ float sigmoid_(float x) {
  return EXACT ? 1.f / (1.f + expf(-x))
               : __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(-x * LOG2E));
}
__device__ __forceinline__ float softplus_(float x) {
  return x > 20.f ? x : log1pf(expf(x));
}
// (r, i pre-activations with bias) -> a and b of S <- a S + b. 1 - a^2 is
// 1 - exp(y) with y = 2 log a <= 0; where that would cancel, the series.
template <bool EXACT>
__device__ __forceinline__ void rglru_pair(float zr, float zi, float u, float rate, float& a,
                                           float& b) {
  const float la = -sigmoid_<EXACT>(zr) * rate;  // rate = c * softplus(lam)
  a = exp_<EXACT>(la);
  const float y = 2.f * la;
  float m;
  if (EXACT) {
    m = -expm1f(y);
  } else {
    const float series =
        -y * (1.f + y * (1.f / 2) *
                        (1.f + y * (1.f / 3) *
                                   (1.f + y * (1.f / 4) *
                                              (1.f + y * (1.f / 5) * (1.f + y * (1.f / 6))))));
    m = y > -0.25f ? series : 1.f - a * a;
  }
  b = (EXACT ? sqrtf(m) : __builtin_amdgcn_sqrtf(m)) * (sigmoid_<EXACT>(zi) * u);
}

// Gates from finished products: zr, zi [blocks, T, n] float (no bias yet).
template <typename T>
__global__ void rglru_pair_k(const float* __restrict__ zr, const float* __restrict__ zi,
                             const T* __restrict__ u, const float* __restrict__ br,
                             const float* __restrict__ bi, const float* __restrict__ lam,
                             float* __restrict__ a, float* __restrict__ b, int Ttok, int blocks,
                             int n, float c) {
  const int W = blocks * n;
  const int64_t total = (int64_t)Ttok * W;
  for (int64_t i = blockIdx.x * (int64_t)blockDim.x + threadIdx.x; i < total;
       i += (int64_t)gridDim.x * blockDim.x) {
    const int64_t t = i / W;
    const int ch = (int)(i - t * W);
    const int blk = ch / n;
    const int64_t z = ((int64_t)blk * Ttok + t) * n + (ch - blk * n);
    float av, bv;
    rglru_pair<true>(zr[z] + br[ch], zi[z] + bi[ch], ld(u + i), c * softplus_(lam[ch]), av, bv);
    a[i] = av;
    b[i] = bv;
  }
}

// Both block-diagonal products and the gates in one pass, 16-bit operands:
// a workgroup of 256 threads owns 16*WM tokens x 16*WN*NN outputs of one
// block (WM * WN = 4 waves) and walks the block's n inputs KC at a time
// through LDS; a wave keeps NN accumulator tiles of 16x16 per gate. Both
// operands are K-contiguous, so tiles are staged as they lie in memory.
constexpr int GK = 64;        // inputs per staged step
constexpr int GKP = GK + 8;   // padded LDS row: 16-byte aligned, spread banks

template <int WM, int WN, int NN>
__global__ __launch_bounds__(NT) void rglru_gates_mfma_k(
    const bf16* __restrict__ u, const bf16* __restrict__ wr, const bf16* __restrict__ wi,
    const float* __restrict__ br, const float* __restrict__ bi, const float* __restrict__ lam,
    float* __restrict__ a, float* __restrict__ b, int Ttok, int n, int W, float c) {
  constexpr int TM = 16 * WM, TN = 16 * WN * NN, ZP = TN + 4;
  constexpr int LDS_IN = (TM + 2 * TN) * GKP * 2, LDS_OUT = 2 * TM * ZP * 4;
  __shared__ __attribute__((aligned(16))) char smem[LDS_IN > LDS_OUT ? LDS_IN : LDS_OUT];
  short* sU = reinterpret_cast<short*>(smem);  // [TM][GKP]
  short* sR = sU + TM * GKP;                   // [TN][GKP]
  short* sI = sR + TN * GKP;                   // [TN][GKP]
  const int t0 = blockIdx.x * TM, blk = blockIdx.y, o0 = blockIdx.z * TN;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int wm = wave % WM, wn = wave / WM;
  const int l15 = lane & 15, quad = lane >> 4;
  const short* ub = reinterpret_cast<const short*>(u) + blk * n;
  const short* rb = reinterpret_cast<const short*>(wr) + (int64_t)blk * n * n;
  const short* ib = reinterpret_cast<const short*>(wi) + (int64_t)blk * n * n;
  const bool vec = (n & 7) == 0;  // rows start 16-byte aligned

  constexpr int G8 = GK / 8;
  constexpr int UPT = (TM * G8 + NT - 1) / NT, WPT = (TN * G8 + NT - 1) / NT;
  short8 pu[UPT], pr[WPT], pi[WPT];
  auto get = [&](const short* row, int k, bool in) {
    short8 x = {0, 0, 0, 0, 0, 0, 0, 0};
    if (in) {
      if (vec) {
        if (k < n) x = *reinterpret_cast<const short8*>(row + k);
      } else {
#pragma unroll
        for (int e = 0; e < 8; ++e)
          if (k + e < n) x[e] = row[k + e];
      }
    }
    return x;
  };
  auto fetch = [&](int k0) {
#pragma unroll
    for (int i = 0; i < UPT; ++i) {
      const int f = threadIdx.x + i * NT;
      const int r = f / G8, k = k0 + (f % G8) * 8;
      pu[i] = get(ub + (int64_t)(t0 + r) * W, k, r < TM && t0 + r < Ttok);
    }
#pragma unroll
    for (int i = 0; i < WPT; ++i) {
      const int f = threadIdx.x + i * NT;
      const int r = f / G8, k = k0 + (f % G8) * 8;
      const bool in = r < TN && o0 + r < n;
      pr[i] = get(rb + (int64_t)(o0 + r) * n, k, in);
      pi[i] = get(ib + (int64_t)(o0 + r) * n, k, in);
    }
  };
  auto stash = [&]() {
#pragma unroll
    for (int i = 0; i < UPT; ++i) {
      const int f = threadIdx.x + i * NT;
      const int r = f / G8, k = (f % G8) * 8;
      if (r < TM) *reinterpret_cast<short8*>(&sU[r * GKP + k]) = pu[i];
    }
#pragma unroll
    for (int i = 0; i < WPT; ++i) {
      const int f = threadIdx.x + i * NT;
      const int r = f / G8, k = (f % G8) * 8;
      if (r < TN) {
        *reinterpret_cast<short8*>(&sR[r * GKP + k]) = pr[i];
        *reinterpret_cast<short8*>(&sI[r * GKP + k]) = pi[i];
      }
    }
  };
  floatx4 ar[NN], ai[NN];
#pragma unroll
  for (int j = 0; j < NN; ++j) {
    ar[j] = (floatx4){0.f, 0.f, 0.f, 0.f};
    ai[j] = (floatx4){0.f, 0.f, 0.f, 0.f};
  }
  fetch(0);
  for (int k0 = 0; k0 < n; k0 += GK) {
    stash();
    __syncthreads();
    if (k0 + GK < n) fetch(k0 + GK);
#pragma unroll
    for (int kk = 0; kk < GK; kk += 32) {
      const short8 fa =
          *reinterpret_cast<const short8*>(&sU[(wm * 16 + l15) * GKP + kk + quad * 8]);
#pragma unroll
      for (int j = 0; j < NN; ++j) {
        const int o = ((wn * NN + j) * 16 + l15) * GKP + kk + quad * 8;
        const short8 fr = *reinterpret_cast<const short8*>(&sR[o]);
        const short8 fi = *reinterpret_cast<const short8*>(&sI[o]);
        ar[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
            __builtin_bit_cast(__attribute__((ext_vector_type(8))) __bf16, fa),
            __builtin_bit_cast(__attribute__((ext_vector_type(8))) __bf16, fr), ar[j], 0, 0, 0);
        ai[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
            __builtin_bit_cast(__attribute__((ext_vector_type(8))) __bf16, fa),
            __builtin_bit_cast(__attribute__((ext_vector_type(8))) __bf16, fi), ai[j], 0, 0, 0);
      }
    }
    __syncthreads();
  }
  if (TN == 64 && (n & 3) == 0) {
    // the products go through LDS once more, so that a thread finishes four
    // neighbouring channels and whole 16-byte groups are stored
    float* zr = reinterpret_cast<float*>(smem);  // [TM][ZP]
    float* zi = zr + TM * ZP;
#pragma unroll
    for (int j = 0; j < NN; ++j)
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int at = (wm * 16 + quad * 4 + e) * ZP + (wn * NN + j) * 16 + l15;
        zr[at] = ar[j][e];
        zi[at] = ai[j][e];
      }
    __syncthreads();
    const int o4 = (threadIdx.x & 15) * 4;
    if (o0 + o4 >= n) return;
    const int ch = blk * n + o0 + o4;
    float rate[4], cr[4], ci[4];
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      rate[e] = c * softplus_(lam[ch + e]);
      cr[e] = br[ch + e];
      ci[e] = bi[ch + e];
    }
#pragma unroll
    for (int r = threadIdx.x >> 4; r < TM; r += NT / 16) {
      const int64_t t = t0 + r;
      if (t >= Ttok) break;
      const float4 xr = *reinterpret_cast<const float4*>(zr + r * ZP + o4);
      const float4 xi = *reinterpret_cast<const float4*>(zi + r * ZP + o4);
      const uint2 xu = *reinterpret_cast<const uint2*>(u + t * W + ch);
      float4 av, bv;
      rglru_pair<false>(xr.x + cr[0], xi.x + ci[0], __uint_as_float(xu.x << 16), rate[0], av.x,
                        bv.x);
      rglru_pair<false>(xr.y + cr[1], xi.y + ci[1], __uint_as_float(xu.x & 0xffff0000u), rate[1],
                        av.y, bv.y);
      rglru_pair<false>(xr.z + cr[2], xi.z + ci[2], __uint_as_float(xu.y << 16), rate[2], av.z,
                        bv.z);
      rglru_pair<false>(xr.w + cr[3], xi.w + ci[3], __uint_as_float(xu.y & 0xffff0000u), rate[3],
                        av.w, bv.w);
      *reinterpret_cast<float4*>(a + t * W + ch) = av;
      *reinterpret_cast<float4*>(b + t * W + ch) = bv;
    }
    return;
  }
#pragma unroll
  for (int j = 0; j < NN; ++j) {
    const int o = o0 + (wn * NN + j) * 16 + l15;  // this lane's output column
    if (o >= n) continue;
    const int ch = blk * n + o;
    const float rate = c * softplus_(lam[ch]), cr = br[ch], ci = bi[ch];
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int t = t0 + wm * 16 + quad * 4 + e;
      if (t < Ttok) {
        float av, bv;
        rglru_pair<false>(ar[j][e] + cr, ai[j][e] + ci, ld(u + (int64_t)t * W + ch), rate, av,
                          bv);
        a[(int64_t)t * W + ch] = av;
        b[(int64_t)t * W + ch] = bv;
      }
    }
  }
}

// ------------------------------------------------- scan of S <- a S + b
// out = S * act(gate), act: 0 tanh GELU (as z * sigmoid(2 sqrt(2/pi) (z +
// 0.044715 z^3))), 1 SiLU, gate null: none.
template <bool EXACT>
__device__ __forceinline__ float gate_act(float z, int act) {
  const float arg = act == 0 ? 1.5957691216057308f * (z + 0.044715f * z * z * z) : z;
  return z * sigmoid_<EXACT>(arg);
}

// Prompt portions: a workgroup of DS_T threads owns CPB channels of one
// sequence. Its DS_T / CPB segments take DS_L consecutive tokens each (a tile
// is all of them); every segment first reduces its tokens to one (A, B) pair,
// the pairs pass through LDS, and every segment composes the pairs before it
// with the tile's incoming state (a segment's partial sums are at most DS_L
// tokens long, so the rounding differs from a token-by-token walk only in the
// order of additions). The next tile's operands are in flight meanwhile.
// Tokens beyond the end act as a = 1, b = 0.
constexpr int DS_T = 1024, DS_L = 8;

template <typename T, int CPB>
__global__ __launch_bounds__(DS_T) void diagonal_scan_k(
    const float* __restrict__ a, const float* __restrict__ b, const T* __restrict__ gate,
    int ld_gate, int act, float* __restrict__ state, const int* __restrict__ cu,
    const int* __restrict__ seq_slot, T* __restrict__ out, int W) {
  constexpr int NSEG = DS_T / CPB;
  constexpr bool EXACT = sizeof(T) == 4;
  __shared__ float sA[2][NSEG][CPB], sB[2][NSEG][CPB];
  const int s = blockIdx.x;
  const int cl = threadIdx.x % CPB, seg = threadIdx.x / CPB;
  const int ch = blockIdx.y * CPB + cl;
  const bool live = ch < W;
  const int c = live ? ch : W - 1;  // idle lanes shadow the last channel
  const int t0 = cu[s], n = cu[s + 1] - t0;
  float* Sg = state + (int64_t)seq_slot[s] * W + c;
  float S = *Sg;
  float na[DS_L], nb[DS_L], ng[DS_L];
  auto fetch = [&](int base) {
#pragma unroll
    for (int i = 0; i < DS_L; ++i) {
      const int j = base + seg * DS_L + i;
      const int64_t t = t0 + j;
      const bool in = j < n;
      na[i] = in ? a[t * W + c] : 1.f;
      nb[i] = in ? b[t * W + c] : 0.f;
      ng[i] = in && gate ? ld(gate + t * ld_gate + c) : 0.f;
    }
  };
  fetch(0);
  int buf = 0;
  for (int base = 0; base < n; base += NSEG * DS_L, buf ^= 1) {
    float va[DS_L], vb[DS_L], vg[DS_L];
    float A = 1.f, B = 0.f;
#pragma unroll
    for (int i = 0; i < DS_L; ++i) {
      va[i] = na[i];
      vb[i] = nb[i];
      vg[i] = ng[i];
      A *= va[i];
      B = va[i] * B + vb[i];
    }
    sA[buf][seg][cl] = A;
    sB[buf][seg][cl] = B;
    __syncthreads();
    if (base + NSEG * DS_L < n) fetch(base + NSEG * DS_L);
    float x = S;
#pragma unroll 8
    for (int k = 0; k < NSEG; ++k) {
      if (k == seg) x = S;  // the state this segment starts from
      S = sA[buf][k][cl] * S + sB[buf][k][cl];
    }
#pragma unroll
    for (int i = 0; i < DS_L; ++i) {
      x = va[i] * x + vb[i];
      const int j = base + seg * DS_L + i;
      if (live && j < n)
        st(out + (int64_t)(t0 + j) * W + c, gate ? x * gate_act<EXACT>(vg[i], act) : x);
    }
  }
  // every segment ends with the same S
  __syncthreads();
  if (live && seg == 0 && n > 0) *Sg = S;
}

// Steps of few tokens per sequence: a thread owns a channel and walks them.
template <typename T>
__global__ __launch_bounds__(NT) void diagonal_scan_short_k(
    const float* __restrict__ a, const float* __restrict__ b, const T* __restrict__ gate,
    int ld_gate, int act, float* __restrict__ state, const int* __restrict__ cu,
    const int* __restrict__ seq_slot, T* __restrict__ out, int W) {
  constexpr bool EXACT = sizeof(T) == 4;
  const int s = blockIdx.x;
  const int c = blockIdx.y * NT + threadIdx.x;
  if (c >= W) return;
  const int t0 = cu[s], t1 = cu[s + 1];
  if (t1 <= t0) return;
  float* Sg = state + (int64_t)seq_slot[s] * W + c;
  float S = *Sg;
  for (int64_t t = t0; t < t1; ++t) {
    S = a[t * W + c] * S + b[t * W + c];
    st(out + t * W + c, gate ? S * gate_act<EXACT>(ld(gate + t * ld_gate + c), act) : S);
  }
  *Sg = S;
}

// One token per sequence, 16-bit: convolution, tail shift, both gate products,
// gates, state update and gated read-out of one block of channels of up to 16
// sequences in one workgroup (it owns the block's channels: nobody else reads
// or shifts their tails). proj row = [ y (W) | x (W) ].
constexpr int RS_W = 16;  // waves
constexpr int RS_K = 6;   // 32-wide input steps whose weights are fetched ahead
constexpr int RS_U = 2;   // channels of a thread whose loads are issued together

// TAPS > 0: that many taps, a channel's tail in registers; 0: any number.
// VEC: n a multiple of 8 (rows of the weights start 16-byte aligned).
template <int TAPS, bool VEC>
__global__ __launch_bounds__(64 * RS_W) void rglru_step_k(
    const bf16* __restrict__ proj, int ld_proj, const bf16* __restrict__ cw,
    const float* __restrict__ cb, bf16* __restrict__ tail, int64_t tail_stride, int taps,
    const bf16* __restrict__ wr, const bf16* __restrict__ wi, const float* __restrict__ br,
    const float* __restrict__ bi, const float* __restrict__ lam, float* __restrict__ state,
    const int* __restrict__ seq_slot, const int* __restrict__ seq_start, bf16* __restrict__ out,
    int nseq, int n, int W, float c) {
  typedef __attribute__((ext_vector_type(8))) __bf16 frag;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  __shared__ int s_slot[16], s_pos[16];
  bf16* sU = reinterpret_cast<bf16*>(smem);  // [16][pitch]
  const int pitch = (n + 31) / 32 * 32 + 8;
  const int t0 = blockIdx.x * 16, blk = blockIdx.y;
  const int nt = min(16, nseq - t0);
  const int kept = taps - 1;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int l15 = lane & 15, quad = lane >> 4;
  if (threadIdx.x < 16) {
    const int t = t0 + min((int)threadIdx.x, nt - 1);
    s_slot[threadIdx.x] = seq_slot[t];
    s_pos[threadIdx.x] = seq_start[t];
  }
  // this wave's first tile of both weights: in flight over the convolution
  auto get = [&](const bf16* base, int o, int k) {
    const short* row = reinterpret_cast<const short*>(base) + ((int64_t)blk * n + o) * n;
    short8 x = {0, 0, 0, 0, 0, 0, 0, 0};
    if (o < n) {
      if (VEC) {
        if (k < n) x = *reinterpret_cast<const short8*>(row + k);
      } else {
#pragma unroll
        for (int e = 0; e < 8; ++e)
          if (k + e < n) x[e] = row[k + e];
      }
    }
    return x;
  };
  short8 pr[RS_K], pi[RS_K];
#pragma unroll
  for (int i = 0; i < (VEC ? RS_K : 0); ++i) {
    pr[i] = get(wr, wave * 16 + l15, i * 32 + quad * 8);
    pi[i] = get(wi, wave * 16 + l15, i * 32 + quad * 8);
  }
  for (int i = nt * pitch + threadIdx.x; i < 16 * pitch; i += 64 * RS_W) st(sU + i, 0.f);
  for (int i = threadIdx.x; i < nt * (pitch - n); i += 64 * RS_W) {
    const int tk = i / (pitch - n);
    st(sU + tk * pitch + n + i - tk * (pitch - n), 0.f);
  }
  __syncthreads();
  // what the wave's first tile needs at its end, in flight over the rest
  float pS[4], pz[4], prate, pcr, pci;
  {
    const int ch = blk * n + min(wave * 16 + l15, n - 1);
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int tk = min(quad * 4 + e, nt - 1);
      pS[e] = state[(int64_t)s_slot[tk] * W + ch];
      pz[e] = ld(proj + (int64_t)(t0 + tk) * ld_proj + ch);
    }
    prate = lam[ch];
    pcr = br[ch];
    pci = bi[ch];
  }
  if (TAPS > 0) {
    constexpr int K = TAPS > 1 ? TAPS - 1 : 1;
    for (int i0 = threadIdx.x; i0 < nt * n; i0 += 64 * RS_W * RS_U) {
      float x[RS_U], cbv[RS_U], wv[RS_U][K + 1], tv[RS_U][K];
#pragma unroll
      for (int q = 0; q < RS_U; ++q) {
        const int i = min(i0 + q * 64 * RS_W, nt * n - 1);
        const int tk = i / n, ch = blk * n + i - tk * n;
        x[q] = ld(proj + (int64_t)(t0 + tk) * ld_proj + W + ch);
        cbv[q] = cb[ch];
#pragma unroll
        for (int j = 0; j < TAPS; ++j) wv[q][j] = ld(cw + (int64_t)ch * TAPS + j);
#pragma unroll
        for (int j = 0; j + 1 < TAPS; ++j)
          tv[q][j] = ld(tail + (int64_t)s_slot[tk] * tail_stride + (int64_t)j * W + ch);
      }
#pragma unroll
      for (int q = 0; q < RS_U; ++q) {
        const int i = i0 + q * 64 * RS_W;
        if (i >= nt * n) break;
        const int tk = i / n, ch = blk * n + i - tk * n;
        float u = wv[q][TAPS > 0 ? TAPS - 1 : 0] * x[q];
#pragma unroll
        for (int j = 1; j < TAPS; ++j)
          if (s_pos[tk] - j >= 0) u += wv[q][TAPS - 1 - j] * tv[q][TAPS - 1 - j];
        st(sU + tk * pitch + i - tk * n, u + cbv[q]);
        bf16* tl = tail + (int64_t)s_slot[tk] * tail_stride + ch;
#pragma unroll
        for (int j = 0; j + 1 < TAPS; ++j)
          st(tl + (int64_t)j * W, j + 2 < TAPS ? tv[q][j + 1 < K ? j + 1 : 0] : x[q]);
      }
    }
  } else {
    for (int i = threadIdx.x; i < nt * n; i += 64 * RS_W) {
      const int tk = i / n, k = i - tk * n;
      const int ch = blk * n + k;
      const bf16 xin = proj[(int64_t)(t0 + tk) * ld_proj + W + ch];
      bf16* tl = tail + (int64_t)s_slot[tk] * tail_stride + ch;
      const bf16* w = cw + (int64_t)ch * taps;
      float u = ld(w + kept) * ld(&xin);
      for (int j = 1; j <= kept; ++j)
        if (s_pos[tk] - j >= 0) u += ld(w + kept - j) * ld(tl + (int64_t)(kept - j) * W);
      st(sU + tk * pitch + k, u + cb[ch]);
      for (int j = 0; j + 1 < kept; ++j) tl[(int64_t)j * W] = tl[(int64_t)(j + 1) * W];
      if (kept > 0) tl[(int64_t)(kept - 1) * W] = xin;
    }
  }
  __syncthreads();
  for (int ot = wave; ot * 16 < n; ot += RS_W) {
    const int o = ot * 16 + l15;
    const int ch = blk * n + min(o, n - 1);
    if (ot != wave) {
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int tk = min(quad * 4 + e, nt - 1);
        pS[e] = state[(int64_t)s_slot[tk] * W + ch];
        pz[e] = ld(proj + (int64_t)(t0 + tk) * ld_proj + ch);
      }
      prate = lam[ch];
      pcr = br[ch];
      pci = bi[ch];
    }
    floatx4 ar = {0.f, 0.f, 0.f, 0.f}, ai = {0.f, 0.f, 0.f, 0.f};
    auto step = [&](int kk, short8 r, short8 i) {
      const frag fa = *reinterpret_cast<const frag*>(sU + l15 * pitch + kk + quad * 8);
      ar = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fa, __builtin_bit_cast(frag, r), ar, 0, 0, 0);
      ai = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fa, __builtin_bit_cast(frag, i), ai, 0, 0, 0);
    };
    int k0 = 0;
    if (VEC && ot == wave) {
#pragma unroll
      for (int i = 0; i < RS_K; ++i)
        if (i * 32 < n) step(i * 32, pr[i], pi[i]);
      k0 = RS_K * 32;
    }
#pragma unroll 2
    for (int kk = k0; kk < n; kk += 32)
      step(kk, get(wr, o, kk + quad * 8), get(wi, o, kk + quad * 8));
    if (o >= n) continue;
    const float rate = c * softplus_(prate);
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int tk = quad * 4 + e;
      if (tk < nt) {
        float a, b;
        rglru_pair<false>(ar[e] + pcr, ai[e] + pci, ld(sU + tk * pitch + o), rate, a, b);
        const float Sn = a * pS[e] + b;
        state[(int64_t)s_slot[tk] * W + ch] = Sn;
        st(out + (int64_t)(t0 + tk) * W + ch, Sn * gate_act<false>(pz[e], 0));
      }
    }
  }
}

// ------------------------------ retention, one token per sequence, in one pass
// A workgroup owns one head of one sequence: rotation of q and k (HALF
// pairing, keys then times k_scale), S <- g S + k v^T, o = S^T q, RMS norm of
// o over the head, times SiLU(gate) and out_scale. CW neighbouring threads
// hold neighbouring columns; RT_T / CW groups share the rows.
constexpr int RT_T = 1024;

template <typename T, int CW>
__global__ __launch_bounds__(RT_T) void retention_step_k(
    const T* __restrict__ qk, int ld_qk, const T* __restrict__ v, int ld_v,
    const T* __restrict__ gate, int ld_gate, const float* __restrict__ cosT,
    const float* __restrict__ sinT, const int* __restrict__ tok_pos,
    const float* __restrict__ decay, float* __restrict__ state, const int* __restrict__ seq_slot,
    T* __restrict__ out, int ld_out, int H, int dim, int vdim, int rot_dims, float k_scale,
    float eps, float out_scale) {
  constexpr bool EXACT = sizeof(T) == 4;
  constexpr int RG = RT_T / CW;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  float* sq = reinterpret_cast<float*>(smem);  // [dim]
  float* sk = sq + dim;                        // [dim]
  float* so = sk + dim;                        // [vdim]
  float* sp = so + vdim;                       // [RT_T]
  const int t = blockIdx.x, h = blockIdx.y;
  const int half = rot_dims >> 1;
  const float* cs = cosT + (int64_t)tok_pos[t] * half;
  const float* sn = sinT + (int64_t)tok_pos[t] * half;
  for (int i = threadIdx.x; i < 2 * dim; i += RT_T) {
    const bool is_k = i >= dim;
    const int c = is_k ? i - dim : i;
    const T* hd = qk + (int64_t)t * ld_qk + (is_k ? (H + h) * dim : h * dim);
    float x = ld(hd + c);
    if (c < rot_dims) {
      const bool second = c >= half;
      const int f = second ? c - half : c;
      const float y = ld(hd + (second ? f : c + half));
      x = second ? x * cs[f] + y * sn[f] : x * cs[f] - y * sn[f];
    }
    sq[i] = is_k ? x * k_scale : x;
  }
  __syncthreads();
  const float g = decay[h];
  float* Sh = state + ((int64_t)seq_slot[t] * H + h) * dim * (int64_t)vdim;
  const int cl = threadIdx.x % CW, rg = threadIdx.x / CW;
  for (int c0 = 0; c0 < vdim; c0 += CW) {
    const int c = c0 + cl;
    float acc = 0.f;
    if (c < vdim) {
      const float vc = ld(v + (int64_t)t * ld_v + h * vdim + c);
      // eight rows at a time: all loads before the first store
      for (int d0 = rg; d0 < dim; d0 += 8 * RG) {
        float S[8];
#pragma unroll
        for (int i = 0; i < 8; ++i) {
          const int d = d0 + i * RG;
          S[i] = d < dim ? Sh[(int64_t)d * vdim + c] : 0.f;
        }
#pragma unroll
        for (int i = 0; i < 8; ++i) {
          const int d = d0 + i * RG;
          if (d < dim) {
            S[i] = g * S[i] + sk[d] * vc;
            Sh[(int64_t)d * vdim + c] = S[i];
            acc += sq[d] * S[i];
          }
        }
      }
    }
    sp[threadIdx.x] = acc;
    __syncthreads();
    if (rg == 0 && c < vdim) {
      float o = 0.f;
      for (int r = 0; r < RG; ++r) o += sp[r * CW + cl];
      so[c] = o;
    }
    __syncthreads();
  }
  float ss = 0.f;
  for (int c = threadIdx.x; c < vdim; c += RT_T) ss += so[c] * so[c];
  const float inv = rsqrtf(block_sum(ss, sp) / (float)vdim + eps) * out_scale;
  for (int c = threadIdx.x; c < vdim; c += RT_T) {
    const float z = ld(gate + (int64_t)t * ld_gate + h * vdim + c);
    st(out + (int64_t)t * ld_out + h * vdim + c, so[c] * inv * gate_act<EXACT>(z, 1));
  }
}

// ------------------------- matrix-state recurrence with a fixed decay, chunks
// S <- g S + k v^T, o = S^T q per head, RC tokens at a time on matrix cores:
// with a chunk's tokens 0..n-1 and the state S0 before it,
//   o_t = g^(t+1) S0^T q_t + sum_{s<=t} g^(t-s) (q_t . k_s) v_s
//   S   = g^n S0 + sum_s (g^(n-1-s) k_s) v_s^T.
// q and k are float, v bf16. Every float operand of a product (q, k, the
// decayed keys, the masked scores, the state) enters as a bf16 head plus a
// bf16 remainder, i.e. with 16 bits of mantissa, and the product of the two
// remainders is dropped; sums and the state itself (accumulators, RN columns
// of one head per workgroup, kept over all chunks) are float.
//
// 4 waves: wave w owns tokens 16w..16w+15 of the chunk and rows
// w*DP/4..(w+1)*DP/4-1 of the state. LDS holds the keys by token, the decayed
// keys and the values by coordinate (token-contiguous) and the state by value
// column; rows are split into 16-byte groups whose order is permuted by the
// row, which spreads both the writes (rows 4i + e over lanes i) and the reads
// (16 neighbouring rows) over the banks. The scores are made transposed (keys
// as rows), so that a lane's accumulators are four neighbouring keys of its
// own token: they are the A operand of the product with v as they are, with
// the key order of both operands permuted alike. The next chunk's q, k, v are
// in flight while a chunk is computed.
typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;
typedef __attribute__((ext_vector_type(4))) __bf16 bf16x4;
constexpr int RC = 64;  // tokens per chunk
constexpr int RN = 64;  // value columns per workgroup

// offset of element (row, col) in rows of `pitch` elements (whole 64s)
__device__ __forceinline__ int swz(int row, int col, int pitch) {
  return row * pitch + (((col >> 3) ^ ((row ^ (row >> 2)) & 7)) << 3) + (col & 7);
}
__device__ __forceinline__ void split2(float x, __bf16& hi, __bf16& lo) {
  hi = static_cast<__bf16>(x);
  lo = static_cast<__bf16>(x - static_cast<float>(hi));
}
__device__ __forceinline__ floatx4 mma(bf16x8 a, bf16x8 b, floatx4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0);
}

template <int DP>
__global__ __launch_bounds__(256) void retention_chunk_k(
    const float* __restrict__ q, const float* __restrict__ k, const bf16* __restrict__ v,
    int ld_v, const float* __restrict__ decay, float* __restrict__ state,
    const int* __restrict__ cu, const int* __restrict__ seq_slot, float* __restrict__ out, int G,
    int H, int dim, int vdim, float q_scale) {
  constexpr int KS = DP / 32;   // 32-wide steps over a head's coordinates
  constexpr int MT = DP / 64;   // 16-row tiles of the state per wave
  constexpr int NT4 = RN / 16;  // 16-column tiles
  constexpr int KQ = DP / 4;    // groups of four coordinates
  extern __shared__ __attribute__((aligned(16))) char smem[];
  __bf16* Kh = reinterpret_cast<__bf16*>(smem);  // [RC][DP]
  __bf16* Kl = Kh + RC * DP;
  __bf16* Dh = Kl + RC * DP;  // [DP][RC] keys times their decay to the chunk's end
  __bf16* Dl = Dh + DP * RC;
  __bf16* Sh = Dl + DP * RC;  // [RN][DP]
  __bf16* Sl = Sh + RN * DP;
  __bf16* Vt = Sl + RN * DP;  // [RN][RC]
  const int s = blockIdx.x, h = blockIdx.y, c0 = blockIdx.z * RN;
  const int t0 = cu[s], cnt = cu[s + 1] - t0;
  if (cnt <= 0) return;  // whole workgroup
  const int g = h / (H / G);
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6;
  const int l15 = lane & 15, quad = lane >> 4;
  const float lg = fmaxf(log2f(decay[h]), -1000.f);
  auto pw = [&](int e) { return __builtin_amdgcn_exp2f(lg * (float)e); };
  const int ldq = G * dim;
  const float* qb = q + (int64_t)t0 * ldq + g * dim;
  const float* kb = k + (int64_t)t0 * ldq + g * dim;
  const bf16* vb = v + (int64_t)t0 * ld_v + h * vdim + c0;

  // this lane's part of the state, accumulator layout: row (coordinate)
  // w*DP/4 + 16 mt + 4 quad + j, column c0 + 16 nt + l15
  float* Sg = state + (((int64_t)seq_slot[s] * H + h) * dim) * vdim + c0;
  floatx4 S[MT][NT4];
#pragma unroll
  for (int mt = 0; mt < MT; ++mt)
#pragma unroll
    for (int nt = 0; nt < NT4; ++nt)
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int d = w * (DP / 4) + mt * 16 + quad * 4 + j, c = nt * 16 + l15;
        S[mt][nt][j] = d < dim && c0 + c < vdim ? Sg[(int64_t)d * vdim + c] : 0.f;
      }

  // staging: a thread moves four coordinates of eight tokens of k, and four
  // columns of eight tokens of v; of q a lane holds its token's A operands
  const int kq = threadIdx.x % KQ, kg = threadIdx.x / KQ;
  const bool kin = kg < RC / 8;
  const int vq = (threadIdx.x - 128) & 15, vg = (threadIdx.x - 128) >> 4;
  const bool vin = threadIdx.x >= 128;
  float4 rk[8], rq[KS][2];
  uint2 rv[8];
  auto fetch = [&](int base) {
    const int n = min(RC, cnt - base);
    const float4 z4 = make_float4(0.f, 0.f, 0.f, 0.f);
    if (kin) {
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        const int t = kg * 8 + i;
        rk[i] = t < n && kq * 4 < dim
                    ? *reinterpret_cast<const float4*>(kb + (int64_t)(base + t) * ldq + kq * 4)
                    : z4;
      }
    }
    if (vin) {
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        const int t = vg * 8 + i;
        rv[i] = t < n && c0 + vq * 4 < vdim
                    ? *reinterpret_cast<const uint2*>(vb + (int64_t)(base + t) * ld_v + vq * 4)
                    : make_uint2(0u, 0u);
      }
    }
    const int t = w * 16 + l15;
#pragma unroll
    for (int ks = 0; ks < KS; ++ks)
#pragma unroll
      for (int e = 0; e < 2; ++e) {
        const int d = ks * 32 + quad * 8 + e * 4;
        rq[ks][e] = t < n && d < dim
                        ? *reinterpret_cast<const float4*>(qb + (int64_t)(base + t) * ldq + d)
                        : z4;
      }
  };
  auto stash = [&](int n) {
    if (kin) {
      float f[8];
#pragma unroll
      for (int i = 0; i < 8; ++i) f[i] = pw(max(n - 1 - (kg * 8 + i), 0));
      bf16x8 th[4], tl[4];
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        const float x[4] = {rk[i].x, rk[i].y, rk[i].z, rk[i].w};
        bf16x4 hi, lo;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          __bf16 a, b;
          split2(x[e], a, b);
          hi[e] = a;
          lo[e] = b;
          split2(x[e] * f[i], a, b);
          th[e][i] = a;
          tl[e][i] = b;
        }
        const int at = swz(kg * 8 + i, kq * 4, DP);
        *reinterpret_cast<bf16x4*>(Kh + at) = hi;
        *reinterpret_cast<bf16x4*>(Kl + at) = lo;
      }
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int at = swz(kq * 4 + e, kg * 8, RC);
        *reinterpret_cast<bf16x8*>(Dh + at) = th[e];
        *reinterpret_cast<bf16x8*>(Dl + at) = tl[e];
      }
    }
    if (vin) {
      bf16x8 tv[4];
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        const bf16x4 x = __builtin_bit_cast(bf16x4, rv[i]);
#pragma unroll
        for (int e = 0; e < 4; ++e) tv[e][i] = x[e];
      }
#pragma unroll
      for (int e = 0; e < 4; ++e)
        *reinterpret_cast<bf16x8*>(Vt + swz(vq * 4 + e, vg * 8, RC)) = tv[e];
    }
#pragma unroll
    for (int mt = 0; mt < MT; ++mt)
#pragma unroll
      for (int nt = 0; nt < NT4; ++nt) {
        bf16x4 hi, lo;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          __bf16 a, b;
          split2(S[mt][nt][j], a, b);
          hi[j] = a;
          lo[j] = b;
        }
        const int at = swz(nt * 16 + l15, w * (DP / 4) + mt * 16 + quad * 4, DP);
        *reinterpret_cast<bf16x4*>(Sh + at) = hi;
        *reinterpret_cast<bf16x4*>(Sl + at) = lo;
      }
  };

  fetch(0);
  for (int base = 0; base < cnt; base += RC) {
    const int n = min(RC, cnt - base);
    stash(n);
    bf16x8 qh[KS], ql[KS];
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      const float x[8] = {rq[ks][0].x, rq[ks][0].y, rq[ks][0].z, rq[ks][0].w,
                          rq[ks][1].x, rq[ks][1].y, rq[ks][1].z, rq[ks][1].w};
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        __bf16 a, b;
        split2(x[e] * q_scale, a, b);
        qh[ks][e] = a;
        ql[ks][e] = b;
      }
    }
    __syncthreads();
    if (base + RC < cnt) fetch(base + RC);

    // masked, decayed scores: p[jt][j] for key 16 jt + 4 quad + j, token l15
    // (tiles above the diagonal are made and masked too: four independent
    // chains of products fill the pipe better than a wave-dependent number)
    floatx4 p[4];
#pragma unroll
    for (int jt = 0; jt < 4; ++jt) p[jt] = (floatx4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      bf16x8 kh[4], kl[4];
#pragma unroll
      for (int jt = 0; jt < 4; ++jt) {
        const int at = swz(jt * 16 + l15, ks * 32 + quad * 8, DP);
        kh[jt] = *reinterpret_cast<const bf16x8*>(Kh + at);
        kl[jt] = *reinterpret_cast<const bf16x8*>(Kl + at);
      }
#pragma unroll
      for (int jt = 0; jt < 4; ++jt) p[jt] = mma(kh[jt], qh[ks], p[jt]);
#pragma unroll
      for (int jt = 0; jt < 4; ++jt) p[jt] = mma(kl[jt], qh[ks], p[jt]);
#pragma unroll
      for (int jt = 0; jt < 4; ++jt) p[jt] = mma(kh[jt], ql[ks], p[jt]);
    }
#pragma unroll
    for (int jt = 0; jt < 4; ++jt)
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int dt = (w - jt) * 16 + l15 - quad * 4 - j;
        p[jt][j] = dt >= 0 ? p[jt][j] * pw(dt) : 0.f;
      }
    // what the earlier chunks' state gives, then this chunk's own tokens
    floatx4 o[NT4];
#pragma unroll
    for (int nt = 0; nt < NT4; ++nt) o[nt] = (floatx4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      bf16x8 sh[NT4], sl[NT4];
#pragma unroll
      for (int nt = 0; nt < NT4; ++nt) {
        const int at = swz(nt * 16 + l15, ks * 32 + quad * 8, DP);
        sh[nt] = *reinterpret_cast<const bf16x8*>(Sh + at);
        sl[nt] = *reinterpret_cast<const bf16x8*>(Sl + at);
      }
#pragma unroll
      for (int nt = 0; nt < NT4; ++nt) o[nt] = mma(qh[ks], sh[nt], o[nt]);
#pragma unroll
      for (int nt = 0; nt < NT4; ++nt) o[nt] = mma(ql[ks], sh[nt], o[nt]);
#pragma unroll
      for (int nt = 0; nt < NT4; ++nt) o[nt] = mma(qh[ks], sl[nt], o[nt]);
    }
    float f[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) f[j] = pw(w * 16 + quad * 4 + j + 1);
#pragma unroll
    for (int nt = 0; nt < NT4; ++nt)
#pragma unroll
      for (int j = 0; j < 4; ++j) o[nt][j] *= f[j];
#pragma unroll
    for (int kp = 0; kp < 2; ++kp) {
      if (2 * kp > w) continue;  // wave-uniform
      bf16x8 ph, pl;
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        __bf16 a, b;
        split2(p[2 * kp + (e >> 2)][e & 3], a, b);
        ph[e] = a;
        pl[e] = b;
      }
#pragma unroll
      for (int nt = 0; nt < NT4; ++nt) {
        const int r = nt * 16 + l15;
        const bf16x4 a =
            *reinterpret_cast<const bf16x4*>(Vt + swz(r, (2 * kp) * 16 + quad * 4, RC));
        const bf16x4 b =
            *reinterpret_cast<const bf16x4*>(Vt + swz(r, (2 * kp + 1) * 16 + quad * 4, RC));
        const bf16x8 vf = __builtin_shufflevector(a, b, 0, 1, 2, 3, 4, 5, 6, 7);
        o[nt] = mma(ph, vf, o[nt]);
        o[nt] = mma(pl, vf, o[nt]);
      }
    }
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int t = w * 16 + quad * 4 + j;
      if (t < n) {
        float* row = out + ((int64_t)(t0 + base + t) * H + h) * vdim + c0;
#pragma unroll
        for (int nt = 0; nt < NT4; ++nt)
          if (c0 + nt * 16 + l15 < vdim) row[nt * 16 + l15] = o[nt][j];
      }
    }
    // the state after the chunk
    const float gn = pw(n);
#pragma unroll
    for (int mt = 0; mt < MT; ++mt)
#pragma unroll
      for (int nt = 0; nt < NT4; ++nt)
#pragma unroll
        for (int j = 0; j < 4; ++j) S[mt][nt][j] *= gn;
#pragma unroll
    for (int kk = 0; kk < 2; ++kk) {
      bf16x8 vf[NT4];
#pragma unroll
      for (int nt = 0; nt < NT4; ++nt)
        vf[nt] = *reinterpret_cast<const bf16x8*>(
            Vt + swz(nt * 16 + l15, kk * 32 + quad * 8, RC));
#pragma unroll
      for (int mt = 0; mt < MT; ++mt) {
        const int at = swz(w * (DP / 4) + mt * 16 + l15, kk * 32 + quad * 8, RC);
        const bf16x8 dh = *reinterpret_cast<const bf16x8*>(Dh + at);
        const bf16x8 dl = *reinterpret_cast<const bf16x8*>(Dl + at);
#pragma unroll
        for (int nt = 0; nt < NT4; ++nt) {
          S[mt][nt] = mma(dh, vf[nt], S[mt][nt]);
          S[mt][nt] = mma(dl, vf[nt], S[mt][nt]);
        }
      }
    }
    __syncthreads();  // every read of this chunk's LDS is done
  }
#pragma unroll
  for (int mt = 0; mt < MT; ++mt)
#pragma unroll
    for (int nt = 0; nt < NT4; ++nt)
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int d = w * (DP / 4) + mt * 16 + quad * 4 + j, c = nt * 16 + l15;
        if (d < dim && c0 + c < vdim) Sg[(int64_t)d * vdim + c] = S[mt][nt][j];
      }
}

template <int DP>
int launch_retention_chunk(const float* q, const float* k, const void* v, int ld_v,
                           const float* decay, float* state, const int* cu, const int* seq_slot,
                           float* out, int nseq, int G, int H, int dim, int vdim, float q_scale,
                           hipStream_t s) {
  const int lds = (4 * RC * DP + 2 * RN * DP + RN * RC) * 2;
  auto kern = retention_chunk_k<DP>;
  if (lds > 48 * 1024) {
    hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(kern),
                                       hipFuncAttributeMaxDynamicSharedMemorySize, lds);
    if (e != hipSuccess) return (int)e;
  }
  kern<<<dim3(nseq, H, (vdim + RN - 1) / RN), 256, lds, s>>>(
      q, k, (const bf16*)v, ld_v, decay, state, cu, seq_slot, out, G, H, dim, vdim, q_scale);
  return (int)hipGetLastError();
}

}  // namespace

extern "C" {

int dsv_rglru_pair(const float* zr, const float* zi, const void* u, const float* br,
                   const float* bi, const float* lam, float* a, float* b, int dt, int Ttok,
                   int blocks, int n, float c, hipStream_t s) {
  if (Ttok <= 0) return 0;
  if (blocks < 1 || n < 1) return -1;
  BY_DTYPE(dt, (rglru_pair_k<T><<<nblocks((int64_t)Ttok * blocks * n, 256), 256, 0, s>>>(
                   zr, zi, (const T*)u, br, bi, lam, a, b, Ttok, blocks, n, c)));
  return (int)hipGetLastError();
}

// bf16 u [T, blocks*n] (contiguous), wr/wi [blocks, n, n]
int dsv_rglru_gates(const void* u, const void* wr, const void* wi, const float* br,
                    const float* bi, const float* lam, float* a, float* b, int Ttok, int blocks,
                    int n, float c, hipStream_t s) {
  if (Ttok <= 0) return 0;
  if (blocks < 1 || blocks > 65535 || n < 1) return -1;
  if ((uintptr_t)u % 16 || (uintptr_t)wr % 16 || (uintptr_t)wi % 16) return -2;
#define GATES(WM, WN, NN)                                                                       \
  rglru_gates_mfma_k<WM, WN, NN>                                                                 \
      <<<dim3((Ttok + 16 * WM - 1) / (16 * WM), blocks,                                          \
              (n + 16 * WN * NN - 1) / (16 * WN * NN)),                                          \
         NT, 0, s>>>((const bf16*)u, (const bf16*)wr, (const bf16*)wi, br, bi, lam, a, b, Ttok,  \
                     n, blocks * n, c)
  if (Ttok >= 512) GATES(4, 1, 4);
  else if (Ttok > 16) GATES(2, 2, 1);
  else GATES(1, 4, 1);
#undef GATES
  return (int)hipGetLastError();
}

// max_count: most tokens any sequence brings
int dsv_diagonal_scan(const float* a, const float* b, const void* gate, int ld_gate, int act,
                      float* state, const int* cu, const int* seq_slot, void* out, int dt,
                      int nseq, int W, int max_count, hipStream_t s) {
  if (nseq <= 0 || max_count <= 0) return 0;
  if (W < 1 || (act != 0 && act != 1)) return -1;
  if (max_count <= 8) {
    BY_DTYPE(dt, (diagonal_scan_short_k<T><<<dim3(nseq, (W + NT - 1) / NT), NT, 0, s>>>(
                     a, b, (const T*)gate, ld_gate, act, state, cu, seq_slot, (T*)out, W)));
    return (int)hipGetLastError();
  }
  // narrow channel groups while the launch would not fill the chip
  if ((int64_t)nseq * ((W + 63) / 64) >= 512)
    BY_DTYPE(dt, (diagonal_scan_k<T, 64><<<dim3(nseq, (W + 63) / 64), DS_T, 0, s>>>(
                     a, b, (const T*)gate, ld_gate, act, state, cu, seq_slot, (T*)out, W)));
  else
    BY_DTYPE(dt, (diagonal_scan_k<T, 32><<<dim3(nseq, (W + 31) / 32), DS_T, 0, s>>>(
                     a, b, (const T*)gate, ld_gate, act, state, cu, seq_slot, (T*)out, W)));
  return (int)hipGetLastError();
}

// largest head size of keys the chunked form covers
int dsv_retention_chunk_max_dim() { return 128; }

// float q, k [T, G*dim] (contiguous), bf16 v (row stride ld_v), decay [H];
// dim, vdim and ld_v multiples of 4, q and k 16-byte and v 8-byte aligned
int dsv_retention_chunk(const float* q, const float* k, const void* v, int ld_v,
                        const float* decay, float* state, const int* cu, const int* seq_slot,
                        float* out, int nseq, int G, int H, int dim, int vdim, float q_scale,
                        hipStream_t s) {
  if (dim < 1 || dim > dsv_retention_chunk_max_dim() || vdim < 1 || G < 1 || H % G) return -1;
  if (dim % 4 || vdim % 4 || ld_v % 4 || (uintptr_t)q % 16 || (uintptr_t)k % 16 ||
      (uintptr_t)v % 8)
    return -2;
  if (nseq <= 0) return 0;
  if (dim <= 64)
    return launch_retention_chunk<64>(q, k, v, ld_v, decay, state, cu, seq_slot, out, nseq, G, H,
                                      dim, vdim, q_scale, s);
  return launch_retention_chunk<128>(q, k, v, ld_v, decay, state, cu, seq_slot, out, nseq, G, H,
                                     dim, vdim, q_scale, s);
}

// one token per sequence: flat token i is sequence i's
int dsv_rglru_step(const void* proj, int ld_proj, const void* cw, const float* cb, void* tail,
                   int64_t tail_stride, int taps, const void* wr, const void* wi, const float* br,
                   const float* bi, const float* lam, float* state, const int* seq_slot,
                   const int* seq_start, void* out, int nseq, int blocks, int n, float c,
                   hipStream_t s) {
  if (nseq <= 0) return 0;
  if (blocks < 1 || blocks > 65535 || n < 1 || taps < 1 || ld_proj < 2 * blocks * n) return -1;
  if ((uintptr_t)wr % 16 || (uintptr_t)wi % 16) return -2;
  const size_t lds = (size_t)16 * ((n + 31) / 32 * 32 + 8) * 2;
  if (lds > 48 * 1024) return -3;
#define RGSTEP(TAPS, VEC)                                                                       \
  rglru_step_k<TAPS, VEC><<<dim3((nseq + 15) / 16, blocks), 64 * RS_W, lds, s>>>(                \
      (const bf16*)proj, ld_proj, (const bf16*)cw, cb, (bf16*)tail, tail_stride, taps,          \
      (const bf16*)wr, (const bf16*)wi, br, bi, lam, state, seq_slot, seq_start, (bf16*)out,    \
      nseq, n, blocks * n, c)
  if (n % 8) RGSTEP(0, false);
  else if (taps == 4) RGSTEP(4, true);
  else if (taps == 3) RGSTEP(3, true);
  else if (taps == 2) RGSTEP(2, true);
  else RGSTEP(0, true);
#undef RGSTEP
  return (int)hipGetLastError();
}

// one token per sequence; qk row = [ q (H x dim) | k (H x dim) ]
int dsv_retention_step(const void* qk, int ld_qk, const void* v, int ld_v, const void* gate,
                       int ld_gate, const float* cosT, const float* sinT, const int* tok_pos,
                       const float* decay, float* state, const int* seq_slot, void* out,
                       int ld_out, int dt, int nseq, int H, int dim, int vdim, int rot_dims,
                       float k_scale, float eps, float out_scale, hipStream_t s) {
  if (nseq <= 0) return 0;
  if (H < 1 || H > 65535 || dim < 1 || vdim < 1) return -1;
  if (rot_dims < 0 || (rot_dims & 1) || rot_dims > dim) return -2;
  if (rot_dims > 0 && (!cosT || !sinT)) return -2;
  const size_t lds = ((size_t)2 * dim + vdim + RT_T) * 4;
  if (lds > 48 * 1024) return -3;
#define RSTEP(CW)                                                                               \
  BY_DTYPE(dt, (retention_step_k<T, CW><<<dim3(nseq, H), RT_T, lds, s>>>(                        \
                   (const T*)qk, ld_qk, (const T*)v, ld_v, (const T*)gate, ld_gate, cosT, sinT,  \
                   tok_pos, decay, state, seq_slot, (T*)out, ld_out, H, dim, vdim, rot_dims,     \
                   k_scale, eps, out_scale)))
  if (vdim <= 64) RSTEP(64);
  else if (vdim <= 128) RSTEP(128);
  else RSTEP(256);
#undef RSTEP
  return (int)hipGetLastError();
}

}  // extern "C"
