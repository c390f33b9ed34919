// Gated diagonal recurrences over ragged batches for MI355X (gfx950): the
// block-diagonal gates of a real-gated linear recurrent unit and the scan of
// a recurrence with one state per channel.
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
// 1 - exp(y) for y <= 0: the series where the difference would cancel
template <bool EXACT>
__device__ __forceinline__ float one_minus_exp(float y) {
  if (EXACT) return -expm1f(y);
  const float series =
      -y * (1.f + y * (1.f / 2) *
                      (1.f + y * (1.f / 3) *
                                 (1.f + y * (1.f / 4) *
                                            (1.f + y * (1.f / 5) *
                                                       (1.f + y * (1.f / 6) *
                                                                  (1.f + y * (1.f / 7)))))));
  return y > -0.4f ? series : 1.f - exp_<false>(y);
}

// (r, i pre-activations with bias) -> a and b of S <- a S + b
template <bool EXACT>
__device__ __forceinline__ void rglru_pair(float zr, float zi, float u, float rate, float& a,
                                           float& b) {
  const float la = -sigmoid_<EXACT>(zr) * rate;  // rate = c * softplus(lam)
  a = exp_<EXACT>(la);
  b = sqrtf(one_minus_exp<EXACT>(2.f * la)) * (sigmoid_<EXACT>(zi) * u);
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
  constexpr int TM = 16 * WM, TN = 16 * WN * NN;
  __shared__ __attribute__((aligned(16))) short sU[TM * GKP];
  __shared__ __attribute__((aligned(16))) short sR[TN * GKP];
  __shared__ __attribute__((aligned(16))) short sI[TN * GKP];
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

}  // extern "C"
