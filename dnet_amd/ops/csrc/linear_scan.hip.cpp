// Linear-attention recurrences with input-dependent gates (gfx950), fp32 state
// per slot and head:
//
//   gla_scan    S <- diag(alpha_t) S + k v^T ; o = S^T q, a decay per key
//               channel alpha = sigmoid(A2 a1 + b)^(1/tau) (low-rank A2 a1)
//   mlstm_scan  matrix memory with exponential gates and a running maximum m:
//               m' = max(f + m, i); S <- e^(f+m-m') S + e^(i-m') k v^T, n like
//               S with k alone; o = S^T q / (max(|n . q|, e^-m') + 1e-6);
//               i = cap tanh(./cap), f = logsigmoid(cap tanh(./cap))
//
// Geometry is the cache's: token (b,t) = row b*T+t sits at position pos[b]+t of
// slot slots[b] (default b); tokens t >= lens[b] are padding. State is taken as
// zero at position 0 and written only by rows with real tokens. Gates, decays,
// states and results are fp32 whatever the activation dtype ("short" stands
// for bf16 bits).
//
// Prompts (linear_chunk_kernel): a workgroup owns a tile of value columns of one
// head of one batch row and walks the tokens in chunks of 16. With w_s(t) = the
// key of token s carried to token t (k_s times every decay after s up to t),
// a chunk is
//     A[t][s] = q_t . w_s(t)  (s <= t)
//     O = A V + (q_t times the chunk's decays up to t) S
//     S <- (all the chunk's decays) S + w_s(last)^T V
// A comes from walking w token by token in registers (products of decays only,
// never a quotient, so that strong decays underflow instead of overflowing);
// the matrix products run on v_mfma_f32_16x16x4_f32 (fp32 operands: the state,
// the decays and what they multiply stay 32-bit), the state tile stays in the
// accumulator fragments. The next chunk's rows are in flight meanwhile.
// The matrix memory's normalizer n and maximum m ride along; every 64 value
// columns have their own copy of both in the state, so that no workgroup reads
// what another one writes.
//
// The decays of gated linear attention are formed for all tokens at once by a
// kernel in front (low_rank_decay_kernel).
//
// Key sizes above 256 (and low-rank inputs above 1024) take linear_scan_kernel,
// a walk over the tokens one by one: thread (column j, slice s) keeps rows
// [R s, R s + R) of column j in registers, the slices of a column are
// neighbouring lanes, tokens are staged through LDS in chunks with every gate
// evaluated once, and n is one more column (of ones) on a wave of its own.
//
// Decode steps (one token per row) have a kernel of their own: a workgroup owns
// a head of a batch row, streams its state once through 16 B accesses, and goes
// on with what follows the recurrence: RMS norm of the head, weight, output
// gate, one rounding into the next product's operand.
#include "common.h"

namespace dnet {

namespace {

template <typename T> __device__ __forceinline__ float ldx(const T* p);
template <> __device__ __forceinline__ float ldx<float>(const float* p) { return *p; }
template <> __device__ __forceinline__ float ldx<short>(const short* p) { return bits2f(*p); }

bool is_bf16(const torch::Tensor& t) { return t.scalar_type() == torch::kBFloat16; }
bool is_f32(const torch::Tensor& t) { return t.scalar_type() == torch::kFloat32; }

__device__ __forceinline__ float log_sigmoid(float z) {
  return fminf(z, 0.f) - log1pf(expf(-fabsf(z)));
}

// sigmoid(z)^p; the hardware exponential and logarithm are within a few 1e-7 of
// the decay here (the logarithm's argument lies in [1, 2])
__device__ __forceinline__ float decay_of(float z, float p) {
  const float ls = fminf(z, 0.f) - __logf(1.f + __expf(-fabsf(z)));
  return __expf(ls * p);
}

constexpr int kGla = 0, kMlstm = 1;
constexpr float kDenEps = 1e-6f;

struct ScanArgs {
  const void* src;           // projection rows [B*T, ld]
  float* state;              // [Bc, H, d, dv]
  float* o;                  // [B*T, H*dv]
  const int* pos;
  const int* lens;
  const int* slots;
  // gla: low-rank input at column a0, a2t [rank][H*d], bias [H*d]
  const float* a2t;
  const float* ab;
  const float* alpha;        // prompts: the decays, [B*T, H*d]
  // mlstm: gate columns i0, f0 with biases, n [Bc, H, NT, d], m [Bc, H, NT]
  const float* ib;
  const float* fb;
  float* nst;
  float* mst;
  int64_t ld;
  int q0, k0, v0, a0, rank, i0, f0, T, Bc, H, d, dv, JB, NS, TC, NT;
  float qscale, inv_tau, cap;
};

template <typename T, int R, int KIND>
__global__ __launch_bounds__(1024) void linear_scan_kernel(const ScanArgs a) {
  const int h = blockIdx.x / a.NT, tile = blockIdx.x % a.NT, b = blockIdx.y;
  const int n = a.lens ? min(a.lens[b], a.T) : a.T;
  const int slot = a.slots ? a.slots[b] : b;
  const int p0 = a.pos[b];
  if (n <= 0 || slot < 0 || slot >= a.Bc || p0 < 0) return;   // uniform
  const int d = a.d, dv = a.dv, JB = a.JB, NS = a.NS, TC = a.TC;
  const int j0 = tile * JB;
  const int DR = NS * R;                    // key rows incl. padding
  const int DP = NS * (R + 4);              // LDS pitch of one token: slices
                                            // four banks apart
  const int JP = JB + 1;                    // columns and the normalizer's
  const int nmain = JB * NS, lane = threadIdx.x & 63;
  const bool ncol = KIND == kMlstm && (int)threadIdx.x >= nmain;  // wave-uniform
  const int jl = ncol ? JB : threadIdx.x / NS;
  const int sl = ncol ? lane % NS : threadIdx.x % NS;
  const int j = j0 + jl;
  const bool col_ok = !ncol && j < dv;

  extern __shared__ __attribute__((aligned(16))) float sm[];
  float* sQ = sm;                           // [TC][DP]
  float* sK = sQ + TC * DP;
  float* sA = sK + TC * DP;                 // gla: decays
  float* sV = sA + (KIND == kGla ? TC * DP : 0);   // [TC][JP]
  float* sO = sV + TC * JP;                 // [TC][JP]
  float* sKeep = sO + TC * JP;              // mlstm: [TC] each; gla: [TC][rank]
  float* sPut = sKeep + TC;
  float* sEm = sPut + TC;
  float* sZ = sKeep;

  float S[R];
  float* sp = a.state + (((int64_t)slot * a.H + h) * d) * dv;
  float* np = nullptr;
  float* mp = nullptr;
  float m = 0.f;
  if constexpr (KIND == kMlstm) {
    np = a.nst + (((int64_t)slot * a.H + h) * a.NT + tile) * d;
    mp = a.mst + ((int64_t)slot * a.H + h) * a.NT + tile;
    if (p0 > 0) m = *mp;
  }
#pragma unroll
  for (int r = 0; r < R; ++r) {
    const int row = sl * R + r;
    S[r] = 0.f;
    if (p0 > 0 && row < d) {
      if (ncol) S[r] = np[row];
      else if (col_ok) S[r] = sp[(int64_t)row * dv + j];
    }
  }
  const T* src = reinterpret_cast<const T*>(a.src) + (int64_t)b * a.T * a.ld;

  for (int t0 = 0; t0 < n; t0 += TC) {
    const int tc = min(TC, n - t0);
    __syncthreads();                        // previous chunk consumed
    if (ncol) {
      float lf = 0.f, li = 0.f;
      if (lane < tc) {
        const T* sr = src + (int64_t)(t0 + lane) * a.ld;
        const float iv = ldx<T>(sr + a.i0 + h) + a.ib[h];
        const float fv = ldx<T>(sr + a.f0 + h) + a.fb[h];
        li = a.cap * tanhf(iv / a.cap);
        lf = log_sigmoid(a.cap * tanhf(fv / a.cap));
      }
      float before = 0.f, after = 0.f;
      for (int t = 0; t < tc; ++t) {        // the running maximum, in order
        const float f = __shfl(lf, t, 64), i = __shfl(li, t, 64);
        const float mn = fmaxf(f + m, i);
        if (lane == t) {
          before = f + m;
          after = mn;
        }
        m = mn;
      }
      if (lane < tc) {
        sKeep[lane] = expf(before - after);
        sPut[lane] = expf(li - after);
        sEm[lane] = expf(-after);
        sV[lane * JP + JB] = 1.f;
      }
    } else {
      for (int idx = threadIdx.x; idx < tc * DR; idx += nmain) {
        const int tt = idx / DR, i = idx % DR;
        const T* sr = src + (int64_t)(t0 + tt) * a.ld + h * d + i;
        const int at = tt * DP + (i / R) * (R + 4) + (i % R);
        sQ[at] = i < d ? ldx<T>(sr + a.q0) * a.qscale : 0.f;
        sK[at] = i < d ? ldx<T>(sr + a.k0) : 0.f;
      }
      for (int idx = threadIdx.x; idx < tc * JB; idx += nmain) {
        const int tt = idx / JB, c = idx % JB;
        sV[tt * JP + c] =
            j0 + c < dv ? ldx<T>(src + (int64_t)(t0 + tt) * a.ld + a.v0 +
                                 h * dv + j0 + c)
                        : 0.f;
      }
      if constexpr (KIND == kGla)
        for (int idx = threadIdx.x; idx < tc * a.rank; idx += nmain) {
          const int tt = idx / a.rank, r = idx % a.rank;
          sZ[idx] = ldx<T>(src + (int64_t)(t0 + tt) * a.ld + a.a0 + r);
        }
    }
    __syncthreads();
    if constexpr (KIND == kGla) {
      // decays of four tokens per work item (a weight is read once for them)
      const int groups = (tc + 3) / 4;
      for (int idx = threadIdx.x; idx < DR * groups; idx += nmain) {
        const int i = idx % DR, tg = (idx / DR) * 4;
        float z[4] = {0.f, 0.f, 0.f, 0.f};
        if (i < d) {
          const float* wp = a.a2t + h * d + i;
#pragma unroll
          for (int u = 0; u < 4; ++u) z[u] = a.ab[h * d + i];
#pragma unroll 4
          for (int r = 0; r < a.rank; ++r) {
            const float w = wp[(int64_t)r * a.H * d];
#pragma unroll
            for (int u = 0; u < 4; ++u)
              z[u] = fmaf(w, sZ[min(tg + u, tc - 1) * a.rank + r], z[u]);
          }
        }
        const int at = (i / R) * (R + 4) + (i % R);
#pragma unroll
        for (int u = 0; u < 4; ++u)
          if (tg + u < tc)
            sA[(tg + u) * DP + at] =
                i < d ? decay_of(z[u], a.inv_tau) : 0.f;
      }
      __syncthreads();
    }
    for (int tt = 0; tt < tc; ++tt) {
      const int base = tt * DP + sl * (R + 4);
      const float4* kp = reinterpret_cast<const float4*>(sK + base);
      const float4* qp = reinterpret_cast<const float4*>(sQ + base);
      float vj = sV[tt * JP + jl], acc = 0.f;
      if constexpr (KIND == kGla) {
        const float4* ap = reinterpret_cast<const float4*>(sA + base);
#pragma unroll
        for (int r4 = 0; r4 < R / 4; ++r4) {
          const float4 kv = kp[r4], qv = qp[r4], av = ap[r4];
          S[4 * r4 + 0] = fmaf(kv.x, vj, av.x * S[4 * r4 + 0]);
          S[4 * r4 + 1] = fmaf(kv.y, vj, av.y * S[4 * r4 + 1]);
          S[4 * r4 + 2] = fmaf(kv.z, vj, av.z * S[4 * r4 + 2]);
          S[4 * r4 + 3] = fmaf(kv.w, vj, av.w * S[4 * r4 + 3]);
          acc = fmaf(S[4 * r4 + 0], qv.x, acc);
          acc = fmaf(S[4 * r4 + 1], qv.y, acc);
          acc = fmaf(S[4 * r4 + 2], qv.z, acc);
          acc = fmaf(S[4 * r4 + 3], qv.w, acc);
        }
      } else {
        const float keep = sKeep[tt];
        vj *= sPut[tt];
#pragma unroll
        for (int r4 = 0; r4 < R / 4; ++r4) {
          const float4 kv = kp[r4], qv = qp[r4];
          S[4 * r4 + 0] = fmaf(kv.x, vj, keep * S[4 * r4 + 0]);
          S[4 * r4 + 1] = fmaf(kv.y, vj, keep * S[4 * r4 + 1]);
          S[4 * r4 + 2] = fmaf(kv.z, vj, keep * S[4 * r4 + 2]);
          S[4 * r4 + 3] = fmaf(kv.w, vj, keep * S[4 * r4 + 3]);
          acc = fmaf(S[4 * r4 + 0], qv.x, acc);
          acc = fmaf(S[4 * r4 + 1], qv.y, acc);
          acc = fmaf(S[4 * r4 + 2], qv.z, acc);
          acc = fmaf(S[4 * r4 + 3], qv.w, acc);
        }
      }
      for (int off = NS >> 1; off > 0; off >>= 1)
        acc += __shfl_xor(acc, off, 64);
      if (sl == 0) sO[tt * JP + jl] = acc;
    }
    __syncthreads();
    for (int idx = threadIdx.x; idx < tc * JB; idx += blockDim.x) {
      const int tt = idx / JB, c = idx % JB;
      if (j0 + c >= dv) continue;
      float v = sO[tt * JP + c];
      if constexpr (KIND == kMlstm)
        v /= fmaxf(fabsf(sO[tt * JP + JB]), sEm[tt]) + kDenEps;
      a.o[((int64_t)b * a.T + t0 + tt) * (int64_t)a.H * dv + h * dv + j0 + c] = v;
    }
  }
#pragma unroll
  for (int r = 0; r < R; ++r) {
    const int row = sl * R + r;
    if (row >= d) continue;
    if (ncol) {
      if (lane < NS) np[row] = S[r];
    } else if (col_ok) {
      sp[(int64_t)row * dv + j] = S[r];
    }
  }
  if (ncol && lane == 0) *mp = m;
}

// ---- prompts in chunks on the matrix cores -------------------------------------
using f32x4 = __attribute__((ext_vector_type(4))) float;

// sum over the 16 lanes of a row, in every lane
template <int CTRL> __device__ __forceinline__ float row_rot(float x) {
  union { float f; int i; } u;
  u.f = x;
  u.i = __builtin_amdgcn_update_dpp(0, u.i, CTRL, 0xf, 0xf, true);
  return u.f;
}
__device__ __forceinline__ float row16_sum(float x) {
  x += row_rot<0x128>(x);                   // row_ror:8, 4, 2, 1
  x += row_rot<0x124>(x);
  x += row_rot<0x122>(x);
  x += row_rot<0x121>(x);
  return x;
}

// x times the values of the lower lanes of its row of 16 (inclusive product)
template <int CTRL> __device__ __forceinline__ float row_shift1(float x) {
  union { float f; int i; } u, one;
  u.f = x;
  one.f = 1.f;                              // lanes without a source
  u.i = __builtin_amdgcn_update_dpp(one.i, u.i, CTRL, 0xf, 0xf, false);
  return u.f;
}
__device__ __forceinline__ float row16_prod_upto(float x) {
  x *= row_shift1<0x111>(x);                // row_shr:1, 2, 4, 8
  x *= row_shift1<0x112>(x);
  x *= row_shift1<0x114>(x);
  x *= row_shift1<0x118>(x);
  return x;
}
__device__ __forceinline__ float from_lane(float x, int l) {
  union { float f; int i; } u;
  u.f = x;
  u.i = __builtin_amdgcn_readlane(u.i, l);
  return u.f;
}

constexpr int kTok = 16;                    // tokens of a chunk
constexpr int kAP = 20;                     // LDS pitch of a row of A

// LDS floats of a chunk kernel with DPAD key rows and JB columns
__host__ __device__ constexpr int chunk_lds(int kind, int DPAD, int JB) {
  return kTok * (DPAD + 4) * (kind == kGla ? 3 : 2) + kTok * (JB + 4) +
         kTok * kAP + DPAD + (kind == kGla ? 4 * DPAD : 9 * kTok);
}

// decays of a prompt's tokens: grid (channel tiles, token tiles), a thread walks
// 16 tokens of one channel, every weight read once for them
template <typename T>
__global__ __launch_bounds__(256) void low_rank_decay_kernel(
    const ScanArgs a, float* __restrict__ alpha, const int64_t M) {
  extern __shared__ __attribute__((aligned(16))) float sm[];   // [rank][16]
  const int64_t m0 = (int64_t)blockIdx.y * kTok;
  const int mt = (int)min((int64_t)kTok, M - m0);
  const int HD = a.H * a.d, c = blockIdx.x * 256 + threadIdx.x;
  const T* src = reinterpret_cast<const T*>(a.src);
  for (int idx = threadIdx.x; idx < kTok * a.rank; idx += 256) {
    const int tt = idx / a.rank, r = idx % a.rank;
    sm[r * kTok + tt] = ldx<T>(src + (m0 + min(tt, mt - 1)) * a.ld + a.a0 + r);
  }
  __syncthreads();
  if (c >= HD) return;
  float z[kTok];
  const float ab = a.ab[c];
#pragma unroll
  for (int t = 0; t < kTok; ++t) z[t] = ab;
#pragma unroll 4
  for (int r = 0; r < a.rank; ++r) {
    const float w = a.a2t[(int64_t)r * HD + c];
#pragma unroll
    for (int q = 0; q < kTok / 4; ++q) {
      const float4 x = *reinterpret_cast<const float4*>(sm + r * kTok + q * 4);
      z[4 * q + 0] = fmaf(w, x.x, z[4 * q + 0]);
      z[4 * q + 1] = fmaf(w, x.y, z[4 * q + 1]);
      z[4 * q + 2] = fmaf(w, x.z, z[4 * q + 2]);
      z[4 * q + 3] = fmaf(w, x.w, z[4 * q + 3]);
    }
  }
#pragma unroll
  for (int t = 0; t < kTok; ++t)
    if (t < mt) alpha[(m0 + t) * HD + c] = decay_of(z[t], a.inv_tau);
}

// grid (H * column blocks, B), 4 waves of CF x 16 columns; the matrix memory has
// a fifth wave that forms the next chunk's gates and running maximum while the
// others work on the current one. M4 = key rows / 64. Fragments of
// v_mfma_f32_16x16x4_f32: lane (c = lane & 15, hi = lane >> 4) holds A[c][hi],
// B[hi][c] and rows hi*4 + r of column c of the result. The sum over k may run
// in any order: step r takes rows hi*4 + r, which are what a lane's state
// fragment holds in register r, and one 16 B read of an A row.
template <typename T, int M4, int CF, int KIND>
__global__ __launch_bounds__(M4 == 4 && KIND == kGla ? 256 : 320)
void linear_chunk_kernel(const ScanArgs a) {
  constexpr int DPAD = M4 * 64, DF = M4 * 4, DP = DPAD + 4;
  constexpr int JB = 64 * CF, VP = JB + 4;
  constexpr int QN = kTok * DPAD / 256, VN = kTok * JB / 256;
  const int NB = (a.dv + JB - 1) / JB;      // column blocks
  const int h = blockIdx.x / NB, blk = blockIdx.x % NB, b = blockIdx.y;
  const int n = a.lens ? min(a.lens[b], a.T) : a.T;
  const int slot = a.slots ? a.slots[b] : b;
  const int p0 = a.pos[b];
  if (n <= 0 || slot < 0 || slot >= a.Bc || p0 < 0) return;   // uniform
  const int d = a.d, dv = a.dv, j0 = blk * JB, tid = threadIdx.x;
  const int wave = tid >> 6, lane = tid & 63, c16 = lane & 15, hi = lane >> 4;
  const bool work = wave < 4;               // else: the gates' wave

  extern __shared__ __attribute__((aligned(16))) float sm[];
  float* sQ = sm;                           // [16][DP]
  float* sK = sQ + kTok * DP;               // [16][DP]
  float* sAl = sK + kTok * DP;              // gla: decays [16][DP]
  float* sV = sAl + (KIND == kGla ? kTok * DP : 0);   // [16][VP]
  float* sAm = sV + kTok * VP;              // [16][kAP]
  float* sE = sAm + kTok * kAP;             // gla: the chunk's decays; mlstm: n
  float* sGp = sE + DPAD;                   // gla: decays of 4 tokens [4][DPAD]
  float* sGate = sE + DPAD;                 // mlstm: 2 x (keep, put, e^-m, keeps
                                            // up to t) [16]
  float* sDen = sGate + 8 * kTok;           // mlstm: 1 / denominator [16]

  f32x4 S[CF][DF];
  float* sp = a.state + (((int64_t)slot * a.H + h) * d) * dv;
#pragma unroll
  for (int f = 0; f < CF; ++f) {
    const int j = j0 + (wave * CF + f) * 16 + c16;
#pragma unroll
    for (int g = 0; g < DF; ++g)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int row = g * 16 + hi * 4 + r;
        S[f][g][r] = work && p0 > 0 && row < d && j < dv
                         ? sp[(int64_t)row * dv + j] : 0.f;
      }
  }
  // copies of n and m that belong to this block
  const int tile0 = blk * CF, tile1 = min(tile0 + CF, a.NT);
  float m = 0.f, ib = 0.f, fb = 0.f;
  const int ci = tid % DPAD;                // a thread's channel when staging
  if constexpr (KIND == kMlstm) {
    const float* np = a.nst + (((int64_t)slot * a.H + h) * a.NT + tile0) * d;
    if (work)
      for (int i = tid; i < DPAD; i += 256)
        sE[i] = p0 > 0 && i < d ? np[i] : 0.f;
    if (p0 > 0) m = a.mst[((int64_t)slot * a.H + h) * a.NT + tile0];
    ib = a.ib[h];
    fb = a.fb[h];
  }

  // The next chunk's projection values travel into registers: loads without
  // conditions (out-of-range ones repeat a valid element and are dropped where
  // they are stored to LDS).
  const T* src = reinterpret_cast<const T*>(a.src) + (int64_t)b * a.T * a.ld;
  T rq[QN], rk[QN], rv[VN];
  float ra[M4][4];                          // gla: decays of four tokens
  const int qc = h * d + min(ci, d - 1);
  const int vcol = tid % JB, vc = h * dv + min(j0 + vcol, dv - 1);
  const int ldi = (int)a.ld;
  auto fetch = [&](const int t0) {
    const int last = min(kTok, n - t0) - 1;
    const T* row = src + (int64_t)t0 * a.ld;
    const T* q = row + a.q0 + qc;
    const T* k = row + a.k0 + qc;
    const T* v = row + a.v0 + vc;
#pragma unroll
    for (int u = 0; u < QN; ++u) {
      const int at = min((tid + u * 256) / DPAD, last) * ldi;
      rq[u] = q[at];
      rk[u] = k[at];
    }
#pragma unroll
    for (int u = 0; u < VN; ++u)
      rv[u] = v[min((tid + u * 256) / JB, last) * ldi];
    if constexpr (KIND == kGla) {
      const float* al = a.alpha + ((int64_t)b * a.T + t0) * a.H * d + qc;
#pragma unroll
      for (int u0 = 0; u0 < M4; ++u0)
#pragma unroll
        for (int u = 0; u < 4; ++u)
          ra[u0][u] = al[min(((tid + u0 * 256) / DPAD) * 4 + u, last) *
                         (a.H * d)];
    }
  };
  // gates of the chunk at t0 into buffer buf (mlstm, the fifth wave)
  auto gates = [&](const int t0, float* g) {
    const int tc = min(kTok, n - t0);
    const T* sr = src + (int64_t)(t0 + min(lane, tc - 1)) * a.ld + h;
    const float gi = ldx<T>(sr + a.i0), gf = ldx<T>(sr + a.f0);
    const float li = a.cap * tanhf((gi + ib) / a.cap);
    const float lf = log_sigmoid(a.cap * tanhf((gf + fb) / a.cap));
    float before = 0.f, after = 0.f;
#pragma unroll
    for (int t = 0; t < kTok; ++t) {        // the running maximum, in order
      const float f = from_lane(lf, t), i = from_lane(li, t);
      const float mn = fmaxf(f + m, i);
      if (lane == t) {
        before = f + m;
        after = mn;
      }
      if (t < tc) m = mn;
    }
    const bool real = lane < tc;            // neutral tokens behind the last
    const float keep = real ? expf(before - after) : 1.f;
    const float prod = row16_prod_upto(keep);
    if (lane < kTok) {
      g[lane] = keep;
      g[kTok + lane] = real ? expf(li - after) : 0.f;
      g[2 * kTok + lane] = expf(-after);
      g[3 * kTok + lane] = prod;
    }
  };
  if (work) fetch(0);
  else gates(0, sGate);

  int buf = 0;
  for (int t0 = 0; t0 < n; t0 += kTok, buf ^= 1) {
    const int tc = min(kTok, n - t0);
    const float* sKeep = sGate + buf * 4 * kTok;
    const float* sPut = sKeep + kTok;
    const float* sEm = sPut + kTok;
    const float* sP = sEm + kTok;           // products of keep up to t
    float al[M4][4];                        // gla: own decays
    __syncthreads();                        // previous chunk consumed
    if (work) {
#pragma unroll
      for (int u = 0; u < QN; ++u) {
        const int tt = (tid + u * 256) / DPAD, at = tt * DP + ci;
        const bool in = tt < tc && ci < d;
        sQ[at] = in ? ldx<T>(&rq[u]) * a.qscale : 0.f;
        sK[at] = in ? ldx<T>(&rk[u]) : 0.f;
      }
#pragma unroll
      for (int u = 0; u < VN; ++u) {
        const int tt = (tid + u * 256) / JB;
        sV[tt * VP + vcol] =
            tt < tc && j0 + vcol < dv ? ldx<T>(&rv[u]) : 0.f;
      }
      if constexpr (KIND == kGla) {
#pragma unroll
        for (int u0 = 0; u0 < M4; ++u0) {
          const int tg = ((tid + u0 * 256) / DPAD) * 4;
          float p = 1.f;
#pragma unroll
          for (int u = 0; u < 4; ++u) {
            al[u0][u] = tg + u < tc ? ra[u0][u] : 1.f;
            sAl[(tg + u) * DP + ci] = al[u0][u];
            p *= al[u0][u];
          }
          sGp[(tg / 4) * DPAD + ci] = p;
        }
      }
    }
    __syncthreads();
    if (work && t0 + kTok < n) fetch(t0 + kTok);
    if (work) {
      // A, and the keys carried to the chunk's end: 16 lanes per key s, four
      // channels of every 64 per lane; lane sl keeps A[sl][s]
      const int s = tid >> 4, sl = tid & 15;
      float4 k4[M4], w4[M4];
      const float put = KIND == kMlstm ? sPut[s] : 1.f;
      float carried = 0.f, mine = 0.f;      // mlstm: the key's scalar factor
#pragma unroll
      for (int q = 0; q < M4; ++q) {
        k4[q] = *reinterpret_cast<const float4*>(sK + s * DP + q * 64 + sl * 4);
        w4[q] = make_float4(0.f, 0.f, 0.f, 0.f);
      }
#pragma unroll 1
      for (int tg = 0; tg < kTok; tg += 4) {
#pragma unroll
        for (int u = 0; u < 4; ++u) {
          const int t = tg + u;
          const bool own = t == s;
          float acc = 0.f;
#pragma unroll
          for (int q = 0; q < M4; ++q) {
            const int at = t * DP + q * 64 + sl * 4;
            const float4 qv = *reinterpret_cast<const float4*>(sQ + at);
            float4 w = k4[q];
            if constexpr (KIND == kGla) {
              const float4 av = *reinterpret_cast<const float4*>(sAl + at);
              w.x = own ? k4[q].x : w4[q].x * av.x;
              w.y = own ? k4[q].y : w4[q].y * av.y;
              w.z = own ? k4[q].z : w4[q].z * av.z;
              w.w = own ? k4[q].w : w4[q].w * av.w;
              w4[q] = w;
            }
            acc = fmaf(qv.x, w.x, acc);
            acc = fmaf(qv.y, w.y, acc);
            acc = fmaf(qv.z, w.z, acc);
            acc = fmaf(qv.w, w.w, acc);
          }
          if constexpr (KIND == kMlstm) {
            carried = own ? put : carried * sKeep[t];
            acc *= carried;
          }
          acc = row16_sum(acc);
          if (sl == t) mine = acc;
        }
      }
      sAm[sl * kAP + s] = mine;
#pragma unroll
      for (int q = 0; q < M4; ++q) {
        if constexpr (KIND == kMlstm)
          w4[q] = make_float4(k4[q].x * carried, k4[q].y * carried,
                              k4[q].z * carried, k4[q].w * carried);
        *reinterpret_cast<float4*>(sK + s * DP + q * 64 + sl * 4) = w4[q];
      }
    } else if (t0 + kTok < n) {
      gates(t0 + kTok, sGate + (buf ^ 1) * 4 * kTok);
    }
    __syncthreads();
    if constexpr (KIND == kGla) {
      // queries times the decays up to them; the whole chunk's decays
#pragma unroll
      for (int u0 = 0; u0 < M4; ++u0) {
        const int g = (tid + u0 * 256) / DPAD;
        const float g0 = sGp[ci], g1 = sGp[DPAD + ci], g2 = sGp[2 * DPAD + ci];
        float p = (g > 0 ? g0 : 1.f) * (g > 1 ? g1 : 1.f) * (g > 2 ? g2 : 1.f);
#pragma unroll
        for (int u = 0; u < 4; ++u) {
          p *= al[u0][u];
          sQ[(g * 4 + u) * DP + ci] *= p;
        }
        if (g == 3) sE[ci] = p;
      }
    } else if (work) {
      // n . q of every token: 16 lanes per token
      const int t = tid >> 4, l = tid & 15;
      const float at = sAm[t * kAP + l];
      float nq = 0.f;
#pragma unroll
      for (int q = 0; q < M4; ++q) {
        const float4 qv =
            *reinterpret_cast<const float4*>(sQ + t * DP + q * 64 + l * 4);
        const float4 nv = *reinterpret_cast<const float4*>(sE + q * 64 + l * 4);
        nq = fmaf(qv.x, nv.x, nq);
        nq = fmaf(qv.y, nv.y, nq);
        nq = fmaf(qv.z, nv.z, nq);
        nq = fmaf(qv.w, nv.w, nq);
      }
      nq = row16_sum(fmaf(nq, sP[t], at));  // (A is zero above the diagonal)
      if (l == 0) sDen[t] = 1.f / (fmaxf(fabsf(nq), sEm[t]) + kDenEps);
    }
    __syncthreads();
    if (work) {
      const float pq = KIND == kMlstm ? sP[c16] : 1.f;
      const float pc = KIND == kMlstm ? sP[kTok - 1] : 1.f;
      // A row c16, entries hi*4 .. +3
      const float4 a4 =
          *reinterpret_cast<const float4*>(sAm + c16 * kAP + hi * 4);
      const float am[4] = {a4.x, a4.y, a4.z, a4.w};
      float bv[CF][4];
      f32x4 o[CF];
#pragma unroll
      for (int f = 0; f < CF; ++f) {
        o[f] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int r = 0; r < 4; ++r)
          bv[f][r] = sV[(hi * 4 + r) * VP + (wave * CF + f) * 16 + c16];
      }
#pragma unroll
      for (int r = 0; r < 4; ++r)
#pragma unroll
        for (int f = 0; f < CF; ++f)
          o[f] = __builtin_amdgcn_mfma_f32_16x16x4f32(am[r], bv[f][r], o[f], 0,
                                                      0, 0);
#pragma unroll
      for (int g = 0; g < DF; ++g) {
        const float4 q4 =
            *reinterpret_cast<const float4*>(sQ + c16 * DP + g * 16 + hi * 4);
        const float qr[4] = {q4.x * pq, q4.y * pq, q4.z * pq, q4.w * pq};
        float e[4] = {pc, pc, pc, pc};
        if constexpr (KIND == kGla) {
          const float4 e4 =
              *reinterpret_cast<const float4*>(sE + g * 16 + hi * 4);
          e[0] = e4.x; e[1] = e4.y; e[2] = e4.z; e[3] = e4.w;
        }
        float ka[4];
#pragma unroll
        for (int r = 0; r < 4; ++r)
          ka[r] = sK[(hi * 4 + r) * DP + g * 16 + c16];
#pragma unroll
        for (int r = 0; r < 4; ++r)
#pragma unroll
          for (int f = 0; f < CF; ++f)
            o[f] = __builtin_amdgcn_mfma_f32_16x16x4f32(qr[r], S[f][g][r], o[f],
                                                        0, 0, 0);
#pragma unroll
        for (int f = 0; f < CF; ++f) {
#pragma unroll
          for (int r = 0; r < 4; ++r) S[f][g][r] *= e[r];
#pragma unroll
          for (int r = 0; r < 4; ++r)
            S[f][g] = __builtin_amdgcn_mfma_f32_16x16x4f32(ka[r], bv[f][r],
                                                           S[f][g], 0, 0, 0);
        }
      }
#pragma unroll
      for (int f = 0; f < CF; ++f) {
        const int j = j0 + (wave * CF + f) * 16 + c16;
        float* op = a.o + ((int64_t)b * a.T + t0 + hi * 4) * a.H * dv + h * dv + j;
        float4 den = make_float4(1.f, 1.f, 1.f, 1.f);
        if constexpr (KIND == kMlstm)
          den = *reinterpret_cast<const float4*>(sDen + hi * 4);
        const float dn[4] = {den.x, den.y, den.z, den.w};
#pragma unroll
        for (int r = 0; r < 4; ++r)
          if (hi * 4 + r < tc && j < dv)
            op[(int64_t)r * a.H * dv] =
                KIND == kMlstm ? o[f][r] * dn[r] : o[f][r];
      }
      if constexpr (KIND == kMlstm)         // n was last read before the barrier
        for (int i = tid; i < DPAD; i += 256) {
          float v = sE[i] * pc;
#pragma unroll
          for (int t = 0; t < kTok; ++t) v += sK[t * DP + i];
          sE[i] = v;
        }
    }
  }
#pragma unroll
  for (int f = 0; f < CF; ++f) {
    const int j = j0 + (wave * CF + f) * 16 + c16;
#pragma unroll
    for (int g = 0; g < DF; ++g)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int row = g * 16 + hi * 4 + r;
        if (work && row < d && j < dv) sp[(int64_t)row * dv + j] = S[f][g][r];
      }
  }
  if constexpr (KIND == kMlstm) {
    for (int tile = tile0; tile < tile1; ++tile) {
      float* np = a.nst + (((int64_t)slot * a.H + h) * a.NT + tile) * d;
      if (work)
        for (int i = tid; i < d; i += 256) np[i] = sE[i];   // own elements
      else if (lane == 0)
        a.mst[((int64_t)slot * a.H + h) * a.NT + tile] = m;
    }
  }
}

// ---- one decode step -----------------------------------------------------------
// grid (H, B). Thread (row group, column lane): V neighbouring columns of every
// RG-th state row, the first rows in flight while the gates are formed.
struct StepTail {
  const float* w;            // norm weight [H*dv]
  void* out;                 // [B, H*dv], row stride out_ld
  int64_t out_ld;
  int g0, silu;              // gate columns of src
  float eps;
};

template <typename T> __device__ __forceinline__ void stx(T* p, float v);
template <> __device__ __forceinline__ void stx<float>(float* p, float v) { *p = v; }
template <> __device__ __forceinline__ void stx<short>(short* p, float v) { *p = f2bits(v); }

template <int V> struct vecf { float v[V]; };
template <int V> __device__ __forceinline__ vecf<V> ldf(const float* p) {
  vecf<V> r;
  if constexpr (V == 4) {
    const float4 t = *reinterpret_cast<const float4*>(p);
    r.v[0] = t.x; r.v[1] = t.y; r.v[2] = t.z; r.v[3] = t.w;
  } else {
    r.v[0] = *p;
  }
  return r;
}
template <int V> __device__ __forceinline__ void stf(float* p, const vecf<V>& r) {
  if constexpr (V == 4)
    *reinterpret_cast<float4*>(p) = make_float4(r.v[0], r.v[1], r.v[2], r.v[3]);
  else *p = r.v[0];
}

constexpr int kStepRows = 8;   // state rows of a thread in flight

template <typename T, int V, int KIND>
__global__ __launch_bounds__(256) void linear_step_kernel(const ScanArgs a,
                                                          const StepTail e) {
  const int h = blockIdx.x, b = blockIdx.y, tid = threadIdx.x;
  const int d = a.d, dv = a.dv;
  T* op = reinterpret_cast<T*>(e.out) + b * e.out_ld + (int64_t)h * dv;
  const int slot = a.slots ? a.slots[b] : b;
  const int p0 = a.pos[b];
  if ((a.lens && a.lens[b] <= 0) || slot < 0 || slot >= a.Bc || p0 < 0) {
    for (int c = tid; c < dv; c += 256) stx<T>(op + c, 0.f);   // idle row
    return;
  }
  extern __shared__ __attribute__((aligned(16))) float sm[];
  float* sQ = sm;                           // [d]
  float* sK = sQ + d;
  float* sA = sK + d;                       // gla: decays
  float* sP = sm + (3 * d + 3) / 4 * 4;     // [RG][columns of one pass]
  __shared__ float red[8];
  const T* src = reinterpret_cast<const T*>(a.src) + (int64_t)b * a.ld;
  const int CT = (dv + V - 1) / V;          // column lanes of the head
  const int CL = min(CT, 256);              // ... of one pass
  const int RG = 256 / CL;
  const int rg = tid / CL, cl = tid % CL;
  float* sO = sP + RG * CL * V;             // [dv]
  float* st = a.state + ((int64_t)slot * a.H + h) * d * dv;
  const bool old = p0 > 0;

  vecf<V> pre[kStepRows];
#pragma unroll
  for (int u = 0; u < kStepRows; ++u) {
    const int row = rg + u * RG;
#pragma unroll
    for (int j = 0; j < V; ++j) pre[u].v[j] = 0.f;
    if (old && rg < RG && row < d)
      pre[u] = ldf<V>(st + (int64_t)row * dv + cl * V);
  }
  float keep = 1.f, put = 1.f, floor_ = 0.f, nq = 0.f;
  if constexpr (KIND == kMlstm) {
    float* mp = a.mst + ((int64_t)slot * a.H + h) * a.NT;
    const float m = old ? *mp : 0.f;
    const float i = a.cap * tanhf((ldx<T>(src + a.i0 + h) + a.ib[h]) / a.cap);
    const float f = log_sigmoid(
        a.cap * tanhf((ldx<T>(src + a.f0 + h) + a.fb[h]) / a.cap));
    const float mn = fmaxf(f + m, i);
    keep = expf(f + m - mn);
    put = expf(i - mn);
    floor_ = expf(-mn);
    __syncthreads();                        // every thread has read m
    if (tid < a.NT) mp[tid] = mn;
    for (int t = tid + 256; t < a.NT; t += 256) mp[t] = mn;
  }
  for (int i = tid; i < d; i += 256) {
    const float q = ldx<T>(src + a.q0 + h * d + i) * a.qscale;
    const float k = ldx<T>(src + a.k0 + h * d + i);
    sQ[i] = q;
    sK[i] = k;
    if constexpr (KIND == kGla) {
      float z = a.ab[h * d + i];
      const float* wp = a.a2t + h * d + i;
#pragma unroll 16
      for (int r = 0; r < a.rank; ++r)
        z = fmaf(wp[(int64_t)r * a.H * d], ldx<T>(src + a.a0 + r), z);
      sA[i] = decay_of(z, a.inv_tau);
    } else {
      // the normalizer, every column tile's copy
      float* np = a.nst + ((int64_t)slot * a.H + h) * a.NT * d + i;
      const float nn = fmaf(put, k, keep * (old ? *np : 0.f));
      for (int t = 0; t < a.NT; ++t) np[(int64_t)t * d] = nn;
      nq = fmaf(nn, q, nq);
    }
  }
  if constexpr (KIND == kMlstm) nq = block_reduce_sum(nq, red);
  __syncthreads();
  for (int c0 = 0; c0 < CT; c0 += CL) {     // one pass up to 256 V columns
    const int col = (c0 + cl) * V;
    const bool on = rg < RG && c0 + cl < CT;
    vecf<V> v, acc;
#pragma unroll
    for (int j = 0; j < V; ++j) {
      v.v[j] = on ? ldx<T>(src + a.v0 + h * dv + col + j) * put : 0.f;
      acc.v[j] = 0.f;
    }
    if (on)
      for (int r0 = rg; r0 < d; r0 += RG * kStepRows) {
        vecf<V> s[kStepRows];
        const bool first = c0 == 0 && r0 == rg;
#pragma unroll
        for (int u = 0; u < kStepRows; ++u) {
          const int row = r0 + u * RG;
          s[u] = pre[u];
          if (!first && row < d) {
#pragma unroll
            for (int j = 0; j < V; ++j) s[u].v[j] = 0.f;
            if (old) s[u] = ldf<V>(st + (int64_t)row * dv + col);
          }
        }
#pragma unroll
        for (int u = 0; u < kStepRows; ++u) {
          const int row = r0 + u * RG;
          if (row >= d) continue;
          const float k = sK[row], q = sQ[row];
          const float g = KIND == kGla ? sA[row] : keep;
#pragma unroll
          for (int j = 0; j < V; ++j) {
            s[u].v[j] = fmaf(k, v.v[j], g * s[u].v[j]);
            acc.v[j] = fmaf(s[u].v[j], q, acc.v[j]);
          }
          stf<V>(st + (int64_t)row * dv + col, s[u]);
        }
      }
    __syncthreads();                        // sP of the last pass consumed
    if (on)
#pragma unroll
      for (int j = 0; j < V; ++j) sP[(rg * CL + cl) * V + j] = acc.v[j];
    __syncthreads();
    for (int c = tid; c < CL * V && c0 * V + c < dv; c += 256) {
      float o = 0.f;
      for (int r = 0; r < RG; ++r) o += sP[r * CL * V + c];
      sO[c0 * V + c] = o;
    }
  }
  __syncthreads();
  float inv = 1.f;
  if constexpr (KIND == kMlstm) inv = 1.f / (fmaxf(fabsf(nq), floor_) + kDenEps);
  float ss = 0.f;
  for (int c = tid; c < dv; c += 256) {
    const float o = sO[c] * inv;
    ss = fmaf(o, o, ss);
  }
  ss = block_reduce_sum(ss, red);
  const float r = inv / sqrtf(ss / (float)dv + e.eps);
  for (int c = tid; c < dv; c += 256) {
    const float g = ldx<T>(src + e.g0 + h * dv + c);
    float s = 1.f / (1.f + expf(-g));
    if (e.silu) s *= g;
    stx<T>(op + c, sO[c] * r * e.w[h * dv + c] * s);
  }
}

const int* idx32(const torch::Tensor& t, int64_t n) {
  DNET_CHECK(t.scalar_type() == torch::kInt32 && t.is_contiguous() &&
                 t.numel() >= n, "int32 index tensor [B]");
  return t.data_ptr<int>();
}

const float* f32p(const torch::Tensor& t, int64_t n, const char* what) {
  DNET_CHECK(is_f32(t) && t.is_contiguous() && t.numel() == n, what);
  return t.data_ptr<float>();
}

// shared part of the entry points: checks and geometry
void fill_args(ScanArgs& a, const torch::Tensor& src, int64_t q0, int64_t k0,
               int64_t v0, double qscale, torch::Tensor& state,
               const torch::Tensor& pos,
               const c10::optional<torch::Tensor>& lens,
               const c10::optional<torch::Tensor>& slots, int64_t T,
               int64_t NT) {
  const int64_t M = src.size(0), ld = src.size(1);
  DNET_CHECK(src.dim() == 2 && src.is_contiguous() &&
                 (is_bf16(src) || is_f32(src)), "src [B*T, ld]");
  DNET_CHECK(T > 0 && M % T == 0, "rows = B*T");
  const int64_t B = M / T;
  DNET_CHECK(is_f32(state) && state.is_contiguous() && state.dim() == 4,
             "state fp32 [Bc, H, d, dv]");
  const int64_t H = state.size(1), d = state.size(2), dv = state.size(3);
  DNET_CHECK(q0 >= 0 && k0 >= 0 && v0 >= 0 && q0 + H * d <= ld &&
                 k0 + H * d <= ld && v0 + H * dv <= ld, "src columns");
  DNET_CHECK(d >= 1 && d <= 512 && dv >= 1, "1 <= head size <= 512");
  if (!slots.has_value()) DNET_CHECK(B <= state.size(0), "more rows than slots");
  a.src = src.data_ptr();
  a.state = state.data_ptr<float>();
  a.pos = idx32(pos, B);
  a.lens = lens.has_value() ? idx32(*lens, B) : nullptr;
  a.slots = slots.has_value() ? idx32(*slots, B) : nullptr;
  a.ld = ld; a.q0 = (int)q0; a.k0 = (int)k0; a.v0 = (int)v0;
  a.T = (int)T; a.Bc = (int)state.size(0); a.H = (int)H; a.d = (int)d;
  a.dv = (int)dv; a.qscale = (float)qscale; a.NT = (int)NT;
}

void scan_launch(ScanArgs& a, int kind, const torch::Tensor& src,
                 torch::Tensor& o) {
  const int64_t M = src.size(0), B = M / a.T, T = a.T, NT = a.NT;
  const int64_t H = a.H, d = a.d, dv = a.dv;
  DNET_CHECK(is_f32(o) && o.is_contiguous() && o.size(0) == M &&
                 o.size(1) == H * dv, "o fp32 [B*T, H*dv]");
  if (M == 0) return;
  a.o = o.data_ptr<float>();
  auto st = current_stream();
  // the copies of n and m belong to 64 columns each there
  const bool tiles64 = NT == (dv + 63) / 64;
  const int M4 = d <= 64 ? 1 : (d <= 128 ? 2 : 4);
  // two column fragments per wave when that still fills the chip
  const int CF = dv > 64 && M4 < 4 && H * B * ((dv + 127) / 128) >= 256 ? 2 : 1;
  const size_t clds =
      (size_t)chunk_lds(kind, M4 * 64, 64 * CF) * sizeof(float);
  const size_t dlds = (size_t)kTok * a.rank * sizeof(float);
  if (d <= 256 && tiles64 && clds <= 64 * 1024 && dlds <= 64 * 1024) {
    torch::Tensor alpha;
    if (kind == kGla) {
      alpha = torch::empty({M, H * d}, o.options());
      a.alpha = alpha.data_ptr<float>();
      const dim3 dgrid((unsigned)((H * d + 255) / 256),
                       (unsigned)((M + kTok - 1) / kTok));
      if (is_bf16(src))
        hipLaunchKernelGGL((low_rank_decay_kernel<short>), dgrid, dim3(256),
                           dlds, st, a, alpha.data_ptr<float>(), M);
      else
        hipLaunchKernelGGL((low_rank_decay_kernel<float>), dgrid, dim3(256),
                           dlds, st, a, alpha.data_ptr<float>(), M);
    }
    const dim3 cgrid((unsigned)(H * ((dv + 64 * CF - 1) / (64 * CF))),
                     (unsigned)B);
#define LC(TT, MM, CC, KK)                                                    \
  hipLaunchKernelGGL((linear_chunk_kernel<TT, MM, CC, KK>), cgrid,            \
                     dim3(KK == kMlstm ? 320 : 256), clds, st, a)
#define LC_M(TT, KK)                                                          \
  do {                                                                        \
    if (M4 == 4) LC(TT, 4, 1, KK);                                            \
    else if (M4 == 2) { if (CF == 2) LC(TT, 2, 2, KK); else LC(TT, 2, 1, KK); } \
    else { if (CF == 2) LC(TT, 1, 2, KK); else LC(TT, 1, 1, KK); }            \
  } while (0)
#define LC_K(TT) do { if (kind == kGla) LC_M(TT, kGla); else LC_M(TT, kMlstm); } while (0)
    if (is_bf16(src)) LC_K(short); else LC_K(float);
#undef LC_K
#undef LC_M
#undef LC
    return;
  }
  const int R = d <= 32 ? 8 : (d <= 128 ? 16 : 32);
  a.NS = 1;
  while (a.NS * R < d) a.NS *= 2;           // power of two, <= 16
  const int cols = (int)((dv + NT - 1) / NT);
  const int unit = kWave / a.NS;            // whole waves
  a.JB = (cols + unit - 1) / unit * unit;
  const int threads = a.JB * a.NS + (kind == kMlstm ? kWave : 0);
  DNET_CHECK(threads <= 1024, "column tiles too wide");
  const int DP = a.NS * (R + 4);
  auto floats = [&](int tc) {
    return (size_t)tc * ((kind == kGla ? 3 : 2) * DP + 2 * (a.JB + 1) +
                         (kind == kGla ? a.rank : 3));
  };
  a.TC = (int)std::min<int64_t>(16, T);
  while (a.TC > 1 && floats(a.TC) * sizeof(float) > 56 * 1024) a.TC /= 2;
  const size_t lds = floats(a.TC) * sizeof(float);
  DNET_CHECK(lds <= 64 * 1024, "linear_scan: sizes exceed LDS");
  const dim3 grid((unsigned)(H * NT), (unsigned)B);
#define LS(TT, RR, KK)                                                        \
  hipLaunchKernelGGL((linear_scan_kernel<TT, RR, KK>), grid, dim3(threads),   \
                     lds, st, a)
#define LS_R(TT, KK)                        \
  do {                                      \
    if (R == 8) LS(TT, 8, KK);              \
    else if (R == 16) LS(TT, 16, KK);       \
    else LS(TT, 32, KK);                    \
  } while (0)
#define LS_K(TT) do { if (kind == kGla) LS_R(TT, kGla); else LS_R(TT, kMlstm); } while (0)
  if (is_bf16(src)) LS_K(short); else LS_K(float);
#undef LS_K
#undef LS_R
#undef LS
}

// decode step of either kind with the head's norm, weight and output gate
void step_launch(ScanArgs& a, int kind, const torch::Tensor& src,
                 const torch::Tensor& w, int64_t g0, bool silu, double eps,
                 torch::Tensor& out) {
  const int64_t B = src.size(0), n = (int64_t)a.H * a.dv;
  StepTail e;
  e.w = f32p(w, n, "norm weight fp32 [H*dv]");
  DNET_CHECK(g0 >= 0 && g0 + n <= src.size(1), "gate columns");
  DNET_CHECK(out.dim() == 2 && out.size(0) == B && out.size(1) == n &&
                 out.stride(1) == 1 && (B <= 1 || out.stride(0) >= n) &&
                 out.scalar_type() == src.scalar_type(), "out [B, H*dv]");
  if (B == 0) return;
  e.out = out.data_ptr();
  e.out_ld = out.stride(0);
  e.g0 = (int)g0;
  e.silu = silu ? 1 : 0;
  e.eps = (float)eps;
  const bool v4 = a.dv % 4 == 0;
  const int V = v4 ? 4 : 1;
  const int CL = std::min((a.dv + V - 1) / V, 256);
  const size_t lds =
      ((3 * a.d + 3) / 4 * 4 + (256 / CL) * CL * V + a.dv) * sizeof(float);
  DNET_CHECK(lds <= 60 * 1024, "linear_step: sizes exceed LDS");
  const dim3 grid((unsigned)a.H, (unsigned)B);
  auto st = current_stream();
#define LP(TT, VV, KK)                                                        \
  hipLaunchKernelGGL((linear_step_kernel<TT, VV, KK>), grid, dim3(256), lds,  \
                     st, a, e)
#define LP_K(TT, VV) do { if (kind == kGla) LP(TT, VV, kGla); else LP(TT, VV, kMlstm); } while (0)
#define LP_V(TT) do { if (v4) LP_K(TT, 4); else LP_K(TT, 1); } while (0)
  if (is_bf16(src)) LP_V(short); else LP_V(float);
#undef LP_V
#undef LP_K
#undef LP
}

ScanArgs gla_args(const torch::Tensor& src, int64_t q0, int64_t k0, int64_t v0,
                  int64_t a0, const torch::Tensor& a2t, const torch::Tensor& ab,
                  double inv_tau, double qscale, torch::Tensor& state,
                  const torch::Tensor& pos,
                  const c10::optional<torch::Tensor>& lens,
                  const c10::optional<torch::Tensor>& slots, int64_t T) {
  ScanArgs a = {};
  // column tiles of up to 64
  fill_args(a, src, q0, k0, v0, qscale, state, pos, lens, slots, T,
            (state.size(3) + 63) / 64);
  const int64_t n = (int64_t)a.H * a.d;
  DNET_CHECK(a2t.dim() == 2 && a2t.size(1) == n, "a2t fp32 [rank, H*d]");
  a.rank = (int)a2t.size(0);
  DNET_CHECK(a.rank >= 1 && a.rank <= 2048 && a0 >= 0 &&
                 a0 + a.rank <= src.size(1), "low-rank columns");
  a.a2t = f32p(a2t, a.rank * n, "a2t fp32 [rank, H*d]");
  a.ab = f32p(ab, n, "ab fp32 [H*d]");
  a.a0 = (int)a0;
  a.inv_tau = (float)inv_tau;
  return a;
}

ScanArgs mlstm_args(const torch::Tensor& src, int64_t q0, int64_t k0,
                    int64_t v0, int64_t i0, int64_t f0, const torch::Tensor& ib,
                    const torch::Tensor& fb, double cap, double qscale,
                    torch::Tensor& state, torch::Tensor& nst,
                    torch::Tensor& mst, const torch::Tensor& pos,
                    const c10::optional<torch::Tensor>& lens,
                    const c10::optional<torch::Tensor>& slots, int64_t T) {
  ScanArgs a = {};
  DNET_CHECK(nst.dim() == 4, "n fp32 [Bc, H, tiles, d]");
  const int64_t NT = nst.size(2);
  fill_args(a, src, q0, k0, v0, qscale, state, pos, lens, slots, T, NT);
  const int64_t Bc = a.Bc, H = a.H, d = a.d;
  DNET_CHECK(nst.size(0) == Bc && nst.size(1) == H && nst.size(3) == d &&
                 NT >= 1 && (a.dv + NT - 1) / NT <= 64,
             "n fp32 [Bc, H, tiles, d], tiles of up to 64 columns");
  f32p(nst, Bc * H * NT * d, "n fp32 [Bc, H, tiles, d]");
  f32p(mst, Bc * H * NT, "m fp32 [Bc, H, tiles]");
  a.nst = nst.data_ptr<float>();
  a.mst = mst.data_ptr<float>();
  a.ib = f32p(ib, H, "gate bias fp32 [H]");
  a.fb = f32p(fb, H, "gate bias fp32 [H]");
  DNET_CHECK(i0 >= 0 && f0 >= 0 && i0 + H <= src.size(1) &&
                 f0 + H <= src.size(1), "gate columns");
  DNET_CHECK(cap > 0, "gate cap");
  a.i0 = (int)i0; a.f0 = (int)f0; a.cap = (float)cap;
  return a;
}

}  // namespace

void gla_scan(torch::Tensor src, int64_t q0, int64_t k0, int64_t v0, int64_t a0,
              torch::Tensor a2t, torch::Tensor ab, double inv_tau,
              double qscale, torch::Tensor state, torch::Tensor o,
              torch::Tensor pos, c10::optional<torch::Tensor> lens,
              c10::optional<torch::Tensor> slots, int64_t T) {
  ScanArgs a = gla_args(src, q0, k0, v0, a0, a2t, ab, inv_tau, qscale, state,
                        pos, lens, slots, T);
  scan_launch(a, kGla, src, o);
}

void gla_step(torch::Tensor src, int64_t q0, int64_t k0, int64_t v0, int64_t a0,
              torch::Tensor a2t, torch::Tensor ab, double inv_tau,
              double qscale, torch::Tensor state, torch::Tensor w, int64_t g0,
              bool silu, double eps, torch::Tensor out, torch::Tensor pos,
              c10::optional<torch::Tensor> lens,
              c10::optional<torch::Tensor> slots) {
  ScanArgs a = gla_args(src, q0, k0, v0, a0, a2t, ab, inv_tau, qscale, state,
                        pos, lens, slots, 1);
  step_launch(a, kGla, src, w, g0, silu, eps, out);
}

void mlstm_scan(torch::Tensor src, int64_t q0, int64_t k0, int64_t v0,
                int64_t i0, int64_t f0, torch::Tensor ib, torch::Tensor fb,
                double cap, double qscale, torch::Tensor state,
                torch::Tensor nst, torch::Tensor mst, torch::Tensor o,
                torch::Tensor pos, c10::optional<torch::Tensor> lens,
                c10::optional<torch::Tensor> slots, int64_t T) {
  ScanArgs a = mlstm_args(src, q0, k0, v0, i0, f0, ib, fb, cap, qscale, state,
                          nst, mst, pos, lens, slots, T);
  scan_launch(a, kMlstm, src, o);
}

void mlstm_step(torch::Tensor src, int64_t q0, int64_t k0, int64_t v0,
                int64_t i0, int64_t f0, torch::Tensor ib, torch::Tensor fb,
                double cap, double qscale, torch::Tensor state,
                torch::Tensor nst, torch::Tensor mst, torch::Tensor w,
                int64_t g0, bool silu, double eps, torch::Tensor out,
                torch::Tensor pos, c10::optional<torch::Tensor> lens,
                c10::optional<torch::Tensor> slots) {
  ScanArgs a = mlstm_args(src, q0, k0, v0, i0, f0, ib, fb, cap, qscale, state,
                          nst, mst, pos, lens, slots, 1);
  step_launch(a, kMlstm, src, w, g0, silu, eps, out);
}

}  // namespace dnet
