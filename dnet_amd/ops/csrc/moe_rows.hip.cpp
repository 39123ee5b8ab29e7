// Mixtures of sigmoid-routed experts, the routing weight on an expert's input or
// on its result (gfx950):
//
//   moe_router       fp32 sigmoid scores, the `top` largest kept times a
//                    constant (plus an optional shared-expert gate as the last
//                    row), optionally chosen by score + correction inside the
//                    best groups of neighbouring experts;
//                    the products themselves are part of the kernel for few
//                    rows, prompts hand in the logits of a library product
//   moe_plan         entries (row, choice) sorted by expert, without host work
//   moe_gather       the sorted entries' rows and scales
//   moe_gateup_rows  every expert on every row of a decode batch, matrix
//   moe_down_rows    cores (moe_up_rows: ungated experts, squared ReLU;
//                    moe_clamped_rows: clamped gate, routing weight on the
//                    result): an expert's weights are read once for all rows,
//                    experts that no row chose are skipped on the device
//   moe_merge        sum of each row's chosen results + gate * shared
//
// The scale w of a gated expert's input commutes with the product, so it is applied to the
// fp32 accumulators: silu(w g) * (w u). A row that did not choose an expert
// has w = 0 and therefore act = 0. "short" stands for bf16 bits.
#include "common.h"

namespace dnet {

namespace {

using bf16x8 = __attribute__((ext_vector_type(8))) __bf16;
using f32x4 = __attribute__((ext_vector_type(4))) float;

template <typename T> __device__ __forceinline__ float ldx(const T* p);
template <> __device__ __forceinline__ float ldx<float>(const float* p) { return *p; }
template <> __device__ __forceinline__ float ldx<short>(const short* p) { return bits2f(*p); }
template <typename T> __device__ __forceinline__ void stx(T* p, float v);
template <> __device__ __forceinline__ void stx<float>(float* p, float v) { *p = v; }
template <> __device__ __forceinline__ void stx<short>(short* p, float v) { *p = f2bits(v); }

bool is_bf16(const torch::Tensor& t) { return t.scalar_type() == torch::kBFloat16; }
bool is_f32(const torch::Tensor& t) { return t.scalar_type() == torch::kFloat32; }
bool is_i32(const torch::Tensor& t) { return t.scalar_type() == torch::kInt32; }

// ---- router ------------------------------------------------------------------
// One workgroup per row. x given: its waves form the R = E (+1) dot products
// (wave per router row, up to 16 waves); else one wave starts from logits [T, R]. Then the
// first wave picks by the logits (the sigmoid keeps their order, and does not
// tell large ones apart in fp32): they sit in LDS, every lane scans its
// experts, ties go to the lower expert.
template <typename T> __device__ __forceinline__ float4 ld4(const T* p);
template <> __device__ __forceinline__ float4 ld4<float>(const float* p) {
  return *reinterpret_cast<const float4*>(p);
}
template <> __device__ __forceinline__ float4 ld4<short>(const short* p) {
  const short4v v = *reinterpret_cast<const short4v*>(p);
  return make_float4(bits2f(v.x[0]), bits2f(v.x[1]), bits2f(v.x[2]),
                     bits2f(v.x[3]));
}

template <typename T>
__global__ __launch_bounds__(1024) void moe_router_kernel(
    const T* __restrict__ x, const float* __restrict__ w,
    const float* __restrict__ logits, int* __restrict__ idx,
    float* __restrict__ val, float* __restrict__ we, float* __restrict__ gate,
    const float* __restrict__ corr, const int W, const int E, const int R,
    const int top, const int groups, const int keep, const float scale) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  float* sc = sm;                                   // [R] logits, then choice
  float* ss = sm + R;                               // [E] scores (biased choice)
  float* gs = ss + E;                               // [groups]
  // choice by score + correction and by groups; else by the logits
  const bool biased = corr != nullptr || groups > 1;
  const int t = blockIdx.x;
  const int wid = threadIdx.x >> 6, lane = threadIdx.x & 63;
  if (x != nullptr) {
    const T* xr = x + (int64_t)t * W;
    const int nw = blockDim.x >> 6;
    for (int e = wid; e < R; e += nw) {
      const float* wr = w + (int64_t)e * W;
      float s = 0.f;
      if ((W & 3) == 0) {
        // 4 pieces in flight
        float4 a = {0.f, 0.f, 0.f, 0.f};
        int i = lane * 4;
        for (; i + 768 < W; i += 1024) {
          float4 wv[4], xv[4];
#pragma unroll
          for (int u = 0; u < 4; ++u) {
            wv[u] = *reinterpret_cast<const float4*>(wr + i + u * 256);
            xv[u] = ld4<T>(xr + i + u * 256);
          }
#pragma unroll
          for (int u = 0; u < 4; ++u) {
            a.x = fmaf(xv[u].x, wv[u].x, a.x);
            a.y = fmaf(xv[u].y, wv[u].y, a.y);
            a.z = fmaf(xv[u].z, wv[u].z, a.z);
            a.w = fmaf(xv[u].w, wv[u].w, a.w);
          }
        }
        for (; i < W; i += 256) {
          const float4 wv = *reinterpret_cast<const float4*>(wr + i);
          const float4 xv = ld4<T>(xr + i);
          a.x = fmaf(xv.x, wv.x, a.x);
          a.y = fmaf(xv.y, wv.y, a.y);
          a.z = fmaf(xv.z, wv.z, a.z);
          a.w = fmaf(xv.w, wv.w, a.w);
        }
        s = (a.x + a.y) + (a.z + a.w);
      } else {
        for (int i = lane; i < W; i += 64) s = fmaf(ldx<T>(xr + i), wr[i], s);
      }
      s = wave_reduce_sum(s);
      if (lane == 0) sc[e] = s;
    }
  } else {
    for (int e = threadIdx.x; e < R; e += blockDim.x)
      sc[e] = logits[(int64_t)t * R + e];
  }
  __syncthreads();
  for (int e = threadIdx.x; e < R; e += blockDim.x) {
    const float zr = sc[e];
    const float z = zr > -1e30f ? zr : -1e30f;   // (padding rows may hold NaN)
    sc[e] = z;
    if (biased && e < E) {
      const float s = 1.f / (1.f + expf(-z));
      ss[e] = s;
      sc[e] = corr ? s + corr[e] : s;
    }
    if (e == E && gate) gate[t] = 1.f / (1.f + expf(-z));
    if (e < E) we[(int64_t)t * E + e] = 0.f;
  }
  __syncthreads();
  if (wid != 0) return;
  if (groups > 1) {
    // a group's score: the sum of its two largest choice scores; experts of
    // all but the `keep` best groups (lower index first) drop out
    const int gsz = E / groups;
    for (int g = lane; g < groups; g += 64) {
      float a = -1e37f, c = -1e37f;
      for (int e = g * gsz; e < (g + 1) * gsz; ++e) {
        const float s = sc[e];
        if (s > a) {
          c = a;
          a = s;
        } else if (s > c) {
          c = s;
        }
      }
      gs[g] = gsz > 1 ? a + c : a;
    }
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");   // one wave only
    for (int g = lane; g < groups; g += 64) {
      const float s = gs[g];
      int better = 0;
      for (int o = 0; o < groups; ++o)
        better += gs[o] > s || (gs[o] == s && o < g);
      if (better >= keep)
        for (int e = g * gsz; e < (g + 1) * gsz; ++e) sc[e] = -3e38f;
    }
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
  }
  for (int k = 0; k < top; ++k) {
    float bv = -2e38f;
    int bi = E;                             // chosen logits are set to -3e38
    for (int e = lane; e < E; e += 64) {
      const float s = sc[e];
      if (s > bv) {
        bv = s;
        bi = e;
      }
    }
#pragma unroll
    for (int off = 32; off > 0; off >>= 1) {
      const float ov = __shfl_xor(bv, off, 64);
      const int oi = __shfl_xor(bi, off, 64);
      if (ov > bv || (ov == bv && oi < bi)) {
        bv = ov;
        bi = oi;
      }
    }
    // top <= experts that can be chosen: bi is always one of them
    if (lane == 0) {
      const float s = (biased ? ss[bi] : 1.f / (1.f + expf(-bv))) * scale;
      idx[(int64_t)t * top + k] = bi;
      val[(int64_t)t * top + k] = s;
      // never 0: a chosen expert must not look skipped to the row kernels
      we[(int64_t)t * E + bi] = s != 0.f ? s : 1e-38f;
      sc[bi] = -3e38f;
    }
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");   // one wave only
  }
}

// ---- plan ----------------------------------------------------------------------
// grid (E), 1024 threads: workgroup e counts the entries of lower experts (its
// base) and places its own in ascending order (ballot prefix inside a wave,
// wave sums through LDS).
__global__ __launch_bounds__(1024) void moe_plan_kernel(
    const int* __restrict__ idx, int* __restrict__ order, int* __restrict__ at,
    int* __restrict__ counts, const int n) {
  __shared__ int wsum[16], wlow[16];
  const int e = blockIdx.x;
  const int wid = threadIdx.x >> 6, lane = threadIdx.x & 63;
  int low = 0, own = 0;
  for (int i = threadIdx.x; i < n; i += 1024) {
    const int v = idx[i];
    low += v < e;
    own += v == e;
  }
#pragma unroll
  for (int off = 32; off > 0; off >>= 1) {
    low += __shfl_down(low, off, 64);
    own += __shfl_down(own, off, 64);
  }
  if (lane == 0) {
    wlow[wid] = low;
    wsum[wid] = own;
  }
  __syncthreads();
  int base = 0, total = 0;
#pragma unroll
  for (int w = 0; w < 16; ++w) {
    base += wlow[w];
    total += wsum[w];
  }
  if (threadIdx.x == 0) counts[e] = total;
  if (total == 0) return;                         // workgroup-uniform
  for (int i0 = 0; i0 < n; i0 += 1024) {
    const int i = i0 + threadIdx.x;
    const bool mine = i < n && idx[i] == e;
    const unsigned long long m = __ballot(mine);
    __syncthreads();                              // wsum of the last round
    if (lane == 0) wsum[wid] = __popcll(m);
    __syncthreads();
    int before = 0, all = 0;
#pragma unroll
    for (int w = 0; w < 16; ++w) {
      if (w < wid) before += wsum[w];
      all += wsum[w];
    }
    if (mine) {
      const int p = base + before +
                    __popcll(m & ((1ull << lane) - 1ull));
      order[p] = i;
      at[i] = p;
    }
    base += all;
  }
}

// grid (entries): row order[r] / top of x -> xs[r], scale of the entry
template <int V>
__global__ __launch_bounds__(256) void moe_gather_kernel(
    const char* __restrict__ x, const int* __restrict__ order,
    const float* __restrict__ val, char* __restrict__ xs,
    float* __restrict__ scale, const int top, const int64_t bytes) {
  const int64_t r = blockIdx.x;
  const int en = order[r];
  const char* src = x + (int64_t)(en / top) * bytes;
  char* dst = xs + r * bytes;
  for (int64_t i = (int64_t)threadIdx.x * V; i < bytes; i += 256 * V) {
    if constexpr (V == 16)
      *reinterpret_cast<int4*>(dst + i) = *reinterpret_cast<const int4*>(src + i);
    else
      *reinterpret_cast<short*>(dst + i) = *reinterpret_cast<const short*>(src + i);
  }
  if (threadIdx.x == 0) scale[r] = val[en];
}

// ---- experts on the rows of a decode batch ----------------------------------------
// grid (column tiles, row blocks of 16 MT, E), NW waves. The inner
// dimension goes in groups of NW x U 32-wide steps, U neighbouring ones per
// wave (64 U bytes of every weight row it reads), NF weight fragments x MT row fragments of
// v_mfma_f32_16x16x32_bf16, the next group in flight while one is multiplied;
// the partial sums fold wave by wave through LDS. GLU: the first half of the fragments are gate columns,
// the second half the up columns beside them (8 NF columns of act), inputs
// scaled by the routing weight (ClampGlu: clamped gate, the weight on the
// result); else 16 NF plain or squared-ReLU columns.
constexpr int kPlain = 0, kGlu = 1, kReluSq = 2, kClampGlu = 3;

template <int MT, int NF, int NW, int U, int KIND>
__global__ __launch_bounds__(NW * 64) void moe_rows_kernel(
    const short* __restrict__ x, const short* __restrict__ w,
    const float* __restrict__ we, short* __restrict__ out, const int K,
    const int N, const int E, const int T, const int64_t x_expert,
    const float alpha, const float limit) {
  constexpr bool GLU = KIND == kGlu || KIND == kClampGlu;
  constexpr int NC = GLU ? NF / 2 : NF;      // column fragments of the result
  __shared__ f32x4 part[NW / 2][MT * NF][64];
  const int e = blockIdx.z;
  const int m0 = blockIdx.y * (16 * MT);
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  {
    const int t = m0 + lane;
    const bool hit = lane < 16 * MT && t < T && we[(int64_t)t * E + e] != 0.f;
    if (__ballot(hit) == 0ull) return;       // the same in all waves
  }
  const int c = lane & 15, hi = lane >> 4;
  const int n0 = blockIdx.x * (16 * NC);
  const short* wp[NF];
#pragma unroll
  for (int f = 0; f < NF; ++f) {
    // GLU: w is [E, 2N, K] with the gate rows first
    const int col = min(n0 + (f % NC) * 16 + c, N - 1);
    const int64_t row = GLU ? ((int64_t)e * 2 + f / NC) * N + col
                            : (int64_t)e * N + col;
    wp[f] = w + row * K + hi * 8;
  }
  const short* xp[MT];
#pragma unroll
  for (int m = 0; m < MT; ++m)
    xp[m] = x + e * x_expert + (int64_t)min(m0 + m * 16 + c, T - 1) * K + hi * 8;
  f32x4 acc[MT][NF];
#pragma unroll
  for (int m = 0; m < MT; ++m)
#pragma unroll
    for (int f = 0; f < NF; ++f) acc[m][f] = {0.f, 0.f, 0.f, 0.f};

  const int full = K / 32;                   // whole steps
  short8 z;
#pragma unroll
  for (int j = 0; j < 8; ++j) z.x[j] = 0;
  const bf16x8 zero = *reinterpret_cast<const bf16x8*>(&z);
  struct Batch { bf16x8 wf[U][NF], xf[U][MT]; };
  auto load = [&](Batch& q, const int s) {
    // a row's neighbouring 64 B pieces back to back
#pragma unroll
    for (int f = 0; f < NF; ++f)
#pragma unroll
      for (int u = 0; u < U; ++u)
        q.wf[u][f] =
            *reinterpret_cast<const bf16x8*>(wp[f] + (s + u) * 32);
#pragma unroll
    for (int m = 0; m < MT; ++m)
#pragma unroll
      for (int u = 0; u < U; ++u)
        q.xf[u][m] = *reinterpret_cast<const bf16x8*>(xp[m] + (s + u) * 32);
  };
  auto mul = [&](const Batch& q) {
#pragma unroll
    for (int u = 0; u < U; ++u)
#pragma unroll
      for (int m = 0; m < MT; ++m)
#pragma unroll
        for (int f = 0; f < NF; ++f)
          acc[m][f] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
              q.xf[u][m], q.wf[u][f], acc[m][f], 0, 0, 0);
  };
  // every workgroup starts at another place of the inner dimension: weight
  // rows are often a power of two apart, and workgroups in step would all
  // read from the same few memory channels
  const int groups = full / (NW * U);
  const int turn =
      groups > 1 ? (int)((blockIdx.x * 5 + blockIdx.z * 3) % groups) : 0;
  auto place = [&](int g) {
    g += turn;
    if (g >= groups) g -= groups;
    return (g * NW + wave) * U;
  };
  if (groups > 0) {
    Batch q0, q1;
    load(q0, place(0));
    int g = 0;
    for (; g + 2 <= groups; g += 2) {
      load(q1, place(g + 1));
      __builtin_amdgcn_sched_barrier(0);
      mul(q0);
      if (g + 2 < groups) load(q0, place(g + 2));
      __builtin_amdgcn_sched_barrier(0);
      mul(q1);
    }
    if (g < groups) mul(q0);
  }
  auto tail = [&](const int s, const bool in) {
    bf16x8 wf[NF], xf[MT];
#pragma unroll
    for (int f = 0; f < NF; ++f)
      wf[f] = in ? *reinterpret_cast<const bf16x8*>(wp[f] + s * 32) : zero;
#pragma unroll
    for (int m = 0; m < MT; ++m)
      xf[m] = in ? *reinterpret_cast<const bf16x8*>(xp[m] + s * 32) : zero;
#pragma unroll
    for (int m = 0; m < MT; ++m)
#pragma unroll
      for (int f = 0; f < NF; ++f)
        acc[m][f] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(xf[m], wf[f],
                                                            acc[m][f], 0, 0, 0);
  };
  for (int s = groups * NW * U + wave; s < full; s += NW) tail(s, true);
  if (full * 32 < K && wave == full % NW)    // the last, shorter step
    tail(full, full * 32 + hi * 8 < K);      // (K is a multiple of 8)

#pragma unroll
  for (int half = NW / 2; half > 0; half >>= 1) {
    if (wave >= half && wave < 2 * half)
#pragma unroll
      for (int m = 0; m < MT; ++m)
#pragma unroll
        for (int f = 0; f < NF; ++f)
          part[wave - half][m * NF + f][lane] = acc[m][f];
    __syncthreads();
    if (wave < half)
#pragma unroll
      for (int m = 0; m < MT; ++m)
#pragma unroll
        for (int f = 0; f < NF; ++f) {
          const f32x4 p = part[wave][m * NF + f][lane];
#pragma unroll
          for (int r = 0; r < 4; ++r) acc[m][f][r] += p[r];
        }
    __syncthreads();
  }
  if (wave != 0) return;
#pragma unroll
  for (int m = 0; m < MT; ++m)
#pragma unroll
    for (int f = 0; f < NC; ++f) {
      const int i = n0 + f * 16 + c;
      if (i >= N) continue;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int t = m0 + m * 16 + hi * 4 + r;
        if (t >= T) continue;
        float v = acc[m][f][r];
        if constexpr (KIND == kClampGlu) {
          const float g = fminf(v, limit);
          const float u = fminf(fmaxf(acc[m][NC + f][r], -limit), limit);
          v = g * __builtin_amdgcn_rcpf(1.f + __expf(-alpha * g)) * (u + 1.f) *
              we[(int64_t)t * E + e];
        } else if constexpr (GLU) {
          const float s = we[(int64_t)t * E + e];
          const float g = v * s;
          v = g * __builtin_amdgcn_rcpf(1.f + __expf(-g)) *
              (acc[m][NC + f][r] * s);
        } else if constexpr (KIND == kReluSq) {
          v = fmaxf(v, 0.f);
          v = v * v;
        }
        out[((int64_t)e * T + t) * N + i] = f2bits(v);
      }
    }
}

// ---- merge ----------------------------------------------------------------------
// grid (column tiles, T). er > 0: y is [E, er, W] and at holds experts.
template <typename T, int V>
__global__ __launch_bounds__(256) void moe_merge_kernel(
    const T* __restrict__ y, const int* __restrict__ at,
    const T* __restrict__ shared, const float* __restrict__ gate,
    T* __restrict__ out, const int W, const int top, const int er,
    const int64_t R) {
  const int t = blockIdx.y;
  const int w = (blockIdx.x * blockDim.x + threadIdx.x) * V;
  if (w >= W) return;
  float a[V];
#pragma unroll
  for (int j = 0; j < V; ++j) a[j] = 0.f;
  auto add = [&](const T* p, float k) {
    if constexpr (V == 1) {
      a[0] = fmaf(k, ldx<T>(p), a[0]);
    } else if constexpr (sizeof(T) == 2) {
      const short4v v = *reinterpret_cast<const short4v*>(p);
#pragma unroll
      for (int j = 0; j < 4; ++j) a[j] = fmaf(k, bits2f(v.x[j]), a[j]);
    } else {
      const float4 v = *reinterpret_cast<const float4*>(p);
      a[0] = fmaf(k, v.x, a[0]);
      a[1] = fmaf(k, v.y, a[1]);
      a[2] = fmaf(k, v.z, a[2]);
      a[3] = fmaf(k, v.w, a[3]);
    }
  };
  for (int k = 0; k < top; ++k) {
    int64_t r = at[(int64_t)t * top + k];
    if (er > 0) r = r * er + t;
    if (r >= 0 && r < R) add(y + r * W + w, 1.f);
  }
  if (shared) add(shared + (int64_t)t * W + w, gate[t]);
  T* op = out + (int64_t)t * W + w;
  if constexpr (V == 1) {
    stx<T>(op, a[0]);
  } else if constexpr (sizeof(T) == 2) {
    short4v v;
#pragma unroll
    for (int j = 0; j < 4; ++j) v.x[j] = f2bits(a[j]);
    *reinterpret_cast<short4v*>(op) = v;
  } else {
    *reinterpret_cast<float4*>(op) = make_float4(a[0], a[1], a[2], a[3]);
  }
}

}  // namespace

void moe_router(c10::optional<torch::Tensor> x, torch::Tensor w,
                c10::optional<torch::Tensor> logits, torch::Tensor idx,
                torch::Tensor val, torch::Tensor we,
                c10::optional<torch::Tensor> gate,
                c10::optional<torch::Tensor> corr, int64_t groups,
                int64_t keep, double scale) {
  DNET_CHECK(w.dim() == 2 && is_f32(w) && w.is_contiguous(), "w fp32 [R, W]");
  const int R = w.size(0), W = w.size(1);
  const int64_t T = we.size(0), E = we.size(1);
  DNET_CHECK(x.has_value() != logits.has_value(), "rows or logits");
  DNET_CHECK(E >= 1 && R == E + (gate.has_value() ? 1 : 0),
             "router rows = experts (+ the shared gate)");
  DNET_CHECK(we.dim() == 2 && is_f32(we) && we.is_contiguous(), "we fp32 [T, E]");
  DNET_CHECK(idx.dim() == 2 && is_i32(idx) && idx.is_contiguous() &&
                 idx.size(0) == T && val.sizes() == idx.sizes() &&
                 is_f32(val) && val.is_contiguous(), "idx, val [T, top]");
  const int top = idx.size(1);
  DNET_CHECK(top >= 1 && top <= E, "1 <= top <= experts");
  if (gate.has_value())
    DNET_CHECK(is_f32(*gate) && gate->is_contiguous() && gate->numel() == T,
               "gate fp32 [T]");
  DNET_CHECK(groups >= 1 && E % groups == 0 && keep >= 1 && keep <= groups &&
                 top <= keep * (E / groups), "expert groups");
  if (corr.has_value())
    DNET_CHECK(is_f32(*corr) && corr->is_contiguous() && corr->numel() == E,
               "correction fp32 [E]");
  const float* cp = corr.has_value() ? corr->data_ptr<float>() : nullptr;
  const size_t lds = (size_t)(R + E + groups) * sizeof(float);
  DNET_CHECK(lds <= 60 * 1024, "moe_router: too many experts");
  if (T == 0) return;
  float* gp = gate.has_value() ? gate->data_ptr<float>() : nullptr;
  auto st = current_stream();
#define MR(TT, NT, XP, LP)                                                    \
  hipLaunchKernelGGL((moe_router_kernel<TT>), dim3((unsigned)T), dim3(NT),    \
                     lds, st, XP, w.data_ptr<float>(), LP,                    \
                     idx.data_ptr<int>(), val.data_ptr<float>(),              \
                     we.data_ptr<float>(), gp, cp, W, (int)E, R, top,         \
                     (int)groups, (int)keep, (float)scale)
  if (x.has_value()) {
    DNET_CHECK(x->dim() == 2 && x->is_contiguous() && x->size(0) == T &&
                   x->size(1) == W, "x [T, W]");
    const int nt = 64 * std::min(R, 16);
    if (is_bf16(*x)) MR(short, nt, (const short*)x->data_ptr(), nullptr);
    else if (is_f32(*x)) MR(float, nt, (const float*)x->data_ptr(), nullptr);
    else DNET_CHECK(false, "moe_router: dtype");
  } else {
    DNET_CHECK(logits->dim() == 2 && is_f32(*logits) &&
                   logits->is_contiguous() && logits->size(0) == T &&
                   logits->size(1) == R, "logits fp32 [T, R]");
    MR(float, 64, nullptr, logits->data_ptr<float>());
  }
#undef MR
}

void moe_plan(torch::Tensor idx, torch::Tensor order, torch::Tensor at,
              torch::Tensor counts) {
  DNET_CHECK(is_i32(idx) && idx.is_contiguous() && is_i32(order) &&
                 order.is_contiguous() && order.numel() == idx.numel() &&
                 is_i32(at) && at.is_contiguous() &&
                 at.numel() == idx.numel() && is_i32(counts) &&
                 counts.is_contiguous() && counts.numel() >= 1,
             "moe_plan: int32 tensors");
  DNET_CHECK(idx.numel() < (1ll << 31), "moe_plan: too many entries");
  hipLaunchKernelGGL(moe_plan_kernel, dim3((unsigned)counts.numel()),
                     dim3(1024), 0, current_stream(), idx.data_ptr<int>(),
                     order.data_ptr<int>(), at.data_ptr<int>(),
                     counts.data_ptr<int>(), (int)idx.numel());
}

void moe_gather(torch::Tensor x, torch::Tensor order, torch::Tensor val,
                torch::Tensor xs, torch::Tensor scale) {
  DNET_CHECK(x.dim() == 2 && x.is_contiguous() && xs.dim() == 2 &&
                 xs.is_contiguous() && xs.size(1) == x.size(1) &&
                 xs.scalar_type() == x.scalar_type(), "x [T, W], xs [R, W]");
  const int64_t R = xs.size(0);
  DNET_CHECK(val.dim() == 2 && is_f32(val) && val.is_contiguous() &&
                 val.size(0) == x.size(0) && val.numel() == R,
             "val fp32 [T, top]");
  DNET_CHECK(is_i32(order) && order.is_contiguous() && order.numel() == R &&
                 is_f32(scale) && scale.is_contiguous() && scale.numel() == R,
             "order int32 [R], scale fp32 [R]");
  if (R == 0) return;
  const int64_t bytes = x.size(1) * x.element_size();
  const int top = (int)val.size(1);
  auto st = current_stream();
  if (bytes % 16 == 0)
    hipLaunchKernelGGL((moe_gather_kernel<16>), dim3((unsigned)R), dim3(256), 0,
                       st, (const char*)x.data_ptr(), order.data_ptr<int>(),
                       val.data_ptr<float>(), (char*)xs.data_ptr(),
                       scale.data_ptr<float>(), top, bytes);
  else
    hipLaunchKernelGGL((moe_gather_kernel<2>), dim3((unsigned)R), dim3(256), 0,
                       st, (const char*)x.data_ptr(), order.data_ptr<int>(),
                       val.data_ptr<float>(), (char*)xs.data_ptr(),
                       scale.data_ptr<float>(), top, bytes);
}

// Routed rows of `x` [T, K] through the gated experts w [E, 2N, K]: shapes
static void check_gated(const torch::Tensor& x, const torch::Tensor& w,
                        const torch::Tensor& we, const torch::Tensor& act) {
  const int64_t T = x.size(0), K = x.size(1), E = w.size(0), N = w.size(1) / 2;
  DNET_CHECK(is_bf16(x) && is_bf16(w) && is_bf16(act) && is_f32(we) &&
                 x.is_contiguous() && w.is_contiguous() &&
                 act.is_contiguous() && we.is_contiguous(),
             "gated expert rows: contiguous bf16, we fp32");
  DNET_CHECK(x.dim() == 2 && w.dim() == 3 && w.size(1) % 2 == 0 &&
                 w.size(2) == K && we.dim() == 2 && we.size(0) == T &&
                 we.size(1) == E && act.dim() == 3 && act.size(0) == E &&
                 act.size(1) == T && act.size(2) == N && K % 8 == 0 && K > 0 &&
                 N > 0, "gated expert rows: shapes");
}

static void rows_launch(const torch::Tensor& x, const torch::Tensor& w,
                        const torch::Tensor& we, torch::Tensor& out, int64_t T,
                        int64_t K, int64_t N, int kind, int64_t x_expert,
                        float alpha = 0.f, float limit = 0.f) {
  const int64_t E = we.size(1);
  auto st = current_stream();
#define RL(MM, NF, NW, UU, GG)                                                \
  hipLaunchKernelGGL((moe_rows_kernel<MM, NF, NW, UU, GG>),                   \
                     dim3((unsigned)cdiv(N, GG == kGlu || GG == kClampGlu     \
                                                ? NF * 8 : NF * 16),          \
                          (unsigned)cdiv(T, 16 * MM), (unsigned)E),           \
                     dim3(NW * 64), 0, st, (const short*)x.data_ptr(),        \
                     (const short*)w.data_ptr(), we.data_ptr<float>(),        \
                     (short*)out.data_ptr(), (int)K, (int)N, (int)E, (int)T,  \
                     x_expert, alpha, limit)
  // shapes measured at experts of 4096 x 3072 to 5120 x 12800: few rows want
  // more workgroups (narrow column tiles)
#define RL_K(MM, NF, NW, UU)                            \
  do {                                                  \
    if (kind == kGlu) RL(MM, NF, NW, UU, kGlu);         \
    else if (kind == kReluSq) RL(MM, NF, NW, UU, kReluSq); \
    else if (kind == kClampGlu) RL(MM, NF, NW, UU, kClampGlu); \
    else RL(MM, NF, NW, UU, kPlain);                    \
  } while (0)
  if (T <= 2 && kind == kPlain) RL(1, 1, 8, 4, kPlain);
  else if (T <= 16) RL_K(1, 2, 8, 4);
  else if (T <= 32) RL_K(2, 4, 4, 2);
  else RL_K(4, 4, 4, 2);
#undef RL_K
#undef RL
}

void moe_gateup_rows(torch::Tensor x, torch::Tensor w, torch::Tensor we,
                     torch::Tensor act) {
  check_gated(x, w, we, act);
  if (x.size(0) == 0) return;
  rows_launch(x, w, we, act, x.size(0), x.size(1), w.size(1) / 2, kGlu, 0);
}

void moe_clamped_rows(torch::Tensor x, torch::Tensor w, torch::Tensor we,
                      torch::Tensor act, double alpha, double limit) {
  check_gated(x, w, we, act);
  if (x.size(0) == 0) return;
  rows_launch(x, w, we, act, x.size(0), x.size(1), w.size(1) / 2, kClampGlu, 0,
              (float)alpha, (float)limit);
}

void moe_up_rows(torch::Tensor x, torch::Tensor w, torch::Tensor we,
                 torch::Tensor act) {
  const int64_t T = x.size(0), K = x.size(1), E = w.size(0), N = w.size(1);
  DNET_CHECK(is_bf16(x) && is_bf16(w) && is_bf16(act) && is_f32(we) &&
                 x.is_contiguous() && w.is_contiguous() &&
                 act.is_contiguous() && we.is_contiguous(),
             "moe_up_rows: contiguous bf16, we fp32");
  DNET_CHECK(x.dim() == 2 && w.dim() == 3 && w.size(2) == K && we.dim() == 2 &&
                 we.size(0) == T && we.size(1) == E && act.dim() == 3 &&
                 act.size(0) == E && act.size(1) == T && act.size(2) == N &&
                 K % 8 == 0 && K > 0 && N > 0, "moe_up_rows: shapes");
  if (T == 0) return;
  rows_launch(x, w, we, act, T, K, N, kReluSq, 0);
}

void moe_down_rows(torch::Tensor act, torch::Tensor w, torch::Tensor we,
                   torch::Tensor y) {
  const int64_t E = w.size(0), N = w.size(1), K = w.size(2);
  const int64_t T = act.size(1);
  DNET_CHECK(is_bf16(act) && is_bf16(w) && is_bf16(y) && is_f32(we) &&
                 act.is_contiguous() && w.is_contiguous() &&
                 y.is_contiguous() && we.is_contiguous(),
             "moe_down_rows: contiguous bf16, we fp32");
  DNET_CHECK(act.dim() == 3 && act.size(0) == E && act.size(2) == K &&
                 w.dim() == 3 && we.dim() == 2 && we.size(0) == T &&
                 we.size(1) == E && y.dim() == 3 && y.size(0) == E &&
                 y.size(1) == T && y.size(2) == N && K % 8 == 0 && K > 0,
             "moe_down_rows: shapes");
  if (T == 0) return;
  rows_launch(act, w, we, y, T, K, N, kPlain, T * K);
}

void moe_merge(torch::Tensor y, torch::Tensor at,
               c10::optional<torch::Tensor> shared,
               c10::optional<torch::Tensor> gate, torch::Tensor out) {
  DNET_CHECK(out.dim() == 2 && out.is_contiguous() && y.is_contiguous() &&
                 y.scalar_type() == out.scalar_type() &&
                 y.size(-1) == out.size(1), "y [.., W], out [T, W]");
  const int64_t T = out.size(0);
  const int W = out.size(1);
  DNET_CHECK(at.dim() == 2 && is_i32(at) && at.is_contiguous() &&
                 at.size(0) == T, "at int32 [T, top]");
  DNET_CHECK(y.dim() == 2 || (y.dim() == 3 && y.size(1) == T),
             "y [R, W] or [E, T, W]");
  DNET_CHECK(shared.has_value() == gate.has_value(), "shared with its gate");
  if (shared.has_value())
    DNET_CHECK(shared->is_contiguous() && shared->sizes() == out.sizes() &&
                   shared->scalar_type() == out.scalar_type() &&
                   is_f32(*gate) && gate->is_contiguous() && gate->numel() == T,
               "shared [T, W], gate fp32 [T]");
  if (T == 0) return;
  const int er = y.dim() == 3 ? (int)T : 0;
  const int64_t R = y.numel() / W;
  auto st = current_stream();
#define MM(TT, VV)                                                            \
  hipLaunchKernelGGL((moe_merge_kernel<TT, VV>),                              \
                     dim3((unsigned)cdiv(W, 256 * VV), (unsigned)T),          \
                     dim3(256), 0, st, (const TT*)y.data_ptr(),               \
                     at.data_ptr<int>(),                                      \
                     shared.has_value() ? (const TT*)shared->data_ptr()       \
                                        : nullptr,                            \
                     gate.has_value() ? gate->data_ptr<float>() : nullptr,    \
                     (TT*)out.data_ptr(), W, (int)at.size(1), er, R)
  if (is_bf16(out)) { if (W % 4 == 0) MM(short, 4); else MM(short, 1); }
  else if (is_f32(out)) { if (W % 4 == 0) MM(float, 4); else MM(float, 1); }
  else DNET_CHECK(false, "moe_merge: dtype");
#undef MM
}

}  // namespace dnet
