// Norm + token shift, minGRU recurrence and their small companions (gfx950):
//
//   norm_token_shift  h = rms(x) * wn;  y = h + (h' - h) * mu with h' the
//                     previous token's h; optionally x += rms(a) * wa first
//                     (decode steps: residual update, norm and shift in one
//                     launch). The slot's last h is its state (fp32).
//   mingru_scan       S <- (1 - z) S + z * candidate per channel, z and the
//                     candidate from the step's projections alone (no state
//                     feedback); y = S * silu(gate)
//   cache_append      projection columns as they are into cache rows
//   gated_act         act(s gate) * (s up) over [gate | up] rows, act = silu
//                     or tanh-gelu, s an optional factor per row
//
// Geometry is the cache's: token (b,t) = row b*T+t sits at position pos[b]+t
// of slot slots[b] (default b); tokens t >= lens[b] are padding. State is
// taken as zero at position 0 and written only by rows with real tokens.
// Sums, statistics, gates and states are fp32 whatever the activation dtype
// ("short" stands for bf16 bits).
#include "common.h"

namespace dnet {

namespace {

template <typename T> __device__ __forceinline__ float ldx(const T* p);
template <> __device__ __forceinline__ float ldx<float>(const float* p) { return *p; }
template <> __device__ __forceinline__ float ldx<short>(const short* p) { return bits2f(*p); }
template <typename T> __device__ __forceinline__ void stx(T* p, float v);
template <> __device__ __forceinline__ void stx<float>(float* p, float v) { *p = v; }
template <> __device__ __forceinline__ void stx<short>(short* p, float v) { *p = f2bits(v); }

// N consecutive elements (N = 1, 4 or 8 bf16 / 4 fp32: one access)
template <int N> struct vec { float v[N]; };
template <int N, typename T>
__device__ __forceinline__ vec<N> ldv(const T* p) {
  vec<N> r;
  if constexpr (N == 1) {
    r.v[0] = ldx<T>(p);
  } else if constexpr (sizeof(T) == 4) {
#pragma unroll
    for (int j = 0; j < N; j += 4) {
      const float4 t = *reinterpret_cast<const float4*>(p + j);
      r.v[j] = t.x; r.v[j + 1] = t.y; r.v[j + 2] = t.z; r.v[j + 3] = t.w;
    }
  } else if constexpr (N == 8) {
    const short8 t = *reinterpret_cast<const short8*>(p);
#pragma unroll
    for (int j = 0; j < 8; ++j) r.v[j] = bits2f(t.x[j]);
  } else {
    const short4v t = *reinterpret_cast<const short4v*>(p);
#pragma unroll
    for (int j = 0; j < 4; ++j) r.v[j] = bits2f(t.x[j]);
  }
  return r;
}
template <int N, typename T>
__device__ __forceinline__ void stv(T* p, const vec<N>& r) {
  if constexpr (N == 1) {
    stx<T>(p, r.v[0]);
  } else if constexpr (sizeof(T) == 4) {
#pragma unroll
    for (int j = 0; j < N; j += 4)
      *reinterpret_cast<float4*>(p + j) =
          make_float4(r.v[j], r.v[j + 1], r.v[j + 2], r.v[j + 3]);
  } else if constexpr (N == 8) {
    short8 t;
#pragma unroll
    for (int j = 0; j < 8; ++j) t.x[j] = f2bits(r.v[j]);
    *reinterpret_cast<short8*>(p) = t;
  } else {
    short4v t;
#pragma unroll
    for (int j = 0; j < 4; ++j) t.x[j] = f2bits(r.v[j]);
    *reinterpret_cast<short4v*>(p) = t;
  }
}

// transcendental flavours: fp32 models use the accurate library functions,
// bf16 models the hardware approximations (error far below bf16 rounding)
template <bool FAST> __device__ __forceinline__ float sigmoid_x(float x) {
  return FAST ? __builtin_amdgcn_rcpf(1.f + __expf(-x))
              : 1.f / (1.f + expf(-x));
}
template <bool FAST> __device__ __forceinline__ float tanh_x(float x) {
  return FAST ? 1.f - 2.f * __builtin_amdgcn_rcpf(__expf(2.f * x) + 1.f)
              : tanhf(x);
}

struct Rows {
  const int* pos;
  const int* lens;
  const int* slots;
  int T, Bc;
};

__device__ __forceinline__ bool row_of(const Rows& g, int b, int& p0, int& n,
                                       int& slot) {
  n = g.lens ? min(g.lens[b], g.T) : g.T;
  slot = g.slots ? g.slots[b] : b;
  p0 = g.pos[b];
  return n > 0 && slot >= 0 && slot < g.Bc && p0 >= 0;
}

const int* i32_or_null(const c10::optional<torch::Tensor>& t, int64_t n) {
  if (!t.has_value()) return nullptr;
  DNET_CHECK(t->scalar_type() == torch::kInt32 && t->is_contiguous() &&
                 t->numel() >= n, "int32 index tensor [B]");
  return t->data_ptr<int>();
}

Rows make_rows(const torch::Tensor& pos,
               const c10::optional<torch::Tensor>& lens,
               const c10::optional<torch::Tensor>& slots, int64_t B, int64_t T,
               int64_t Bc) {
  DNET_CHECK(pos.scalar_type() == torch::kInt32 && pos.is_contiguous() &&
                 pos.numel() >= B, "pos int32 [B]");
  if (!slots.has_value()) DNET_CHECK(B <= Bc, "more rows than cache slots");
  Rows g;
  g.pos = pos.data_ptr<int>();
  g.lens = i32_or_null(lens, B);
  g.slots = i32_or_null(slots, B);
  g.T = (int)T;
  g.Bc = (int)Bc;
  return g;
}

bool is_bf16(const torch::Tensor& t) { return t.scalar_type() == torch::kBFloat16; }
bool is_f32(const torch::Tensor& t) { return t.scalar_type() == torch::kFloat32; }

// ---- norm + token shift ------------------------------------------------------
// grid (B * strips): a workgroup walks a strip of consecutive tokens of one
// row with the previous token's h in LDS (every thread reads and writes its
// own elements only). The strip's first predecessor is the token before it
// (its norm is recomputed), the slot's state, or zero at position 0. With
// `a` (one token per row): x += rms(a) * wa first.
template <typename T, int V, bool RES>
__global__ __launch_bounds__(1024) void norm_shift_kernel(
    float* __restrict__ x, const T* __restrict__ a,
    const float* __restrict__ wa, const float* __restrict__ wn,
    const float* __restrict__ mu, float* prev, T* __restrict__ y,
    const Rows g, const int W, const float eps, const int strip,
    const int write_state) {
  extern __shared__ __attribute__((aligned(16))) float hp[];    // [W]
  __shared__ float red[16];
  const int nstrip = (g.T + strip - 1) / strip;
  const int b = blockIdx.x / nstrip;
  const int t0 = (blockIdx.x % nstrip) * strip;
  const int t1 = min(t0 + strip, g.T);
  int p0, n, slot;
  const bool valid = row_of(g, b, p0, n, slot);
  const int step = blockDim.x * V;
  const int i0 = threadIdx.x * V;

  // h of the token before the strip
  if (t0 > 0) {
    const float* xr = x + ((int64_t)b * g.T + t0 - 1) * W;
    float ss = 0.f;
    for (int i = i0; i < W; i += step) {
      const vec<V> v = ldv<V, float>(xr + i);
#pragma unroll
      for (int j = 0; j < V; ++j) ss = fmaf(v.v[j], v.v[j], ss);
    }
    ss = block_reduce_sum(ss, red);
    const float r = 1.0f / sqrtf(ss / (float)W + eps);
    for (int i = i0; i < W; i += step) {
      vec<V> v = ldv<V, float>(xr + i);
      const vec<V> wv = ldv<V, float>(wn + i);
#pragma unroll
      for (int j = 0; j < V; ++j) v.v[j] = v.v[j] * r * wv.v[j];
      stv<V, float>(hp + i, v);
    }
  } else {
    const bool keep = valid && p0 > 0;
    for (int i = i0; i < W; i += step) {
      vec<V> v;
#pragma unroll
      for (int j = 0; j < V; ++j) v.v[j] = 0.f;
      if (keep) v = ldv<V, float>(prev + (int64_t)slot * W + i);
      stv<V, float>(hp + i, v);
    }
  }

  for (int t = t0; t < t1; ++t) {
    const int64_t row = (int64_t)b * g.T + t;
    float* xr = x + row * W;
    float ra = 0.f;
    if constexpr (RES) {
      const T* ar = a + row * W;
      float sa = 0.f;
      for (int i = i0; i < W; i += step) {
        const vec<V> v = ldv<V, T>(ar + i);
#pragma unroll
        for (int j = 0; j < V; ++j) sa = fmaf(v.v[j], v.v[j], sa);
      }
      sa = block_reduce_sum(sa, red);
      ra = 1.0f / sqrtf(sa / (float)W + eps);
    }
    float ss = 0.f;
    for (int i = i0; i < W; i += step) {
      vec<V> v = ldv<V, float>(xr + i);
      if constexpr (RES) {
        const vec<V> av = ldv<V, T>(a + row * W + i);
        const vec<V> wv = ldv<V, float>(wa + i);
#pragma unroll
        for (int j = 0; j < V; ++j) v.v[j] += av.v[j] * ra * wv.v[j];
        stv<V, float>(xr + i, v);
      }
#pragma unroll
      for (int j = 0; j < V; ++j) ss = fmaf(v.v[j], v.v[j], ss);
    }
    ss = block_reduce_sum(ss, red);
    const float r = 1.0f / sqrtf(ss / (float)W + eps);
    // each thread re-reads exactly the elements it read or wrote above
    const bool last = write_state && valid && t == n - 1;
    for (int i = i0; i < W; i += step) {
      vec<V> h = ldv<V, float>(xr + i);
      const vec<V> wv = ldv<V, float>(wn + i), m = ldv<V, float>(mu + i);
      const vec<V> q = ldv<V, float>(hp + i);
      vec<V> o;
#pragma unroll
      for (int j = 0; j < V; ++j) {
        h.v[j] = h.v[j] * r * wv.v[j];
        o.v[j] = h.v[j] + (q.v[j] - h.v[j]) * m.v[j];
      }
      stv<V, float>(hp + i, h);
      stv<V, T>(y + row * W + i, o);
      if (last) stv<V, float>(prev + (int64_t)slot * W + i, h);
    }
  }
}

// grid (B), prompts of several strips: the slot's state becomes the h of its
// last real token. A separate launch: the first strip reads the old state.
template <int V>
__global__ __launch_bounds__(256) void shift_state_kernel(
    const float* __restrict__ x, const float* __restrict__ wn,
    float* __restrict__ prev, const Rows g, const int W, const float eps) {
  __shared__ float red[8];
  const int b = blockIdx.x;
  int p0, n, slot;
  if (!row_of(g, b, p0, n, slot)) return;
  const float* xr = x + ((int64_t)b * g.T + n - 1) * W;
  const int step = blockDim.x * V, i0 = threadIdx.x * V;
  float ss = 0.f;
  for (int i = i0; i < W; i += step) {
    const vec<V> v = ldv<V, float>(xr + i);
#pragma unroll
    for (int j = 0; j < V; ++j) ss = fmaf(v.v[j], v.v[j], ss);
  }
  ss = block_reduce_sum(ss, red);
  const float r = 1.0f / sqrtf(ss / (float)W + eps);
  for (int i = i0; i < W; i += step) {
    vec<V> v = ldv<V, float>(xr + i);
    const vec<V> wv = ldv<V, float>(wn + i);
#pragma unroll
    for (int j = 0; j < V; ++j) v.v[j] = v.v[j] * r * wv.v[j];
    stv<V, float>(prev + (int64_t)slot * W + i, v);
  }
}

// ---- minGRU ---------------------------------------------------------------
template <bool FAST>
__device__ __forceinline__ void gru_gates(float zc, float xc, float& keep,
                                          float& add) {
  const float z = sigmoid_x<FAST>(zc);
  const float cand = xc >= 0.f ? xc + 0.5f : sigmoid_x<FAST>(xc);
  keep = 1.f - z;
  add = z * cand;
}

// decode: one thread per channel; grid (channel tiles, B)
template <typename T>
__global__ __launch_bounds__(256) void mingru_step_kernel(
    const T* __restrict__ src, const int64_t ld, const int z0, const int x0,
    const int g0, const float* __restrict__ bz, const float* __restrict__ bx,
    float* __restrict__ state, T* __restrict__ y, const Rows g, const int N) {
  constexpr bool FAST = sizeof(T) == 2;
  const int c = blockIdx.x * blockDim.x + threadIdx.x;
  if (c >= N) return;
  const int b = blockIdx.y;
  int p0, n, slot;
  if (!row_of(g, b, p0, n, slot)) return;
  const T* sr = src + (int64_t)b * ld;
  float keep, add;
  gru_gates<FAST>(ldx<T>(sr + z0 + c) + bz[c], ldx<T>(sr + x0 + c) + bx[c],
                  keep, add);
  float* sp = state + (int64_t)slot * N + c;
  const float S = fmaf(keep, p0 > 0 ? *sp : 0.f, add);
  *sp = S;
  const float gv = ldx<T>(sr + g0 + c);
  stx<T>(y + (int64_t)b * N + c, S * gv * sigmoid_x<FAST>(gv));
}

// prompts: grid (channel tiles of 64, B), NW waves. A tile of NW * TW tokens
// is cut into TW consecutive tokens per wave, lane = channel: each wave reads
// its tokens' gates once into registers and folds them into one affine map
// S -> A S + C; the maps meet in LDS, every wave applies those before its own
// to the carried state and replays its tokens from registers.
constexpr int kGruTW = 16;

template <typename T, int NW>
__global__ __launch_bounds__(NW * 64) void mingru_scan_kernel(
    const T* __restrict__ src, const int64_t ld, const int z0, const int x0,
    const int g0, const float* __restrict__ bz, const float* __restrict__ bx,
    float* __restrict__ state, T* __restrict__ y, const Rows g, const int N) {
  constexpr bool FAST = sizeof(T) == 2;
  constexpr int TW = kGruTW;
  __shared__ float sA[2][NW][64], sC[2][NW][64];
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int c = blockIdx.x * 64 + lane;
  const int b = blockIdx.y;
  int p0, n, slot;
  if (!row_of(g, b, p0, n, slot)) return;          // workgroup-uniform
  const bool on = c < N;
  const int cc = on ? c : N - 1;
  const float bzc = bz[cc], bxc = bx[cc];
  float* sp = state + (int64_t)slot * N + cc;
  float carry = p0 > 0 ? *sp : 0.f;
  const T* base = src + (int64_t)b * g.T * ld + cc;
  int buf = 0;
  for (int tile = 0; tile < n; tile += NW * TW, buf ^= 1) {
    const int t0 = tile + wave * TW;
    float keep[TW], add[TW], gv[TW];
#pragma unroll
    for (int i = 0; i < TW; ++i) {
      const int t = min(t0 + i, n - 1);
      const T* sr = base + (int64_t)t * ld;
      keep[i] = ldx<T>(sr + z0);
      add[i] = ldx<T>(sr + x0);
      gv[i] = ldx<T>(sr + g0);
    }
    float A = 1.f, C = 0.f;
#pragma unroll
    for (int i = 0; i < TW; ++i) {
      float k, d;
      gru_gates<FAST>(keep[i] + bzc, add[i] + bxc, k, d);
      if (t0 + i >= n) {                           // past the row's tokens
        k = 1.f;
        d = 0.f;
      }
      keep[i] = k;
      add[i] = d;
      A *= k;
      C = fmaf(k, C, d);
    }
    sA[buf][wave][lane] = A;
    sC[buf][wave][lane] = C;
    __syncthreads();      // (two buffers: the next tile writes the other one)
    float S = carry, mine = carry;
#pragma unroll
    for (int w = 0; w < NW; ++w) {
      if (w == wave) mine = S;
      S = fmaf(sA[buf][w][lane], S, sC[buf][w][lane]);
    }
    carry = S;
    S = mine;
#pragma unroll
    for (int i = 0; i < TW; ++i) {
      S = fmaf(keep[i], S, add[i]);
      if (on && t0 + i < n)
        stx<T>(y + ((int64_t)b * g.T + t0 + i) * N + c,
               S * gv[i] * sigmoid_x<FAST>(gv[i]));
    }
  }
  if (on && wave == 0) *sp = carry;
}

// ---- rows into the cache -----------------------------------------------------
// grid (B*T): src columns [col0, col0 + H*D) -> cache [Bc, H, Smax, D]
template <typename TI, typename TO>
__global__ __launch_bounds__(256) void cache_append_kernel(
    const TI* __restrict__ src, const int64_t ld, const int col0,
    TO* __restrict__ cache, const Rows g, const int H, const int D,
    const int Smax) {
  const int64_t row = blockIdx.x;
  const int b = (int)(row / g.T), t = (int)(row % g.T);
  int p0, n, slot;
  if (!row_of(g, b, p0, n, slot) || t >= n) return;
  const int p = p0 + t;
  if (p >= Smax) return;
  const TI* sr = src + row * ld + col0;
  for (int i = threadIdx.x; i < H * D; i += blockDim.x) {
    const int h = i / D, e = i % D;
    stx<TO>(cache + (((int64_t)slot * H + h) * Smax + p) * D + e,
            ldx<TI>(sr + i));
  }
}

// ---- gated activations ---------------------------------------------------------
constexpr int kActSilu = 0, kActGelu = 1, kActClamp = 2;

template <bool FAST, int KIND> __device__ __forceinline__ float act_x(float g) {
  if constexpr (KIND == kActGelu) {
    const float k = 0.7978845608028654f;           // sqrt(2 / pi)
    return 0.5f * g * (1.f + tanh_x<FAST>(k * (g + 0.044715f * g * g * g)));
  }
  return g * sigmoid_x<FAST>(g);
}

// silu, tanh-gelu: act(s g) * (s u), the row factor s on the inputs. Clamped:
// g' sigmoid(alpha g') (u' + 1) s with g' = min(g, limit), u' = u clamped to
// +-limit, the factor on the result.
template <typename T, int V, int KIND>
__global__ __launch_bounds__(256) void gated_act_kernel(
    const T* __restrict__ gu, const float* __restrict__ scale,
    T* __restrict__ y, const int I, const int64_t total, const float alpha,
    const float limit) {
  constexpr bool FAST = sizeof(T) == 2;
  for (int64_t idx = ((int64_t)blockIdx.x * blockDim.x + threadIdx.x) * V;
       idx < total; idx += (int64_t)gridDim.x * blockDim.x * V) {
    const int64_t row = idx / I;
    const int c = (int)(idx % I);
    const float s = scale ? scale[row] : 1.f;
    const vec<V> gv = ldv<V, T>(gu + row * 2 * I + c);
    vec<V> uv = ldv<V, T>(gu + row * 2 * I + I + c);
#pragma unroll
    for (int j = 0; j < V; ++j) {
      if constexpr (KIND == kActClamp) {
        const float g = fminf(gv.v[j], limit);
        const float u = fminf(fmaxf(uv.v[j], -limit), limit);
        uv.v[j] = g * sigmoid_x<FAST>(alpha * g) * (u + 1.f) * s;
      } else {
        uv.v[j] = act_x<FAST, KIND>(gv.v[j] * s) * (uv.v[j] * s);
      }
    }
    stv<V, T>(y + idx, uv);
  }
}

}  // namespace

void norm_token_shift(torch::Tensor x, c10::optional<torch::Tensor> a,
                      c10::optional<torch::Tensor> wa, torch::Tensor wn,
                      torch::Tensor mu, torch::Tensor prev, torch::Tensor y,
                      torch::Tensor pos, c10::optional<torch::Tensor> lens,
                      c10::optional<torch::Tensor> slots, int64_t T,
                      double eps) {
  DNET_CHECK(x.dim() == 2 && x.is_contiguous() && is_f32(x), "x fp32 [B*T, W]");
  const int64_t M = x.size(0);
  const int W = x.size(1);
  DNET_CHECK(T > 0 && M % T == 0, "rows = B*T");
  const int64_t B = M / T;
  DNET_CHECK(is_f32(wn) && wn.is_contiguous() && wn.numel() == W &&
                 is_f32(mu) && mu.is_contiguous() && mu.numel() == W,
             "wn, mu fp32 [W]");
  DNET_CHECK(is_f32(prev) && prev.is_contiguous() && prev.dim() == 2 &&
                 prev.size(1) == W, "prev fp32 [Bc, W]");
  DNET_CHECK(y.is_contiguous() && y.sizes() == x.sizes() &&
                 (is_f32(y) || is_bf16(y)), "y [B*T, W]");
  DNET_CHECK(a.has_value() == wa.has_value(), "a and wa come together");
  if (a.has_value())
    DNET_CHECK(T == 1 && a->is_contiguous() && a->sizes() == x.sizes() &&
                   a->scalar_type() == y.scalar_type() && is_f32(*wa) &&
                   wa->is_contiguous() && wa->numel() == W,
               "a [B, W] in y's dtype, wa fp32 [W], one token per row");
  const size_t lds = (size_t)W * sizeof(float);
  DNET_CHECK(lds <= 60 * 1024, "norm_token_shift: width <= 15360");
  if (M == 0) return;
  const Rows g = make_rows(pos, lens, slots, B, T, prev.size(0));
  // strips of 16 tokens (one recomputed norm each) once they fill the chip
  int strip = (int)std::min<int64_t>(T, 16);
  while (strip > 4 && B * ((T + strip - 1) / strip) < 512) strip /= 2;
  const int nstrip = (int)((T + strip - 1) / strip);
  const bool v4 = W % 4 == 0;
  // decode: few workgroups, so more waves on each row
  const int nt = T == 1 && W >= 4096 ? 1024 : (T == 1 && W >= 1024 ? 512 : 256);
  auto st = current_stream();
#define NS(TT, VV, RR)                                                        \
  hipLaunchKernelGGL((norm_shift_kernel<TT, VV, RR>),                         \
                     dim3((unsigned)(B * nstrip)), dim3(nt), lds, st,         \
                     x.data_ptr<float>(),                                     \
                     RR ? (const TT*)a->data_ptr() : nullptr,                 \
                     RR ? wa->data_ptr<float>() : nullptr,                    \
                     wn.data_ptr<float>(), mu.data_ptr<float>(),              \
                     prev.data_ptr<float>(), (TT*)y.data_ptr(), g, W,         \
                     (float)eps, strip, nstrip == 1 ? 1 : 0)
#define NS_V(TT, RR) do { if (v4) NS(TT, 4, RR); else NS(TT, 1, RR); } while (0)
  if (is_bf16(y)) {
    if (a.has_value()) NS_V(short, true); else NS_V(short, false);
  } else {
    if (a.has_value()) NS_V(float, true); else NS_V(float, false);
  }
#undef NS_V
#undef NS
  if (nstrip > 1) {
    if (v4)
      hipLaunchKernelGGL((shift_state_kernel<4>), dim3((unsigned)B), dim3(256),
                         0, st, x.data_ptr<float>(), wn.data_ptr<float>(),
                         prev.data_ptr<float>(), g, W, (float)eps);
    else
      hipLaunchKernelGGL((shift_state_kernel<1>), dim3((unsigned)B), dim3(256),
                         0, st, x.data_ptr<float>(), wn.data_ptr<float>(),
                         prev.data_ptr<float>(), g, W, (float)eps);
  }
}

void mingru_scan(torch::Tensor src, int64_t z0, int64_t x0, int64_t g0,
                 torch::Tensor bz, torch::Tensor bx, torch::Tensor state,
                 torch::Tensor y, torch::Tensor pos,
                 c10::optional<torch::Tensor> lens,
                 c10::optional<torch::Tensor> slots, int64_t T) {
  DNET_CHECK(src.dim() == 2 && src.is_contiguous(), "src [B*T, ld]");
  const int64_t M = src.size(0), ld = src.size(1);
  DNET_CHECK(T > 0 && M % T == 0, "rows = B*T");
  const int64_t B = M / T, N = bz.numel();
  DNET_CHECK(N > 0 && z0 >= 0 && x0 >= 0 && g0 >= 0 && z0 + N <= ld &&
                 x0 + N <= ld && g0 + N <= ld, "src columns");
  DNET_CHECK(is_f32(bz) && bz.is_contiguous() && is_f32(bx) &&
                 bx.is_contiguous() && bx.numel() == N, "biases fp32 [N]");
  DNET_CHECK(is_f32(state) && state.is_contiguous() && state.dim() == 2 &&
                 state.size(1) == N, "state fp32 [Bc, N]");
  DNET_CHECK(y.is_contiguous() && y.dim() == 2 && y.size(0) == M &&
                 y.size(1) == N && y.scalar_type() == src.scalar_type(),
             "y [B*T, N] in src's dtype");
  if (M == 0) return;
  const Rows g = make_rows(pos, lens, slots, B, T, state.size(0));
  auto st = current_stream();
#define MG_ARGS(TT)                                                           \
  0, st, (const TT*)src.data_ptr(), ld, (int)z0, (int)x0, (int)g0,            \
      bz.data_ptr<float>(), bx.data_ptr<float>(), state.data_ptr<float>(),    \
      (TT*)y.data_ptr(), g, (int)N
#define MG(TT)                                                                \
  do {                                                                        \
    if (T == 1)                                                               \
      hipLaunchKernelGGL((mingru_step_kernel<TT>),                            \
                         dim3((unsigned)((N + 255) / 256), (unsigned)B),      \
                         dim3(256), MG_ARGS(TT));                             \
    else if (T <= 4 * kGruTW)                                                 \
      hipLaunchKernelGGL((mingru_scan_kernel<TT, 4>),                         \
                         dim3((unsigned)((N + 63) / 64), (unsigned)B),        \
                         dim3(256), MG_ARGS(TT));                             \
    else                                                                      \
      hipLaunchKernelGGL((mingru_scan_kernel<TT, 16>),                        \
                         dim3((unsigned)((N + 63) / 64), (unsigned)B),        \
                         dim3(1024), MG_ARGS(TT));                            \
  } while (0)
  if (is_bf16(src)) MG(short);
  else if (is_f32(src)) MG(float);
  else DNET_CHECK(false, "mingru_scan: dtype");
#undef MG
#undef MG_ARGS
}

void cache_append(torch::Tensor src, int64_t col0, torch::Tensor cache,
                  torch::Tensor pos, c10::optional<torch::Tensor> lens,
                  c10::optional<torch::Tensor> slots, int64_t T) {
  DNET_CHECK(src.dim() == 2 && src.is_contiguous(), "src [B*T, ld]");
  const int64_t M = src.size(0), ld = src.size(1);
  DNET_CHECK(T > 0 && M % T == 0, "rows = B*T");
  DNET_CHECK(cache.dim() == 4 && cache.is_contiguous(), "cache [Bc,H,Smax,D]");
  const int H = cache.size(1), Smax = cache.size(2), D = cache.size(3);
  DNET_CHECK(col0 >= 0 && col0 + (int64_t)H * D <= ld, "src columns");
  if (M == 0) return;
  const Rows g = make_rows(pos, lens, slots, M / T, T, cache.size(0));
  auto st = current_stream();
#define CA(TI, TO)                                                            \
  hipLaunchKernelGGL((cache_append_kernel<TI, TO>), dim3((unsigned)M),        \
                     dim3(256), 0, st, (const TI*)src.data_ptr(), ld,         \
                     (int)col0, (TO*)cache.data_ptr(), g, H, D, Smax)
  if (is_bf16(src) && is_bf16(cache)) CA(short, short);
  else if (is_f32(src) && is_bf16(cache)) CA(float, short);
  else if (is_f32(src) && is_f32(cache)) CA(float, float);
  else DNET_CHECK(false, "cache_append: dtypes");
#undef CA
}

void gated_act(torch::Tensor gu, c10::optional<torch::Tensor> scale,
               torch::Tensor y, int64_t kind, double alpha, double limit) {
  DNET_CHECK(gu.dim() == 2 && gu.is_contiguous() && y.dim() == 2 &&
                 y.is_contiguous() && y.size(0) == gu.size(0) &&
                 gu.size(1) == 2 * y.size(1) &&
                 y.scalar_type() == gu.scalar_type(), "gu [M, 2I], y [M, I]");
  DNET_CHECK(kind >= 0 && kind <= 2, "gated_act: kind");
  const float* sp = nullptr;
  if (scale.has_value()) {
    DNET_CHECK(is_f32(*scale) && scale->is_contiguous() &&
                   scale->numel() == gu.size(0), "scale fp32 [M]");
    sp = scale->data_ptr<float>();
  }
  const int64_t total = y.numel();
  if (total == 0) return;
  const int I = y.size(1);
  auto st = current_stream();
#define GA(TT, VV, GG)                                                        \
  hipLaunchKernelGGL((gated_act_kernel<TT, VV, GG>),                          \
                     dim3((unsigned)std::min<int64_t>(                        \
                         (total / VV + 255) / 256, 8192)),                    \
                     dim3(256), 0, st, (const TT*)gu.data_ptr(), sp,          \
                     (TT*)y.data_ptr(), I, total, (float)alpha, (float)limit)
#define GA_K(TT, VV)                                 \
  do {                                               \
    if (kind == kActGelu) GA(TT, VV, kActGelu);      \
    else if (kind == kActClamp) GA(TT, VV, kActClamp); \
    else GA(TT, VV, kActSilu);                       \
  } while (0)
  if (is_bf16(gu)) { if (I % 8 == 0) GA_K(short, 8); else GA_K(short, 1); }
  else if (is_f32(gu)) { if (I % 4 == 0) GA_K(float, 4); else GA_K(float, 1); }
  else DNET_CHECK(false, "gated_act: dtype");
#undef GA_K
#undef GA
}

}  // namespace dnet
