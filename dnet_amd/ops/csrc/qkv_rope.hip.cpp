// Projection rows -> attention operands in one launch (gfx950).
//
//   qkv_rope_append   columns [q | k | v] of a projection: + bias, short causal
//                     convolution over time (no activation), rotation of q and
//                     k (interleaved or half-split pairs on the first channels
//                     of a head), mixing of v with another layer's values of
//                     the same token; q written out, k and v appended to the
//                     cache. Every step is optional.
//
// Geometry is the cache's: token (b,t) = row b*T+t sits at position pos[b]+t of
// slot slots[b] (default b); tokens t >= lens[b] are padding: nothing of them
// is written. The convolution's last taps-1 inputs of a slot are its state,
// taken as zero before position 0. Sums, angles and the rotation are fp32 and
// a value is rounded once ("short" stands for bf16 bits).
#include "common.h"

namespace dnet {

namespace {

bool is_bf16(const torch::Tensor& t) { return t.scalar_type() == torch::kBFloat16; }
bool is_f32(const torch::Tensor& t) { return t.scalar_type() == torch::kFloat32; }

// E neighbouring channels in one access (E = 2: 4 B bf16 / 8 B fp32)
template <int E> __device__ __forceinline__ void ldc(const float* p, float (&v)[E]) {
  if constexpr (E == 2) {
    const float2 t = *reinterpret_cast<const float2*>(p);
    v[0] = t.x; v[1] = t.y;
  } else {
    v[0] = *p;
  }
}
template <int E> __device__ __forceinline__ void ldc(const short* p, float (&v)[E]) {
  if constexpr (E == 2) {
    const unsigned t = *reinterpret_cast<const unsigned*>(p);
    v[0] = bits2f((short)(t & 0xffffu));
    v[1] = bits2f((short)(t >> 16));
  } else {
    v[0] = bits2f(*p);
  }
}
template <int E> __device__ __forceinline__ void stc(float* p, const float (&v)[E]) {
  if constexpr (E == 2) *reinterpret_cast<float2*>(p) = make_float2(v[0], v[1]);
  else *p = v[0];
}
template <int E> __device__ __forceinline__ void stc(short* p, const float (&v)[E]) {
  if constexpr (E == 2)
    *reinterpret_cast<unsigned*>(p) =
        (unsigned)(unsigned short)f2bits(v[0]) |
        ((unsigned)(unsigned short)f2bits(v[1]) << 16);
  else *p = f2bits(v[0]);
}

struct QkvArgs {
  const void* src;           // [B*T, ld], q at column col0
  const float* bias;         // [C] or null
  const float* cw;           // convolution taps [C, taps] or null
  void* cstate;              // [Bc, taps-1, C]
  const float* freq;         // [nrot]
  void* q;                   // [B*T, nq*d]
  void* kc;                  // [Bc, nkv, Smax, d]
  void* vc;                  // [Bc, nkv, Smax, dv]
  // v <- (1 - lam) v + lam vf; vf: rows of this step (vf_rows: row stride
  // vs_pos) or another layer's value cache (slot / head / position strides)
  const void* vf;
  const float* lam;
  int64_t ld, vs_slot, vs_head, vs_pos;
  const int* pos;
  const int* lens;
  const int* slots;
  int col0, taps, nrot, nq, nkv, d, dv, Smax, T, Bc, tile, tail, vf_rows;
};

__device__ __forceinline__ bool row_of(const QkvArgs& a, int b, int& p0, int& n,
                                       int& slot) {
  n = a.lens ? min(a.lens[b], a.T) : a.T;
  slot = a.slots ? a.slots[b] : b;
  p0 = a.pos[b];
  return n > 0 && slot >= 0 && slot < a.Bc && p0 >= 0;
}

// grid (B * token tiles, channel splits). A work item is four channels of one
// head (two with E = 1) as two groups of E neighbours: the two halves of the
// turning pairs in the half-split layout, neighbours otherwise. A thread walks
// the tile's tokens with the convolution's window in registers, so an input is
// read once. TAPS: register window (the real taps sit at its end).
template <typename T, int E, int TAPS, bool HALF>
__global__ __launch_bounds__(256) void qkv_rope_kernel(const QkvArgs a) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  const int ntile = (a.T + a.tile - 1) / a.tile;
  const int b = blockIdx.x / ntile;
  const int t0 = (blockIdx.x % ntile) * a.tile;
  int p0, n, slot;
  if (!row_of(a, b, p0, n, slot) || t0 >= n) return;   // workgroup-uniform
  const int t1 = min(t0 + a.tile, n);
  float* cs = sm;                          // [tile][nrot]
  float* sn = sm + a.tile * a.nrot;
  for (int i = threadIdx.x; i < (t1 - t0) * a.nrot; i += blockDim.x)
    sincosf((float)(p0 + t0 + i / a.nrot) * a.freq[i % a.nrot], &sn[i], &cs[i]);
  if (a.nrot > 0) __syncthreads();

  const T* src = reinterpret_cast<const T*>(a.src);
  T* cstate = reinterpret_cast<T*>(a.cstate);
  const int NQ = a.nq * a.d, NK = a.nkv * a.d, C = NQ + NK + a.nkv * a.dv;
  const int ih = (a.d + 2 * E - 1) / (2 * E);
  const int iv = (a.dv + 2 * E - 1) / (2 * E);
  const int nqk = (a.nq + a.nkv) * ih, items = nqk + a.nkv * iv;
  for (int it = blockIdx.y * blockDim.x + threadIdx.x; it < items;
       it += gridDim.y * blockDim.x) {
    const bool isv = it >= nqk;
    const int head = isv ? (it - nqk) / iv : it / ih;   // q heads, then k heads
    const int i = isv ? (it - nqk) % iv : it % ih;
    const bool isk = !isv && head >= a.nq;
    const int hd = isv ? a.dv : a.d;
    // the item's two channel groups and, when they turn, their first pair
    int c0 = 2 * E * i, c1 = c0 + E, pr = 0;
    bool turn = false;
    if (!isv) {
      if (HALF) {
        turn = E * i < a.nrot;
        if (turn) {
          pr = c0 = E * i;
          c1 = c0 + a.nrot;
        }
      } else {
        pr = E * i;
        turn = pr < a.nrot;
      }
    }
    const bool on1 = c1 < hd;              // E = 1, odd sizes: one channel left
    const int base = isv ? NQ + NK + head * a.dv : head * a.d;
    const int ch[2] = {base + c0, base + (on1 ? c1 : c0)};

    float w[TAPS][2][E], win[TAPS][2][E], bs[2][E];
#pragma unroll
    for (int g = 0; g < 2; ++g)
#pragma unroll
      for (int e = 0; e < E; ++e) {
        bs[g][e] = a.bias ? a.bias[ch[g] + e] : 0.f;
        if constexpr (TAPS > 1) {
#pragma unroll
          for (int j = 0; j < TAPS; ++j) {
            const int jj = j - (TAPS - a.taps);
            w[j][g][e] =
                jj >= 0 ? a.cw[(int64_t)(ch[g] + e) * a.taps + jj] : 0.f;
          }
        }
      }
    if constexpr (TAPS > 1) {
      // inputs before the tile: earlier rows of this step, the slot's tail, or
      // zero before position 0
#pragma unroll
      for (int j = 0; j < TAPS - 1; ++j) {
        const int tt = t0 - (TAPS - 1) + j, s = a.taps - 1 + tt;
#pragma unroll
        for (int g = 0; g < 2; ++g) {
#pragma unroll
          for (int e = 0; e < E; ++e) win[j][g][e] = 0.f;
          if (j < TAPS - a.taps) continue;             // no such tap
          if (tt >= 0)
            ldc<E>(src + ((int64_t)b * a.T + tt) * a.ld + a.col0 + ch[g],
                   win[j][g]);
          else if (p0 + tt >= 0 && s >= 0)
            ldc<E>(cstate + ((int64_t)slot * (a.taps - 1) + s) * C + ch[g],
                   win[j][g]);
        }
      }
    }
    for (int t = t0; t < t1; ++t) {
      const int64_t row = (int64_t)b * a.T + t;
      const int p = p0 + t;
      float x[2][E];
#pragma unroll
      for (int g = 0; g < 2; ++g) {
        ldc<E>(src + row * a.ld + a.col0 + ch[g], x[g]);
#pragma unroll
        for (int e = 0; e < E; ++e) x[g][e] += bs[g][e];
        if constexpr (TAPS > 1) {
#pragma unroll
          for (int e = 0; e < E; ++e) {
            float s = 0.f;
#pragma unroll
            for (int j = 0; j < TAPS - 1; ++j)
              s = fmaf(w[j][g][e], win[j][g][e], s);
            s = fmaf(w[TAPS - 1][g][e], x[g][e], s);
#pragma unroll
            for (int j = 0; j < TAPS - 2; ++j) win[j][g][e] = win[j + 1][g][e];
            win[TAPS - 2][g][e] = x[g][e];
            x[g][e] = s;
          }
        }
      }
      if (turn) {
        const float* ct = cs + (t - t0) * a.nrot;
        const float* st = sn + (t - t0) * a.nrot;
        if constexpr (HALF) {              // x[0][e] with x[1][e]
#pragma unroll
          for (int e = 0; e < E; ++e) {
            const float c = ct[pr + e], s = st[pr + e];
            const float u = x[0][e], v = x[1][e];
            x[0][e] = u * c - v * s;
            x[1][e] = v * c + u * s;
          }
        } else if constexpr (E == 2) {     // pairs inside each group
#pragma unroll
          for (int g = 0; g < 2; ++g)
            if (pr + g < a.nrot) {
              const float c = ct[pr + g], s = st[pr + g];
              const float u = x[g][0], v = x[g][1];
              x[g][0] = u * c - v * s;
              x[g][1] = v * c + u * s;
            }
        } else {
          const float c = ct[pr], s = st[pr];
          const float u = x[0][0], v = x[1][0];
          x[0][0] = u * c - v * s;
          x[1][0] = v * c + u * s;
        }
      }
      if (isv) {
        if (p >= a.Smax) continue;
        if (a.vf) {
          const float lam = *a.lam;
          const T* vr = reinterpret_cast<const T*>(a.vf) +
                        (a.vf_rows ? row * a.vs_pos
                                   : slot * a.vs_slot + p * a.vs_pos) +
                        head * a.vs_head;
#pragma unroll
          for (int g = 0; g < 2; ++g) {
            float f[E];
            ldc<E>(vr + (g == 0 || !on1 ? c0 : c1), f);
#pragma unroll
            for (int e = 0; e < E; ++e)
              x[g][e] = (1.f - lam) * x[g][e] + lam * f[e];
          }
        }
        T* dst = reinterpret_cast<T*>(a.vc) +
                 (((int64_t)slot * a.nkv + head) * a.Smax + p) * a.dv;
        stc<E>(dst + c0, x[0]);
        if (on1) stc<E>(dst + c1, x[1]);
      } else if (isk) {
        if (p >= a.Smax) continue;
        T* dst = reinterpret_cast<T*>(a.kc) +
                 (((int64_t)slot * a.nkv + head - a.nq) * a.Smax + p) * a.d;
        stc<E>(dst + c0, x[0]);
        if (on1) stc<E>(dst + c1, x[1]);
      } else {
        T* dst = reinterpret_cast<T*>(a.q) + row * NQ + head * a.d;
        stc<E>(dst + c0, x[0]);
        if (on1) stc<E>(dst + c1, x[1]);
      }
    }
    if constexpr (TAPS > 1) {
      // a row's tokens fit one tile: this thread's window is the new tail
      if (a.tail) {
#pragma unroll
        for (int j = 0; j < TAPS - 1; ++j) {
          const int s = j - (TAPS - a.taps);
          if (s < 0) continue;
          T* st = cstate + ((int64_t)slot * (a.taps - 1) + s) * C;
          stc<E>(st + ch[0], win[j][0]);
          if (on1) stc<E>(st + ch[1], win[j][1]);
        }
      }
    }
  }
}

// grid (channel tiles, B), rows of several tiles: the slot's tail moves on, in
// a launch of its own, after every tile has read the old one
template <typename T>
__global__ __launch_bounds__(256) void qkv_tail_kernel(const QkvArgs a,
                                                       const int C) {
  const int c = blockIdx.x * blockDim.x + threadIdx.x;
  if (c >= C) return;
  const int b = blockIdx.y;
  int p0, n, slot;
  if (!row_of(a, b, p0, n, slot)) return;
  const T* src = reinterpret_cast<const T*>(a.src);
  T* st = reinterpret_cast<T*>(a.cstate) + (int64_t)slot * (a.taps - 1) * C + c;
  for (int s = 0; s < a.taps - 1; ++s) {        // ascending: reads run ahead
    const int q = n - (a.taps - 1) + s;         // index among the new tokens
    T v = (T)0;
    if (q >= 0) v = src[((int64_t)b * a.T + q) * a.ld + a.col0 + c];
    else if (p0 + q >= 0) v = st[(int64_t)(s + n) * C];
    st[(int64_t)s * C] = v;
  }
}

const int* idx32(const torch::Tensor& t, int64_t n) {
  DNET_CHECK(t.scalar_type() == torch::kInt32 && t.is_contiguous() &&
                 t.numel() >= n, "int32 index tensor [B]");
  return t.data_ptr<int>();
}

}  // namespace

void qkv_rope_append(torch::Tensor src, int64_t col0, int64_t nq, int64_t nkv,
                     int64_t d, int64_t dv, c10::optional<torch::Tensor> bias,
                     c10::optional<torch::Tensor> conv_w,
                     c10::optional<torch::Tensor> conv_state,
                     c10::optional<torch::Tensor> rot_freq, bool half,
                     c10::optional<torch::Tensor> vf,
                     c10::optional<torch::Tensor> lam, torch::Tensor q,
                     torch::Tensor kcache, torch::Tensor vcache,
                     torch::Tensor pos, c10::optional<torch::Tensor> lens,
                     c10::optional<torch::Tensor> slots, int64_t T) {
  DNET_CHECK(src.dim() == 2 && src.is_contiguous(), "src [B*T, ld]");
  const int64_t M = src.size(0), ld = src.size(1);
  DNET_CHECK(T > 0 && M % T == 0, "rows = B*T");
  const int64_t B = M / T, C = nq * d + nkv * (d + dv);
  DNET_CHECK(nq > 0 && nkv > 0 && d > 0 && dv > 0 && nq % nkv == 0, "heads");
  DNET_CHECK(col0 >= 0 && col0 + C <= ld, "src columns");
  DNET_CHECK(is_bf16(src) || is_f32(src), "bf16 or fp32");
  DNET_CHECK(q.dim() == 2 && q.is_contiguous() && q.size(0) == M &&
                 q.size(1) == nq * d, "q [B*T, nq*d]");
  DNET_CHECK(kcache.dim() == 4 && vcache.dim() == 4 && kcache.is_contiguous() &&
                 vcache.is_contiguous() && kcache.size(1) == nkv &&
                 kcache.size(3) == d && vcache.size(0) == kcache.size(0) &&
                 vcache.size(1) == nkv && vcache.size(2) == kcache.size(2) &&
                 vcache.size(3) == dv, "cache [Bc, nkv, Smax, d | dv]");
  const auto dt = src.scalar_type();
  DNET_CHECK(q.scalar_type() == dt && kcache.scalar_type() == dt &&
                 vcache.scalar_type() == dt, "dtypes");
  QkvArgs a = {};
  a.src = src.data_ptr(); a.q = q.data_ptr();
  a.kc = kcache.data_ptr(); a.vc = vcache.data_ptr();
  a.ld = ld; a.col0 = (int)col0; a.nq = (int)nq; a.nkv = (int)nkv;
  a.d = (int)d; a.dv = (int)dv; a.T = (int)T;
  a.Bc = (int)kcache.size(0); a.Smax = (int)kcache.size(2);
  a.taps = 1;
  if (!slots.has_value()) DNET_CHECK(B <= a.Bc, "more rows than cache slots");
  a.pos = idx32(pos, B);
  a.lens = lens.has_value() ? idx32(*lens, B) : nullptr;
  a.slots = slots.has_value() ? idx32(*slots, B) : nullptr;
  if (bias.has_value()) {
    DNET_CHECK(is_f32(*bias) && bias->is_contiguous() && bias->numel() == C,
               "bias fp32 [C]");
    a.bias = bias->data_ptr<float>();
  }
  if (conv_w.has_value()) {
    DNET_CHECK(!bias.has_value(), "the convolution's inputs take no bias");
    DNET_CHECK(is_f32(*conv_w) && conv_w->is_contiguous() &&
                   conv_w->dim() == 2 && conv_w->size(0) == C,
               "conv_w fp32 [C, taps]");
    a.taps = (int)conv_w->size(1);
    DNET_CHECK(a.taps >= 1 && a.taps <= 16, "1 <= taps <= 16");
    DNET_CHECK(conv_state.has_value() && conv_state->dim() == 3 &&
                   conv_state->is_contiguous() &&
                   conv_state->size(0) == a.Bc &&
                   conv_state->size(1) == a.taps - 1 &&
                   conv_state->size(2) == C && conv_state->scalar_type() == dt,
               "conv_state [Bc, taps-1, C]");
    a.cw = conv_w->data_ptr<float>();
    a.cstate = conv_state->data_ptr();
  }
  if (rot_freq.has_value()) {
    DNET_CHECK(is_f32(*rot_freq) && rot_freq->is_contiguous() &&
                   rot_freq->numel() * 2 <= d, "rot_freq fp32 [<= d/2]");
    a.freq = rot_freq->data_ptr<float>();
    a.nrot = (int)rot_freq->numel();
  }
  DNET_CHECK(vf.has_value() == lam.has_value(), "vf and lam come together");
  if (vf.has_value()) {
    DNET_CHECK(is_f32(*lam) && lam->numel() == 1, "lam fp32 [1]");
    a.lam = lam->data_ptr<float>();
    DNET_CHECK(vf->is_contiguous() && vf->scalar_type() == dt, "vf");
    a.vf = vf->data_ptr();
    if (vf->dim() == 2) {                  // this step's rows
      DNET_CHECK(vf->size(0) == M && vf->size(1) == nkv * dv,
                 "vf rows [B*T, nkv*dv]");
      a.vf_rows = 1;
      a.vs_pos = nkv * dv;
      a.vs_head = dv;
    } else {                               // another layer's value cache
      DNET_CHECK(vf->dim() == 4 && vf->size(0) == a.Bc &&
                     vf->size(2) == a.Smax &&
                     vf->size(1) * vf->size(3) == nkv * dv &&
                     vf->size(3) == dv, "vf cache [Bc, nkv, Smax, dv]");
      a.vs_slot = nkv * (int64_t)a.Smax * dv;
      a.vs_head = (int64_t)a.Smax * dv;
      a.vs_pos = dv;
    }
  }
  if (M == 0) return;
  a.tile = T == 1 ? 1 : 8;
  const int ntile = (int)((T + a.tile - 1) / a.tile);
  a.tail = a.taps > 1 && ntile == 1;
  // neighbouring channels two at a time when everything is aligned for it
  const bool e2 = d % 4 == 0 && dv % 4 == 0 && col0 % 2 == 0 && ld % 2 == 0 &&
                  a.nrot % 2 == 0;
  const int E = e2 ? 2 : 1;
  const int64_t items = (nq + nkv) * ((d + 2 * E - 1) / (2 * E)) +
                        nkv * ((dv + 2 * E - 1) / (2 * E));
  // few rows (decode): spread a row's channels over workgroups
  int gy = 1;
  const int need = (int)((items + 255) / 256);
  while (gy < need && B * ntile * gy < 512) ++gy;
  const dim3 grid((unsigned)(B * ntile), (unsigned)gy);
  const size_t lds = (size_t)a.tile * a.nrot * 2 * sizeof(float);
  auto st = current_stream();
#define QR(TT, EE, TP, HH)                                                    \
  hipLaunchKernelGGL((qkv_rope_kernel<TT, EE, TP, HH>), grid, dim3(256), lds, \
                     st, a)
#define QR_H(TT, EE, TP) do { if (half) QR(TT, EE, TP, true); else QR(TT, EE, TP, false); } while (0)
#define QR_T(TT, EE)                        \
  do {                                      \
    if (a.cw == nullptr) QR_H(TT, EE, 1);   \
    else if (a.taps <= 4) QR_H(TT, EE, 4);  \
    else QR_H(TT, EE, 16);                  \
  } while (0)
#define QR_E(TT) do { if (e2) QR_T(TT, 2); else QR_T(TT, 1); } while (0)
  if (is_bf16(src)) QR_E(short); else QR_E(float);
#undef QR_E
#undef QR_T
#undef QR_H
#undef QR
  if (a.taps > 1 && !a.tail) {
    const dim3 tg((unsigned)((C + 255) / 256), (unsigned)B);
    if (is_bf16(src))
      hipLaunchKernelGGL((qkv_tail_kernel<short>), tg, dim3(256), 0, st, a, (int)C);
    else
      hipLaunchKernelGGL((qkv_tail_kernel<float>), tg, dim3(256), 0, st, a, (int)C);
  }
}

}  // namespace dnet
