// Routed experts over rows sorted by expert, without a host read.
//   expert_plan   stable counting sort of the T * top routed entries by
//                 router output: segment offsets, token of every sorted
//                 entry, sorted place of every entry. The outputs come from
//                 a router (sel) or from a table row per token id; the table
//                 form plans several layers in one launch, one workgroup
//                 each.
//   experts_in    mid_i = act(W_in[e] (scale_i) x[rows[i]]) for the sorted
//                 entries i of every expert e (gate | up rows, or up alone);
//   experts_out   y_i = W_out[e] mid_i;
//   experts_sum   out[t] = sum_k w[t, k] y[pos[t, k]] (+ identity entries,
//                 shared expert), fp32, in order of k.
//
// experts_in / experts_out are weight streams: at decode sizes an expert has
// a handful of rows, so the time is that of reading the chosen experts'
// weights once. A workgroup (4 waves) owns 64 weight rows of one expert
// (experts_in: 32 gate and the matching 32 up rows) and all of the expert's
// rows, up to 48 at a time. The waves split the reduction dimension in
// chunks of 64 entries (one 128-byte line per weight row), weights go from
// memory straight into the operand registers of v_mfma_f32_16x16x32_bf16
// (A = weights, B = rows, so a lane ends up with 4 consecutive outputs of
// one row), with the next chunk's loads in flight during the products, and
// the four partial sums meet in LDS in a fixed order. An expert nobody chose
// costs nothing.
#include "mix_common.h"

typedef __attribute__((ext_vector_type(8))) __bf16 mg_bf16x8;
typedef __attribute__((ext_vector_type(4))) float mg_f32x4;

#define MG_MAX_OUT 1024
#define MG_PLAN_THREADS 512

// ---------------------------------------------------------------------------
// plan
// ---------------------------------------------------------------------------
// Lanes of the wave whose value equals this lane's; v < 2^bits.
PS_DEV unsigned long long mg_peers(int v, bool on, int bits) {
  unsigned long long m = __ballot(on);
  for (int b = 0; b < bits; ++b) {
    const unsigned long long s = __ballot(on && ((v >> b) & 1));
    m &= ((v >> b) & 1) ? s : ~s;
  }
  return m;
}

// One workgroup per layer. Every wave owns a contiguous share of the entries
// and a histogram of its own in LDS; the histograms' prefix sums (by output,
// then by wave) are the places at which the waves then lay down their
// entries in order.
__global__ __launch_bounds__(MG_PLAN_THREADS) void expert_plan_kernel(
    int* __restrict__ offs, int* __restrict__ rows, int* __restrict__ pos,
    const int64_t* __restrict__ sel, const int64_t* __restrict__ tokens,
    const int* __restrict__ tables, int T_, int top, int n_out, int V,
    int bits) {
  extern __shared__ int lds_i[];
  constexpr int NW = MG_PLAN_THREADS / 64;
  int* cnt = lds_i;                 // [NW][n_out]
  int* tot = cnt + NW * n_out;      // [n_out]
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int n = T_ * top;
  offs += (size_t)blockIdx.x * (n_out + 1);
  rows += (size_t)blockIdx.x * n;
  pos += (size_t)blockIdx.x * n;
  const int* table =
      tables != nullptr ? tables + (size_t)blockIdx.x * V * top : nullptr;
  auto output_of = [&](int i) -> int {
    int e;
    if (table != nullptr) {
      const int t = i / top;
      const int64_t tok = tokens[t];
      const int64_t safe = tok < 0 ? 0 : (tok < V ? tok : V - 1);
      e = table[safe * top + (i - t * top)];
    } else {
      e = (int)sel[i];
    }
    return e < 0 ? 0 : (e < n_out ? e : n_out - 1);
  };
  for (int c = threadIdx.x; c < NW * n_out; c += blockDim.x) cnt[c] = 0;
  __syncthreads();
  const int share = ((n + NW * 64 - 1) / (NW * 64)) * 64;
  const int a = wave * share, b = min(n, a + share);
  volatile int* mine = cnt + wave * n_out;
  for (int i0 = a; i0 < b; i0 += 64) {
    const int i = i0 + lane;
    if (i < b) atomicAdd(cnt + wave * n_out + output_of(i), 1);
  }
  __syncthreads();
  for (int e = threadIdx.x; e < n_out; e += blockDim.x) {
    int s = 0;
    for (int w = 0; w < NW; ++w) s += cnt[w * n_out + e];
    tot[e] = s;
  }
  __syncthreads();
  if (wave == 0) {
    // exclusive prefix sum over the outputs, 64 at a time
    int base = 0;
    for (int e0 = 0; e0 < n_out; e0 += 64) {
      const int e = e0 + lane;
      int v = e < n_out ? tot[e] : 0;
      const int own = v;
#pragma unroll
      for (int off = 1; off < 64; off <<= 1) {
        const int u = __shfl_up(v, off, 64);
        if (lane >= off) v += u;
      }
      if (e < n_out) {
        tot[e] = base + v - own;
        offs[e] = base + v - own;
      }
      base += __shfl(v, 63, 64);
    }
    if (lane == 0) offs[n_out] = base;
  }
  __syncthreads();
  for (int e = threadIdx.x; e < n_out; e += blockDim.x) {
    int s = tot[e];
    for (int w = 0; w < NW; ++w) {
      const int c = cnt[w * n_out + e];
      cnt[w * n_out + e] = s;
      s += c;
    }
  }
  __syncthreads();
  for (int i0 = a; i0 < b; i0 += 64) {
    const int i = i0 + lane;
    const bool on = i < b;
    const int e = on ? output_of(i) : 0;
    const unsigned long long peers = mg_peers(e, on, bits);
    const int before = __popcll(peers & ((1ull << lane) - 1ull));
    int at = 0;
    if (on) at = mine[e] + before;
    // every lane has read its base before the first of the peers moves it
    __builtin_amdgcn_wave_barrier();
    if (on && before == 0) mine[e] = at + __popcll(peers);
    __builtin_amdgcn_wave_barrier();
    if (on) {
      pos[i] = at;
      rows[at] = i / top;
    }
  }
}

// ---------------------------------------------------------------------------
// grouped products
// ---------------------------------------------------------------------------
union MgPack {
  mg_bf16x8 v;
  uint4 q;
};

// 16 bytes at p + k, zeros from K on (K is a multiple of 8).
PS_DEV mg_bf16x8 mg_load(const unsigned short* __restrict__ p, int k, int K) {
  MgPack u;
  u.q = k < K ? *(const uint4*)(p + k) : make_uint4(0, 0, 0, 0);
  return u.v;
}

PS_DEV float mg_act(int kind, float g, float u, bool gated, float limit) {
  switch (kind) {
    case 0: return g * mx_sigmoid(g) * u;
    case 1: {
      const float z = 0.7978845608028654f * (g + 0.044715f * g * g * g);
      return 0.5f * g * (1.0f + tanhf(z)) * u;
    }
    case 2: {
      g = fminf(g, limit);
      u = gated ? fminf(fmaxf(u, -limit), limit) : 0.f;
      return g * mx_sigmoid(1.702f * g) * (u + 1.0f);
    }
    case 3: return mx_sigmoid(g) * u;
    case 4: {
      const float r = fmaxf(g, 0.f);
      return r * r * u;
    }
    default: return g;
  }
}

#define MG_ACT_NONE (-1)

PS_DEV float mg_round(float v) {
  return ps_bf16_to_f32(ps_f32_to_bf16(v));
}

// Four 16-row weight tiles (row pointers wp, one per tile and lane) times RT
// 16-row tiles of inputs (row pointers xp): this wave's share of K.
template <int RT>
PS_DEV void mg_product(const unsigned short* const (&wp)[4],
                       const unsigned short* const (&xp)[RT], int K, int wave,
                       int kq, mg_f32x4 (&acc)[4][RT]) {
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int r = 0; r < RT; ++r) acc[i][r] = {0.f, 0.f, 0.f, 0.f};
  auto multiply = [&](const mg_bf16x8(&wa)[4][2], const mg_bf16x8(&xa)[RT][2]) {
#pragma unroll
    for (int s = 0; s < 2; ++s)
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int r = 0; r < RT; ++r)
          acc[i][r] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
              wa[i][s], xa[r][s], acc[i][r], 0, 0, 0);
  };
  auto fetch = [&](mg_bf16x8(&wa)[4][2], mg_bf16x8(&xa)[RT][2], int k) {
#pragma unroll
    for (int s = 0; s < 2; ++s) {
#pragma unroll
      for (int i = 0; i < 4; ++i)
        wa[i][s] = *(const mg_bf16x8*)(wp[i] + k + 32 * s);
#pragma unroll
      for (int r = 0; r < RT; ++r)
        xa[r][s] = *(const mg_bf16x8*)(xp[r] + k + 32 * s);
    }
  };
  // whole chunks of 256 (64 per wave), the next one's loads in flight
  const int whole = K & ~255;
  int k = wave * 64 + kq;
  mg_bf16x8 wa[4][2], xa[RT][2];
  if (whole > 0) fetch(wa, xa, k);
  for (int k0 = 0; k0 < whole; k0 += 256) {
    mg_bf16x8 wn[4][2], xn[RT][2];
    k += 256;
    const bool more = k0 + 256 < whole;
    if (more) fetch(wn, xn, k);
    multiply(wa, xa);
    if (more) {
#pragma unroll
      for (int s = 0; s < 2; ++s) {
#pragma unroll
        for (int i = 0; i < 4; ++i) wa[i][s] = wn[i][s];
#pragma unroll
        for (int r = 0; r < RT; ++r) xa[r][s] = xn[r][s];
      }
    }
  }
  // the rest, zero-filled from K on
  if (whole + wave * 64 < K) {
    k = whole + wave * 64 + kq;
#pragma unroll
    for (int s = 0; s < 2; ++s) {
#pragma unroll
      for (int i = 0; i < 4; ++i) wa[i][s] = mg_load(wp[i], k + 32 * s, K);
#pragma unroll
      for (int r = 0; r < RT; ++r) xa[r][s] = mg_load(xp[r], k + 32 * s, K);
    }
    multiply(wa, xa);
  }
}

// The rows m0 .. m0 + 16 RT of one expert's segment (n rows from entry
// `first` on). PAIR: tiles 0, 1 are gate rows and 2, 3 the matching up rows,
// 32 outputs; otherwise four tiles of 64 outputs. N outputs in all.
template <int RT, bool PAIR>
PS_DEV void mg_rows(unsigned short* __restrict__ out,
                    const unsigned short* __restrict__ x,
                    const unsigned short* __restrict__ w,
                    const int* __restrict__ rows,
                    const float* __restrict__ row_scale, int first, int m0,
                    int n, int n0, int N, int K, int act, bool gated,
                    float limit, mg_f32x4* lds) {
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int lr = lane & 15, kq = 8 * (lane >> 4);
  const unsigned short* wp[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int c = min(n0 + 16 * (PAIR ? (i & 1) : i) + lr, N - 1);
    wp[i] = w + (size_t)(PAIR && i >= 2 ? N + c : c) * K;
  }
  const unsigned short* xp[RT];
#pragma unroll
  for (int r = 0; r < RT; ++r) {
    const int m = first + min(m0 + 16 * r + lr, n - 1);
    xp[r] = x + (size_t)(rows != nullptr ? rows[m] : m) * K;
  }
  mg_f32x4 acc[4][RT];
  mg_product<RT>(wp, xp, K, wave, kq, acc);
  // two rounds: tiles (j, j + 2); partial sums of the four waves
#pragma unroll
  for (int j = 0; j < 2; ++j) {
    __syncthreads();
#pragma unroll
    for (int p = 0; p < 2; ++p)
#pragma unroll
      for (int r = 0; r < RT; ++r)
        lds[((wave * 2 + p) * RT + r) * 64 + lane] = acc[j + 2 * p][r];
    __syncthreads();
    if (wave < RT) {
      const int r = wave;
      mg_f32x4 s[2];
#pragma unroll
      for (int p = 0; p < 2; ++p) {
        s[p] = lds[(p * RT + r) * 64 + lane];
#pragma unroll
        for (int v = 1; v < 4; ++v) s[p] += lds[((v * 2 + p) * RT + r) * 64 + lane];
      }
      const int m = m0 + 16 * r + lr;
      if (m < n) {
        unsigned short* o = out + (size_t)(first + m) * N;
        const float sc = row_scale != nullptr ? row_scale[first + m] : 1.f;
#pragma unroll
        for (int p = 0; p < (PAIR ? 1 : 2); ++p) {
          const int c = n0 + 16 * (PAIR ? j : j + 2 * p) + 4 * (lane >> 4);
          float y[4];
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            // rounded here as a GEMM of its own would round its result, so
            // small and large batches agree
            y[i] = mg_round(sc * s[p][i]);
            if (PAIR)
              y[i] = mg_act(act, y[i], mg_round(sc * s[1][i]), true, limit);
            else if (act != MG_ACT_NONE)
              y[i] = mg_act(act, y[i], 1.f, false, limit);
          }
          // N is a multiple of 8: four outputs are in range together
          if (c < N) {
            uint2 u;
            u.x = (unsigned int)ps_f32_to_bf16(y[0]) |
                  ((unsigned int)ps_f32_to_bf16(y[1]) << 16);
            u.y = (unsigned int)ps_f32_to_bf16(y[2]) |
                  ((unsigned int)ps_f32_to_bf16(y[3]) << 16);
            *(uint2*)(o + c) = u;
          }
        }
      }
    }
  }
}

template <bool PAIR>
__global__ __launch_bounds__(256, 2) void experts_product_kernel(
    unsigned short* __restrict__ out, const unsigned short* __restrict__ x,
    const unsigned short* __restrict__ w, const int* __restrict__ offs,
    const int* __restrict__ rows, const float* __restrict__ row_scale, int N,
    int K, int act, int gated, float limit) {
  __shared__ mg_f32x4 lds[8 * 3 * 64];  // [4 waves][2 tiles][RT][64 lanes]
  const int e = blockIdx.y;
  const int first = offs[e], n = offs[e + 1] - first;
  const int n0 = blockIdx.x * (PAIR ? 32 : 64);
  const unsigned short* we = w + (size_t)e * (PAIR ? 2 * N : N) * K;
  // the branches depend on the workgroup alone
  for (int m0 = 0; m0 < n;) {
    const int left = n - m0;
    if (left <= 16) {
      mg_rows<1, PAIR>(out, x, we, rows, row_scale, first, m0, n, n0, N, K,
                       act, gated != 0, limit, lds);
      m0 += 16;
    } else if (left <= 32) {
      mg_rows<2, PAIR>(out, x, we, rows, row_scale, first, m0, n, n0, N, K,
                       act, gated != 0, limit, lds);
      m0 += 32;
    } else {
      mg_rows<3, PAIR>(out, x, we, rows, row_scale, first, m0, n, n0, N, K,
                       act, gated != 0, limit, lds);
      m0 += 48;
    }
  }
}

// ---------------------------------------------------------------------------
// weighted sum
// ---------------------------------------------------------------------------
// Grid (column chunks, tokens); a thread takes V consecutive columns.
template <typename T, int V>
__global__ __launch_bounds__(256) void experts_sum_kernel(
    float* __restrict__ out, const T* __restrict__ y,
    const int* __restrict__ pos, int top, const float* __restrict__ wts,
    float weight, const int64_t* __restrict__ sel, int E,
    const T* __restrict__ x, int ldx, const T* __restrict__ ys, int ldys,
    const T* __restrict__ sgate, int ldsg, int W) {
  const int t = blockIdx.y;
  const int c = (blockIdx.x * blockDim.x + threadIdx.x) * V;
  if (c >= W) return;
  struct __align__(sizeof(T) * V) Vec {
    T e[V];
  };
  float acc[V];
#pragma unroll
  for (int i = 0; i < V; ++i) acc[i] = 0.f;
  for (int k = 0; k < top; ++k) {
    const int j = t * top + k;
    const float w = wts != nullptr ? wts[j] : weight;
    const bool ident = sel != nullptr && sel[j] >= E;
    const T* src = ident ? x + (size_t)t * ldx : y + (size_t)pos[j] * W;
    const Vec v = *(const Vec*)(src + c);
#pragma unroll
    for (int i = 0; i < V; ++i) acc[i] += w * MxElem<T>::ld(&v.e[i]);
  }
  if (ys != nullptr) {
    const float g = sgate != nullptr
                        ? mx_sigmoid(MxElem<T>::ld(sgate + (size_t)t * ldsg))
                        : 1.f;
    const Vec v = *(const Vec*)(ys + (size_t)t * ldys + c);
#pragma unroll
    for (int i = 0; i < V; ++i) acc[i] += g * MxElem<T>::ld(&v.e[i]);
  }
#pragma unroll
  for (int i = 0; i < V; ++i) out[(size_t)t * W + c + i] = acc[i];
}

extern "C" {

int mx_expert_plan(void* offs, void* rows, void* pos, const void* sel,
                   const void* tokens, const void* tables, int layers, int T_,
                   int top, int n_out, int V, void* stream) {
  if (layers <= 0 || T_ <= 0) return 0;
  if (n_out < 1 || n_out > MG_MAX_OUT || top < 1) return 1;
  int bits = 1;
  while ((1 << bits) < n_out) ++bits;
  const size_t lds = (size_t)(MG_PLAN_THREADS / 64 + 1) * n_out * sizeof(int);
  hipLaunchKernelGGL(expert_plan_kernel, dim3(layers), dim3(MG_PLAN_THREADS),
                     lds, (hipStream_t)stream, (int*)offs, (int*)rows,
                     (int*)pos, (const int64_t*)sel, (const int64_t*)tokens,
                     (const int*)tables, T_, top, n_out, V, bits);
  return 0;
}

void mx_experts_in(void* mid, const void* x, const void* w, const void* offs,
                   const void* rows, const void* row_scale, int E, int W,
                   int ff, int gated, int act, float limit, void* stream) {
  if (E <= 0 || ff <= 0) return;
  typedef unsigned short U;
  if (gated)
    hipLaunchKernelGGL((experts_product_kernel<true>),
                       dim3((ff + 31) / 32, E), dim3(256), 0,
                       (hipStream_t)stream, (U*)mid, (const U*)x, (const U*)w,
                       (const int*)offs, (const int*)rows,
                       (const float*)row_scale, ff, W, act, 1, limit);
  else
    hipLaunchKernelGGL((experts_product_kernel<false>),
                       dim3((ff + 63) / 64, E), dim3(256), 0,
                       (hipStream_t)stream, (U*)mid, (const U*)x, (const U*)w,
                       (const int*)offs, (const int*)rows,
                       (const float*)row_scale, ff, W, act, 0, limit);
}

void mx_experts_out(void* y, const void* mid, const void* w, const void* offs,
                    int E, int W, int ff, void* stream) {
  if (E <= 0 || W <= 0) return;
  typedef unsigned short U;
  hipLaunchKernelGGL((experts_product_kernel<false>), dim3((W + 63) / 64, E),
                     dim3(256), 0, (hipStream_t)stream, (U*)y, (const U*)mid,
                     (const U*)w, (const int*)offs, (const int*)nullptr,
                     (const float*)nullptr, W, ff, MG_ACT_NONE, 0, 0.f);
}

void mx_experts_sum(void* out, const void* y, const void* pos, int top,
                    const void* wts, float weight, const void* sel, int E,
                    const void* x, int ldx, const void* ys, int ldys,
                    const void* sgate, int ldsg, int T_, int W, int dtype,
                    void* stream) {
  if (T_ <= 0 || W <= 0) return;
  const bool aligned =
      W % 4 == 0 && ldx % 4 == 0 && ldys % 4 == 0 &&
      (((size_t)out | (size_t)y | (size_t)x | (size_t)ys) & 15) == 0;
  MX_DISPATCH_DTYPE(dtype, {
    if (aligned) {
      hipLaunchKernelGGL((experts_sum_kernel<T, 4>),
                         dim3((W / 4 + 255) / 256, T_), dim3(256), 0,
                         (hipStream_t)stream, (float*)out, (const T*)y,
                         (const int*)pos, top, (const float*)wts, weight,
                         (const int64_t*)sel, E, (const T*)x, ldx,
                         (const T*)ys, ldys, (const T*)sgate, ldsg, W);
    } else {
      hipLaunchKernelGGL((experts_sum_kernel<T, 1>),
                         dim3((W + 255) / 256, T_), dim3(256), 0,
                         (hipStream_t)stream, (float*)out, (const T*)y,
                         (const int*)pos, top, (const float*)wts, weight,
                         (const int64_t*)sel, E, (const T*)x, ldx,
                         (const T*)ys, ldys, (const T*)sgate, ldsg, W);
    }
  })
}

}  // extern "C"
