// Linear attention with one fixed decay per head and no denominator:
//   S_t = decay S_(t-1) + k_t v_t^T,   o_t = S_t^T q_t,   S [D, V] in 32-bit.
// q, k, v are read from columns of a projection row; on the way in they pass
// an optional SiLU, an optional rotation of the first dims (k also a factor).
//
// Portions of prompts run in chunks of 64 tokens (never across sequences):
//   1. chunk_state: what each chunk adds to the state, in parallel;
//   2. chunk_scan:  a running state over each sequence's chunks, from the
//                   sequence's slot (or zero) and back into it;
//   3. chunk_out:   decayed (q k^T) v inside a chunk plus q times the state
//                   ahead of it, in parallel.
// Products run on the matrix cores: float32 MFMA here, exact to 32-bit.
//
// Single tokens (decode) update the state in place: one workgroup per
// (sequence, head) streams S once through registers.
#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

#include "common.h"

constexpr int CHUNK = 64;
constexpr int VBLK = 64;

DEVINL f32x4 mfma4f(float a, float b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0);
}

// where q/k/v come from and what happens to them on the way in
struct Source {
  long ld;                 // projection row stride
  int H, D, V;
  const float* cs;         // [T, rdims] cos | sin, or null
  int rdims, interleaved, silu;
  float kscale;
};

struct Chunks {
  const int* seq;          // [n] sequence of a chunk
  const int* row;          // [n] its first token row
  const int* len;          // [n] its tokens, 1..CHUNK
  const int* first;        // [B + 1] first chunk of a sequence
};

template <typename T>
DEVINL float load_qk(const T* base, int e, const Source& s, const float* cs) {
  float x = ldf(base + e);
  if (s.silu) x = act_silu(x);
  if (e < s.rdims) {
    const int half = s.rdims >> 1;
    const int p = s.interleaved ? e >> 1 : (e < half ? e : e - half);
    const bool lead = s.interleaved ? !(e & 1) : e < half;
    const int other = s.interleaved ? e ^ 1 : (lead ? e + half : e - half);
    float y = ldf(base + other);
    if (s.silu) y = act_silu(y);
    x = x * cs[p] + (lead ? -y : y) * cs[half + p];
  }
  return x;
}

template <typename T>
DEVINL float load_v(const T* base, int e, const Source& s) {
  const float x = ldf(base + e);
  return s.silu ? act_silu(x) : x;
}

// ------------------------------------------------ 1. what a chunk adds
// U[d][v] = sum_j decay^(n-1-j) k_j[d] v_j[v]; ws [chunks, H, D, V]
template <typename T, int DP>
__global__ __launch_bounds__(256) void chunk_state_kernel(
    const T* __restrict__ k, const T* __restrict__ v, Source s, Chunks ch,
    const float* __restrict__ pw, float* __restrict__ ws) {
  constexpr int KS = DP + 16, VS = VBLK + 16;
  __shared__ float kt[CHUNK * KS], vt[CHUNK * VS];
  const int c = blockIdx.x, h = blockIdx.y, v0 = blockIdx.z * VBLK;
  const int n = ch.len[c];
  const long t0 = ch.row[c];
  const float* pwh = pw + h * (CHUNK + 1);
  for (int i = threadIdx.x; i < CHUNK * DP; i += 256) {
    const int j = i / DP, d = i % DP;
    float x = 0.f;
    if (j < n && d < s.D)
      x = load_qk(k + (t0 + j) * s.ld + h * s.D, d, s, s.cs + (t0 + j) * s.rdims) * s.kscale *
          pwh[n - 1 - j];
    kt[j * KS + d] = x;
  }
  for (int i = threadIdx.x; i < CHUNK * VBLK; i += 256) {
    const int j = i / VBLK, e = i % VBLK;
    vt[j * VS + e] =
        (j < n && v0 + e < s.V) ? load_v(v + (t0 + j) * s.ld + h * s.V, v0 + e, s) : 0.f;
  }
  __syncthreads();
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6;
  const int lo = lane & 15, hi = lane >> 4;
  constexpr int RT = DP / 16;                 // row tiles of U
  constexpr int RW = RT >= 4 ? RT / 4 : RT;   // per wave
  constexpr int CW = RT >= 4 ? 4 : 1;         // column tiles per wave
  const int r0 = RT >= 4 ? w * RW : 0, c0 = RT >= 4 ? 0 : w;
  f32x4 acc[RW][CW];
#pragma unroll
  for (int r = 0; r < RW; r++)
#pragma unroll
    for (int q = 0; q < CW; q++) acc[r][q] = f32x4{0.f, 0.f, 0.f, 0.f};
  for (int st = 0; st < CHUNK / 4; st++) {
    const int j = 4 * st + hi;
    float a[RW], b[CW];
#pragma unroll
    for (int r = 0; r < RW; r++) a[r] = kt[j * KS + (r0 + r) * 16 + lo];
#pragma unroll
    for (int q = 0; q < CW; q++) b[q] = vt[j * VS + (c0 + q) * 16 + lo];
#pragma unroll
    for (int r = 0; r < RW; r++)
#pragma unroll
      for (int q = 0; q < CW; q++) acc[r][q] = mfma4f(a[r], b[q], acc[r][q]);
  }
  float* u = ws + ((long)c * s.H + h) * s.D * s.V;
#pragma unroll
  for (int r = 0; r < RW; r++)
#pragma unroll
    for (int q = 0; q < CW; q++)
#pragma unroll
      for (int i = 0; i < 4; i++) {
        const int d = (r0 + r) * 16 + 4 * hi + i, e = v0 + (c0 + q) * 16 + lo;
        if (d < s.D && e < s.V) u[(long)d * s.V + e] = acc[r][q][i];
      }
}

// ------------------------------------------------------ 2. running state
// ws: in, what a chunk adds; out, the state ahead of the chunk
__global__ __launch_bounds__(256) void chunk_scan_kernel(
    float* __restrict__ ws, float* __restrict__ state, Chunks ch,
    const int* __restrict__ slots, const int* __restrict__ fresh,
    const float* __restrict__ pw, int H, int DV) {
  const int b = blockIdx.x, h = blockIdx.y;
  const int e = blockIdx.z * 256 + threadIdx.x;
  if (e >= DV) return;
  float* st = state + ((long)slots[b] * H + h) * DV + e;
  const float* pwh = pw + h * (CHUNK + 1);
  float s = fresh[b] ? 0.f : *st;
  const int c1 = ch.first[b + 1];
  float* p = ws + ((long)ch.first[b] * H + h) * DV + e;
#pragma unroll 4
  for (int c = ch.first[b]; c < c1; c++, p += (long)H * DV) {
    const float u = *p;
    *p = s;
    s = pwh[ch.len[c]] * s + u;
  }
  *st = s;
}

// ---------------------------------------------------------- 3. the output
template <typename T, int DP>
__global__ __launch_bounds__(256) void chunk_out_kernel(
    const T* __restrict__ q, const T* __restrict__ k, const T* __restrict__ v, Source s,
    Chunks ch, const float* __restrict__ pw, const float* __restrict__ ws, T* __restrict__ o) {
  constexpr int KS = DP + 4, VS = VBLK + 16, PS = CHUNK + 4;
  __shared__ float kt[CHUNK * KS], vt[CHUNK * VS], pt[4][16 * PS], pws[CHUNK + 1];
  const int c = blockIdx.x, h = blockIdx.y, v0 = blockIdx.z * VBLK;
  const int n = ch.len[c];
  const long t0 = ch.row[c];
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6;
  const int lo = lane & 15, hi = lane >> 4;
  if (threadIdx.x <= CHUNK) pws[threadIdx.x] = pw[h * (CHUNK + 1) + threadIdx.x];
  auto stage = [&](const T* x, float mul) {
    for (int i = threadIdx.x; i < CHUNK * DP; i += 256) {
      const int j = i / DP, d = i % DP;
      kt[j * KS + d] = (j < n && d < s.D) ? load_qk(x + (t0 + j) * s.ld + h * s.D, d, s,
                                                    s.cs + (t0 + j) * s.rdims) * mul
                                          : 0.f;
    }
  };
  stage(q, 1.f);
  __syncthreads();
  float qf[DP / 4];
#pragma unroll
  for (int st = 0; st < DP / 4; st++) qf[st] = kt[(16 * w + lo) * KS + 4 * st + hi];
  __syncthreads();
  stage(k, s.kscale);
  for (int i = threadIdx.x; i < CHUNK * VBLK; i += 256) {
    const int j = i / VBLK, e = i % VBLK;
    vt[j * VS + e] =
        (j < n && v0 + e < s.V) ? load_v(v + (t0 + j) * s.ld + h * s.V, v0 + e, s) : 0.f;
  }
  __syncthreads();
  if (16 * w >= n) return;
  f32x4 acc[4];
#pragma unroll
  for (int t = 0; t < 4; t++) acc[t] = f32x4{0.f, 0.f, 0.f, 0.f};
  // q decayed to the chunk's start, times the state ahead of the chunk
  const float* sp = ws + ((long)c * s.H + h) * s.D * s.V;
  const float pq = pws[16 * w + lo + 1];
#pragma unroll 4
  for (int st = 0; st < DP / 4; st++) {
    const int d = 4 * st + hi;
    const float a = qf[st] * pq;
#pragma unroll
    for (int t = 0; t < 4; t++) {
      const int e = v0 + 16 * t + lo;
      const float b = (d < s.D && e < s.V) ? sp[(long)d * s.V + e] : 0.f;
      acc[t] = mfma4f(a, b, acc[t]);
    }
  }
  // inside the chunk
  float* pr = pt[w];
  for (int jt = 0; jt <= w; jt++) {
    f32x4 sc{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int st = 0; st < DP / 4; st++)
      sc = mfma4f(qf[st], kt[(16 * jt + lo) * KS + 4 * st + hi], sc);
#pragma unroll
    for (int r = 0; r < 4; r++) {
      const int i = 16 * w + 4 * hi + r, j = 16 * jt + lo;
      pr[(4 * hi + r) * PS + j] = i >= j ? sc[r] * pws[i - j] : 0.f;
    }
  }
  lds_fence_wave_kv();
  for (int st = 0; st < 4 * (w + 1); st++) {
    const float a = pr[lo * PS + 4 * st + hi];
#pragma unroll
    for (int t = 0; t < 4; t++)
      acc[t] = mfma4f(a, vt[(4 * st + hi) * VS + 16 * t + lo], acc[t]);
  }
#pragma unroll
  for (int t = 0; t < 4; t++)
#pragma unroll
    for (int r = 0; r < 4; r++) {
      const int i = 16 * w + 4 * hi + r, e = v0 + 16 * t + lo;
      if (i < n && e < s.V) stf(o + (t0 + i) * (long)s.H * s.V + h * s.V + e, acc[t][r]);
    }
}

// ------------------------------------------------------------- one token
// One workgroup per (sequence, head).  With a gate, the head's output is
// divided by its root mean square and multiplied by silu(gate) on the way out.
template <typename T, int VEC>
__global__ __launch_bounds__(256) void linear_decode_kernel(
    const T* __restrict__ q, const T* __restrict__ k, const T* __restrict__ v, Source s,
    const float* __restrict__ pw, float* __restrict__ state, const int* __restrict__ slots,
    const int* __restrict__ seq_lens, const T* __restrict__ gate, long ldg, float eps,
    T* __restrict__ o, long ldo) {
  extern __shared__ __attribute__((aligned(16))) float sh[];
  float* qs = sh;                 // [D]
  float* ks = qs + s.D;           // [D]
  float* red = qs + ((2 * s.D + 3) & ~3);   // [rows per pass][V], 16-B aligned
  __shared__ float scratch[4];
  const int b = blockIdx.x, h = blockIdx.y;
  const float* cs = s.cs + (long)b * s.rdims;
  for (int d = threadIdx.x; d < s.D; d += 256) {
    qs[d] = load_qk(q + b * s.ld + h * s.D, d, s, cs);
    ks[d] = load_qk(k + b * s.ld + h * s.D, d, s, cs) * s.kscale;
  }
  __syncthreads();
  const int nv = s.V / VEC, R = 256 / nv;
  const int r0 = threadIdx.x / nv, e0 = (threadIdx.x % nv) * VEC;
  const bool fresh = seq_lens[b] == 1;
  const float decay = pw[h * (CHUNK + 1) + 1];
  float* st = state + ((long)slots[b] * s.H + h) * s.D * s.V;
  float acc[VEC] = {};
  if (r0 < R) {
    float vv[VEC];
#pragma unroll
    for (int i = 0; i < VEC; i++) vv[i] = load_v(v + b * s.ld + h * s.V, e0 + i, s);
#pragma unroll 8
    for (int d = r0; d < s.D; d += R) {
      float x[VEC];
      float* p = st + (long)d * s.V + e0;
      if (fresh) {
#pragma unroll
        for (int i = 0; i < VEC; i++) x[i] = 0.f;
      } else {
        ldv<VEC>(p, x);
      }
      const float kd = ks[d], qd = qs[d];
#pragma unroll
      for (int i = 0; i < VEC; i++) {
        x[i] = decay * x[i] + kd * vv[i];
        acc[i] += qd * x[i];
      }
      stv<VEC>(p, x);
    }
    stv<VEC>(red + r0 * s.V + e0, acc);
  }
  __syncthreads();
  float ss = 0.f;
  for (int e = threadIdx.x; e < s.V; e += 256) {
    float x = 0.f;
    for (int r = 0; r < R; r++) x += red[r * s.V + e];
    red[e] = x;                    // column e is this thread's alone
    ss += x * x;
  }
  float inv = 1.f;
  if (gate) inv = 1.f / sqrtf(block_sum<256>(ss, scratch) / (float)s.V + eps);
  for (int e = threadIdx.x; e < s.V; e += 256) {
    float x = red[e] * inv;
    if (gate) x *= act_silu(ldf(gate + b * ldg + h * s.V + e));
    stf(o + b * ldo + h * s.V + e, x);
  }
}

// ======================================================== host wrappers ==
static Source make_source(const torch::Tensor& q, const torch::Tensor& k, const torch::Tensor& v,
                          const torch::Tensor& pw, const c10::optional<torch::Tensor>& cs,
                          bool interleaved, bool silu, double kscale) {
  const long H = pw.size(0);
  TORCH_CHECK(q.is_cuda() && q.dim() == 2 && k.sizes() == q.sizes() && v.size(0) == q.size(0));
  TORCH_CHECK(q.stride(1) == 1 && k.stride(1) == 1 && v.stride(1) == 1 &&
              q.stride(0) == k.stride(0) && q.stride(0) == v.stride(0),
              "q, k and v are columns of one row-major projection");
  TORCH_CHECK(q.scalar_type() == k.scalar_type() && q.scalar_type() == v.scalar_type());
  TORCH_CHECK(q.size(1) % H == 0 && v.size(1) % H == 0);
  TORCH_CHECK(pw.dim() == 2 && pw.size(1) == CHUNK + 1 && pw.is_contiguous() &&
              pw.scalar_type() == torch::kFloat32, "decay powers are [heads, ", CHUNK + 1, "]");
  Source s;
  s.ld = q.stride(0);
  s.H = H;
  s.D = q.size(1) / H;
  s.V = v.size(1) / H;
  s.cs = cs.has_value() ? cs->data_ptr<float>() : nullptr;
  s.rdims = cs.has_value() ? cs->size(1) : 0;
  s.interleaved = interleaved;
  s.silu = silu;
  s.kscale = kscale;
  TORCH_CHECK(s.D >= 1 && s.D <= 256 && s.V >= 1 && s.rdims <= s.D && s.rdims % 2 == 0);
  if (cs.has_value())
    TORCH_CHECK(cs->scalar_type() == torch::kFloat32 && cs->is_contiguous() && cs->size(0) == q.size(0));
  return s;
}

static void check_state(const torch::Tensor& state, const Source& s) {
  TORCH_CHECK(state.scalar_type() == torch::kFloat32 && state.is_contiguous() && state.dim() == 4 &&
              state.size(1) == s.H && state.size(2) == s.D && state.size(3) == s.V);
}

static void check_ints(const torch::Tensor& t, long n) {
  TORCH_CHECK(t.is_cuda() && t.scalar_type() == torch::kInt && t.is_contiguous() && t.numel() == n);
}

// o [T, H * V] <- portions described by chunks (int32 [3, n]: sequence, first
// row, length), first (int32 [B + 1]), slots and fresh (int32 [B])
void linear_attn_chunked(torch::Tensor q, torch::Tensor k, torch::Tensor v, torch::Tensor pw,
                         c10::optional<torch::Tensor> cs, bool interleaved, bool silu,
                         double kscale, torch::Tensor chunks, torch::Tensor first,
                         torch::Tensor slots, torch::Tensor fresh, torch::Tensor state,
                         torch::Tensor o) {
  const Source s = make_source(q, k, v, pw, cs, interleaved, silu, kscale);
  check_state(state, s);
  const long n = chunks.size(1), B = slots.numel();
  check_ints(chunks, 3 * n);
  check_ints(first, B + 1);
  check_ints(slots, B);
  check_ints(fresh, B);
  TORCH_CHECK(o.is_contiguous() && o.scalar_type() == q.scalar_type() && o.size(0) == q.size(0) &&
              o.size(1) == (long)s.H * s.V);
  if (n == 0) return;
  auto ws = torch::empty({n, s.H, s.D, s.V}, state.options());
  int* cp = chunks.data_ptr<int>();
  const Chunks ch{cp, cp + n, cp + 2 * n, first.data_ptr<int>()};
  auto stream = at::hip::getCurrentHIPStream();
  const dim3 grid(n, s.H, (s.V + VBLK - 1) / VBLK);
  const int DV = s.D * s.V;
  const float* pwp = pw.data_ptr<float>();
  float* wsp = ws.data_ptr<float>();
#define PHASES(TT, DP)                                                                         \
  do {                                                                                         \
    hipLaunchKernelGGL((chunk_state_kernel<TT, DP>), grid, dim3(256), 0, stream,               \
                       (const TT*)k.data_ptr(), (const TT*)v.data_ptr(), s, ch, pwp, wsp);     \
    hipLaunchKernelGGL(chunk_scan_kernel, dim3(B, s.H, (DV + 255) / 256), dim3(256), 0, stream, \
                       wsp, state.data_ptr<float>(), ch, slots.data_ptr<int>(),                \
                       fresh.data_ptr<int>(), pwp, s.H, DV);                                   \
    hipLaunchKernelGGL((chunk_out_kernel<TT, DP>), grid, dim3(256), 0, stream,                 \
                       (const TT*)q.data_ptr(), (const TT*)k.data_ptr(),                       \
                       (const TT*)v.data_ptr(), s, ch, pwp, wsp, (TT*)o.data_ptr());           \
  } while (0)
#define BY_D(TT)                            \
  do {                                      \
    if (s.D <= 32) PHASES(TT, 32);          \
    else if (s.D <= 64) PHASES(TT, 64);     \
    else if (s.D <= 128) PHASES(TT, 128);   \
    else PHASES(TT, 256);                   \
  } while (0)
  if (q.scalar_type() == torch::kBFloat16) BY_D(short);
  else {
    TORCH_CHECK(q.scalar_type() == torch::kFloat32);
    BY_D(float);
  }
#undef BY_D
#undef PHASES
  HIP_CHECK_LAST();
}

// o [B, H * V] (any row stride) <- one token of each of B sequences
void linear_attn_decode(torch::Tensor q, torch::Tensor k, torch::Tensor v, torch::Tensor pw,
                        c10::optional<torch::Tensor> cs, bool interleaved, bool silu,
                        double kscale, torch::Tensor slots, torch::Tensor seq_lens,
                        torch::Tensor state, c10::optional<torch::Tensor> gate, double eps,
                        torch::Tensor o) {
  const Source s = make_source(q, k, v, pw, cs, interleaved, silu, kscale);
  check_state(state, s);
  const long B = q.size(0);
  check_ints(slots, B);
  check_ints(seq_lens, B);
  TORCH_CHECK(o.scalar_type() == q.scalar_type() && o.size(0) == B && o.stride(1) == 1 &&
              o.size(1) == (long)s.H * s.V);
  if (gate.has_value())
    TORCH_CHECK(gate->scalar_type() == q.scalar_type() && gate->size(0) == B &&
                gate->stride(1) == 1 && gate->size(1) == o.size(1));
  if (B == 0) return;
  const bool vec = s.V % 4 == 0;
  TORCH_CHECK(s.V / (vec ? 4 : 1) <= 256, "value width too large");
  const int R = 256 / (s.V / (vec ? 4 : 1));
  const size_t lds = sizeof(float) * (((2 * s.D + 3) & ~3) + (long)R * s.V);
  auto stream = at::hip::getCurrentHIPStream();
#define LAUNCH(TT, VEC)                                                                         \
  hipLaunchKernelGGL((linear_decode_kernel<TT, VEC>), dim3(B, s.H), dim3(256), lds, stream,     \
                     (const TT*)q.data_ptr(), (const TT*)k.data_ptr(), (const TT*)v.data_ptr(), \
                     s, pw.data_ptr<float>(), state.data_ptr<float>(), slots.data_ptr<int>(),   \
                     seq_lens.data_ptr<int>(),                                                  \
                     gate.has_value() ? (const TT*)gate->data_ptr() : nullptr,                  \
                     gate.has_value() ? (long)gate->stride(0) : 0L, (float)eps,                 \
                     (TT*)o.data_ptr(), (long)o.stride(0))
  if (q.scalar_type() == torch::kBFloat16) {
    if (vec) LAUNCH(short, 4); else LAUNCH(short, 1);
  } else {
    TORCH_CHECK(q.scalar_type() == torch::kFloat32);
    if (vec) LAUNCH(float, 4); else LAUNCH(float, 1);
  }
#undef LAUNCH
  HIP_CHECK_LAST();
}
