// Residual-stream kernels of the parallel-block models: the 32-bit residual
// with its grouped norm, the norm-and-gate epilogue of a linear-attention
// mixer, the gated feed-forward activation, per-token rotation tables, and the
// fused query/key/value preparation of a rotary attention layer.
//
// All are templated on the activation type (bf16 or float); sums, norms,
// angles and activations are computed in 32-bit either way.  Rows have
// explicit strides, so every kernel reads its columns of one wide projection
// and writes its columns of one wide concatenation in place.
#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

#include "common.h"

// sum over NW waves of a block (NW == 1: no barrier)
template <int NW>
DEVINL float unit_sum(float v, float* scratch) {
  v = wave_sum(v);
  if constexpr (NW > 1) {
    if ((threadIdx.x & 63) == 0) scratch[threadIdx.x >> 6] = v;
    __syncthreads();
    v = 0.f;
#pragma unroll
    for (int w = 0; w < NW; w++) v += scratch[w];
  }
  return v;
}

// ------------------------------------------------- residual + grouped norm
// One unit = one group of one row; its norm depends on nothing else.
//   ids != null:    x = embed[id]                    (first norm of a model)
//   delta != null:  x = x + mult * delta             (pending sublayer output)
//   y = x / sqrt(mean(x^2) + eps) * w
// NW waves work on a unit; NW == 1 packs four units into a block.
template <typename T, int VEC, int NW>
__global__ __launch_bounds__(256) void residual_group_norm_kernel(
    float* __restrict__ x, const T* __restrict__ delta, const T* __restrict__ embed,
    const long* __restrict__ ids, const T* __restrict__ w, T* __restrict__ y,
    long units, int groups, int part, float mult, float eps) {
  constexpr int REG = 4;          // vectors kept in registers between the passes
  constexpr int NT = NW * 64;
  __shared__ float scratch[4];
  const long unit = NW == 1 ? blockIdx.x * 4L + (threadIdx.x >> 6) : (long)blockIdx.x;
  if (unit >= units) return;
  const int tid = NW == 1 ? (threadIdx.x & 63) : threadIdx.x;
  const long row = unit / groups;
  const int g = (int)(unit % groups);
  const long base = row * (long)groups * part + (long)g * part;
  const int nvec = part / VEC;
  float keep[REG][VEC];
  float ss = 0.f;
  auto fetch = [&](int i, float* v) {
    if (ids) {
      ldv<VEC>(embed + ids[row] * (long)groups * part + (long)g * part + (long)i * VEC, v);
      stv<VEC>(x + base + (long)i * VEC, v);
    } else {
      ldv<VEC>(x + base + (long)i * VEC, v);
      if (delta) {
        float d[VEC];
        ldv<VEC>(delta + base + (long)i * VEC, d);
#pragma unroll
        for (int j = 0; j < VEC; j++) v[j] += mult * d[j];
        stv<VEC>(x + base + (long)i * VEC, v);
      }
    }
#pragma unroll
    for (int j = 0; j < VEC; j++) ss += v[j] * v[j];
  };
#pragma unroll
  for (int r = 0; r < REG; r++) {
    const int i = tid + r * NT;
    if (i < nvec) fetch(i, keep[r]);
  }
  for (int i = tid + REG * NT; i < nvec; i += NT) {
    float v[VEC];
    fetch(i, v);
  }
  ss = unit_sum<NW>(ss, scratch);
  const float inv = 1.f / sqrtf(ss / (float)part + eps);
  auto emit = [&](int i, const float* v) {
    float wv[VEC], o[VEC];
    ldv<VEC>(w + (long)g * part + (long)i * VEC, wv);
#pragma unroll
    for (int j = 0; j < VEC; j++) o[j] = v[j] * inv * wv[j];
    stv<VEC>(y + base + (long)i * VEC, o);
  };
#pragma unroll
  for (int r = 0; r < REG; r++) {
    const int i = tid + r * NT;
    if (i < nvec) emit(i, keep[r]);
  }
  for (int i = tid + REG * NT; i < nvec; i += NT) {
    float v[VEC];
    ldv<VEC>(x + base + (long)i * VEC, v);   // this thread's own store above
    emit(i, v);
  }
}

// ------------------------------------------------------ norm, then a gate
// One unit = one group of one row of `in` [rows, groups * part]:
//   out = in / sqrt(mean(in^2) + eps) * w * act(gate)
// `w` covers the whole row and may be null; gate and out have row strides.
template <typename T, int VEC, int NW, int ACT>
__global__ __launch_bounds__(256) void gated_norm_kernel(
    const T* __restrict__ in, const T* __restrict__ w, const T* __restrict__ gate,
    T* __restrict__ out, long units, int groups, int part, long ldg, long ldo, float eps) {
  constexpr int NT = NW * 64;
  __shared__ float scratch[4];
  const long unit = NW == 1 ? blockIdx.x * 4L + (threadIdx.x >> 6) : (long)blockIdx.x;
  if (unit >= units) return;
  const int tid = NW == 1 ? (threadIdx.x & 63) : threadIdx.x;
  const long row = unit / groups;
  const long col = (unit % groups) * part;
  const T* src = in + row * (long)groups * part + col;
  const int nvec = part / VEC;
  float ss = 0.f;
  for (int i = tid; i < nvec; i += NT) {
    float v[VEC];
    ldv<VEC>(src + (long)i * VEC, v);
#pragma unroll
    for (int j = 0; j < VEC; j++) ss += v[j] * v[j];
  }
  ss = unit_sum<NW>(ss, scratch);
  const float inv = 1.f / sqrtf(ss / (float)part + eps);
  for (int i = tid; i < nvec; i += NT) {
    float v[VEC], gv[VEC], wv[VEC];
    ldv<VEC>(src + (long)i * VEC, v);
    ldv<VEC>(gate + row * ldg + col + (long)i * VEC, gv);
    if (w) ldv<VEC>(w + col + (long)i * VEC, wv);
#pragma unroll
    for (int j = 0; j < VEC; j++) {
      const float a = ACT == 0 ? act_silu(gv[j]) : act_sigmoid(gv[j]);
      v[j] = v[j] * inv * (w ? wv[j] : 1.f) * a;
    }
    stv<VEC>(out + row * ldo + col + (long)i * VEC, v);
  }
}

// ---------------------------------------------------- gated feed-forward
// out[:, 0:pad) = 0 (unused columns ahead of the segment), then
// out[:, pad + i] = gelu_tanh(gate[:, i]) * up[:, i]
template <typename T, int VEC>
__global__ __launch_bounds__(256) void gelu_glu_kernel(
    const T* __restrict__ gate, const T* __restrict__ up, T* __restrict__ out,
    long rows, int ff, int pad, int tail, long ldp, long ldo) {
  const int nvec = (pad + ff + tail) / VEC;
  const long idx = (long)blockIdx.x * 256 + threadIdx.x;
  if (idx >= rows * nvec) return;
  const long row = idx / nvec;
  const int c = (int)(idx % nvec) * VEC - pad;   // column within the segment
  float o[VEC];
  if (c >= 0 && c + VEC <= ff) {
    float g[VEC], u[VEC];
    ldv<VEC>(gate + row * ldp + c, g);
    ldv<VEC>(up + row * ldp + c, u);
#pragma unroll
    for (int j = 0; j < VEC; j++) o[j] = act_gelu_tanh(g[j]) * u[j];
  } else {
#pragma unroll
    for (int j = 0; j < VEC; j++) {
      const int e = c + j;
      o[j] = (e >= 0 && e < ff)
                 ? act_gelu_tanh(ldf(gate + row * ldp + e)) * ldf(up + row * ldp + e)
                 : 0.f;
    }
  }
  stv<VEC>(out + row * ldo + pad + c, o);
}

// ------------------------------------------------------- rotation angles
// cs[t] = cos | sin of positions[t] * freq[i]; the product and its reduction
// to [-pi, pi] are 64-bit, so the result is exact to 32-bit at any position.
__global__ __launch_bounds__(256) void rope_angles_kernel(
    const long* __restrict__ pos, const double* __restrict__ freq,
    float* __restrict__ cs, long T, int n) {
  const long idx = (long)blockIdx.x * 256 + threadIdx.x;
  if (idx >= T * n) return;
  const long t = idx / n;
  const int i = (int)(idx % n);
  const double a = (double)pos[t] * freq[i];
  const double r = a - rint(a * 0.15915494309189535) * 6.283185307179586;
  cs[t * 2 * n + i] = cosf((float)r);
  cs[t * 2 * n + n + i] = sinf((float)r);
}

// ------------------------------------- rotary attention: q, k, v in one go
// One wave per (token, head) of q, k and v, read from columns of the layer's
// projection row:
//   q, k: RMS norm over the head with weight qw/kw (null: no norm), then
//         rotation of the first rdims dimensions by csk;
//   v:    rotation over all its dimensions by csv (null: none).
// q goes to qo [T, H, DKP] (pad columns zeroed); k and v go straight into
// their pages, K [P, ps, G, DKP], V [P, G, DVP, ps].  Pad columns of the pages
// stay zero from the pool's creation.
template <typename T>
__global__ __launch_bounds__(256) void rotary_qkv_kernel(
    const T* __restrict__ proj, long ld, int qoff, int koff, int voff,
    const T* __restrict__ qw, const T* __restrict__ kw,
    const float* __restrict__ csk, const float* __restrict__ csv,
    const long* __restrict__ slots, T* __restrict__ qo, T* __restrict__ kc,
    T* __restrict__ vc, long tokens, int H, int G, int D, int V, int DKP, int DVP,
    int rdims, int interleaved, int ps, float eps) {
  __shared__ float buf[4][256];
  const int lane = threadIdx.x & 63;
  float* wb = buf[threadIdx.x >> 6];
  const int heads = H + 2 * G;
  const long unit = blockIdx.x * 4L + (threadIdx.x >> 6);
  if (unit >= tokens * heads) return;
  const long t = unit / heads;
  const int h = (int)(unit % heads);
  const bool is_q = h < H, is_v = h >= H + G;
  const int n = is_v ? V : D;
  const int rot = is_v ? (csv ? V : 0) : rdims;
  const float* cs = is_v ? csv + t * V : csk + t * (long)rdims;
  const T* src = proj + t * ld +
                 (is_q ? qoff + h * D : is_v ? voff + (h - H - G) * V : koff + (h - H) * D);
  float x[4];
  float ss = 0.f;
#pragma unroll
  for (int r = 0; r < 2; r++) {
    const int e = 2 * lane + 128 * r;
    x[2 * r] = e < n ? ldf(src + e) : 0.f;
    x[2 * r + 1] = e + 1 < n ? ldf(src + e + 1) : 0.f;
    ss += x[2 * r] * x[2 * r] + x[2 * r + 1] * x[2 * r + 1];
  }
  const T* w = is_v ? nullptr : is_q ? qw : kw;
  if (w) {
    ss = wave_sum(ss);
    const float inv = 1.f / sqrtf(ss / (float)n + eps);
#pragma unroll
    for (int r = 0; r < 4; r++) {
      const int e = 2 * lane + 128 * (r >> 1) + (r & 1);
      if (e < n) x[r] = x[r] * inv * ldf(w + e);
    }
  }
  const int half = rot >> 1;
  if (interleaved) {
#pragma unroll
    for (int r = 0; r < 2; r++) {
      const int p = lane + 64 * r;
      if (p < half) {
        const float c = cs[p], s = cs[half + p];
        const float u = x[2 * r], v = x[2 * r + 1];
        x[2 * r] = u * c - v * s;
        x[2 * r + 1] = v * c + u * s;
      }
    }
  } else if (rot) {
#pragma unroll
    for (int r = 0; r < 4; r++) {
      const int e = 2 * lane + 128 * (r >> 1) + (r & 1);
      if (e < n) wb[e] = x[r];
    }
    lds_fence_wave_kv();
#pragma unroll
    for (int r = 0; r < 4; r++) {
      const int e = 2 * lane + 128 * (r >> 1) + (r & 1);
      if (e < half) x[r] = x[r] * cs[e] - wb[e + half] * cs[half + e];
      else if (e < rot) x[r] = x[r] * cs[e - half] + wb[e - half] * cs[e];
    }
  }
  if (is_q) {
    T* dst = qo + (t * H + h) * (long)DKP;
#pragma unroll
    for (int r = 0; r < 4; r++) {
      const int e = 2 * lane + 128 * (r >> 1) + (r & 1);
      if (e < DKP) stf(dst + e, e < n ? x[r] : 0.f);
    }
    return;
  }
  const long slot = slots[t];
  const long page = slot / ps;
  const int off = (int)(slot % ps);
#pragma unroll
  for (int r = 0; r < 4; r++) {
    const int e = 2 * lane + 128 * (r >> 1) + (r & 1);
    if (e >= n) continue;
    if (is_v)
      stf(vc + ((page * G + (h - H - G)) * (long)DVP + e) * ps + off, x[r]);
    else
      stf(kc + (slot * G + (h - H)) * (long)DKP + e, x[r]);
  }
}

// ======================================================== host wrappers ==
template <typename F>
static inline void by_type(const torch::Tensor& t, F f) {
  if (t.scalar_type() == torch::kBFloat16) {
    f(short{});
  } else {
    TORCH_CHECK(t.scalar_type() == torch::kFloat32, "bf16 or float32 expected");
    f(float{});
  }
}

template <typename T>
static inline T* ptr(const torch::Tensor& t) { return (T*)t.data_ptr(); }
template <typename T>
static inline T* optr(const c10::optional<torch::Tensor>& t) {
  return t.has_value() ? (T*)t->data_ptr() : nullptr;
}
static inline bool aligned(const void* p, size_t n) { return ((uintptr_t)p % n) == 0; }

torch::Tensor residual_group_norm(torch::Tensor x, c10::optional<torch::Tensor> delta,
                                  c10::optional<torch::Tensor> embed,
                                  c10::optional<torch::Tensor> ids, torch::Tensor w,
                                  long groups, double mult, double eps) {
  TORCH_CHECK(x.is_cuda() && x.scalar_type() == torch::kFloat32 && x.is_contiguous() && x.dim() == 2,
              "the residual stream is a contiguous float32 matrix");
  const long rows = x.size(0), W = x.size(1);
  TORCH_CHECK(w.is_contiguous() && w.numel() == W && groups > 0 && W % groups == 0);
  TORCH_CHECK(!(delta.has_value() && ids.has_value()));
  if (delta.has_value())
    TORCH_CHECK(delta->is_contiguous() && delta->sizes() == x.sizes() &&
                delta->scalar_type() == w.scalar_type());
  if (ids.has_value())
    TORCH_CHECK(embed.has_value() && embed->is_contiguous() && embed->size(1) == W &&
                embed->scalar_type() == w.scalar_type() && ids->numel() == rows &&
                ids->scalar_type() == torch::kLong && ids->is_contiguous());
  auto y = torch::empty({rows, W}, w.options());
  if (rows == 0) return y;
  const int part = W / groups;
  const long units = rows * groups;
  auto stream = at::hip::getCurrentHIPStream();
  by_type(w, [&](auto tag) {
    using T = decltype(tag);
    const bool vec = part % 4 == 0 && aligned(x.data_ptr(), 16) && aligned(w.data_ptr(), 16) &&
                     aligned(optr<T>(delta), 16) && aligned(optr<T>(embed), 16);
#define RGN(VEC, NW)                                                                      \
  hipLaunchKernelGGL((residual_group_norm_kernel<T, VEC, NW>),                            \
                     dim3(NW == 1 ? (units + 3) / 4 : units), dim3(256), 0, stream,       \
                     x.data_ptr<float>(), optr<T>(delta), optr<T>(embed), optr<long>(ids), \
                     ptr<T>(w), ptr<T>(y), units, (int)groups, part, (float)mult, (float)eps)
    if (!vec) RGN(1, 1);
    else if (part > 1024) RGN(4, 4);
    else RGN(4, 1);
#undef RGN
  });
  HIP_CHECK_LAST();
  return y;
}

void gated_norm(torch::Tensor in, c10::optional<torch::Tensor> w, torch::Tensor gate,
                torch::Tensor out, long groups, long act, double eps) {
  const long rows = in.size(0), W = in.size(1);
  TORCH_CHECK(in.is_cuda() && in.is_contiguous() && in.dim() == 2 && groups > 0 && W % groups == 0);
  TORCH_CHECK(gate.size(0) == rows && gate.size(1) == W && gate.stride(1) == 1);
  TORCH_CHECK(out.size(0) == rows && out.size(1) == W && out.stride(1) == 1);
  TORCH_CHECK(gate.scalar_type() == in.scalar_type() && out.scalar_type() == in.scalar_type());
  if (w.has_value())
    TORCH_CHECK(w->numel() == W && w->is_contiguous() && w->scalar_type() == in.scalar_type());
  TORCH_CHECK(act == 0 || act == 1);
  if (rows == 0) return;
  const int part = W / groups;
  const long units = rows * groups, ldg = gate.stride(0), ldo = out.stride(0);
  auto stream = at::hip::getCurrentHIPStream();
  by_type(in, [&](auto tag) {
    using T = decltype(tag);
    const bool vec = part % 4 == 0 && ldg % 4 == 0 && ldo % 4 == 0 &&
                     aligned(in.data_ptr(), 16) && aligned(gate.data_ptr(), 4 * sizeof(T)) &&
                     aligned(out.data_ptr(), 4 * sizeof(T)) && aligned(optr<T>(w), 16);
#define GN(VEC, NW, ACT)                                                               \
  hipLaunchKernelGGL((gated_norm_kernel<T, VEC, NW, ACT>),                             \
                     dim3(NW == 1 ? (units + 3) / 4 : units), dim3(256), 0, stream,    \
                     ptr<T>(in), optr<T>(w), ptr<T>(gate), ptr<T>(out), units,         \
                     (int)groups, part, ldg, ldo, (float)eps)
#define GNA(VEC, NW) do { if (act == 0) GN(VEC, NW, 0); else GN(VEC, NW, 1); } while (0)
    if (!vec) GNA(1, 1);
    else if (part > 512) GNA(4, 4);
    else GNA(4, 1);
#undef GNA
#undef GN
  });
  HIP_CHECK_LAST();
}

void gelu_glu(torch::Tensor gate, torch::Tensor up, torch::Tensor out, long pad, long tail) {
  // `out` covers [pad | ff | tail] columns
  const long rows = gate.size(0), ff = gate.size(1);
  TORCH_CHECK(gate.is_cuda() && gate.stride(1) == 1 && up.stride(1) == 1 && out.stride(1) == 1);
  TORCH_CHECK(up.size(0) == rows && up.size(1) == ff && gate.stride(0) == up.stride(0));
  TORCH_CHECK(pad >= 0 && tail >= 0 && out.size(0) == rows && out.size(1) == pad + ff + tail);
  TORCH_CHECK(gate.scalar_type() == up.scalar_type() && gate.scalar_type() == out.scalar_type());
  if (rows == 0) return;
  const long ldp = gate.stride(0), ldo = out.stride(0);
  auto stream = at::hip::getCurrentHIPStream();
  by_type(gate, [&](auto tag) {
    using T = decltype(tag);
    constexpr int V = 16 / sizeof(T);
    const bool vec = pad % V == 0 && (pad + ff + tail) % V == 0 && ldp % V == 0 && ldo % V == 0 &&
                     aligned(gate.data_ptr(), 16) && aligned(up.data_ptr(), 16) &&
                     aligned(out.data_ptr(), 16);
    const long n = rows * ((pad + ff + tail) / (vec ? V : 1));
    if (vec)
      hipLaunchKernelGGL((gelu_glu_kernel<T, V>), dim3((n + 255) / 256), dim3(256), 0, stream,
                         ptr<T>(gate), ptr<T>(up), ptr<T>(out), rows, (int)ff, (int)pad,
                         (int)tail, ldp, ldo);
    else
      hipLaunchKernelGGL((gelu_glu_kernel<T, 1>), dim3((n + 255) / 256), dim3(256), 0, stream,
                         ptr<T>(gate), ptr<T>(up), ptr<T>(out), rows, (int)ff, (int)pad,
                         (int)tail, ldp, ldo);
  });
  HIP_CHECK_LAST();
}

torch::Tensor rope_angles(torch::Tensor positions, torch::Tensor freqs) {
  TORCH_CHECK(positions.is_cuda() && positions.scalar_type() == torch::kLong && positions.is_contiguous());
  TORCH_CHECK(freqs.is_cuda() && freqs.scalar_type() == torch::kFloat64 && freqs.is_contiguous());
  const long T = positions.numel(), n = freqs.numel();
  auto cs = torch::empty({T, 2 * n}, freqs.options().dtype(torch::kFloat32));
  if (T * n == 0) return cs;
  hipLaunchKernelGGL(rope_angles_kernel, dim3((T * n + 255) / 256), dim3(256), 0,
                     at::hip::getCurrentHIPStream(), positions.data_ptr<long>(),
                     freqs.data_ptr<double>(), cs.data_ptr<float>(), T, (int)n);
  HIP_CHECK_LAST();
  return cs;
}

torch::Tensor rotary_qkv(torch::Tensor proj, long qoff, long koff, long voff,
                         c10::optional<torch::Tensor> qw, c10::optional<torch::Tensor> kw,
                         c10::optional<torch::Tensor> csk, c10::optional<torch::Tensor> csv,
                         torch::Tensor slots, torch::Tensor kc, torch::Tensor vc,
                         long H, long G, long D, long V, bool interleaved, double eps) {
  TORCH_CHECK(proj.is_cuda() && proj.dim() == 2 && proj.stride(1) == 1);
  TORCH_CHECK(kc.scalar_type() == proj.scalar_type() && vc.scalar_type() == proj.scalar_type(),
              "the cache holds the activation type");
  TORCH_CHECK(kc.dim() == 4 && vc.dim() == 4 && kc.is_contiguous() && vc.is_contiguous());
  const long T = proj.size(0);
  const int ps = kc.size(1), DKP = kc.size(3), DVP = vc.size(2);
  TORCH_CHECK(kc.size(2) == G && vc.size(1) == G && vc.size(3) == ps && kc.size(0) == vc.size(0));
  TORCH_CHECK(D % 2 == 0 && V % 2 == 0 && D <= DKP && V <= DVP && DKP <= 256 && DVP <= 256);
  TORCH_CHECK(qoff >= 0 && koff >= 0 && voff >= 0 && qoff + H * D <= proj.size(1) &&
              koff + G * D <= proj.size(1) && voff + G * V <= proj.size(1));
  TORCH_CHECK(slots.scalar_type() == torch::kLong && slots.is_contiguous() && slots.numel() == T);
  const long rdims = csk.has_value() ? csk->size(1) : 0;
  if (csk.has_value())
    TORCH_CHECK(csk->is_contiguous() && csk->size(0) == T && rdims <= D && rdims % 2 == 0 &&
                csk->scalar_type() == torch::kFloat32);
  if (csv.has_value())
    TORCH_CHECK(csv->is_contiguous() && csv->size(0) == T && csv->size(1) == V &&
                csv->scalar_type() == torch::kFloat32);
  for (auto& w : {qw, kw})
    if (w.has_value())
      TORCH_CHECK(w->is_contiguous() && w->numel() == D && w->scalar_type() == proj.scalar_type());
  auto qo = torch::empty({T, H, (long)DKP}, proj.options());
  if (T == 0) return qo;
  const long units = T * (H + 2 * G);
  by_type(proj, [&](auto tag) {
    using T = decltype(tag);
    hipLaunchKernelGGL((rotary_qkv_kernel<T>), dim3((units + 3) / 4), dim3(256), 0,
                       at::hip::getCurrentHIPStream(), ptr<T>(proj), proj.stride(0), (int)qoff,
                       (int)koff, (int)voff, optr<T>(qw), optr<T>(kw), optr<float>(csk),
                       optr<float>(csv), slots.data_ptr<long>(), ptr<T>(qo), ptr<T>(kc),
                       ptr<T>(vc), (long)proj.size(0), (int)H, (int)G, (int)D, (int)V, DKP, DVP,
                       (int)rdims, (int)interleaved, ps, (float)eps);
  });
  HIP_CHECK_LAST();
  return qo;
}
