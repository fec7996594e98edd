// Heads of an attention whose projections pass a short causal convolution.
//
// conv_qkv takes the fused projection's query, key and value columns through the
// convolution, turns queries and keys in the neighbouring pairs of their first
// dimensions and values, if they turn, in all of theirs, and writes queries to a
// buffer and keys and values to the paged cache, at the cache's head widths.
//
// A thread owns V neighbouring channels of one head (whole pairs, so a rotation never
// leaves the thread) and walks up to CONVQ_ROWS rows of one sequence with the last
// inputs in registers. A sequence's past lies in a ring by position in its state slot;
// the thread that reads a channel's past, in a portion's first block, also stores what
// the portion leaves behind, so a portion never races with itself. Slot -1 marks an
// idle row of a captured batch: it has no past and stores none.
#include "head_turn.h"
#include <torch/extension.h>
#include <c10/hip/HIPStream.h>

#define CUR_STREAM c10::hip::getCurrentHIPStream().stream()
#define CONVQ_ROWS 16      // rows per workgroup
#define CONVQ_MAX_TAPS 16  // a block's past must not reach past the block before it

struct ConvHeadArgs {
  const void* proj;       // [T, stride]
  long stride;
  int q0, k0, v0;         // columns
  const float* w;         // [taps, C], the last row the present
  int taps, C;            // C = Hq d + Hkv (d + dv)
  const float *cs, *vcs;  // [positions, rot], [positions, dv] or null
  int rot;
  void* ring;             // [slots, taps - 1, C]
  const int *kv_slots, *cu, *bseq, *boff, *starts, *slots;
  void *q, *kc, *vc;      // [T, Hq, DK], [pages, Hkv, P, DK | DV]
  int Hq, Hkv, d, dv, DK, DV, P;
};

// VEC: 16-byte accesses of V elements, and d, dv, DK, DV, columns and strides are
// multiples of V (TAPS > 0 only so); else V is 2 and a head's last channel may stand alone. TAPS 0: any
// number, inputs read again for every tap.
template <typename T, int V, int TAPS, bool VEC>
__global__ __launch_bounds__(256) void conv_qkv_kernel(ConvHeadArgs a) {
  const int qu = (a.DK + V - 1) / V, vu = (a.DV + V - 1) / V;  // units per head
  int u = blockIdx.y * 256 + threadIdx.x;
  const int nq = a.Hq * qu, nk = a.Hkv * qu;
  if (u >= nq + nk + a.Hkv * vu) return;
  const bool is_q = u < nq, is_v = u >= nq + nk;
  u -= is_q ? 0 : is_v ? nq + nk : nq;
  const int h = u / (is_v ? vu : qu), c = (u - h * (is_v ? vu : qu)) * V;
  const int width = is_v ? a.DV : a.DK, n = is_v ? a.dv : a.d;  // stored, the model's
  const int col = (is_q ? a.q0 : is_v ? a.v0 : a.k0) + h * n + c;
  const int ch = (is_q ? 0 : is_v ? (a.Hq + a.Hkv) * a.d : a.Hq * a.d) + h * n + c;

  const int seq = a.cu ? a.bseq[blockIdx.x] : blockIdx.x;
  const int off = a.cu ? a.boff[blockIdx.x] : 0;
  const int row0 = a.cu ? a.cu[seq] : seq;
  const int len = a.cu ? a.cu[seq + 1] - row0 : 1;
  const int rows = min(CONVQ_ROWS, len - off);
  const int slot = a.slots[seq], start = a.starts[seq];
  const int taps = TAPS ? TAPS : a.taps, keep = taps - 1, ring_len = max(keep, 1);
  const T* src = (const T*)a.proj + (long)row0 * a.stride + col;
  T* ring = (T*)a.ring + (long)max(slot, 0) * keep * a.C + ch;

  // the unit's channels of local row t (may be negative: the sequence's past)
  auto input = [&](int t, float (&x)[V]) {
    const T* p = nullptr;
    if (t >= 0) p = src + t * a.stride;
    else if (slot >= 0 && start + t >= 0) p = ring + (long)((start + t) % ring_len) * a.C;
    if constexpr (VEC) {
#pragma unroll
      for (int v = 0; v < V; v += 4) {
        floatx4 y = {0.f, 0.f, 0.f, 0.f};
        if (p && c < n) y = ld4(p + v);
#pragma unroll
        for (int i = 0; i < 4; ++i) x[v + i] = y[i];
      }
    } else {
#pragma unroll
      for (int v = 0; v < V; ++v) x[v] = p && c + v < n ? ldf(p + v) : 0.f;
    }
  };
  // rotation and place of local row t
  auto finish = [&](int t, float (&y)[V]) {
    const int turning = is_v ? (a.vcs ? a.dv : 0) : a.rot;
    const float* cs = (is_v ? a.vcs : a.cs) + (long)(start + t) * turning;
    if (VEC && c + V <= turning && (turning & 7) == 0) {
#pragma unroll
      for (int v = 0; v < V; v += 4) {
        const floatx2 cv = *(const floatx2*)(cs + (c + v) / 2);
        const floatx2 sv = *(const floatx2*)(cs + (turning + c + v) / 2);
        turn_pair(y[v], y[v + 1], cv[0], sv[0]);
        turn_pair(y[v + 2], y[v + 3], cv[1], sv[1]);
      }
    } else {
#pragma unroll
      for (int v = 0; v < V; v += 2)
        if (c + v < turning)
          turn_pair(y[v], y[v + 1], cs[(c + v) / 2], cs[(turning + c + v) / 2]);
    }
    T* dst;
    if (is_q) {
      dst = (T*)a.q + ((long)(row0 + t) * a.Hq + h) * a.DK + c;
    } else {
      const int s = a.kv_slots[row0 + t];
      if (s < 0) return;
      dst = (T*)(is_v ? a.vc : a.kc) +
            (((long)(s / a.P) * a.Hkv + h) * a.P + s % a.P) * width + c;
    }
    if constexpr (VEC) {
#pragma unroll
      for (int v = 0; v < V; v += 4) st4(dst + v, floatx4{y[v], y[v + 1], y[v + 2], y[v + 3]});
    } else {
#pragma unroll
      for (int v = 0; v < V; ++v)
        if (c + v < width) stf(dst + v, y[v]);
    }
  };

  if constexpr (TAPS > 0) {
    float win[TAPS][V], wt[TAPS][V];  // win[j]: input TAPS - 1 - j rows back
#pragma unroll
    for (int j = 0; j < TAPS; ++j)
#pragma unroll
      for (int v = 0; v < V; v += 4) {
        floatx4 y = {0.f, 0.f, 0.f, 0.f};
        if (c < n) y = ld4(a.w + (long)j * a.C + ch + v);
#pragma unroll
        for (int i = 0; i < 4; ++i) wt[j][v + i] = y[i];
      }
#pragma unroll
    for (int j = 1; j < TAPS; ++j) input(off - TAPS + j, win[j]);
    for (int t = 0; t < rows; ++t) {
#pragma unroll
      for (int j = 0; j + 1 < TAPS; ++j)
#pragma unroll
        for (int v = 0; v < V; ++v) win[j][v] = win[j + 1][v];
      input(off + t, win[TAPS - 1]);
      float y[V];
#pragma unroll
      for (int v = 0; v < V; ++v) {
        y[v] = 0.f;
#pragma unroll
        for (int j = 0; j < TAPS; ++j) y[v] += wt[j][v] * win[j][v];
      }
      finish(off + t, y);
    }
  } else {
    for (int t = 0; t < rows; ++t) {
      float y[V], x[V];
#pragma unroll
      for (int v = 0; v < V; ++v) y[v] = 0.f;
      for (int j = 0; j < taps; ++j) {
        input(off + t - keep + j, x);
#pragma unroll
        for (int v = 0; v < V; ++v)
          if (c + v < n) y[v] += a.w[(long)j * a.C + ch + v] * x[v];
      }
      finish(off + t, y);
    }
  }
  // only the first block reads the past, and it has
  if (off == 0 && slot >= 0)
    for (int t = max(0, len - keep); t < len; ++t) {
      T* p = ring + (long)((start + t) % ring_len) * a.C;
#pragma unroll
      for (int v = 0; v < V; ++v)
        if (c + v < n) p[v] = src[t * a.stride + v];
    }
}

long conv_qkv_rows() { return CONVQ_ROWS; }

void conv_qkv(torch::Tensor proj, long q0, long k0, long v0, torch::Tensor w,
              torch::Tensor turn, c10::optional<torch::Tensor> value_turn, torch::Tensor ring,
              torch::Tensor kv_slots, c10::optional<torch::Tensor> cu,
              c10::optional<torch::Tensor> bseq, c10::optional<torch::Tensor> boff,
              torch::Tensor starts, torch::Tensor slots, torch::Tensor kc, torch::Tensor vc,
              torch::Tensor q, long d, long dv) {
  const int T_ = proj.size(0), S = slots.numel();
  const long Hq = q.size(1), Hkv = kc.size(1), C = w.size(1), taps = w.size(0);
  TORCH_CHECK(proj.is_cuda() && proj.dim() == 2 && proj.stride(1) == 1);
  TORCH_CHECK(kc.dtype() == proj.dtype() && vc.dtype() == proj.dtype() && kc.is_contiguous() &&
              vc.is_contiguous() && vc.size(1) == Hkv && kc.size(2) == vc.size(2) &&
              kc.size(0) == vc.size(0) && kc.size(3) >= d && vc.size(3) >= dv, "caches");
  TORCH_CHECK(q.is_contiguous() && q.dtype() == proj.dtype() && q.size(0) == T_ &&
              q.size(2) == kc.size(3) && Hkv >= 1 && Hq % Hkv == 0, "queries");
  TORCH_CHECK(q0 + Hq * d <= proj.size(1) && k0 + Hkv * d <= proj.size(1) &&
              v0 + Hkv * dv <= proj.size(1));
  TORCH_CHECK(w.is_contiguous() && w.dtype() == torch::kFloat32 &&
              C == Hq * d + Hkv * (d + dv), "convolution weights");
  TORCH_CHECK(taps >= 1 && taps <= CONVQ_MAX_TAPS, "a convolution of ", taps, " taps");
  TORCH_CHECK(ring.is_contiguous() && ring.dtype() == proj.dtype() && ring.dim() == 3 &&
              ring.size(1) == taps - 1 && ring.size(2) == C, "convolution state");
  TORCH_CHECK(turn.dtype() == torch::kFloat32 && turn.is_contiguous() && turn.dim() == 2 &&
              turn.size(1) % 2 == 0 && turn.size(1) <= d, "rotation");
  if (value_turn)
    TORCH_CHECK(value_turn->dtype() == torch::kFloat32 && value_turn->is_contiguous() &&
                value_turn->dim() == 2 && value_turn->size(1) == dv && dv % 2 == 0,
                "value rotation");
  TORCH_CHECK(kv_slots.numel() == T_ && kv_slots.dtype() == torch::kInt32 &&
              kv_slots.is_contiguous() && starts.numel() == S &&
              starts.dtype() == torch::kInt32 && starts.is_contiguous() &&
              slots.dtype() == torch::kInt32);
  int blocks = T_;
  if (cu) {
    TORCH_CHECK(bseq && boff && bseq->numel() == boff->numel() && cu->numel() == S + 1 &&
                cu->dtype() == torch::kInt32 && bseq->dtype() == torch::kInt32 &&
                boff->dtype() == torch::kInt32);
    blocks = bseq->numel();
  } else {
    TORCH_CHECK(S == T_);
  }
  if (T_ == 0 || blocks == 0) return;
  ConvHeadArgs a = {};
  a.proj = proj.data_ptr();
  a.stride = proj.stride(0);
  a.q0 = q0; a.k0 = k0; a.v0 = v0;
  a.w = w.data_ptr<float>();
  a.taps = taps; a.C = C;
  a.cs = turn.data_ptr<float>();
  a.rot = turn.size(1);
  if (value_turn) a.vcs = value_turn->data_ptr<float>();
  a.ring = ring.data_ptr();
  a.kv_slots = kv_slots.data_ptr<int>();
  if (cu) {
    a.cu = cu->data_ptr<int>();
    a.bseq = bseq->data_ptr<int>();
    a.boff = boff->data_ptr<int>();
  }
  a.starts = starts.data_ptr<int>();
  a.slots = slots.data_ptr<int>();
  a.q = q.data_ptr(); a.kc = kc.data_ptr(); a.vc = vc.data_ptr();
  a.Hq = Hq; a.Hkv = Hkv; a.d = d; a.dv = dv;
  a.DK = kc.size(3); a.DV = vc.size(3); a.P = kc.size(2);
  DISPATCH_ELEM(proj.dtype() == torch::kBFloat16, {
    constexpr int VW = 16 / sizeof(T);
    auto launch = [&](auto kern, int v) {
      const long units = (Hq + Hkv) * ((a.DK + v - 1) / v) + Hkv * ((a.DV + v - 1) / v);
      hipLaunchKernelGGL(kern, dim3(blocks, (units + 255) / 256), dim3(256), 0, CUR_STREAM, a);
    };
    const bool vec = ((d | dv | a.DK | a.DV | q0 | k0 | v0 | C | proj.stride(0)) & (VW - 1)) == 0 &&
                     (reinterpret_cast<uintptr_t>(a.proj) & 15) == 0;
    if (!vec) launch(conv_qkv_kernel<T, 2, 0, false>, 2);
    else if (taps == 2) launch(conv_qkv_kernel<T, VW, 2, true>, VW);
    else if (taps == 3) launch(conv_qkv_kernel<T, VW, 3, true>, VW);
    else if (taps == 4) launch(conv_qkv_kernel<T, VW, 4, true>, VW);
    else launch(conv_qkv_kernel<T, VW, 0, true>, VW);
  });
  HIP_CHECK_KERNEL();
}
