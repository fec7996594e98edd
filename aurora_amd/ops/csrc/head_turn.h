// What may still happen to an attention head's result before it is stored: values
// that were rotated by their own positions turn back by the query's, and every
// channel is multiplied by a sigmoid gate.
#pragma once
#include <torch/extension.h>

#include "elem.h"

struct HeadTurn {
  const float* cs;   // [positions, dv]: cosines, then sines of every pair; null: no turn
  const void* gate;  // [rows, gstride] pre-activations, heads dv apart; null: no gate
  long gstride;
};

// Channel d of a head; the other channel of its pair is the neighbouring lane's, so
// all lanes of a wave take part (d past dv gives nothing useful).
template <typename T>
DEVINL float turned(const HeadTurn& t, float o, long row, int pos, int h, int d, int dv) {
  const int e = min(d, dv - 1);
  if (t.cs) {
    const float other = __shfl_xor(o, 1, WAVE);
    const float* cs = t.cs + (long)pos * dv + e / 2;
    o = o * cs[0] + (d & 1 ? -other : other) * cs[dv / 2];
  }
  if (t.gate) o *= sigmoid_f(ldf((const T*)t.gate + row * t.gstride + h * dv + e));
  return o;
}

// neighbouring dimensions (u, v) of a query or key by the angle of (c, s)
DEVINL void turn_pair(float& u, float& v, float c, float s) {
  const float a = u * c - v * s;
  v = v * c + u * s;
  u = a;
}

// turn and gate of the attention kernels' results; they come without a penalty
inline HeadTurn head_turn(const c10::optional<torch::Tensor>& turn,
                          const c10::optional<torch::Tensor>& gate, bool penalty,
                          const torch::Tensor& q, long Hq, long dv) {
  HeadTurn t = {};
  TORCH_CHECK(!penalty || !(turn || gate), "a penalty beside a turned or gated result");
  if (turn) {
    TORCH_CHECK(turn->dtype() == torch::kFloat32 && turn->is_contiguous() &&
                turn->dim() == 2 && turn->size(1) == dv && dv % 2 == 0, "value rotation");
    t.cs = turn->data_ptr<float>();
  }
  if (gate) {
    TORCH_CHECK(gate->dtype() == q.dtype() && gate->dim() == 2 && gate->stride(1) == 1 &&
                gate->size(0) == q.size(0) && gate->size(1) == Hq * dv, "gate");
    t.gate = gate->data_ptr();
    t.gstride = gate->stride(0);
  }
  return t;
}
