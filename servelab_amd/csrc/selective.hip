// The selective scan: per channel c a state of N places that every token moves on,
//   S[n][c] <- exp(rate[n][c] dt_c) S[n][c] + dt_c u_c B_n,   y_c = sum_n S[n][c] C_n + skip_c u_c,
// and the read-out times silu of a gate leaves as rows in the activation type.  B and C are a
// token's (shared by the channels), dt = softplus(low W^T + bias) per channel.  Everything is float.
//
// State layout: [N][C], so that neighbouring threads, which own neighbouring channels, read and
// write neighbouring values; a thread keeps its channel's N places in registers.
//
//   step      one token a sequence: dt's product, the state, the read-out and the gate in one launch
//   segment   what a segment of tokens leaves behind when it starts from zero, and the sum of its dt
//             (the factor the state before it keeps is exp(rate sum dt))
//   carry     per place and channel, the state every segment starts from, one after the other
//   read      the segment again, from that state, with read-outs and gate
// A prompt is a chain over its tokens; segments make it as many chains as fill the chip, for the price of
// walking it twice.  Steps no longer than a segment take `read` alone, from and to the slot.
#include "common.h"

__device__ __forceinline__ float sel_softplus(float x) { return fmaxf(x, 0.f) + log1pf(expf(-fabsf(x))); }
__device__ __forceinline__ float sel_silu(float z) { return z / (1.f + expf(-z)); }
constexpr float SEL_LOG2E = 1.4426950408889634f;
// exp(rate dt) with the rate already in units of log 2
__device__ __forceinline__ float sel_decay(float rate2, float dt) { return __builtin_amdgcn_exp2f(rate2 * dt); }

constexpr int SEL_PARTS = 4, SEL_STEP_KEEP = 8;

// Four wavefronts per (token, 64 channels): each takes a quarter of the rank for the step size, then a quarter
// of the places; the partial sums meet in LDS and are added in the wavefronts' order.
__global__ __launch_bounds__(64 * SEL_PARTS) void selective_step_kernel(
    const float* __restrict__ u, int C, const float* __restrict__ proj, int width, int R, int N,
    const float* __restrict__ wt, const float* __restrict__ bias, const float* __restrict__ rates,
    const float* __restrict__ skip, const float* __restrict__ gate, int gate_stride, int gate_col,
    float* __restrict__ state, long long state_stride, const int* __restrict__ positions,
    const int* __restrict__ tok_seq, const int* __restrict__ slots, int write, act_t* __restrict__ out) {
  __shared__ float zs[SEL_PARTS][64], ys[SEL_PARTS][64];
  const size_t t = blockIdx.x;
  const int lane = threadIdx.x & 63, part = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int at = blockIdx.y * 64 + lane;
  const bool live = at < C;
  const int c = live ? at : C - 1;                      // (a lane past the last channel computes it and stores nothing)
  const float* row = proj + t * width;                  // (the same for the whole wavefront)
  const float *B = row + R, *Cn = row + R + N;
  const bool fresh = positions[t] == 0;
  float* S = state + (size_t)slots[tok_seq[t]] * state_stride + c;
  float old[SEL_STEP_KEEP], rate[SEL_STEP_KEEP];        // the first places' values are on their way meanwhile
#pragma unroll
  for (int k = 0; k < SEL_STEP_KEEP; ++k) {
    const int n = part + SEL_PARTS * k;
    old[k] = n < N && !fresh ? S[(size_t)n * C] : 0.f;
    rate[k] = n < N ? rates[(size_t)n * C + c] : 0.f;
  }
  const float x = u[t * C + c];
  float z = 0.f;
#pragma unroll 16
  for (int r = part; r < R; r += SEL_PARTS) z += row[r] * wt[(size_t)r * C + c];
  zs[part][lane] = z;
  __syncthreads();
  z = (zs[0][lane] + zs[1][lane]) + (zs[2][lane] + zs[3][lane]);
  const float dt = sel_softplus(z + bias[c]);
  const float dx = dt * x;
  float y = 0.f;
  auto place = [&](int n, float before, float r) {
    const float s = sel_decay(r * SEL_LOG2E, dt) * before + dx * B[n];
    if (write && live) S[(size_t)n * C] = s;
    y += s * Cn[n];
  };
#pragma unroll
  for (int k = 0; k < SEL_STEP_KEEP; ++k)
    if (part + SEL_PARTS * k < N) place(part + SEL_PARTS * k, old[k], rate[k]);
  for (int n = part + SEL_PARTS * SEL_STEP_KEEP; n < N; n += SEL_PARTS)
    place(n, fresh ? 0.f : S[(size_t)n * C], rates[(size_t)n * C + c]);
  ys[part][lane] = y;
  __syncthreads();
  if (part != 0 || !live) return;
  y = ((ys[0][lane] + ys[1][lane]) + (ys[2][lane] + ys[3][lane])) + skip[c] * x;
  out[t * C + c] = from_f<act_t>(y * sel_silu(gate[t * gate_stride + gate_col + c]));
}

extern "C" const char* sl_selective_step(const float* u, int C, const float* proj, int width, int R, int N,
                                         const float* wt, const float* bias, const float* rates, const float* skip,
                                         const float* gate, int gate_stride, int gate_col, float* state,
                                         long long state_stride, const int* positions, const int* tok_seq,
                                         const int* slots, int T, int write, void* out, hipStream_t stream) {
  SL_CHECK(T >= 0 && C > 0 && R > 0 && N > 0, "selective_step: sizes must be positive");
  SL_CHECK(R + 2 * N <= width && gate_col >= 0 && gate_col + C <= gate_stride, "selective_step: the rows are too short");
  SL_CHECK((long long)N * C <= state_stride, "selective_step: the state does not fit its slot");
  if (T == 0) return nullptr;
  selective_step_kernel<<<dim3(T, (C + 63) / 64), 64 * SEL_PARTS, 0, stream>>>(
      u, C, proj, width, R, N, wt, bias, rates, skip, gate, gate_stride, gate_col, state, state_stride, positions,
      tok_seq, slots, write, (act_t*)out);
  return sl_launch_status();
}

// A thread takes a channel of a (sequence, segment) with its N places: NB exactly (EXACT) or at most.
//   PASS 0: from zero, what it leaves into part and sums.
//   PASS 1: from part (several segments) or the slot, read-outs, gate; one segment: the state into the slot.
template <int NB, bool EXACT, int PASS>
__global__ __launch_bounds__(64) void selective_segment_kernel(
    const float* __restrict__ u, const float* __restrict__ dts, int C, const float* __restrict__ proj, int width,
    int R, int N, const float* __restrict__ rates, const float* __restrict__ skip, const float* __restrict__ gate,
    int gate_stride, int gate_col, float* state, long long state_stride, const int* __restrict__ cu_q,
    const int* __restrict__ positions, const int* __restrict__ slots, int seg, int segs, int write, float* part,
    float* sums, act_t* __restrict__ out) {
  const int s = blockIdx.z, g = blockIdx.y, c = blockIdx.x * 64 + threadIdx.x;
  const int first = cu_q[s], last = cu_q[s + 1];
  const int t0 = first + g * seg;
  if (t0 >= last || c >= C) return;
  const int t1 = min(t0 + seg, last);
  float S[NB], A[NB];
  float* keep = part != nullptr ? part + (((size_t)s * segs + g) * N) * C + c : nullptr;
  float* slot = state + (size_t)slots[s] * state_stride + c;
  const bool fresh = positions[first] == 0;
#pragma unroll
  for (int n = 0; n < NB; ++n) {
    const bool in = EXACT || n < N;
    A[n] = in ? rates[(size_t)n * C + c] * SEL_LOG2E : 0.f;
    S[n] = 0.f;
    if (PASS == 1 && in) {
      if (segs > 1) S[n] = keep[(size_t)n * C];
      else if (!fresh) S[n] = slot[(size_t)n * C];
    }
  }
  const float sk = PASS == 1 ? skip[c] : 0.f;
  float total = 0.f;
  float x = u[(size_t)t0 * C + c], dt = dts[(size_t)t0 * C + c];
  float z = PASS == 1 ? gate[(size_t)t0 * gate_stride + gate_col + c] : 0.f;
  for (int t = t0; t < t1; ++t) {
    // (the next token's values are asked for before this one's are used)
    const int tn = t + 1 < t1 ? t + 1 : t;
    const float xn = u[(size_t)tn * C + c], dn = dts[(size_t)tn * C + c];
    const float zn = PASS == 1 ? gate[(size_t)tn * gate_stride + gate_col + c] : 0.f;
    const float* B = proj + (size_t)t * width + R;      // (the same for the whole wavefront)
    const float* Cn = B + N;
    const float dx = dt * x;
    float y0 = 0.f, y1 = 0.f;
#pragma unroll
    for (int n = 0; n < NB; ++n) {
      if (!EXACT && n >= N) continue;
      S[n] = sel_decay(A[n], dt) * S[n] + dx * B[n];
      if (PASS == 1) {
        if (n & 1) y1 += S[n] * Cn[n];
        else y0 += S[n] * Cn[n];
      }
    }
    if (PASS == 0) total += dt;
    else out[(size_t)t * C + c] = from_f<act_t>(((y0 + y1) + sk * x) * sel_silu(z));
    x = xn;
    dt = dn;
    z = zn;
  }
  if (PASS == 0) {
    sums[((size_t)s * segs + g) * C + c] = total;
#pragma unroll
    for (int n = 0; n < NB; ++n)
      if (EXACT || n < N) keep[(size_t)n * C] = S[n];
  } else if (write && segs == 1) {
#pragma unroll
    for (int n = 0; n < NB; ++n)
      if (EXACT || n < N) slot[(size_t)n * C] = S[n];
  }
}

// A thread takes a place of a channel of a sequence and walks the segments: part holds what each left from
// zero and receives what it starts from; the last state goes to the slot.
__global__ __launch_bounds__(256) void selective_carry_kernel(
    int C, int N, const float* __restrict__ rates, float* __restrict__ state, long long state_stride,
    const int* __restrict__ cu_q, const int* __restrict__ positions, const int* __restrict__ slots, int seg, int segs,
    int write, float* __restrict__ part, const float* __restrict__ sums) {
  const int s = blockIdx.z, n = blockIdx.y, c = blockIdx.x * 256 + threadIdx.x;
  if (c >= C) return;
  const int first = cu_q[s], len = cu_q[s + 1] - first;
  const int used = (len + seg - 1) / seg;
  float* slot = state + (size_t)slots[s] * state_stride + (size_t)n * C + c;
  const float rate2 = rates[(size_t)n * C + c] * SEL_LOG2E;
  float h = positions[first] == 0 ? 0.f : *slot;
  float* p = part + (((size_t)s * segs) * N + n) * C + c;
  const float* sm = sums + (size_t)s * segs * C + c;
  const size_t step = (size_t)N * C;
#pragma unroll 4
  for (int g = 0; g < used; ++g) {
    const float left = p[g * step], f = sel_decay(rate2, sm[(size_t)g * C]);
    p[g * step] = h;
    h = f * h + left;
  }
  if (write) *slot = h;
}

// Any number of places: a wavefront's lanes share the places of 1 channel (lane n takes places n, n + 64, ..,
// at most SEL_WIDE of them), a token's read-out is a sum over the wavefront.  Segments are not used.
constexpr int SEL_WIDE = 16;
__global__ __launch_bounds__(64) void selective_wide_kernel(
    const float* __restrict__ u, const float* __restrict__ dts, int C, const float* __restrict__ proj, int width,
    int R, int N, const float* __restrict__ rates, const float* __restrict__ skip, const float* __restrict__ gate,
    int gate_stride, int gate_col, float* __restrict__ state, long long state_stride, const int* __restrict__ cu_q,
    const int* __restrict__ positions, const int* __restrict__ slots, int write, act_t* __restrict__ out) {
  const int c = blockIdx.x, s = blockIdx.y, lane = threadIdx.x;
  const int first = cu_q[s], last = cu_q[s + 1];
  float* slot = state + (size_t)slots[s] * state_stride + c;
  const bool fresh = positions[first] == 0;
  float S[SEL_WIDE], A[SEL_WIDE];
#pragma unroll
  for (int i = 0; i < SEL_WIDE; ++i) {
    const int n = lane + 64 * i;
    A[i] = n < N ? rates[(size_t)n * C + c] * SEL_LOG2E : 0.f;
    S[i] = n < N && !fresh ? slot[(size_t)n * C] : 0.f;
  }
  for (int t = first; t < last; ++t) {
    const float* B = proj + (size_t)t * width + R;
    const float x = u[(size_t)t * C + c], dt = dts[(size_t)t * C + c];
    float y = 0.f;
#pragma unroll
    for (int i = 0; i < SEL_WIDE; ++i) {
      const int n = lane + 64 * i;
      if (n < N) {
        S[i] = sel_decay(A[i], dt) * S[i] + dt * x * B[n];
        y += S[i] * B[N + n];
      }
    }
    y = wave_sum(y) + skip[c] * x;
    if (lane == 0)
      out[(size_t)t * C + c] = from_f<act_t>(y * sel_silu(gate[(size_t)t * gate_stride + gate_col + c]));
  }
#pragma unroll
  for (int i = 0; i < SEL_WIDE; ++i)
    if (write && lane + 64 * i < N) slot[(size_t)(lane + 64 * i) * C] = S[i];
}

extern "C" const char* sl_selective_scan(const float* u, const float* dts, int C, const float* proj, int width, int R,
                                         int N, const float* rates, const float* skip, const float* gate,
                                         int gate_stride, int gate_col, float* state, long long state_stride,
                                         const int* cu_q, const int* positions, const int* slots, int S, int T,
                                         int max_q_len, int seg, int write, float* part, float* sums, void* out,
                                         hipStream_t stream) {
  SL_CHECK(T >= 0 && S >= 0 && C > 0 && R > 0 && N > 0 && seg > 0, "selective_scan: sizes must be positive");
  SL_CHECK(N <= 64 * SEL_WIDE, "selective_scan: at most 1,024 places a channel");
  SL_CHECK(R + 2 * N <= width && gate_col >= 0 && gate_col + C <= gate_stride, "selective_scan: the rows are too short");
  SL_CHECK((long long)N * C <= state_stride, "selective_scan: the state does not fit its slot");
  SL_CHECK(S <= 65535 && N <= 65535, "selective_scan: grid too large");
  if (T == 0 || S == 0) return nullptr;
  if (N > 64) {
    selective_wide_kernel<<<dim3(C, S), 64, 0, stream>>>(u, dts, C, proj, width, R, N, rates, skip, gate, gate_stride,
                                                         gate_col, state, state_stride, cu_q, positions, slots, write,
                                                         (act_t*)out);
    return sl_launch_status();
  }
  const int segs = (max_q_len + seg - 1) / seg;
  SL_CHECK(segs <= 65535, "selective_scan: too many segments");
  SL_CHECK(segs == 1 || (part != nullptr && sums != nullptr), "selective_scan: segments need their buffers");
  if (segs == 1) part = nullptr;
  const dim3 grid((C + 63) / 64, segs, S);
#define SEL_PASS(NB, EXACT, PASS)                                                                                  \
  selective_segment_kernel<NB, EXACT, PASS><<<grid, 64, 0, stream>>>(u, dts, C, proj, width, R, N, rates, skip, gate, \
                                                                     gate_stride, gate_col, state, state_stride,   \
                                                                     cu_q, positions, slots, seg, segs, write, part, sums, \
                                                                     (act_t*)out)
#define SEL_RUN(NB, EXACT)                                                                                         \
  do {                                                                                                             \
    if (segs > 1) {                                                                                                \
      SEL_PASS(NB, EXACT, 0);                                                                                      \
      selective_carry_kernel<<<dim3((C + 255) / 256, N, S), 256, 0, stream>>>(C, N, rates, state, state_stride,    \
                                                                              cu_q, positions, slots, seg, segs,   \
                                                                              write, part, sums);                  \
    }                                                                                                              \
    SEL_PASS(NB, EXACT, 1);                                                                                        \
  } while (0)
  if (N == 8) SEL_RUN(8, true);
  else if (N == 16) SEL_RUN(16, true);
  else if (N == 24) SEL_RUN(24, true);
  else if (N == 32) SEL_RUN(32, true);
  else if (N == 64) SEL_RUN(64, true);
  else if (N < 16) SEL_RUN(16, false);
  else if (N < 32) SEL_RUN(32, false);
  else SEL_RUN(64, false);
#undef SEL_RUN
#undef SEL_PASS
  return sl_launch_status();
}
