// What every entry point of the library shares: the error text and the HIP graph helpers.  See include/vui_amd.h.
#include <stdarg.h>
#include <stdio.h>

#include <new>

#include "internal.h"

static thread_local char g_err[512] = "";

void vui_set_error(const char* fmt, ...) {
  va_list ap;
  va_start(ap, fmt);
  vsnprintf(g_err, sizeof(g_err), fmt, ap);
  va_end(ap);
}

extern "C" {

const char* vui_last_error(void) { return g_err; }
int vui_version(void) { return 1; }

// ---- HIP graphs ----
struct vui_graph {
  hipGraph_t graph;
  hipGraphExec_t exec;
};

int vui_graph_begin(vui_stream_t stream) {
  HIP_TRY(hipStreamBeginCapture((hipStream_t)stream, hipStreamCaptureModeThreadLocal));
  return VUI_OK;
}

int vui_graph_end(vui_stream_t stream, vui_graph** out) {
  hipGraph_t g = nullptr;
  HIP_TRY(hipStreamEndCapture((hipStream_t)stream, &g));
  if (!out || !g) { if (g) (void)hipGraphDestroy(g); vui_set_error("capture produced no graph"); return VUI_EINVAL; }
  hipGraphExec_t e = nullptr;
  hipError_t err = hipGraphInstantiate(&e, g, nullptr, nullptr, 0);
  if (err != hipSuccess) { (void)hipGraphDestroy(g); vui_set_error("hipGraphInstantiate failed: %s", hipGetErrorString(err)); return VUI_EHIP; }
  vui_graph* vg = new (std::nothrow) vui_graph();
  if (!vg) { (void)hipGraphExecDestroy(e); (void)hipGraphDestroy(g); vui_set_error("out of host memory"); return VUI_ENOMEM; }
  vg->graph = g; vg->exec = e;
  *out = vg;
  return VUI_OK;
}

int vui_graph_launch(vui_graph* g, vui_stream_t stream) {
  if (!g) { vui_set_error("NULL graph"); return VUI_EINVAL; }
  HIP_TRY(hipGraphLaunch(g->exec, (hipStream_t)stream));
  return VUI_OK;
}

void vui_graph_destroy(vui_graph* g) {
  if (!g) return;
  (void)hipGraphExecDestroy(g->exec);
  (void)hipGraphDestroy(g->graph);
  delete g;
}

}  // extern "C"
