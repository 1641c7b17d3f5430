// Which class runs a pipeline type.  Every schedule's source file registers its types, so a program
// links the schedules it serves and no others.
#pragma once
#include <functional>
#include <map>
#include <memory>

#include "computeBound.h"

using PipelineFactory = std::function<std::unique_ptr<PipelineBase>(vortexInitData* input, int rank, int nranks, int vnranks)>;
std::map<Worker::PipelineType, PipelineFactory>& pipelineFactories();
struct RegisterPipeline {
  RegisterPipeline(Worker::PipelineType type, PipelineFactory make) { pipelineFactories()[type] = std::move(make); }
};
